"""TEST INFRASTRUCTURE ONLY — plain, slow torch statement of the Beronex design, one function per mechanism, evaluated on the
CPU in fp64 (or fp32).  It shares no code with ktransformers_amd: the product's operators, cache and kernels are compared
with it.  Whole sequences only: no cache, no batching, no portions — a sequence is a list of token ids.

Notation: x is the residual at all positions (positions count from 0), W a weight stored [out, in] and applied as W @ h,
`P[name]` a tensor of the checkpoint, `cfg` the parsed config.json."""
from __future__ import annotations

import math

import torch


def unit_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def yarn(base, dims, scaling):
    """(angular frequency of every turning pair, factor on cosines and sines).  Pairs that turn more than `fast` times within `original`
    positions keep their frequency, those that turn less than `slow` times have it divided by `factor`, a linear ramp between."""
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freq, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])
    turns_at = lambda t: dims * math.log(original / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo = max(math.floor(turns_at(float(scaling["fast"]))), 0)
    hi = min(math.ceil(turns_at(float(scaling["slow"]))), dims - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(v, rot, half):
    """v [T, heads, n]: the first rot.dims entries of the last axis turn by position x frequency; `half`: entry i pairs with i + dims / 2,
    otherwise 2i with 2i + 1."""
    if not rot:
        return v
    n = int(rot["dims"])
    freq, amp = yarn(float(rot["base"]), n, rot.get("scaling"))
    pos = torch.arange(v.shape[0], dtype=torch.float64)
    out = v.clone()
    for i, f in enumerate(freq):
        c, s = ((fn(pos * f) * amp).to(v.dtype).view(-1, 1) for fn in (torch.cos, torch.sin))
        a, b = (i, i + n // 2) if half else (2 * i, 2 * i + 1)
        out[..., a] = v[..., a] * c - v[..., b] * s
        out[..., b] = v[..., b] * c + v[..., a] * s
    return out


def softmax_attention(q, k, v, scale, window=None):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]; position i sees j <= i, with a window only 0 <= i - j < window; query head h
    reads key / value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    hidden = j > i
    if window:
        hidden = hidden | (i - j >= window)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(hidden, float("-inf"))
        out[:, h] = torch.softmax(s, dim=1) @ v[:, g]
    return out


def window_attention(P, pre, c, h, eps, kept):
    """Grouped-query window attention, rotated then unit-RMS q and k, one gate per head.  `kept`: {layer: (k, v)} of the layers run so far;
    with kv_from the keys and values are another layer's.  Returns (output, k, v)."""
    T = h.shape[0]
    H, G, D, V = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    rot = c.get("rot") or None
    q = unit_rms(rotate((h @ P[pre + "q"].T).view(T, H, D), rot, False), eps)
    if c.get("kv_from") is not None:
        k, v = kept[c["kv_from"]]
    else:
        k = unit_rms(rotate((h @ P[pre + "k"].T).view(T, G, D), rot, False), eps)
        v = (h @ P[pre + "v"].T).view(T, G, V)
    o = softmax_attention(q, k, v, c["scale"], (c.get("mask") or {}).get("size"))
    o = o * torch.sigmoid(h @ P[pre + "g"].T).view(T, H, 1)
    return o.reshape(T, H * V) @ P[pre + "o"].T, k, v


def latent_attention(P, pre, c, h, eps):
    """Keys and values are projections of a normed latent; one rotated key part is shared by the heads; queries go through a normed latent."""
    T = h.shape[0]
    H, D, R, V, L = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    rot = c.get("rot") or None
    cq = rms_norm(h @ P[pre + "dq"].T, P[pre + "dq.norm"], eps)
    q = (cq @ P[pre + "uq"].T).view(T, H, D + R)
    down = h @ P[pre + "dkv"].T
    lat = rms_norm(down[:, :L], P[pre + "dkv.norm"], eps)
    kr = rotate(down[:, L:].view(T, 1, R), rot, True).expand(T, H, R)
    k = torch.cat([(lat @ P[pre + "uk"].T).view(T, H, D), kr], dim=-1)
    q = torch.cat([q[..., :D], rotate(q[..., D:], rot, True)], dim=-1)
    v = (lat @ P[pre + "uv"].T).view(T, H, V)
    return softmax_attention(q, k, v, c["scale"]).reshape(T, H * V) @ P[pre + "o"].T


def decayed_scan(q, k, v, decay):
    """One head: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t; q, k [T, D], v [T, V], decay a number."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype)
    out = []
    for t in range(q.shape[0]):
        S = decay * S + k[t].view(-1, 1) * v[t].view(1, -1)
        out.append(S.T @ q[t])
    return torch.stack(out)


def lightning_attention(P, pre, c, h, eps):
    T = h.shape[0]
    H, D, V = c["heads"], c["dim"], c["vdim"]
    q = silu(h @ P[pre + "q"].T).view(T, H, D)
    k = silu(h @ P[pre + "k"].T).view(T, H, D)
    v = silu(h @ P[pre + "v"].T).view(T, H, V)
    o = torch.stack([decayed_scan(q[:, i], k[:, i], v[:, i], float(c["decay"][i])) for i in range(H)], dim=1).reshape(T, H * V)
    return (rms_norm(o, P[pre + "norm"], eps) * torch.sigmoid(h @ P[pre + "g"].T)) @ P[pre + "o"].T


def dense_feed_forward(P, pre, h):
    return (gelu_tanh(h @ P[pre + "gate"].T) * (h @ P[pre + "up"].T)) @ P[pre + "down"].T


def bounded_expert(P, pre, limit, h):
    g = torch.clamp(h @ P[pre + "gate"].T, max=limit)
    u = torch.clamp(h @ P[pre + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ P[pre + "down"].T


def routed(z, top):
    """[T, experts] router scores -> (chosen [T, top], softmax over the chosen scores)."""
    zs, idx = torch.sort(z, dim=-1, descending=True, stable=True)
    return idx[:, :top], torch.softmax(zs[:, :top], dim=-1)


def mixture(P, pre, c, h):
    idx, w = routed(h @ P[pre + "router"].T + P[pre + "router.b"], c["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(c["router"]["experts"]):
        tok, k = torch.nonzero(idx == e, as_tuple=True)
        if tok.numel():
            out[tok] += w[tok, k].view(-1, 1) * bounded_expert(P, f"{pre}e{e}.", float(c["expert"]["limit"]), h[tok])
    return out


def run(P, cfg, tokens, dtype=torch.float64):
    """(logits [T, vocab], residual after every layer [layers, T, width])."""
    P = {n: (t if t.dtype == torch.int32 else t.to(dtype)) for n, t in P.items()}
    eps = float(cfg["norm"]["eps"])
    x = P["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    kept, trail = {}, []
    for i, L in enumerate(cfg["layers"]):
        pre, c = f"l{i}.", L["mixer"]
        h = rms_norm(x, P[pre + "norm1"], eps)
        if L["type"] == "attention":
            y, k, v = window_attention(P, pre + "mix.", c, h, eps, kept)
            kept[i] = (k, v)
        elif L["type"] == "latent_attention":
            y = latent_attention(P, pre + "mix.", c, h, eps)
        else:
            y = lightning_attention(P, pre + "mix.", c, h, eps)
        x = x + rms_norm(y, P[pre + "norm1b"], eps)
        m = L.get("mlp")
        if m is not None:
            h = rms_norm(x, P[pre + "norm2"], eps)
            y = dense_feed_forward(P, pre + "mlp.", h) if m["kind"] == "dense" else mixture(P, pre + "mlp.", m, h)
            x = x + rms_norm(y, P[pre + "norm2b"], eps)
        trail.append(x)
    return rms_norm(x, P["final.norm"], eps) @ P["head"].T, torch.stack(trail)
