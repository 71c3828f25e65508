"""TEST INFRASTRUCTURE ONLY — plain, slow torch statement of the Beronex design, one function per mechanism, evaluated on the
CPU in fp64 (or fp32).  It shares no code with ktransformers_amd: the product's operators, cache and kernels are compared
with it.  Whole sequences only: no cache, no batching, no portions — a sequence is a list of token ids.

Notation: x is the residual at all positions (positions count from 0), W a weight stored [out, in] and applied as W @ h,
`P[name]` a tensor of the checkpoint, `cfg` the parsed config.json."""
from __future__ import annotations

import copy
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


def router_scores(P, pre, h):
    return h @ P[pre + "router"].T + P[pre + "router.b"]


def mixture(P, pre, c, h):
    idx, w = routed(router_scores(P, pre, h), c["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(c["router"]["experts"]):
        tok, k = torch.nonzero(idx == e, as_tuple=True)
        if tok.numel():
            out[tok] += w[tok, k].view(-1, 1) * bounded_expert(P, f"{pre}e{e}.", float(c["expert"]["limit"]), h[tok])
    return out


def forward(P, cfg, tokens, dtype=torch.float64, return_layers=False, return_gaps=False):
    """tokens: list of ids -> logits [T, vocab]; if asked also the residual after every layer [layers, T, width], and per position the
    smallest distance between the last chosen and the first left-out router score of any mixture (how close a call the routing was)."""
    P = {n: (t.to(dtype) if t.is_floating_point() else t) for n, t in P.items()}
    eps = float(cfg["norm"]["eps"])
    x = P["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    kept, trail, gaps = {}, [], torch.full((len(tokens),), float("inf"), dtype=dtype)
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
            if m["kind"] == "dense":
                y = dense_feed_forward(P, pre + "mlp.", h)
            else:
                y = mixture(P, pre + "mlp.", m, h)
                top = m["router"]["top"]
                if top < m["router"]["experts"]:
                    z = torch.sort(router_scores(P, pre + "mlp.", h), dim=-1, descending=True).values
                    gaps = torch.minimum(gaps, z[:, top - 1] - z[:, top])
            x = x + rms_norm(y, P[pre + "norm2b"], eps)
        trail.append(x)
    logits = rms_norm(x, P["final.norm"], eps) @ P["head"].T
    extra = ([torch.stack(trail)] if return_layers else []) + ([gaps] if return_gaps else [])
    return (logits, *extra) if extra else logits


# ---- small configurations and random checkpoints for the tests ---------------------------------------------------------------------
def rot_of(dims, base=500.0, factor=6.0, original=64, fast=8.0, slow=1.0, scaled=True):
    if not dims:
        return None
    return {"base": base, "dims": dims, "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow} if scaled else None}


def dense_mlp(ff=40):
    return {"kind": "dense", "ff": ff}


def moe_mlp(experts=6, top=2, ff=20, limit=1.5):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def attention_layer(heads=4, kv_heads=2, dim=12, vdim=10, window=9, scale=None, rot=rot_of(8), kv_from=None, mlp="dense"):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window} if window else None,
         "scale": scale if scale is not None else 1.7 * dim ** -0.5, "rot": copy.deepcopy(rot)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": dense_mlp() if mlp == "dense" else mlp}


def latent_layer(heads=3, dim=10, rot_dim=8, vdim=14, q_rank=18, kv_rank=20, scale=None, rot=rot_of(8, base=300.0, factor=4.0), mlp="dense"):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": scale if scale is not None else 1.3 * (dim + rot_dim) ** -0.5, "rot": copy.deepcopy(rot)}
    return {"type": "latent_attention", "mixer": m, "mlp": dense_mlp() if mlp == "dense" else mlp}


def lightning_layer(heads=3, dim=8, vdim=12, decay=None, mlp="dense"):
    decay = [0.5 + 0.49 * (i + 1) / heads for i in range(heads)] if decay is None else list(decay)
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": dense_mlp() if mlp == "dense" else mlp}


def make_config(layers, width=32, vocab=61, eps=1e-5, embed_scale=3.0):
    return {"architecture": "Beronex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": embed_scale}, "layers": layers}


def random_checkpoint(cfg: dict, seed: int = 0) -> dict:
    """Random bf16-representable weights with the checkpoint's tensor names for a config of the design."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def mat(o, i, s=None):
        return (torch.randn(o, i, generator=g) * (s if s is not None else 1.0 / math.sqrt(i))).to(torch.bfloat16)

    def vec(k, mean=1.0, s=0.2):
        return (mean + torch.randn(k, generator=g) * s).to(torch.bfloat16)

    P = {"embed": mat(cfg["vocab"], W, 0.4), "head": mat(cfg["vocab"], W, 2.0 / math.sqrt(W)), "final.norm": vec(W)}
    for li, layer in enumerate(cfg["layers"]):
        p, m, c = f"l{li}.", layer["mixer"], layer.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if c else ()):
            P[p + n] = vec(W, 0.7 if n.endswith("b") else 1.0)
        H, V = m["heads"], m["vdim"]
        if layer["type"] == "attention":
            D, G = m["dim"], m["kv_heads"]
            for t, rows in (("q", H * D), ("k", G * D), ("v", G * V)) if m.get("kv_from") is None else (("q", H * D),):
                P[p + f"mix.{t}"] = mat(rows, W)
            P[p + "mix.g"] = mat(H, W, 1.5 / math.sqrt(W))
        elif layer["type"] == "latent_attention":
            D, R, Q, L = m["dim"], m["rot_dim"], m["q_rank"], m["kv_rank"]
            P[p + "mix.dq"], P[p + "mix.dq.norm"], P[p + "mix.uq"] = mat(Q, W), vec(Q), mat(H * (D + R), Q, 1.3 / math.sqrt(Q))
            P[p + "mix.dkv"], P[p + "mix.dkv.norm"] = mat(L + R, W), vec(L)
            P[p + "mix.uk"], P[p + "mix.uv"] = mat(H * D, L), mat(H * V, L)
        else:
            for t, rows in (("q", H * m["dim"]), ("k", H * m["dim"]), ("v", H * V), ("g", H * V)):
                P[p + f"mix.{t}"] = mat(rows, W)
            P[p + "mix.norm"] = vec(H * V)
        P[p + "mix.o"] = mat(W, H * V)
        if c and c["kind"] == "dense":
            P[p + "mlp.gate"], P[p + "mlp.up"], P[p + "mlp.down"] = mat(c["ff"], W), mat(c["ff"], W), mat(W, c["ff"])
        elif c:
            P[p + "mlp.router"], P[p + "mlp.router.b"] = mat(c["router"]["experts"], W, 2.5 / math.sqrt(W)), vec(c["router"]["experts"], 0.0, 1.0)
            for e in range(c["router"]["experts"]):
                for t, o, i in (("gate", c["expert"]["ff"], W), ("up", c["expert"]["ff"], W), ("down", W, c["expert"]["ff"])):
                    P[p + f"mlp.e{e}.{t}"] = mat(o, i, (1.5 if t != "down" else 1.0) / math.sqrt(i))
    return P


def as_double(P: dict) -> dict:
    return {k: (v.double() if v.is_floating_point() else v) for k, v in P.items()}
