"""TEST INFRASTRUCTURE ONLY — plain, slow torch statement of the Dunusun design, one function per mechanism, evaluated on the
CPU in fp64 (or fp32).  It shares no code with ktransformers_amd: the product's operators, cache and kernels are compared
with it.  Whole sequences only: no cache, no batching, no chunking — a sequence is a list of token ids.

Notation: X[s] are the residual copies at all positions (positions count from 0), W a weight stored [out, in] and applied as
W @ h, `P[name]` a tensor of the checkpoint, `cfg` the parsed config.json."""
from __future__ import annotations

import math

import torch


def layer_norm(x, w, b, eps):
    mu = x.mean(dim=-1, keepdim=True)
    var = (x - mu).pow(2).mean(dim=-1, keepdim=True)
    return (x - mu) / torch.sqrt(var + eps) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


def causal_conv(u, w, b=None):
    """u [T, C], w [C, K]: y[t, c] = b[c] + sum_j w[c, j] u[t - K + 1 + j, c] (the last column multiplies the current token), zeros
    before position 0."""
    T, C = u.shape
    K = w.shape[1]
    y = torch.zeros_like(u) if b is None else b.expand(T, C).clone()
    for j in range(K):
        back = K - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y


def rotate_pairs(v, pos, base, dims):
    """v [T, heads, n]: entries (2i, 2i + 1) of the last axis, i < dims / 2, turn together by pos[t] * base^(-2i / dims)."""
    out = v.clone()
    for i in range(dims // 2):
        ang = (pos.to(v.dtype) * float(base) ** (-2.0 * i / dims)).view(-1, 1)
        c, s = torch.cos(ang), torch.sin(ang)
        a, b = v[..., 2 * i], v[..., 2 * i + 1]
        out[..., 2 * i] = a * c - b * s
        out[..., 2 * i + 1] = b * c + a * s
    return out


def soft_cap(x, cap):
    return x if cap is None else cap * torch.tanh(x / cap)


def capped_attention_core(q, k, v, scale, cap):
    """q [T, H, D], k [T, G, D], v [T, G, V] of ONE sequence -> [T, H, V]: softmax over j <= i of cap * tanh(scale q_i.k_j / cap);
    query head h reads key / value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = soft_cap((q[:, h] @ k[:, g].T) * scale, cap)
        out[:, h] = torch.softmax(s.masked_fill(j > i, float("-inf")), dim=1) @ v[:, g]
    return out


def gated_capped_attention(P, pre, c, h):
    """The left mixer: convolved, partly rotated grouped-query attention with capped scores and a sigmoid output gate."""
    T = h.shape[0]
    H, G, D, V = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (h @ P[pre + n].T for n in "qkv")
    if int(c.get("conv") or 0) > 0:
        q, k, v = (causal_conv(u, P[pre + n + ".conv"]) for u, n in ((q, "q"), (k, "k"), (v, "v")))
    q, k, v = q.view(T, H, D), k.view(T, G, D), v.view(T, G, V)
    rot = c.get("rot") or None
    if rot:
        pos = torch.arange(T)
        q, k = rotate_pairs(q, pos, rot["base"], rot["dims"]), rotate_pairs(k, pos, rot["base"], rot["dims"])
    o = capped_attention_core(q, k, v, c["scale"], c.get("softcap")).reshape(T, H * V)
    return (o * torch.sigmoid(h @ P[pre + "g"].T)) @ P[pre + "o"].T


def decayed_outer_scan(q, k, v, decay):
    """One head: S_t = diag(decay_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t; q, k, decay [T, D], v [T, V] -> [T, V]; S starts at 0."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype)
    out = []
    for t in range(q.shape[0]):
        S = decay[t].view(-1, 1) * S + k[t].view(-1, 1) * v[t].view(1, -1)
        out.append(S.T @ q[t])
    return torch.stack(out)


def gated_linear_attention(P, pre, c, h, eps):
    """The right mixer: a matrix state whose key rows decay by sigmoid(z)^(1 / tau), z a low-rank projection plus a bias."""
    T = h.shape[0]
    H, D, V, tau = c["heads"], c["dim"], c["vdim"], float(c["tau"])
    q = (h @ P[pre + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ P[pre + "k"].T).view(T, H, D)
    v = (h @ P[pre + "v"].T).view(T, H, V)
    z = (h @ P[pre + "a1"].T) @ P[pre + "a2"].T + P[pre + "a2.b"]
    alpha = torch.exp(torch.nn.functional.logsigmoid(z) / tau).view(T, H, D)
    o = torch.stack([decayed_outer_scan(q[:, i], k[:, i], v[:, i], alpha[:, i]) for i in range(H)], dim=1)
    o = unit_rms(o, eps) * P[pre + "norm"]
    return (o.reshape(T, H * V) * silu(h @ P[pre + "g"].T)) @ P[pre + "o"].T


def parallel_mixer(P, pre, c, h, eps):
    return float(c["left_scale"]) * gated_capped_attention(P, pre + "left.", c["left"], h) + \
        float(c["right_scale"]) * gated_linear_attention(P, pre + "right.", c["right"], h, eps)


def state_space_mixer(P, pre, c, h, eps):
    """State-space duality (Mamba-2): one decay per head and token, keys B and queries C shared by the heads of a group."""
    T = h.shape[0]
    H, V, N, G, parts = c["heads"], c["vdim"], c["state"], c["groups"], c["norm_groups"]
    I = H * V
    z, xbc, dt = torch.split(h @ P[pre + "in"].T, [I, I + 2 * G * N, H], dim=1)
    xbc = silu(causal_conv(xbc, P[pre + "conv"], P[pre + "conv.b"]))
    x, B, C = xbc[:, :I].view(T, H, V), xbc[:, I:I + G * N].view(T, G, N), xbc[:, I + G * N:].view(T, G, N)
    dt = torch.nn.functional.softplus(dt + P[pre + "dt_bias"], threshold=1000.0)
    y = torch.zeros(T, H, V, dtype=h.dtype)
    for i in range(H):
        g = i // (H // G)
        decay = torch.exp(-torch.exp(P[pre + "A_log"][i]) * dt[:, i]).view(T, 1).expand(T, N)
        y[:, i] = decayed_outer_scan(C[:, g], B[:, g], dt[:, i:i + 1] * x[:, i], decay) + P[pre + "D"][i] * x[:, i]
    y = y.reshape(T, I) * silu(z)
    y = unit_rms(y.view(T, parts, I // parts), eps).reshape(T, I) * P[pre + "norm"]
    return y @ P[pre + "o"].T


def squared_relu_mlp(P, pre, h):
    return torch.relu(h @ P[pre + "up"].T).pow(2) @ P[pre + "down"].T


def hyper_read(X, w):
    """u = sum_s w[s] X[s]; X [streams, T, W]."""
    return sum(w[s] * X[s] for s in range(X.shape[0]))


def hyper_write(X, y, mix, out):
    """X'[t] = sum_s mix[s, t] X[s] + out[t] y, every t from the old X."""
    n = X.shape[0]
    return torch.stack([sum(mix[s, t] * X[s] for s in range(n)) + out[t] * y for t in range(n)])


def run_order(n_layers, loop):
    if not loop:
        return list(range(n_layers))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n_layers))


def forward(P, cfg, tokens, dtype=torch.float64, return_layers=False):
    """tokens: list of ids -> logits [T, vocab] (and, if asked, the streams' sum after every layer run [runs, T, width])."""
    P = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in P.items()}
    eps = cfg["norm"]["eps"]
    x = P["embed"][torch.tensor(tokens)]
    X = torch.stack([x] * cfg["streams"])
    trail = []
    for i in run_order(len(cfg["layers"]), cfg.get("loop")):
        L, pre = cfg["layers"][i], f"l{i}."
        for q in (1, 2):
            if q == 2 and L.get("mlp") is None:
                continue
            u = layer_norm(hyper_read(X, P[f"{pre}hc{q}.in"]), P[f"{pre}norm{q}"], P[f"{pre}norm{q}.b"], eps)
            if q == 2:
                y = squared_relu_mlp(P, pre + "mlp.", u)
            elif L["type"] == "parallel":
                y = parallel_mixer(P, pre + "mix.", L["mixer"], u, eps)
            elif L["type"] == "mamba2":
                y = state_space_mixer(P, pre + "mix.", L["mixer"], u, eps)
            else:
                raise ValueError(L["type"])
            X = hyper_write(X, y, P[f"{pre}hc{q}.mix"], P[f"{pre}hc{q}.out"])
        trail.append(X.sum(dim=0))
    logits = layer_norm(X.sum(dim=0), P["final.norm"], P["final.norm.b"], eps) @ P["head"].T
    logits = soft_cap(logits, cfg.get("logit_softcap"))
    return (logits, torch.stack(trail)) if return_layers else logits


# ---- small configurations and random checkpoints for the tests ---------------------------------------------------------------------
def parallel_layer(heads=4, kv_heads=2, dim=16, vdim=24, conv=3, rot_dims=8, base=1000.0, scale=None, softcap=5.0, r_heads=3, r_dim=8, r_vdim=12,
                   tau=4.0, left_scale=0.7, right_scale=1.3, rank=6, mlp="dense"):
    """(`rank` of the decay's low-rank projection is a tensor size: random_checkpoint reads it, the model takes it from the tensors)"""
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale if scale is not None else dim ** -0.5,
            "softcap": softcap, "rot": {"base": base, "dims": rot_dims} if rot_dims else None}
    right = {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "tau": tau}
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale, "_rank": rank},
            "mlp": dense_mlp() if mlp == "dense" else mlp}


def ssd_layer(heads=4, vdim=12, state=8, groups=2, conv=4, norm_groups=2, mlp="dense"):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups},
            "mlp": dense_mlp() if mlp == "dense" else mlp}


def dense_mlp(ff=40):
    return {"kind": "dense", "ff": ff}


def make_config(layers, width=32, vocab=61, eps=1e-5, streams=2, loop=None, logit_softcap=8.0):
    return {"architecture": "Dunusun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "streams": streams, "loop": loop,
            "logit_softcap": logit_softcap, "layers": layers}


def random_checkpoint(cfg: dict, seed: int = 0) -> dict:
    """Random bf16-representable weights with the checkpoint's tensor names for a config of the design."""
    g = torch.Generator().manual_seed(seed)
    W, n = cfg["width"], cfg["streams"]

    def mat(o, i, s=None):
        return (torch.randn(o, i, generator=g) * (s if s is not None else 1.0 / math.sqrt(i))).to(torch.bfloat16)

    def vec(k, mean=0.0, s=0.1):
        return (mean + torch.randn(k, generator=g) * s).to(torch.bfloat16)

    P = {"embed": mat(cfg["vocab"], W, 1.0), "head": mat(cfg["vocab"], W, 2.0 / math.sqrt(W)), "final.norm": vec(W, 1.0, 0.2), "final.norm.b": vec(W)}
    for li, layer in enumerate(cfg["layers"]):
        p, m = f"l{li}.", layer["mixer"]
        for q in (1, 2) if layer.get("mlp") else (1,):
            P[p + f"norm{q}"], P[p + f"norm{q}.b"] = vec(W, 1.0, 0.2), vec(W)
            P[p + f"hc{q}.in"], P[p + f"hc{q}.out"] = vec(n, 1.0 / n, 0.3), vec(n, 0.8, 0.3)
            P[p + f"hc{q}.mix"] = (torch.eye(n) * 0.8 + torch.randn(n, n, generator=g) * 0.2).to(torch.bfloat16)
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, D, V, K = a["heads"], a["kv_heads"], a["dim"], a["vdim"], int(a.get("conv") or 0)
            for t, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
                P[p + f"mix.left.{t}"] = mat(rows, W, 1.5 / math.sqrt(W))
                if K:
                    P[p + f"mix.left.{t}.conv"] = mat(rows, K, 0.6)
            P[p + "mix.left.g"], P[p + "mix.left.o"] = mat(H * V, W), mat(W, H * V)
            h, d, v, R = r["heads"], r["dim"], r["vdim"], m.get("_rank", 4)
            for t, rows in (("q", h * d), ("k", h * d), ("v", h * v), ("g", h * v), ("a1", R)):
                P[p + f"mix.right.{t}"] = mat(rows, W)
            P[p + "mix.right.a2"], P[p + "mix.right.a2.b"] = mat(h * d, R, 2.0 / math.sqrt(R)), vec(h * d, 1.0, 1.0)
            P[p + "mix.right.norm"], P[p + "mix.right.o"] = vec(v, 1.0, 0.3), mat(W, h * v)
        else:
            h, v, N, G, K = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
            I = h * v
            P[p + "mix.in"] = mat(2 * I + 2 * G * N + h, W)
            P[p + "mix.conv"], P[p + "mix.conv.b"] = mat(I + 2 * G * N, K, 0.6), vec(I + 2 * G * N, 0.0, 0.3)
            P[p + "mix.dt_bias"], P[p + "mix.A_log"], P[p + "mix.D"] = vec(h, -1.0, 1.0), vec(h, -0.5, 1.0), vec(h, 0.5, 0.5)
            P[p + "mix.norm"], P[p + "mix.o"] = vec(I, 1.0, 0.3), mat(W, I)
        if layer.get("mlp"):
            P[p + "mlp.up"], P[p + "mlp.down"] = mat(layer["mlp"]["ff"], W), mat(W, layer["mlp"]["ff"])
    return P


def as_double(P: dict) -> dict:
    return {k: (v.double() if v.is_floating_point() else v) for k, v in P.items()}
