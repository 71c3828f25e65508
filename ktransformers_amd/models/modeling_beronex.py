"""Module skeleton of Beronex — a pre- and post-normed decoder (RMS norms) with an fp32 residual stream whose layers mix tokens with lightning
attention (a matrix state per head under a constant decay), with a full latent attention whose queries pass a latent of their own, or with a
grouped-query window attention (unit-RMS queries and keys, one sigmoid gate per head) that may read an earlier layer's keys and values; rotations are
YaRN-scaled.  The feed-forward is a dense GELU-gated one or a softmax-routed mixture of bounded gated experts.

Like the other skeletons of this package it only holds the structure the optimize rules inject into (optimize_rules/Beronex.yaml) and
the glue (the layer's residual arrangement); every module that does arithmetic is a leaf that raises until an operator replaces it.  Module paths
equal the checkpoint's tensor prefixes:

    embed | l<i>.{norm1,mix,norm1b,norm2,mlp,norm2b} | final.norm | head

config.json: {"architecture": "Beronex", "width", "vocab", "norm": {"eps"}, "embedding": {"scale"},
"layers": [{"type": "lightning", "mixer": {"heads", "dim", "vdim", "decay": [per head]}, "mlp": ...} |
           {"type": "latent_attention", "mixer": {"heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale", "rot": ROT}, "mlp": ...} |
           {"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": {"size"}, "rot": ROT, "kv_from": j (optional)},
            "mlp": ...}],
 ROT: {"base", "dims", "scaling": {"factor", "original", "fast", "slow"}},
 mlp: null | {"kind": "dense", "ff"} | {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top"}}}.
Sizes and the constants listed there come from the file; what the design fixes is a constant here."""
from __future__ import annotations

import json
import os
from types import SimpleNamespace

import torch
from torch import nn

from ktransformers_amd.models.modeling_deepseek import _Leaf

# fixed by the design
EXPERT_SIGMOID_SLOPE = 1.702   # an expert's gate is g * sigmoid(1.702 g)
EXPERT_UP_SHIFT = 1.0          # ... times (u + 1)
DENSE_ACTIVATION = "gelu_tanh"
MIXER_TYPES = ("lightning", "latent_attention", "attention")
MLP_KINDS = ("dense", "moe")


def _rotation(c: dict, span: int, where: str):
    """(turning entries, base, YaRN scaling or None) of a mixer's "rot"."""
    rot = c.get("rot") or None
    if rot is None:
        return 0, 1.0, None
    dims = int(rot["dims"])
    if dims % 2 or not 0 < dims <= span:
        raise ValueError(f"{where}: rot.dims ({dims}) must be even and at most {span}")
    return dims, float(rot["base"]), rot.get("scaling") or None


def make_beronex_config(d: dict | str, compute_dtype=torch.bfloat16) -> SimpleNamespace:
    """config.json (a dict or a path) -> the namespace the skeleton and the operators read."""
    if isinstance(d, str):
        with open(os.path.join(d, "config.json") if os.path.isdir(d) else d, encoding="utf-8") as f:
            d = json.load(f)
    if d.get("architecture") != "Beronex":
        raise ValueError(f"not a Beronex config: architecture = {d.get('architecture')!r}")
    layers = list(d["layers"])
    for i, L in enumerate(layers):
        if L.get("type") not in MIXER_TYPES:
            raise ValueError(f"layer {i}: unknown layer type {L.get('type')!r}")
        m = L["mixer"]
        if L["type"] == "lightning":
            if len(m["decay"]) != m["heads"] or not all(0.0 <= float(a) <= 1.0 for a in m["decay"]):
                raise ValueError(f"layer {i}: decay takes one number in [0, 1] per head")
        elif L["type"] == "latent_attention":
            _rotation(m, int(m["rot_dim"]), f"layer {i}")
        else:
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: heads ({m['heads']}) must be a multiple of kv_heads ({m['kv_heads']})")
            _rotation(m, int(m["dim"]), f"layer {i}")
            src = m.get("kv_from")
            if src is not None:
                s = layers[src]["mixer"] if 0 <= src < i and layers[src]["type"] == "attention" else None
                if s is None or s.get("kv_from") is not None or any(s.get(k) != m.get(k) for k in ("kv_heads", "dim", "vdim", "rot")):
                    raise ValueError(f"layer {i}: kv_from ({src}) must name an earlier attention layer with projections of its own and equal "
                                     "kv_heads, sizes and rotation")
        c = L.get("mlp")
        if c is not None:
            if c.get("kind") not in MLP_KINDS:
                raise ValueError(f"layer {i}: unknown feed-forward kind {c.get('kind')!r}")
            if c["kind"] == "moe" and not 0 < c["router"]["top"] <= c["router"]["experts"]:
                raise ValueError(f"layer {i}: top ({c['router']['top']}) must lie in 1 .. experts ({c['router']['experts']})")
    return SimpleNamespace(architectures=["Beronex"], width=int(d["width"]), vocab=int(d["vocab"]), eps=float(d["norm"]["eps"]),
                           embed_scale=float((d.get("embedding") or {}).get("scale", 1.0)), layers=layers, num_hidden_layers=len(layers),
                           vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), compute_dtype=compute_dtype, max_position_embeddings=None,
                           raw=d)


def beronex_layer_specs(config) -> list:
    """What KHybridCache needs, one entry per layer: state slots, paged latent rows, paged key / value rows — or nothing for an attention
    layer that reads another layer's."""
    specs = []
    for L in config.layers:
        m = L["mixer"]
        if L["type"] == "lightning":
            specs.append({"decay": tuple(int(m[k]) for k in ("heads", "dim", "vdim"))})
        elif L["type"] == "latent_attention":
            specs.append({"latent": int(m["kv_rank"]) + int(m["rot_dim"])})
        else:
            specs.append({} if m.get("kv_from") is not None else {"kv": tuple(int(m[k]) for k in ("kv_heads", "dim", "vdim"))})
    return specs


class BeronexEmbedding(_Leaf):
    def __init__(self, config):
        super().__init__()
        self.vocab, self.width, self.scale = config.vocab, config.width, config.embed_scale


class BeronexNorm(_Leaf):
    def __init__(self, width, eps):
        super().__init__()
        self.width, self.eps, self.one_plus = width, eps, False


class BeronexLightning(_Leaf):
    """The options KLightningAttention reads."""

    def __init__(self, config, c):
        super().__init__()
        self.width, self.eps = config.width, config.eps
        self.heads, self.dim, self.vdim = (int(c[k]) for k in ("heads", "dim", "vdim"))
        self.decay = [float(a) for a in c["decay"]]


class BeronexLatentAttention(_Leaf):
    """The options KLatentWindowAttention reads."""

    def __init__(self, config, c):
        super().__init__()
        self.width, self.eps = config.width, config.eps
        self.heads, self.dim, self.rot_dim, self.vdim, self.q_rank, self.kv_rank = (int(c[k]) for k in ("heads", "dim", "rot_dim", "vdim", "q_rank",
                                                                                                      "kv_rank"))
        self.scale, self.window = float(c["scale"]), 0
        self.rot_dims, self.rot_base, self.rot_scaling = _rotation(c, self.rot_dim, "latent_attention")
        self.rot_half, self.has_sink = True, False


class BeronexAttention(_Leaf):
    """The options KWindowGQAttention reads."""

    def __init__(self, config, c):
        super().__init__()
        self.width, self.eps = config.width, config.eps
        self.heads, self.kv_heads, self.dim, self.vdim = (int(c[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
        self.scale, self.window = float(c["scale"]), int((c.get("mask") or {}).get("size") or 0)
        self.rot_dims, self.rot_base, self.rot_scaling = _rotation(c, self.dim, "attention")
        self.rot_values, self.qk_norm, self.sink_score, self.gated = False, True, None, "per_head"
        self.kv_from = None if c.get("kv_from") is None else int(c["kv_from"])


class BeronexMLP(_Leaf):
    def __init__(self, config, c):
        super().__init__()
        self.width, self.ff, self.limit, self.activation = config.width, int(c["ff"]), None, DENSE_ACTIVATION


class BeronexMoE(_Leaf):
    def __init__(self, config, c):
        super().__init__()
        self.width, self.ff = config.width, int(c["expert"]["ff"])
        self.experts, self.top, self.identity = int(c["router"]["experts"]), int(c["router"]["top"]), 0
        self.sum_eps, self.router_bias = 0.0, True       # the weights are the softmax over the chosen logits
        self.glu = (float(c["expert"]["limit"]), EXPERT_SIGMOID_SLOPE, EXPERT_UP_SHIFT)


_MIXERS = {"lightning": BeronexLightning, "latent_attention": BeronexLatentAttention, "attention": BeronexAttention}


class BeronexLayer(nn.Module):
    def __init__(self, config, layer_idx):
        super().__init__()
        L = config.layers[layer_idx]
        W, eps = config.width, config.eps
        self.norm1, self.norm1b = BeronexNorm(W, eps), BeronexNorm(W, eps)
        self.mix, self.latent = _MIXERS[L["type"]](config, L["mixer"]), L["type"] == "latent_attention"
        c = L.get("mlp")
        self.mlp = None if c is None else (BeronexMLP if c["kind"] == "dense" else BeronexMoE)(config, c)
        self.routed = c is not None and c["kind"] == "moe"
        if self.mlp is not None:
            self.norm2, self.norm2b = BeronexNorm(W, eps), BeronexNorm(W, eps)

    def forward(self, x, h, batch, cache, cache_idx, next_norm=None):
        """x <- x + norm1b(mix(h)), h = norm1(x) (given);  x <- x + norm2b(mlp(norm2(x))).  x is the fp32 residual and is updated in place.
        The post-norm, the mixture's weighted sum, the residual add AND the pre-norm of whatever follows are the post-norm's one launch;
        returns next_norm(x) or None."""
        y = self.mix(h, batch, cache, cache_idx)
        pending = {"y": y[0] if self.latent else y}
        post = self.norm1b
        if self.mlp is not None:
            h = post.gated_add(x, next_norm=self.norm2, **pending)[1]
            post, y = self.norm2b, self.mlp(h)
            pending = {"expert_rows": y[0], "pair_pos": y[1], "topk_w": y[3]} if self.routed else {"y": y}
        out = post.gated_add(x, next_norm=next_norm, **pending)
        return out[1] if next_norm is not None else None


class _Final(nn.Module):
    def __init__(self, config):
        super().__init__()
        self.norm = BeronexNorm(config.width, config.eps)


class BeronexHead(_Leaf):
    def __init__(self, config):
        super().__init__()
        self.in_features, self.out_features = config.width, config.vocab


class BeronexForCausalLM(nn.Module):
    """forward(input_ids, position_ids, past_key_values, cache_position, batch=, logits_rows=, last_token_only=) -> fp32 logits.

    With `batch` (a ForwardBatch planned by the KHybridCache in `past_key_values`): input_ids is the flattened token list of the
    step and the result is [len(logits_rows) or T, vocab].  Without it, the call is the single-sequence form the generation loop
    uses (util/generate.py): input_ids [1, T] at position_ids [1, T]; the result is [1, T or 1, vocab]."""

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.embed = BeronexEmbedding(config)
        for i in range(config.num_hidden_layers):
            self.add_module(f"l{i}", BeronexLayer(config, i))
        self.final = _Final(config)
        self.head = BeronexHead(config)

    def forward(self, input_ids=None, position_ids=None, past_key_values=None, cache_position=None, batch=None, logits_rows=None,
                last_token_only: bool = False, return_layers: bool = False):
        cache = past_key_values
        single = batch is None
        if single:
            batch = cache.single_request_batch(position_ids)
            if last_token_only and batch.T > 1:
                logits_rows = torch.tensor([batch.T - 1], dtype=torch.int32, device=cache.device)
        x = self.embed(input_ids, batch.positions)
        cd, layers, trail = self.config.compute_dtype, [getattr(self, f"l{i}") for i in range(self.config.num_hidden_layers)], []
        h = layers[0].norm1(x, out_dtype=cd) if layers else None
        for i, layer in enumerate(layers):
            h = layer(x, h, batch, cache, i, next_norm=layers[i + 1].norm1 if i + 1 < len(layers) else None)
            if return_layers:
                trail.append(x.clone())
        logits = self.head(self.final.norm(x, rows=logits_rows, out_dtype=cd))
        if single:
            logits = logits.unsqueeze(0)
        return (logits, torch.stack(trail)) if return_layers else logits
