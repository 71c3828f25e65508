"""Module skeleton of Dunusun — a pre-normed decoder whose fp32 residual is several parallel streams that learned weights mix around every
sublayer (hyper-connections), with layer norms that have a bias.  A layer mixes tokens either with two mixers side by side — a grouped-query
softmax attention behind short causal convolutions, partly rotated (interleaved pairs), its scores soft-capped and its heads gated, and a
gated linear attention whose matrix state decays per key channel — or with a state-space-dual scan (Mamba-2); the feed-forward is a
two-matrix relu^2 one, the logits are soft-capped, and a block of layers may run several times in a row with the same weights.

Like the other skeletons of this package it only holds the structure the optimize rules inject into (optimize_rules/Dunusun.yaml) and
the glue (the streams: what a sublayer produced is written in the launch that reads and norms them for the next one); every module that does
arithmetic is a leaf that raises until an operator replaces it.  Module paths equal the checkpoint's tensor prefixes:

    embed | l<i>.{hc1,norm1,mix,hc2,norm2,mlp} (l<i>.mix.{left,right} in a parallel layer) | final.norm | head

config.json: {"architecture": "Dunusun", "width", "vocab", "norm": {"eps"}, "streams", "logit_softcap", "loop": {"start", "stop", "times"} | null,
"layers": [{"type": "parallel", "mixer": {"left": {"heads", "kv_heads", "dim", "vdim", "conv", "scale", "softcap", "rot": {"base", "dims"}},
                                          "right": {"heads", "dim", "vdim", "tau"}, "left_scale", "right_scale"}, "mlp": ...} |
           {"type": "mamba2", "mixer": {"heads", "vdim", "state", "groups", "conv", "norm_groups"}, "mlp": ...}],
 mlp: null | {"kind": "dense", "ff"}}.
Sizes and the constants listed there come from the file (the rank of the decay's projection from the tensors)."""
from __future__ import annotations

import json
import os
from types import SimpleNamespace

import torch
from torch import nn

from ktransformers_amd.models.modeling_deepseek import _Leaf
from ktransformers_amd.models.modeling_pilavik import layer_runs

MIXER_TYPES = ("parallel", "mamba2")
MLP_KINDS = ("dense",)


def make_dunusun_config(d: dict | str, compute_dtype=torch.bfloat16) -> SimpleNamespace:
    """config.json (a dict or a path) -> the namespace the skeleton and the operators read."""
    if isinstance(d, str):
        with open(os.path.join(d, "config.json") if os.path.isdir(d) else d, encoding="utf-8") as f:
            d = json.load(f)
    if d.get("architecture") != "Dunusun":
        raise ValueError(f"not a Dunusun config: architecture = {d.get('architecture')!r}")
    layers = list(d["layers"])
    for i, L in enumerate(layers):
        if L.get("type") not in MIXER_TYPES:
            raise ValueError(f"layer {i}: unknown layer type {L.get('type')!r}")
        m = L["mixer"]
        if L["type"] == "parallel":
            a = m["left"]
            if a["heads"] % a["kv_heads"]:
                raise ValueError(f"layer {i}: heads ({a['heads']}) must be a multiple of kv_heads ({a['kv_heads']})")
            rot = a.get("rot") or None
            if rot and (rot["dims"] % 2 or rot["dims"] > a["dim"]):
                raise ValueError(f"layer {i}: rot.dims ({rot['dims']}) must be even and at most dim ({a['dim']})")
        else:
            if m["heads"] % m["groups"]:
                raise ValueError(f"layer {i}: heads ({m['heads']}) must be a multiple of groups ({m['groups']})")
            if (m["heads"] * m["vdim"]) % m["norm_groups"]:
                raise ValueError(f"layer {i}: norm_groups ({m['norm_groups']}) must divide heads * vdim ({m['heads'] * m['vdim']})")
        c = L.get("mlp")
        if c is not None and c.get("kind") not in MLP_KINDS:
            raise ValueError(f"layer {i}: unknown feed-forward kind {c.get('kind')!r}")
    loop = d.get("loop") or None
    if loop is not None:
        loop = {"start": int(loop["start"]), "stop": int(loop["stop"]), "times": int(loop["times"])}
        if not (0 <= loop["start"] < loop["stop"] <= len(layers)) or loop["times"] < 1:
            raise ValueError(f"loop {loop} does not fit {len(layers)} layers")
    streams = int(d.get("streams", 1))
    if streams < 1:
        raise ValueError(f"streams ({streams}) must be at least 1")
    cap = d.get("logit_softcap")
    return SimpleNamespace(architectures=["Dunusun"], width=int(d["width"]), vocab=int(d["vocab"]), eps=float(d["norm"]["eps"]), streams=streams,
                           logit_softcap=float(cap) if cap else None, layers=layers, loop=loop,
                           runs=[i for i, _ in layer_runs(len(layers), loop)], num_hidden_layers=len(layers), vocab_size=int(d["vocab"]),
                           hidden_size=int(d["width"]), compute_dtype=compute_dtype, max_position_embeddings=None, raw=d)


def dunusun_layer_specs(config) -> list:
    """What KHybridCache needs, one entry per layer RUN (each pass of the repeated block has its own cache and state)."""
    specs = []
    for i in config.runs:
        L = config.layers[i]
        m = L["mixer"]
        if L["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, D, V, taps = (int(a.get(k) or 0) for k in ("heads", "kv_heads", "dim", "vdim", "conv"))
            specs.append({"kv": (G, D, V), "conv": (H * D + G * (D + V), taps), "decay": (int(r["heads"]), int(r["dim"]), int(r["vdim"]))})
        else:
            H, V, N, G = (int(m[k]) for k in ("heads", "vdim", "state", "groups"))
            specs.append({"decay": (H, N, V), "conv": (H * V + 2 * G * N, int(m["conv"]))})
    return specs


class DunusunEmbedding(_Leaf):
    def __init__(self, config):
        super().__init__()
        self.vocab, self.width = config.vocab, config.width


class DunusunNorm(_Leaf):
    def __init__(self, width, eps):
        super().__init__()
        self.width, self.eps = width, eps


class DunusunHyperConnection(_Leaf):
    def __init__(self, streams):
        super().__init__()
        self.streams = streams


class DunusunAttention(_Leaf):
    """The left mixer: the options KWindowGQAttention reads."""

    def __init__(self, config, c):
        super().__init__()
        self.width, self.eps = config.width, config.eps
        self.heads, self.kv_heads, self.dim, self.vdim = (int(c[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
        self.scale, self.softcap = float(c["scale"]), float(c["softcap"]) if c.get("softcap") else None
        rot = c.get("rot") or None
        self.rot_dims, self.rot_base = (int(rot["dims"]), float(rot["base"])) if rot else (0, 1.0)
        self.rot_values, self.qk_norm, self.sink_score, self.window = False, False, None, 0
        self.conv_taps, self.gated = int(c.get("conv") or 0), True


class DunusunLinearAttention(_Leaf):
    def __init__(self, config, c):
        super().__init__()
        self.width, self.eps = config.width, config.eps
        self.heads, self.dim, self.vdim, self.tau = int(c["heads"]), int(c["dim"]), int(c["vdim"]), float(c["tau"])


class DunusunParallelMixer(_Leaf):
    def __init__(self, config, c):
        super().__init__()
        self.left, self.right = DunusunAttention(config, c["left"]), DunusunLinearAttention(config, c["right"])
        self.left_scale, self.right_scale = float(c["left_scale"]), float(c["right_scale"])


class DunusunStateSpaceMixer(_Leaf):
    def __init__(self, config, c):
        super().__init__()
        self.width, self.eps = config.width, config.eps
        self.heads, self.vdim, self.state, self.groups, self.norm_groups = (int(c[k]) for k in ("heads", "vdim", "state", "groups", "norm_groups"))
        self.taps = int(c["conv"])


class DunusunMLP(_Leaf):
    def __init__(self, config, c):
        super().__init__()
        self.width, self.ff = config.width, int(c["ff"])


class DunusunLayer(nn.Module):
    def __init__(self, config, layer_idx):
        super().__init__()
        L = config.layers[layer_idx]
        self.hc1, self.norm1 = DunusunHyperConnection(config.streams), DunusunNorm(config.width, config.eps)
        self.mix = (DunusunParallelMixer if L["type"] == "parallel" else DunusunStateSpaceMixer)(config, L["mixer"])
        self.mlp = None if L.get("mlp") is None else DunusunMLP(config, L["mlp"])
        if self.mlp is not None:
            self.hc2, self.norm2 = DunusunHyperConnection(config.streams), DunusunNorm(config.width, config.eps)

    def forward(self, streams, batch, cache, cache_idx, dtype):
        """Both sublayers read and write the streams (operators/hyper.py KHyperStreams): one launch in front of each sublayer writes what the
        one before it produced, reads the weighted sum and norms it."""
        h = streams.enter(self.hc1, self.norm1, dtype)
        streams.leave(self.hc1, self.mix(h, batch, cache, cache_idx))
        if self.mlp is not None:
            h = streams.enter(self.hc2, self.norm2, dtype)
            streams.leave(self.hc2, self.mlp(h))


class _Final(nn.Module):
    def __init__(self, config):
        super().__init__()
        self.norm = DunusunNorm(config.width, config.eps)


class DunusunHead(_Leaf):
    def __init__(self, config):
        super().__init__()
        self.in_features, self.out_features, self.soft_cap = config.width, config.vocab, config.logit_softcap


class DunusunForCausalLM(nn.Module):
    """forward(input_ids, position_ids, past_key_values, cache_position, batch=, logits_rows=, last_token_only=) -> fp32 logits.

    With `batch` (a ForwardBatch planned by the KHybridCache in `past_key_values`): input_ids is the flattened token list of the
    step and the result is [len(logits_rows) or T, vocab].  Without it, the call is the single-sequence form the generation loop
    uses (util/generate.py): input_ids [1, T] at position_ids [1, T]; the result is [1, T or 1, vocab]."""

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.embed = DunusunEmbedding(config)
        for i in range(config.num_hidden_layers):
            self.add_module(f"l{i}", DunusunLayer(config, i))
        self.final = _Final(config)
        self.head = DunusunHead(config)

    def forward(self, input_ids=None, position_ids=None, past_key_values=None, cache_position=None, batch=None, logits_rows=None,
                last_token_only: bool = False, return_layers: bool = False):
        from ktransformers_amd.operators.hyper import KHyperStreams
        cache = past_key_values
        single = batch is None
        if single:
            batch = cache.single_request_batch(position_ids)
            if last_token_only and batch.T > 1:
                logits_rows = torch.tensor([batch.T - 1], dtype=torch.int32, device=cache.device)
        cd = self.config.compute_dtype
        streams = KHyperStreams(self.embed(input_ids, batch.positions), self.config.streams)
        trail = []
        for run, i in enumerate(self.config.runs):
            getattr(self, f"l{i}")(streams, batch, cache, run, cd)
            if return_layers:
                trail.append(streams.total())
        logits = self.head(streams.close(self.final.norm, logits_rows, cd))
        if single:
            logits = logits.unsqueeze(0)
        return (logits, torch.stack(trail)) if return_layers else logits
