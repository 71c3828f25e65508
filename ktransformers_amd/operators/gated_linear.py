"""Gated linear attention — an injected recurrent operator beside the mLSTM, delta-rule and selective-scan mixers: a matrix state per head
whose key rows decay by learned, input-dependent factors,

    q = W_q h dim^-1/2, k = W_k h (heads x dim), v = W_v h (heads x vdim);
    alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau), one decay per head and key entry (W_a1, W_a2 low-rank);
    S <- diag(alpha) S + k v^T;  o = S^T q;
    per head o / rms(o) (eps) * norm (one weight per value entry, shared by the heads) * silu(W_g h);  W_o.

S (fp32 [heads, dim, vdim] per sequence) lives in the KHybridCache's slots (spec "decay"); decays, the state and the output norm are fp32
(include/ktx_gla.h `ktx_lowrank_decay`, `ktx_decay_scan`, `ktx_gate_segments`).  All input projections are one GEMM; inside a parallel
mixer (operators/mixers.py) it is shared with the other mixer's, and so is the output product.  tau and eps are constructor arguments (read from
the replaced module).  Checkpoint tensors: `<key>.q`, `.k`, `.v`, `.g`, `.a1` [rank, width], `.a2` [heads dim, rank], `.a2.b`, `.norm` [vdim], `.o`."""
from __future__ import annotations

import torch
from torch import nn

from ktransformers_amd.operators.base_operator import BaseInjectedModule
from ktransformers_amd.operators.linear import padded_rows


class KGatedLinearAttention(BaseInjectedModule):
    IN_ORDER = ("q", "k", "v", "g", "a1")

    def __init__(self, key: str, gguf_loader, config, orig_module: nn.Module, prefill_device: str = "cuda", generate_device: str = "cuda",
                 **kwargs):
        BaseInjectedModule.__init__(self, key, gguf_loader, config, orig_module, prefill_device, generate_device, **kwargs)
        for name in ("heads", "dim", "vdim", "tau", "eps", "width"):
            object.__setattr__(self, name, getattr(orig_module, name))
        object.__setattr__(self, "compute_dtype", getattr(config, "compute_dtype", torch.bfloat16))
        object.__setattr__(self, "w", {})

    def in_weight_names(self):
        H, D, V = self.heads, self.dim, self.vdim
        return [("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V), ("a1", self.w["a1"].shape[0])]

    @property
    def out_columns(self) -> int:
        return self.heads * self.vdim

    def state_spec(self) -> dict:
        return {"decay": (self.heads, self.dim, self.vdim)}

    def load(self):
        ld, dev, cd = self.gguf_loader, torch.device(self.device), self.compute_dtype
        for n in self.IN_ORDER + ("o",):
            self.w[n] = ld.load_tensor(f"{self.key}.{n}", device=dev).to(cd).contiguous()
        f32 = lambda n: ld.load_tensor(f"{self.key}.{n}", device=dev).to(torch.float32).contiguous()
        self.w.update(a2_t=f32("a2").T.contiguous(), a2_b=f32("a2.b"), norm=f32("norm"))
        HD, HV = self.heads * self.dim, self.heads * self.vdim
        if any(tuple(self.w[n].shape) != (rows, self.width) for n, rows in self.in_weight_names()) or tuple(self.w["o"].shape) != (self.width, HV) or \
                tuple(self.w["a2_t"].shape) != (self.w["a1"].shape[0], HD) or self.w["a2_b"].numel() != HD or self.w["norm"].numel() != self.vdim:
            raise ValueError(f"{self.key}: tensor shapes do not fit heads={self.heads} dim={self.dim} vdim={self.vdim} width={self.width}")

    def gated_segment(self, proj: torch.Tensor, base: int, batch, cache, cache_idx: int, scale: float = 1.0):
        """proj fp32 rows holding the input projections from column `base` in IN_ORDER: runs the recurrence (the slots' state moves on) and
        returns the segment of gate_segments that norms and gates its read-out (times `scale`)."""
        from ktransformers_amd._native_gla import decay_scan, gate_seg, lowrank_decay
        cols, c = {}, base
        for n, rows in self.in_weight_names():
            cols[n] = proj[:, c:c + rows]
            c += rows
        alpha = lowrank_decay(cols["a1"], self.w["a2_t"], self.w["a2_b"], self.tau)
        o = decay_scan(cols["q"], cols["k"], cols["v"], alpha, batch, cache.S[cache_idx], q_scale=self.dim ** -0.5)
        return gate_seg(o, cols["g"], "silu", norm=(self.w["norm"], self.vdim, self.eps), scale=scale)

    def forward(self, h: torch.Tensor, batch, cache, cache_idx: int) -> torch.Tensor:
        """h [T, width] in the compute type -> W_o(...) fp32 [T, width]; the slot states of the batch's requests advance in place."""
        from ktransformers_amd._native_gla import gate_segments
        from ktransformers_amd._native_seq import dense_gemm
        if "in" not in self.w:       # used on its own: all input projections as one product
            self.w["in"] = padded_rows([self.w[n] for n in self.IN_ORDER])
        seg = self.gated_segment(dense_gemm(h, self.w["in"]), 0, batch, cache, cache_idx)
        return dense_gemm(gate_segments([seg], h.shape[0], h.device, out_dtype=self.compute_dtype), self.w["o"])
