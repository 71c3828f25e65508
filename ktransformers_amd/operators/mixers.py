"""Token-mixer combinators: two injected mixers side by side on the same input.

KScaledParallelMixer returns left_scale * left(h) + right_scale * right(h) for children that end in a gate and an output product.  All
input projections of both are ONE GEMM; both children's gated heads, each times its scale, are laid side by side by one launch
(include/ktx_gla.h `ktx_gate_segments`) and W_o of both is ONE product over the concatenation: the sum costs nothing.

KParallelMixer runs two injected mixers side by side on the same input and returns half the sum of
their outputs, each first RMS-normed over the model width with its own plain weight:

    y = 0.5 * (rms(left(h)) * w_left + rms(right(h)) * w_right)

All input projections of both children are ONE GEMM (their weights are concatenated at load; the children read their columns of
its fp32 output), and with the fusion hooks of the decoder layer the combination, the layer's post-norm and the residual add are
one launch (`ktx_rms_combine`)."""
from __future__ import annotations

import torch
from torch import nn

from ktransformers_amd.operators.base_operator import BaseInjectedModule
from ktransformers_amd.operators.linear import padded_rows


class KParallelMixer(BaseInjectedModule):
    SUPPORTS_FUSION = True

    def __init__(self, key: str, gguf_loader, config, orig_module: nn.Module, prefill_device: str = "cuda", generate_device: str = "cuda",
                 **kwargs):
        BaseInjectedModule.__init__(self, key, gguf_loader, config, orig_module, prefill_device, generate_device, **kwargs)
        object.__setattr__(self, "eps", orig_module.eps)
        object.__setattr__(self, "w", {})

    def load(self):
        left, right = self.orig_module.left, self.orig_module.right
        for child in (left, right):
            if not hasattr(child, "in_weight_names"):
                raise RuntimeError(f"{self.key}: {type(child).__name__} was not replaced by an injected mixer (check the optimize rules)")
            child.load()
        ld, dev = self.gguf_loader, torch.device(self.device)
        self.w["in"] = torch.cat([left.w[n] for n, _ in left.in_weight_names()] + [right.w[n] for n, _ in right.in_weight_names()]).contiguous()
        self.w["right_base"] = sum(r for _, r in left.in_weight_names())
        self.w["left_out"] = ld.load_tensor(self.key + ".left.out", device=dev).to(torch.float32).contiguous()
        self.w["right_out"] = ld.load_tensor(self.key + ".right.out", device=dev).to(torch.float32).contiguous()

    def forward(self, h: torch.Tensor, batch, cache, post_norm=None, residual: torch.Tensor | None = None):
        """h fp32 [T, width].  Without hooks: the combined output fp32 [T, width].  With post_norm (a KResidualRMSNorm) and residual:
        residual += post_norm(combined), in place, returned."""
        from ktransformers_amd._native_seq import dense_gemm, rms_combine
        left, right = self.orig_module.left, self.orig_module.right
        proj = dense_gemm(h, self.w["in"])
        yl = left(h, batch, cache, proj=proj, q_off=0, k_off=left.heads * left.dim)
        yr = right(h, batch, cache, proj=proj, base=self.w["right_base"])
        if post_norm is not None and residual is not None:
            return rms_combine(yl, post_norm.weight_f32, self.eps, one_plus=post_norm.one_plus, residual=residual, y2=yr,
                               w1=self.w["left_out"], w2=self.w["right_out"])
        return rms_combine(yl, None, self.eps, y2=yr, w1=self.w["left_out"], w2=self.w["right_out"])


class KScaledParallelMixer(BaseInjectedModule):
    def __init__(self, key: str, gguf_loader, config, orig_module: nn.Module, prefill_device: str = "cuda", generate_device: str = "cuda",
                 **kwargs):
        BaseInjectedModule.__init__(self, key, gguf_loader, config, orig_module, prefill_device, generate_device, **kwargs)
        object.__setattr__(self, "scales", (float(orig_module.left_scale), float(orig_module.right_scale)))
        object.__setattr__(self, "compute_dtype", getattr(config, "compute_dtype", torch.bfloat16))
        object.__setattr__(self, "w", {})

    def load(self):
        children = (self.orig_module.left, self.orig_module.right)
        for child in children:
            if not hasattr(child, "gated_segment"):
                raise RuntimeError(f"{self.key}: {type(child).__name__} was not replaced by an injected mixer (check the optimize rules)")
            child.load()
        self.w["in"] = padded_rows([c.w[n] for c in children for n, _ in c.in_weight_names()])
        self.w["o"] = torch.cat([c.w["o"] for c in children], dim=1).contiguous()
        self.w["right_base"] = sum(rows for _, rows in children[0].in_weight_names())
        for c in children:           # (the merged copies serve; the children's own are dropped)
            for n in [n for n, _ in c.in_weight_names() if n != "a1"] + ["o"]:
                c.w[n] = c.w[n].to("meta")

    def forward(self, h: torch.Tensor, batch, cache, cache_idx: int) -> torch.Tensor:
        """h [T, width] in the compute type -> the weighted sum of both mixers, fp32 [T, width]."""
        from ktransformers_amd._native_gla import gate_segments
        from ktransformers_amd._native_seq import dense_gemm
        proj = dense_gemm(h, self.w["in"])
        left = self.orig_module.left.gated_segment(proj, 0, batch, cache, cache_idx, scale=self.scales[0])
        right = self.orig_module.right.gated_segment(proj, self.w["right_base"], batch, cache, cache_idx, scale=self.scales[1])
        return dense_gemm(gate_segments([left, right], h.shape[0], h.device, out_dtype=self.compute_dtype), self.w["o"])
