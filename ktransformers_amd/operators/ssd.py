"""State-space-dual mixer (Mamba-2) — an injected recurrent operator beside the selective scan (operators/selective_scan.py): one decay
per head and token instead of one per channel and state entry, and a state with the shape of a linear attention's,

    W_in h = [z | x | B | C | dt] (z, x: heads vdim; B, C: groups state; dt: heads);
    x, B, C <- silu(conv(.) + b) with a causal convolution per channel;  dt = softplus(dt + dt_bias);
    per head h of group g = h // (heads / groups):  S <- exp(-exp(A_log_h) dt) S + B_g (dt x_h)^T;  y = S^T C_g + D_h x_h;
    y * silu(z), divided by its RMS in `norm_groups` equal parts (eps), times norm;  W_o.

S (fp32 [heads, state, vdim] per sequence) and the convolution's last taps - 1 inputs live in the KHybridCache's slots (specs "decay",
"conv"); steps, decays, the state and the norm are fp32 (include/ktx_gla.h `ktx_ssd_prep`, `ktx_decay_scan`, `ktx_gate_segments`).
Checkpoint tensors: `<key>.in`, `.conv` [channels, taps], `.conv.b`, `.dt_bias`, `.A_log`, `.D` [heads], `.norm`, `.o`."""
from __future__ import annotations

import torch
from torch import nn

from ktransformers_amd.operators.base_operator import BaseInjectedModule
from ktransformers_amd.operators.linear import padded_rows


class KStateSpaceDualMixer(BaseInjectedModule):
    def __init__(self, key: str, gguf_loader, config, orig_module: nn.Module, prefill_device: str = "cuda", generate_device: str = "cuda",
                 **kwargs):
        BaseInjectedModule.__init__(self, key, gguf_loader, config, orig_module, prefill_device, generate_device, **kwargs)
        for name in ("heads", "vdim", "state", "groups", "taps", "norm_groups", "eps", "width"):
            object.__setattr__(self, name, getattr(orig_module, name))
        object.__setattr__(self, "compute_dtype", getattr(config, "compute_dtype", torch.bfloat16))
        object.__setattr__(self, "w", {})

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def conv_channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    def state_spec(self) -> dict:
        return {"decay": (self.heads, self.state, self.vdim), "conv": (self.conv_channels, self.taps)}

    def load(self):
        ld, dev, cd = self.gguf_loader, torch.device(self.device), self.compute_dtype
        get = lambda n: ld.load_tensor(f"{self.key}.{n}", device=dev)
        f32 = lambda n: get(n).to(torch.float32).contiguous()
        win, I, C, H = get("in").to(cd), self.inner, self.conv_channels, self.heads
        if tuple(win.shape) != (I + C + H, self.width):
            raise ValueError(f"{self.key}.in: expected {(I + C + H, self.width)}, got {tuple(win.shape)}")
        self.w.update({"in": padded_rows([win]), "o": get("o").to(cd).contiguous(), "conv": f32("conv"), "conv_b": f32("conv.b"),
                       "dt_bias": f32("dt_bias").reshape(-1), "A_log": f32("A_log").reshape(-1), "D": f32("D").reshape(-1), "norm": f32("norm").reshape(-1)})
        if tuple(self.w["o"].shape) != (self.width, I) or tuple(self.w["conv"].shape) != (C, self.taps) or self.w["norm"].numel() != I or \
                any(self.w[n].numel() != H for n in ("dt_bias", "A_log", "D")):
            raise ValueError(f"{self.key}: tensor shapes do not fit heads={H} vdim={self.vdim} state={self.state} groups={self.groups} taps={self.taps}")

    def forward(self, h: torch.Tensor, batch, cache, cache_idx: int) -> torch.Tensor:
        """h [T, width] in the compute type -> W_o(gated, normed read-out) fp32 [T, width]; the slots' state moves on."""
        from ktransformers_amd._native_gla import decay_scan, gate_seg, gate_segments, ssd_prep
        from ktransformers_amd._native_seq import dense_gemm
        I, H, GN = self.inner, self.heads, self.groups * self.state
        proj = dense_gemm(h, self.w["in"])
        u, gates = ssd_prep(proj, I, I + self.conv_channels, self.w["conv"], self.w["conv_b"], self.w["dt_bias"], self.w["A_log"], batch,
                            cache.conv[cache_idx])
        y = decay_scan(u[:, I + GN:], u[:, I:I + GN], u[:, :I], gates[:, H:], batch, cache.S[cache_idx], heads_per_key=H // self.groups,
                       vmul=gates[:, :H], skip=self.w["D"])
        seg = gate_seg(y, proj[:, :I], "silu", norm=(self.w["norm"], I // self.norm_groups, self.eps), gate_first=True)
        return dense_gemm(gate_segments([seg], h.shape[0], h.device, out_dtype=self.compute_dtype), self.w["o"])
