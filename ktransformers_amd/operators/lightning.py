"""Lightning attention — an injected recurrent operator beside gated linear attention (operators/gated_linear.py) and the state-space-dual
mixer: a matrix state per head that decays by a constant,

    q = silu(W_q h), k = silu(W_k h) (heads x dim), v = silu(W_v h) (heads x vdim);
    S <- decay_head S + k v^T;  o = S^T q;
    the concatenated heads / rms(o) over ALL of them (eps) * norm [heads vdim] * sigmoid(W_g h);  W_o.

S (fp32 [heads, dim, vdim] per sequence) lives in the KHybridCache's slots (spec "decay"); decays, the state and the output norm are fp32.  All input
projections are one GEMM; the activations of q, k and v happen where the scan reads them, and the decays are one row that every token reads
(include/ktx_gla.h `ktx_decay_scan`, `ktx_gate_segments`).  decay (a number per head) and eps are constructor arguments (read from the
replaced module).  Checkpoint tensors: `<key>.q`, `.k`, `.v`, `.g` [heads vdim, width], `.norm` [heads vdim], `.o`."""
from __future__ import annotations

import torch
from torch import nn

from ktransformers_amd.operators.base_operator import BaseInjectedModule
from ktransformers_amd.operators.linear import padded_rows


class KLightningAttention(BaseInjectedModule):
    IN_ORDER = ("q", "k", "v", "g")

    def __init__(self, key: str, gguf_loader, config, orig_module: nn.Module, prefill_device: str = "cuda", generate_device: str = "cuda",
                 **kwargs):
        BaseInjectedModule.__init__(self, key, gguf_loader, config, orig_module, prefill_device, generate_device, **kwargs)
        for name in ("heads", "dim", "vdim", "decay", "eps", "width"):
            object.__setattr__(self, name, getattr(orig_module, name))
        object.__setattr__(self, "compute_dtype", getattr(config, "compute_dtype", torch.bfloat16))
        object.__setattr__(self, "w", {})

    def in_weight_names(self):
        H, D, V = self.heads, self.dim, self.vdim
        return [("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V)]

    def state_spec(self) -> dict:
        return {"decay": (self.heads, self.dim, self.vdim)}

    def load(self):
        ld, dev, cd = self.gguf_loader, torch.device(self.device), self.compute_dtype
        get = lambda n: ld.load_tensor(f"{self.key}.{n}", device=dev)
        parts = [get(n).to(cd) for n in self.IN_ORDER]
        HV = self.heads * self.vdim
        self.w.update({"o": get("o").to(cd).contiguous(), "norm": get("norm").to(torch.float32).reshape(-1).contiguous(),
                       "decay": torch.tensor([float(d) for d in self.decay], dtype=torch.float64).to(torch.float32).to(dev).view(1, -1)})
        if any(tuple(t.shape) != (rows, self.width) for t, (_, rows) in zip(parts, self.in_weight_names())) or \
                tuple(self.w["o"].shape) != (self.width, HV) or self.w["norm"].numel() != HV or self.w["decay"].numel() != self.heads:
            raise ValueError(f"{self.key}: tensor shapes do not fit heads={self.heads} dim={self.dim} vdim={self.vdim} width={self.width}")
        self.w["in"] = padded_rows(parts)

    def forward(self, h: torch.Tensor, batch, cache, cache_idx: int) -> torch.Tensor:
        """h [T, width] in the compute type -> W_o(...) fp32 [T, width]; the slot states of the batch's requests advance in place."""
        from ktransformers_amd._native_gla import decay_scan, gate_seg, gate_segments
        from ktransformers_amd._native_seq import dense_gemm
        proj = dense_gemm(h, self.w["in"])
        cols, c = {}, 0
        for n, rows in self.in_weight_names():
            cols[n] = proj[:, c:c + rows]
            c += rows
        o = decay_scan(cols["q"], cols["k"], cols["v"], self.w["decay"].expand(h.shape[0], -1), batch, cache.S[cache_idx], qkv_silu=True)
        seg = gate_seg(o, cols["g"], "sigmoid", norm=(self.w["norm"], self.heads * self.vdim, self.eps))
        return dense_gemm(gate_segments([seg], h.shape[0], h.device, out_dtype=self.compute_dtype), self.w["o"])
