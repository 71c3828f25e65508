"""Hyper-connections — injected operators for decoders whose residual is n parallel streams instead of one row per token:

    u = sum_s in[s] x_s;   y = sublayer(norm(u));   x_j <- sum_s mix[s, j] x_s + out[j] y   (all j from the old streams)

KHyperConnection holds one sublayer's weights (`<key>.in` [n], `<key>.mix` [n, n] indexed [from, to], `<key>.out` [n]; fp32).  The
arithmetic is KHyperStreams': what a sublayer produced stays PENDING until the next sublayer asks for its input, so that writing the
streams, reading them for the next sublayer and that sublayer's layer norm are one launch (include/ktx_gla.h `ktx_hyper_mix`).  While no
sublayer has written yet all streams equal the embedding output and only that one row is kept."""
from __future__ import annotations

import torch

from ktransformers_amd.operators.base_operator import BaseInjectedModule


class KHyperConnection(BaseInjectedModule):
    def __init__(self, key: str, gguf_loader, config, orig_module, prefill_device: str = "cuda", generate_device: str = "cuda", **kwargs):
        BaseInjectedModule.__init__(self, key, gguf_loader, config, orig_module, prefill_device, generate_device, **kwargs)
        object.__setattr__(self, "streams", int(orig_module.streams))
        object.__setattr__(self, "w", {})

    def load(self):
        n, dev = self.streams, torch.device(self.device)
        for name, shape in (("in", (n,)), ("out", (n,)), ("mix", (n, n))):
            t = self.gguf_loader.load_tensor(f"{self.key}.{name}", device=dev).to(torch.float32).contiguous()
            if tuple(t.shape) != shape:
                raise ValueError(f"{self.key}.{name}: expected {shape}, got {tuple(t.shape)}")
            self.w[name] = t

    def forward(self, *args, **kwargs):
        raise RuntimeError(f"{self.key}: hyper-connections run inside KHyperStreams.enter / leave")


class KHyperStreams:
    """The residual streams of one step: x fp32 [T, W] while they are all equal, [T, n, W] afterwards (updated in place)."""

    def __init__(self, x0: torch.Tensor, n: int):
        self.x, self.n, self.pending = x0, int(n), None

    def _write(self):
        """(what the next launch writes, where the streams go); the pending result is taken."""
        if self.pending is None:
            return None, None
        y, hc = self.pending
        self.pending = None
        out = self.x if self.x.dim() == 3 else torch.empty((self.x.shape[0], self.n, self.x.shape[1]), dtype=torch.float32, device=self.x.device)
        return (y, hc.w["mix"], hc.w["out"]), out

    def enter(self, hc: KHyperConnection, norm, out_dtype) -> torch.Tensor:
        """-> norm(sum_s in[s] x_s) behind the pending write: what the sublayer of `hc` reads (norm: a KLayerNormBias)."""
        from ktransformers_amd._native_gla import hyper_mix
        write, out = self._write()
        h = hyper_mix(self.x, self.n, write=write, out=out, read=(hc.w["in"], norm.weight_f32, norm.bias_f32, norm.eps), out_dtype=out_dtype)
        if out is not None:
            self.x = out
        return h

    def leave(self, hc: KHyperConnection, y: torch.Tensor) -> None:
        """The sublayer of `hc` produced y fp32 [T, W]."""
        self.pending = (y, hc)

    def close(self, norm, rows, out_dtype) -> torch.Tensor:
        """-> norm(sum of the streams) of the given rows (None: all) behind the pending write; the streams themselves are not kept."""
        from ktransformers_amd._native_gla import hyper_mix
        write, _ = self._write()
        return hyper_mix(self.x, self.n, write=write, rows=rows, read=(None, norm.weight_f32, norm.bias_f32, norm.eps), out_dtype=out_dtype)

    def total(self) -> torch.Tensor:
        """The sum of the streams, fp32 [T, W] (the pending write done first): what a caller that looks at the residual between layers sees."""
        from ktransformers_amd._native_gla import hyper_mix
        write, out = self._write()
        if write is not None:
            hyper_mix(self.x, self.n, write=write, out=out)
            self.x = out
        return self.x.sum(dim=1) if self.x.dim() == 3 else self.x * self.n
