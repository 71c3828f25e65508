"""ctypes binding of include/ktx_gla.h — the hyper-connection step, the decay of gated linear attention, the inputs of the state-space-dual
scan, the decayed outer-product scan both share and the gate / norm segments in front of an output product.  Same library and calling
rules as ktransformers_amd._native_seq: device pointers and the caller's current HIP stream cross the boundary, every call is
graph-capturable, there is no CPU fallback."""
from __future__ import annotations

import ctypes as C

import torch

from ktransformers_amd._native_seq import SEQ_DTYPE, KtxError, _seq_dev, _stream_ptr, check, lib

_P, _I, _L, _F, _I32 = C.c_void_p, C.c_int, C.c_int64, C.c_float, C.c_int32


class _HyperArgs(C.Structure):       # include/ktx_gla.h: ktx_hyper_args
    _fields_ = [("x", _P), ("x_tok", _L), ("x_str", _L), ("y", _P), ("ldy", _L), ("mix", _P), ("out", _P), ("x_out", _P), ("in", _P),
                ("norm_w", _P), ("norm_b", _P), ("eps", _F), ("rows", _P), ("h", _P), ("out_dtype", _I32)]


class _DecayScanArgs(C.Structure):   # include/ktx_gla.h: ktx_decay_scan_args
    _fields_ = [("heads", _I32), ("dim", _I32), ("vdim", _I32), ("heads_per_key", _I32), ("q", _P), ("k", _P), ("v", _P), ("a", _P),
                ("vmul", _P), ("skip", _P), ("ldq", _L), ("ldk", _L), ("ldv", _L), ("lda", _L), ("ldm", _L), ("a_per_head", _I32),
                ("q_scale", _F), ("qkv_act", _I32), ("S", _P), ("o", _P), ("scratch", _P), ("chunk_len", _I32)]


class _GateSeg(C.Structure):         # include/ktx_gla.h: ktx_gate_seg
    _fields_ = [("o", _P), ("ldo", _L), ("o_dtype", _I32), ("gate", _P), ("ldg", _L), ("w", _P), ("n", _I32), ("group", _I32), ("w_mod", _I32),
                ("act", _I32), ("gate_first", _I32), ("eps", _F), ("scale", _F), ("out_off", _I32)]


if not hasattr(lib, "ktx_decay_scan"):
    raise ImportError("the loaded kernel library predates include/ktx_gla.h: rebuild with `python -m ktransformers_amd.build [--seq]`")
lib.ktx_hyper_mix.argtypes = [_I, _I, _I, C.POINTER(_HyperArgs), _P]
lib.ktx_lowrank_decay.argtypes = [_I, _I, _I, _P, _L, _P, _P, _F, _P, _P]
lib.ktx_ssd_prep.argtypes = [_I, _I, _I, _I, _I, _I, _P, _L, _I, _I] + [_P] * 12
lib.ktx_decay_scan_scratch.argtypes = [C.POINTER(_DecayScanArgs), _I, _I]
lib.ktx_decay_scan_scratch.restype = C.c_size_t
lib.ktx_decay_scan.argtypes = [_I, _I, _I, _P, _P, _P, C.POINTER(_DecayScanArgs), _P]
lib.ktx_gate_segments.argtypes = [_I, _I, C.POINTER(_GateSeg), _P, _I, _L, _P]


def _ptr(t):
    return t.data_ptr() if t is not None else None


def _f32(t, what):
    return None if t is None else _seq_dev(t, torch.float32, what)


def _rows_f32(t, what):
    """fp32 rows with unit inner stride (a column slice of a GEMM's output is fine) -> (pointer, row stride)."""
    if t is None:
        return None, 0
    if not t.is_cuda or t.dtype != torch.float32 or t.dim() != 2 or t.stride(1) != 1:
        raise KtxError(f"{what}: expected fp32 rows on a HIP device, got {t.dtype} {tuple(t.shape)} strides {t.stride()}")
    return t.data_ptr(), t.stride(0)


def hyper_mix(x: torch.Tensor, n: int, write: tuple | None = None, read: tuple | None = None, out: torch.Tensor | None = None,
              rows: torch.Tensor | None = None, out_dtype=torch.float32) -> torch.Tensor | None:
    """One launch (ktx_hyper_mix).  x fp32 [T, W] (all n streams equal it) or [T, n, W].  write = (y fp32 rows [T, W], mix [n, n] indexed
    [from, to], out weights [n]): x'_j = sum_s mix[s, j] x_s + out[j] y.  `out` (fp32 [T, n, W], may be x) receives the streams.
    read = (in weights [n] or None for the plain sum, norm weight, norm bias or None, eps): returns layer_norm(sum_s in[s] x'_s), [T or
    len(rows), W] of out_dtype."""
    _f32(x, "hyper_mix x")
    T, W = x.shape[0], x.shape[-1]
    if x.dim() not in (2, 3) or (x.dim() == 3 and x.shape[1] != n):
        raise KtxError("hyper_mix: x must be [T, W] or [T, streams, W]")
    a = _HyperArgs()
    a.x, a.x_tok, a.x_str = x.data_ptr(), x.stride(0), W if x.dim() == 3 else 0
    if write is not None:
        y, mix, ow = write
        _f32(mix, "hyper_mix mix"), _f32(ow, "hyper_mix out weights")
        a.y, a.ldy = _rows_f32(y, "hyper_mix y")
        if tuple(y.shape) != (T, W) or tuple(mix.shape) != (n, n) or ow.numel() != n:
            raise KtxError("hyper_mix: y must be [T, W], mix [n, n], out [n]")
        a.mix, a.out = mix.data_ptr(), ow.data_ptr()
    if out is not None:
        _f32(out, "hyper_mix out")
        if tuple(out.shape) != (T, n, W):
            raise KtxError("hyper_mix: out must be [T, n, W]")
        a.x_out = out.data_ptr()
    h = None
    n_out = T
    if rows is not None:
        _seq_dev(rows, torch.int32, "hyper_mix rows")
        a.rows, n_out = rows.data_ptr(), rows.numel()
    if read is not None:
        iw, nw, nb, eps = read
        _f32(iw, "hyper_mix in weights"), _f32(nw, "hyper_mix norm weight"), _f32(nb, "hyper_mix norm bias")
        if (iw is not None and iw.numel() != n) or nw.numel() != W or (nb is not None and nb.numel() != W):
            raise KtxError("hyper_mix: in weights [n], norm weight and bias [W]")
        h = torch.empty((n_out, W), dtype=out_dtype, device=x.device)
        setattr(a, "in", _ptr(iw))
        a.norm_w, a.norm_b, a.eps, a.h, a.out_dtype = nw.data_ptr(), _ptr(nb), float(eps), h.data_ptr(), SEQ_DTYPE[out_dtype]
    check(lib.ktx_hyper_mix(n_out, W, int(n), C.byref(a), _stream_ptr(x.device)))
    return h


def lowrank_decay(low: torch.Tensor, w_t: torch.Tensor, bias: torch.Tensor | None, tau: float) -> torch.Tensor:
    """low fp32 rows [T, R], w_t fp32 [R, C] (transposed factor) -> sigmoid(low w_t + bias)^(1 / tau), fp32 [T, C] (ktx_lowrank_decay)."""
    lp, ldl = _rows_f32(low, "lowrank_decay low")
    _f32(w_t, "lowrank_decay w"), _f32(bias, "lowrank_decay bias")
    T, (R, Cn) = low.shape[0], w_t.shape
    if low.shape[1] != R or (bias is not None and bias.numel() != Cn):
        raise KtxError("lowrank_decay: shapes do not fit")
    alpha = torch.empty((T, Cn), dtype=torch.float32, device=low.device)
    check(lib.ktx_lowrank_decay(T, Cn, R, lp, ldl, w_t.data_ptr(), _ptr(bias), 1.0 / float(tau), alpha.data_ptr(), _stream_ptr(low.device)))
    return alpha


def ssd_prep(proj: torch.Tensor, c_off: int, dt_off: int, w: torch.Tensor, bias: torch.Tensor | None, dt_bias: torch.Tensor,
             A_log: torch.Tensor, batch, conv_state: torch.Tensor | None):
    """proj fp32 rows; w fp32 [C, taps] -> (u = silu(conv + bias) fp32 [T, C], gates fp32 [T, 2 heads] = steps | decays); the slots'
    convolution state moves on (ktx_ssd_prep)."""
    pp, ldp = _rows_f32(proj, "ssd_prep proj")
    for t_, what in ((w, "w"), (bias, "bias"), (dt_bias, "dt_bias"), (A_log, "A_log"), (conv_state, "conv_state")):
        _f32(t_, "ssd_prep " + what)
    T, (Cn, taps), H = proj.shape[0], w.shape, dt_bias.numel()
    if A_log.numel() != H or (bias is not None and bias.numel() != Cn) or batch.T != T or proj.shape[1] < max(c_off + Cn, dt_off + H) or \
            (taps > 1 and (conv_state is None or tuple(conv_state.shape[1:]) != (taps - 1, Cn))):
        raise KtxError("ssd_prep: shapes do not fit")
    u = torch.empty((T, Cn), dtype=torch.float32, device=proj.device)
    gates = torch.empty((T, 2 * H), dtype=torch.float32, device=proj.device)
    check(lib.ktx_ssd_prep(batch.B, T, int(batch.max_q_len), Cn, taps, H, pp, ldp, int(c_off), int(dt_off), w.data_ptr(), _ptr(bias),
                           dt_bias.data_ptr(), A_log.data_ptr(), batch.q_indptr.data_ptr(), batch.pos0.data_ptr(), batch.slot.data_ptr(),
                           batch.tok_req.data_ptr(), _ptr(conv_state), u.data_ptr(), gates.data_ptr(), _stream_ptr(proj.device)))
    return u, gates


SCAN_CHUNK = 64      # tokens per chunk of a prompt (chunks run side by side); twice as many where that still leaves SCAN_GROUPS workgroups
SCAN_GROUPS = 512


def scan_chunk(heads: int, vdim: int, batch) -> int:
    groups = heads * ((vdim + 127) // 128) * (batch.T // (2 * SCAN_CHUNK))
    return 2 * SCAN_CHUNK if groups >= SCAN_GROUPS else SCAN_CHUNK


def decay_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, batch, S: torch.Tensor, heads_per_key: int = 1,
               vmul: torch.Tensor | None = None, skip: torch.Tensor | None = None, q_scale: float = 1.0, chunk_len: int | None = None, qkv_silu: bool = False) -> torch.Tensor:
    """The decayed outer-product scan (ktx_decay_scan): q, k fp32 rows [T, (heads / heads_per_key) * dim], v [T, heads * vdim] (column
    slices are fine), decay [T, heads * dim] (per key channel) or [T, heads] (rows may be one row expanded: a decay that never changes);
    qkv_silu: q, k and v are silu of what the rows hold; vmul [T, heads]: multiplies the values that enter the state;
    skip fp32 [heads]: adds skip[h] v_t to the read-out.  S fp32 [slots, heads, dim, vdim] moves on -> o fp32 [T, heads * vdim]."""
    _f32(S, "decay_scan S"), _f32(skip, "decay_scan skip")
    H, D, V = S.shape[1:]
    T = q.shape[0]
    a = _DecayScanArgs()
    a.heads, a.dim, a.vdim, a.heads_per_key = H, D, V, int(heads_per_key)
    for name, ld, t_, cols in (("q", "ldq", q, H // heads_per_key * D), ("k", "ldk", k, H // heads_per_key * D), ("v", "ldv", v, H * V),
                               ("a", "lda", decay, decay.shape[1]), ("vmul", "ldm", vmul, H)):
        p, s = _rows_f32(t_, "decay_scan " + name)
        if t_ is not None and (t_.shape[0] != T or t_.shape[1] != cols):
            raise KtxError(f"decay_scan: {name} must be [{T}, {cols}], got {tuple(t_.shape)}")
        setattr(a, name, p), setattr(a, ld, s)
    if decay.shape[1] not in (H, H * D) or batch.T != T or (skip is not None and skip.numel() != H):
        raise KtxError("decay_scan: a decay per head or per key channel, one token per row")
    a.a_per_head = 1 if decay.shape[1] == H and D > 1 else 0
    a.skip, a.q_scale, a.S, a.qkv_act = _ptr(skip), float(q_scale), S.data_ptr(), 1 if qkv_silu else 0
    o = torch.empty((T, H * V), dtype=torch.float32, device=q.device)
    a.o, a.chunk_len = o.data_ptr(), int(scan_chunk(H, V, batch) if chunk_len is None else chunk_len)
    need = lib.ktx_decay_scan_scratch(C.byref(a), batch.B, int(batch.max_q_len))
    scratch = torch.empty(need, dtype=torch.float32, device=q.device) if need else None
    a.scratch = _ptr(scratch)
    check(lib.ktx_decay_scan(batch.B, T, int(batch.max_q_len), batch.q_indptr.data_ptr(), batch.pos0.data_ptr(), batch.slot.data_ptr(),
                             C.byref(a), _stream_ptr(q.device)))
    return o


def gate_seg(o: torch.Tensor, gate: torch.Tensor, act: str, norm: tuple | None = None, gate_first: bool = False, scale: float = 1.0):
    """One segment of gate_segments: o [T, n] (fp32 | bf16 rows), gate fp32 rows [T, n]; norm = (weight fp32, group, eps): RMS norm over
    groups of `group` columns, weight of `group` (shared by the groups) or n entries; gate_first: the gate multiplies before the norm."""
    gp, ldg = _rows_f32(gate, "gate_seg gate")
    if not o.is_cuda or o.dtype not in SEQ_DTYPE or o.dim() != 2 or o.stride(1) != 1 or tuple(o.shape) != tuple(gate.shape):
        raise KtxError("gate_seg: o must be rows of the gate's shape")
    s = _GateSeg()
    s.tensors = [o, gate]            # (the struct holds addresses only: the segment keeps what it points to alive)
    s.o, s.ldo, s.o_dtype, s.gate, s.ldg, s.n = o.data_ptr(), o.stride(0), SEQ_DTYPE[o.dtype], gp, ldg, o.shape[1]
    s.act, s.gate_first, s.scale = {"sigmoid": 0, "silu": 1}[act], int(bool(gate_first)), float(scale)
    if norm is not None:
        w, group, eps = norm
        _f32(w, "gate_seg norm weight")
        if w.numel() not in (group, o.shape[1]) or o.shape[1] % group:
            raise KtxError("gate_seg: the norm's groups divide the columns, its weight has a group's or all columns' entries")
        s.tensors.append(w)
        s.w, s.group, s.w_mod, s.eps = w.data_ptr(), int(group), w.numel(), float(eps)
    return s


def gate_segments(segs, T: int, device, out_dtype=torch.float32) -> torch.Tensor:
    """The segments side by side -> [T, sum n] of out_dtype, one launch (ktx_gate_segments)."""
    arr = (_GateSeg * len(segs))(*segs)
    cols = 0
    for s in arr:
        s.out_off = cols
        cols += s.n
    out = torch.empty((T, cols), dtype=out_dtype, device=device)
    check(lib.ktx_gate_segments(T, len(segs), arr, out.data_ptr(), SEQ_DTYPE[out_dtype], out.stride(0), _stream_ptr(out.device)))
    return out
