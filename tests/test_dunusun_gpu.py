"""Dunusun on the GPU against the plain CPU statement of the design (oracle/dunusun_ref.py, fp64): every mechanism alone through its
kernels and operator, then the model through the framework's registry, cache manager, step function and generation loops — whole
prompts, token-by-token decoding, portions, unequal batches, reused pages and slots, far keys, keys at page borders and chunk edges, odd
sizes.  Small random configurations; fp32 runs are held to rounding, bf16 runs to bf16 rounding."""
import math
from types import SimpleNamespace

import pytest
import torch

from oracle import dunusun_ref as R

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF16, F64 = torch.float32, torch.bfloat16, torch.float64
TOL = {F32: 3e-4, BF16: 6e-2}


def rel(got, ref):
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    return float((got - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


def rows_rel(got, ref):
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    return float(((got - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt().clamp_min(1e-30)).max())


def row_errors(got, ref):
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    return (got - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt().clamp_min(1e-30)


def held(got, ref, limit):
    """Largest ratio of a row's relative error to its limit."""
    return float((row_errors(got, ref) / limit).max())


def limits(P, cfg, toks, ref, dtype, draws=4):
    """What a row of logits may be off by: fp32 TOL; bf16 TOL, or four times what random relative noise of bf16's unit roundoff on the weights
    moves this row in the plain statement — normed recurrences and powers of relu amplify rounding at some positions more than at others."""
    lim = torch.full((len(toks),), TOL[dtype], dtype=F64)
    if dtype == F32:
        return lim
    g = torch.Generator().manual_seed(99)
    for _ in range(draws):
        noisy = {k: (v.double() * (1 + torch.randn(v.shape, generator=g, dtype=F64) * 2.0 ** -9) if v.dim() == 2 and ".hc" not in k else v) for k, v in P.items()}
        lim = torch.maximum(lim, 4 * row_errors(R.forward(noisy, cfg, toks), ref))
    return lim


def build(cfg, seed, dtype, max_tokens=2048, max_requests=8, page_size=16, P=None):
    from ktransformers_amd.models import load_model
    from ktransformers_amd.models.custom_cache import KHybridCache
    from ktransformers_amd.models.modeling_dunusun import dunusun_layer_specs
    from ktransformers_amd.util.loader import DictLoader
    P = R.random_checkpoint(cfg, seed) if P is None else P
    model, config, _ = load_model(cfg, dtype=dtype, device=DEV, loader=DictLoader(P))
    cache = KHybridCache(dunusun_layer_specs(config), max_tokens, max_requests=max_requests, page_size=page_size, dtype=dtype, device=DEV)
    return model, cache, R.as_double(P)


def tokens_of(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def engine_of(model, cache, **kw):
    from ktransformers_amd.util.batch_engine import BatchEngine
    return BatchEngine(model, cache, **kw)


def steps(eng, rid, toks, sizes, end=True):
    """Feed toks in portions of the given sizes; logits of every position."""
    got, at = [], 0
    for n in sizes:
        last = at + n == len(toks)
        got.append(eng.step([{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}], [rid] if last and end else []))
        at += n
    assert at == len(toks)
    return torch.cat(got)


def batch_of(cache, entries):
    for rid, _ in entries:
        if rid not in cache.requests:
            cache.admit(rid)
    return cache.plan(entries)


def f32d(t):
    return t.float().contiguous().to(DEV)


# ---- hyper-connections --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("W,n", [(32, 1), (32, 2), (48, 3), (320, 4), (1024, 4), (1028, 5), (2048, 8), (2052, 6), (4096, 3), (4096, 5), (4100, 2),
                                 (7, 3), (1500, 7), (33, 16), (260, 9)])
def test_hyper_step_writes_and_reads_the_streams(W, n):
    """ktx_hyper_mix in all its argument combinations: with and without a write, from equal streams (one stored row) or from n, in place
    and out of place, a bf16 or fp32 result, no norm bias, the plain sum, a row gather; rows held in registers and in LDS."""
    from ktransformers_amd._native_gla import hyper_mix
    g = torch.Generator().manual_seed(W + n)
    T, eps = 5, 1e-5
    X, y = torch.randn(T, n, W, generator=g), torch.randn(T, W + 3, generator=g)[:, :W]
    mix, ow, iw = torch.randn(n, n, generator=g), torch.randn(n, generator=g), torch.randn(n, generator=g)
    nw, nb = 1 + 0.3 * torch.randn(W, generator=g), torch.randn(W, generator=g)
    yd = torch.empty(T, W + 3, device=DEV)
    yd[:, :W] = y.to(DEV)
    yd = yd[:, :W]
    for equal in (False, True):
        src = X[:, 0].contiguous() if equal else X
        old = (X[:, :1].expand(T, n, W) if equal else X).double().transpose(0, 1)
        for write in (False, True):
            new = R.hyper_write(old, y.double(), mix.double(), ow.double()) if write else old
            for lp, bias, plain in ((F32, True, False), (BF16, True, False), (F32, False, True)):
                u = new.sum(0) if plain else R.hyper_read(new, iw.double())
                want = R.layer_norm(u, nw.double(), nb.double() if bias else 0.0, eps)
                xd = src.clone().to(DEV)
                read = (None if plain else iw.to(DEV), nw.to(DEV), nb.to(DEV) if bias else None, eps)
                wr = (yd, mix.to(DEV), ow.to(DEV)) if write else None
                out = torch.full((T, n, W), float("nan"), device=DEV) if equal or not write else xd      # in place where the streams are stored
                h = hyper_mix(xd, n, write=wr, read=read, out=out, out_dtype=lp)
                assert h.dtype == lp and rel(h, want) < (4e-6 if lp == F32 else 4e-3), (equal, write, lp)
                assert rel(out.transpose(0, 1), new) < 2e-6
                if out is not xd:
                    assert torch.equal(xd.cpu(), src)
            rows = torch.tensor([4, 0, 2], dtype=torch.int32, device=DEV)
            xd = src.clone().to(DEV)
            h = hyper_mix(xd, n, write=wr, read=(None, nw.to(DEV), nb.to(DEV), eps), rows=rows)
            assert rel(h, R.layer_norm(new.sum(0), nw.double(), nb.double(), eps)[[4, 0, 2]]) < 4e-6 and torch.equal(xd.cpu(), src)
    out = torch.empty(T, n, W, device=DEV)
    assert hyper_mix(X.to(DEV), n, write=(yd, mix.to(DEV), ow.to(DEV)), out=out) is None
    assert rel(out.transpose(0, 1), R.hyper_write(X.double().transpose(0, 1), y.double(), mix.double(), ow.double())) < 2e-6


def test_hyper_mix_matrix_is_indexed_from_to():
    from ktransformers_amd._native_gla import hyper_mix
    X = torch.tensor([[[1.0] * 4, [10.0] * 4]], device=DEV)
    out = torch.empty(1, 2, 4, device=DEV)
    hyper_mix(X, 2, write=(torch.zeros(1, 4, device=DEV), torch.tensor([[0.0, 1.0], [0.0, 0.0]], device=DEV), torch.ones(2, device=DEV)), out=out)
    assert out[0, 0].tolist() == [0.0] * 4 and out[0, 1].tolist() == [1.0] * 4


def test_hyper_streams_object_keeps_one_row_until_the_first_write():
    from ktransformers_amd.operators.hyper import KHyperStreams
    g = torch.Generator().manual_seed(4)
    T, W, n = 3, 24, 3
    x0, y1, y2 = (torch.randn(T, W, generator=g) for _ in range(3))
    w = [{"in": torch.randn(n, generator=g), "out": torch.randn(n, generator=g), "mix": torch.randn(n, n, generator=g)} for _ in range(2)]
    nw, nb = torch.randn(W, generator=g), torch.randn(W, generator=g)
    hc = [SimpleNamespace(w={k: v.to(DEV) for k, v in d.items()}) for d in w]
    norm = SimpleNamespace(weight_f32=nw.to(DEV), bias_f32=nb.to(DEV), eps=1e-5)
    s = KHyperStreams(x0.to(DEV), n)
    assert rel(s.total(), n * x0.double()) < 1e-6
    X = x0.double().expand(n, T, W)
    for d, c, y in zip(w, hc, (y1, y2)):
        h = s.enter(c, norm, F32)
        assert rel(h, R.layer_norm(R.hyper_read(X, d["in"].double()), nw.double(), nb.double(), 1e-5)) < 4e-6
        s.leave(c, y.to(DEV))
        X = R.hyper_write(X, y.double(), d["mix"].double(), d["out"].double())
    assert s.x.shape == (T, n, W)
    assert rel(s.close(norm, None, F32), R.layer_norm(X.sum(0), nw.double(), nb.double(), 1e-5)) < 4e-6


# ---- the recurrences' inputs ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("T,C,Rk,tau", [(1, 24, 6, 4.0), (37, 300, 1, 16.0), (9, 256, 33, 1.0), (64, 1024, 16, 16.0), (3, 5, 200, 0.5)])
def test_low_rank_decay(T, C, Rk, tau):
    from ktransformers_amd._native_gla import lowrank_decay
    g = torch.Generator().manual_seed(T + C)
    wide = torch.randn(T, Rk + 11, generator=g) * 3
    w, b = torch.randn(C, Rk, generator=g) * 4, torch.randn(C, generator=g) * 4
    low = wide[:, 5:5 + Rk].double()
    z = low @ w.double().T
    for bias in (b, None):
        want = torch.sigmoid(z + (bias.double() if bias is not None else 0.0)).pow(1.0 / tau)
        got = lowrank_decay(wide.to(DEV)[:, 5:5 + Rk], f32d(w.T), None if bias is None else f32d(bias), tau)
        assert float((got.double().cpu() - want).abs().max()) < 2e-5 and got.shape == (T, C)
    assert torch.isfinite(lowrank_decay(f32d(torch.full((2, 1), -300.0)), f32d(torch.ones(1, 3)), None, 16.0)).all()


@pytest.mark.parametrize("C,taps,H,c_off", [(48, 4, 4, 8), (64, 2, 3, 0), (44, 3, 5, 12), (36, 1, 2, 4), (37, 4, 3, 5), (64, 5, 2, 8), (1100, 4, 6, 40),
                                            (20, 9, 1, 4), (1, 2, 1, 1)])
def test_ssd_inputs_whole_and_carried(C, taps, H, c_off):
    """The convolved inputs, steps and decays of two requests: whole, in portions shorter than the taps, one token at a time."""
    from ktransformers_amd._native_gla import ssd_prep
    from ktransformers_amd.models.custom_cache import KHybridCache
    g = torch.Generator().manual_seed(C + taps)
    lens = {"a": 23, "b": 9}
    width = (c_off + C + H + 7) // 8 * 8
    proj = {r: torch.randn(n, width, generator=g) for r, n in lens.items()}
    w, b = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
    dtb, al = torch.randn(H, generator=g) * 2, torch.randn(H, generator=g)
    want_u = {r: R.silu(R.causal_conv(p[:, c_off:c_off + C].double(), w.double(), b.double())) for r, p in proj.items()}
    want_dt = {r: torch.nn.functional.softplus(p[:, c_off + C:c_off + C + H].double() + dtb.double()) for r, p in proj.items()}
    for cut in ([(23, 9)], [(20, 7), (1, 1), (2, 1)], [(2, 2)] * 4 + [(15, 1)], [(1, 1)] * 9 + [(1, 0)] * 14):
        cache = KHybridCache([{"conv": (C, taps)}], 256, max_requests=3, page_size=8, dtype=F32, device=DEV)
        if cache.conv[0] is not None:
            cache.conv[0].fill_(7.0)          # what an earlier request left: position 0 starts from zeros all the same
        at = {"a": 0, "b": 0}
        for na, nb_ in cut:
            part = [(r, n) for r, n in (("b", nb_), ("a", na)) if n]
            bt = batch_of(cache, part)
            rows = torch.cat([proj[r][at[r]:at[r] + n] for r, n in part])
            u, gates = ssd_prep(rows.to(DEV), c_off, c_off + C, f32d(w), f32d(b), f32d(dtb), f32d(al), bt, cache.conv[0])
            wu = torch.cat([want_u[r][at[r]:at[r] + n] for r, n in part])
            wd = torch.cat([want_dt[r][at[r]:at[r] + n] for r, n in part])
            assert rel(u, wu) < 2e-6 and rel(gates[:, :H], wd) < 2e-6
            assert float((gates[:, H:].double().cpu() - torch.exp(-torch.exp(al.double()) * wd)).abs().max()) < 2e-6
            for r, n in part:
                at[r] += n


# ---- the decayed outer-product scan ---------------------------------------------------------------------------------------------------
def run_scan(q, k, v, a, per_head, hpk, q_scale, vmul, skip, cut, chunk_len, garbage=3.0):
    """Two copies of the sequence plus a longer neighbour in one batch, in portions `cut`; output of the second copy's request."""
    from ktransformers_amd._native_gla import decay_scan
    from ktransformers_amd.models.custom_cache import KHybridCache
    T, H, V = v.shape
    D = k.shape[2]
    cache = KHybridCache([{"decay": (H, D, V)}], 4096, max_requests=4, page_size=8, dtype=F32, device=DEV)
    cache.S[0].fill_(garbage)
    flat = lambda t: f32d(t.reshape(t.shape[0], -1))
    fq, fk, fv, fa = flat(q), flat(k), flat(v), flat(a)
    fm = None if vmul is None else f32d(vmul)
    got, at = [], 0
    for n in cut:
        other = n + 3 if at + n + 3 <= T else n
        bt = batch_of(cache, [("x", other), ("r", n)])
        sel = torch.tensor(list(range(other)) + list(range(at, at + n)), device=DEV)
        o = decay_scan(fq[sel], fk[sel], fv[sel], fa[sel], bt, cache.S[0], heads_per_key=hpk, vmul=None if fm is None else fm[sel],
                       skip=None if skip is None else f32d(skip), q_scale=q_scale, chunk_len=chunk_len)
        got.append(o[other:])
        at += n
    assert at == T
    untouched = [s for s in range(cache.max_requests) if s not in (cache.requests["x"]["slot"], cache.requests["r"]["slot"])]
    assert float((cache.S[0][untouched] - garbage).abs().max()) == 0.0
    return torch.cat(got).view(T, H, V), cache.S[0][cache.requests["r"]["slot"]]


SCAN_SIZES = [
    # heads, dim, vdim, per head, heads per key
    (3, 8, 12, False, 1), (4, 8, 12, True, 2), (2, 32, 64, False, 1), (6, 32, 32, True, 3), (2, 128, 128, False, 1), (4, 128, 64, True, 4),
    (1, 256, 70, False, 1), (2, 100, 65, False, 1), (1, 300, 16, True, 1), (2, 1, 1, False, 1), (2, 1, 5, True, 2), (1, 512, 130, False, 1),
    (3, 17, 33, True, 1), (2, 64, 96, True, 1), (2, 48, 200, False, 1),
]


@pytest.mark.parametrize("H,D,V,per_head,hpk", SCAN_SIZES)
def test_decayed_scan_whole_portions_and_chunks(H, D, V, per_head, hpk):
    g = torch.Generator().manual_seed(D + V)
    T, G = 75, H // hpk
    q, k, v = (torch.randn(T, n, d, generator=g) for n, d in ((G, D), (G, D), (H, V)))
    a = torch.sigmoid(torch.randn(T, H, 1 if per_head else D, generator=g) * 2 + 2)
    a[::11] = 1.0
    a[5::29] = 0.0                                    # a decay of 0 forgets everything, of 1 nothing
    vmul, skip = (torch.rand(T, H, generator=g) + 0.2, torch.randn(H, generator=g)) if per_head else (None, None)
    q_scale = 0.37
    want, d64 = torch.zeros(T, H, V, dtype=F64), lambda t: t.double()
    for h in range(H):
        vin = d64(v[:, h]) * (d64(vmul[:, h:h + 1]) if vmul is not None else 1.0)
        want[:, h] = R.decayed_outer_scan(d64(q[:, h // hpk]) * q_scale, d64(k[:, h // hpk]), vin, d64(a[:, h]).expand(T, D))
        if skip is not None:
            want[:, h] += d64(skip[h]) * d64(v[:, h])
    final = None
    for cut, chunk in (([T], 0), ([T], 8), ([T], 64), ([T], 75), ([T], 5), ([1] * T, 64), ([40, 2, 1, 2, 30], 16), ([2] * 37 + [1], 64), ([64, 11], 64),
                       ([9, 66], 32), ([5] * 15, 64), ([17, 16, 15, 27], 64)):
        got, S = run_scan(q, k, v, a, per_head, hpk, q_scale, vmul, skip, cut, chunk)
        assert rel(got, want) < 5e-6, (cut[:4], chunk)
        assert rows_rel(got.reshape(T, -1), want.reshape(T, -1)) < 5e-5, (cut[:4], chunk)
        final = S if final is None else final
        assert rel(S, final) < 5e-6


@pytest.mark.parametrize("per_head", [False, True])
def test_decayed_scan_remembers_one_far_token(per_head):
    """No decay: a pair written at position j is read back at the last position, however many chunks lie between, and at the edges of chunks;
    with ONE decay of 0 behind it it is gone."""
    T, H, D, V = 200, 2, 16, 8
    g = torch.Generator().manual_seed(1)
    v = torch.zeros(T, H, V)
    k = torch.zeros(T, H, D)
    q = torch.zeros(T, H, D)
    q[-1, :, 3] = 1.0
    for j in (0, 15, 16, 63, 64, 127, 128, 198, 199):
        kk, vv = k.clone(), v.clone()
        kk[j, :, 3] = 1.0
        vv[j] = torch.randn(H, V, generator=g)
        a = torch.ones(T, H, 1 if per_head else D)
        for chunk in (16, 64, 128, 0):
            got, _ = run_scan(q, kk, vv, a, per_head, 1, 1.0, None, None, [T], chunk)
            assert rel(got[-1], vv[j]) < 1e-6 and float(got[:-1].abs().max()) == 0.0, j
        if j < T - 1:
            a[j + 1] = 0.0
            got, _ = run_scan(q, kk, vv, a, per_head, 1, 1.0, None, None, [T - 1, 1], 16)
            assert float(got.abs().max()) == 0.0, j


# ---- gates, norms, activations ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T", [1, 3, 70])
def test_gate_segments_side_by_side(dtype, T):
    from ktransformers_amd._native_gla import gate_seg, gate_segments
    g = torch.Generator().manual_seed(T)
    eps = 1e-4
    cases = [  # columns, norm group (None: no norm), shared weight, gate first, activation, o type
        (96, None, False, False, "sigmoid", BF16), (40, 8, True, False, "silu", F32), (72, 24, False, True, "silu", F32), (1300, None, False, False, "silu", F32),
        (1300, 650, False, True, "sigmoid", F32), (2048, 512, True, False, "silu", F32), (2 * 513, 513, True, True, "silu", F32), (5, 1, True, True, "silu", F32),
        (3, 3, False, False, "sigmoid", F32), (1100, 1100, False, True, "silu", BF16)]
    for i, first in enumerate(cases):
        picked = [first, cases[(i + 3) % len(cases)]] if i % 3 else [first]
        segs, want = [], []
        for (n, group, shared, gfirst, act, odt) in picked:
            o, gate = torch.randn(T, n, generator=g).to(odt), torch.randn(T, n + 9, generator=g)
            w = torch.randn((group if shared else n) if group else 1, generator=g)
            scale = 0.7 if gfirst else 1.3
            od, gd, wd = o.to(DEV), gate.to(DEV), w.to(DEV)
            segs.append(gate_seg(od, gd[:, 4:4 + n], act, norm=(wd, group, eps) if group else None, gate_first=gfirst, scale=scale))
            z = gate[:, 4:4 + n].double()
            f = R.silu(z) if act == "silu" else torch.sigmoid(z)
            p = o.double() * (f if gfirst or not group else 1.0)
            if group:
                p = R.unit_rms(p.view(T, n // group, group), eps).reshape(T, n) * (w.double().repeat(n // group) if shared else w.double())
                p = p if gfirst else p * f
            want.append(p * scale)
        got = gate_segments(segs, T, DEV, out_dtype=dtype)
        assert got.dtype == dtype and rel(got, torch.cat(want, dim=1)) < (2e-6 if dtype == F32 else 4e-3), picked


@pytest.mark.parametrize("M,N,K", [(1, 48, 64), (7, 37, 40), (16, 64, 96), (70, 61, 33), (130, 264, 128), (3, 5, 7)])
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("act,arg", [("relu_sq", 0.0), ("soft_cap", 3.0), ("soft_cap", 30.0)])
def test_dense_product_with_squared_relu_and_soft_cap(M, N, K, dtype, act, arg):
    from ktransformers_amd._native_seq import dense_gemm
    g = torch.Generator().manual_seed(M + N)
    a, w = torch.randn(M, K, generator=g).to(dtype), (torch.randn(N, K, generator=g) * 3 / math.sqrt(K)).to(dtype)
    z = a.double() @ w.double().T
    want = torch.relu(z).pow(2) if act == "relu_sq" else R.soft_cap(z, arg)
    got = dense_gemm(a.to(DEV), w.to(DEV), act=act, act_arg=arg)
    assert rel(got, want) < 2e-5
    if dtype == BF16:
        assert rel(dense_gemm(a.to(DEV), w.to(DEV), act=act, act_arg=arg, out_dtype=BF16), want) < 6e-3


# ---- convolved, rotated projections and capped attention ----------------------------------------------------------------------------
PREP_SIZES = [
    # heads, key heads, dim, vdim, taps, rot_dims
    (4, 2, 16, 24, 3, 8), (3, 1, 10, 6, 2, 10), (2, 2, 32, 16, 4, 32), (4, 1, 8, 4, 4, 2), (2, 1, 6, 5, 3, 4), (1, 1, 2, 1, 1, 2), (4, 2, 64, 80, 9, 16),
    (2, 1, 16, 8, 5, 0), (6, 3, 12, 20, 4, 6), (8, 2, 128, 128, 4, 64),
]


@pytest.mark.parametrize("H,G,D,V,taps,rot", PREP_SIZES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_convolved_projections_turn_with_the_position(H, G, D, V, taps, rot, dtype):
    """q, k and v behind the convolution, q and k turned: two requests whole, in portions and one token at a time; the key and value rows the
    cache holds afterwards, in the pages' order."""
    from ktransformers_amd._native_swa import swa_config, swa_conv_prep
    from ktransformers_amd.models.custom_cache import KHybridCache
    g = torch.Generator().manual_seed(D + taps)
    C, base, scale, ps = H * D + G * (D + V), 1000.0, 0.3, 8
    lens = {"a": 21, "b": 10}
    u = {r: torch.randn(n, C + 5, generator=g)[:, :C] for r, n in lens.items()}
    w = torch.randn(C, taps, generator=g)
    want = {}
    for r, n in lens.items():
        y = R.causal_conv(u[r].double(), w.double())
        q, k, v = y[:, :H * D].view(n, H, D), y[:, H * D:(H + G) * D].view(n, G, D), y[:, (H + G) * D:].view(n, G, V)
        pos = torch.arange(n)
        want[r] = (R.rotate_pairs(q, pos, base, rot) * scale, R.rotate_pairs(k, pos, base, rot), v)
    cfg = swa_config(H, G, D, V, rot, False, False, 1e-6, scale, 0, ps, dtype)
    inv = (base ** (-2.0 * torch.arange(rot // 2, dtype=F64) / max(rot, 1))).to(DEV) if rot else None
    for cut in ([(21, 10)], [(17, 4), (2, 2), (2, 4)], [(1, 1)] * 10 + [(1, 0)] * 11):
        cache = KHybridCache([{"kv": (G, D, V), "conv": (C, taps)}], 128, max_requests=3, page_size=ps, dtype=dtype, device=DEV)
        if cache.conv[0] is not None:
            cache.conv[0].fill_(5.0)
        at, got = {"a": 0, "b": 0}, {"a": [], "b": []}
        for na, nb_ in cut:
            part = [(r, n) for r, n in (("b", nb_), ("a", na)) if n]
            bt = batch_of(cache, part)
            rows = torch.cat([u[r][at[r]:at[r] + n] for r, n in part])
            wide = torch.empty(rows.shape[0], C + (-C) % 4, device=DEV)
            wide[:, :C] = rows.to(DEV)
            q = swa_conv_prep(cfg, wide[:, :C], None, f32d(w), None, None, bt, cache.conv[0], cache.k_caches[0], cache.v_caches[0], inv_freq=inv)
            i = 0
            for r, n in part:
                got[r].append(q[i:i + n])
                i, at[r] = i + n, at[r] + n
        for r, n in lens.items():
            pages = cache.requests[r]["pages"]
            loc = torch.tensor([pages[p // ps] * ps + p % ps for p in range(n)], device=DEV)
            assert rel(torch.cat(got[r]).view(n, H, D), want[r][0]) < 2e-6
            assert rel(cache.k_caches[0][loc], want[r][1]) < (2e-6 if dtype == F32 else 4e-3)
            assert rel(cache.v_caches[0][loc], want[r][2]) < (2e-6 if dtype == F32 else 4e-3)


def run_attention(q, k, v, scale, cap, dtype, kernel, nsplit=1, page_size=8, t_new=None):
    """The attention kernels on keys and values written straight into paged caches; the last t_new positions are the queries."""
    from ktransformers_amd._native_swa import swa_config, swa_forward, swa_mfma, swa_mfma_eligible
    from ktransformers_amd.models.custom_cache import KHybridCache
    T, H, D = q.shape
    G, V = k.shape[1], v.shape[2]
    cache = KHybridCache([{"kv": (G, D, V)}], 4 * T + 64, max_requests=4, page_size=page_size, dtype=dtype, device=DEV)
    cache.admit("pad"), cache.plan([("pad", page_size + 3)])          # the request's pages do not start at row 0
    t_new = T if t_new is None else t_new
    cache.admit("r")
    if T > t_new:
        cache.plan([("r", T - t_new)])
    b = cache.plan([("r", t_new)])
    pages = cache.requests["r"]["pages"]
    loc = torch.tensor([pages[p // page_size] * page_size + p % page_size for p in range(T)], device=DEV)
    cache.k_caches[0][loc] = k.to(DEV).to(dtype)
    cache.v_caches[0][loc] = v.to(DEV).to(dtype)
    cfg = swa_config(H, G, D, V, 0, False, False, 1e-6, 1.0, 0, page_size, dtype, softcap=cap)
    qn = f32d((q * scale)[T - t_new:].reshape(t_new, H * D))
    if kernel == "mfma":
        assert swa_mfma_eligible(cfg)
        o = swa_mfma(cfg, qn, cache.k_caches[0], cache.v_caches[0], b, None, None, nsplit=nsplit, out_dtype=F32)
    else:
        o = swa_forward(cfg, qn, cache.k_caches[0], cache.v_caches[0], b, None, None, nsplit=nsplit, out_dtype=F32)
    return o.view(t_new, H, V)


@pytest.mark.parametrize("kernel,dtype", [("valu", F32), ("valu", BF16), ("mfma", BF16)])
@pytest.mark.parametrize("H,G,D,V,T,cap", [(4, 2, 32, 16, 70, 2.0), (3, 1, 10, 6, 45, 0.5), (6, 3, 64, 128, 140, 20.0), (2, 2, 32, 48, 90, None),
                                           (8, 1, 64, 80, 33, 5.0), (1, 1, 1, 1, 9, 1.0)])
@pytest.mark.parametrize("nsplit", [1, 3])
def test_capped_attention_kernels(kernel, dtype, H, G, D, V, T, cap, nsplit):
    if kernel == "mfma" and (D % 32 or V % 16):
        pytest.skip("sizes the matrix-core form does not take")
    g = torch.Generator().manual_seed(T)
    q, k, v = (torch.randn(T, n, d, generator=g).to(dtype).double() for n, d in ((H, D), (G, D), (G, V)))
    q = (q * 2).to(dtype).double()
    scale = 2.0 ** round(math.log2(D ** -0.5))                 # (exact in bf16: the kernels take q already scaled)
    want = R.capped_attention_core(q, k, v, scale, cap)
    for t_new in (T, 1, 5):
        got = run_attention(q, k, v, scale, cap, dtype, kernel, nsplit=nsplit, t_new=t_new)
        assert rel(got, want[T - t_new:]) < (2e-5 if kernel == "valu" else 1.5e-2), t_new


@pytest.mark.parametrize("kernel,dtype", [("valu", F32), ("mfma", BF16)])
@pytest.mark.parametrize("t_new", [None, 1, 2])
def test_one_boosted_key_far_away_and_at_page_borders(kernel, dtype, t_new):
    """ONE key with a score far above the rest takes nearly all the weight wherever it lies — the first position, both sides of page borders
    and of key tiles, the query's own — and none when it lies behind the query."""
    H, G, D, V, T, ps, cap = 2, 1, 32, 16, 203, 8, 40.0
    g = torch.Generator().manual_seed(11)
    base_q, base_k = torch.randn(T, H, D, generator=g) * 0.05, torch.randn(T, G, D, generator=g) * 0.05
    v = torch.randn(T, G, V, generator=g).to(BF16).double()
    i = T - 1
    for j in (0, 1, 7, 8, 31, 32, 63, 64, 127, 128, 191, 192, 199, 200, i - 1, i):
        q, k = base_q.clone(), base_k.clone()
        q[:, :, 3], k[:, 0, 3] = 0.0, 0.0
        q[i, :, 3] = 6.0
        k[j, 0, 3] = 6.0                                        # score 36, capped to 28.6, against ~0 elsewhere
        q, k = q.to(BF16).double(), k.to(BF16).double()
        want = R.capped_attention_core(q, k, v, 1.0, cap)
        assert float((want[i, 0] - v[j, 0]).abs().max()) < 1e-6
        n = T if t_new is None else t_new
        got = run_attention(q, k, v, 1.0, cap, dtype, kernel, page_size=ps, t_new=n)
        assert rel(got, want[T - n:]) < (2e-5 if kernel == "valu" else 1.5e-2), j
    q = base_q.clone()
    q[i - 1, :, 3] = 6.0
    k = base_k.clone()
    k[i, 0, 3] = 6.0                                            # the boosted key lies behind the query: it must not be seen
    q, k = q.to(BF16).double(), k.to(BF16).double()
    got = run_attention(q, k, v, 1.0, cap, dtype, kernel, page_size=ps, t_new=T if t_new is None else 2)
    assert float((got[-2, 0].double().cpu() - v[i, 0]).abs().max()) > 0.3


@pytest.mark.parametrize("kernel,dtype", [("valu", F32), ("mfma", BF16)])
def test_the_cap_makes_huge_scores_equal(kernel, dtype):
    """Scores 60 and 600 differ by everything without the cap and by nothing under a cap of 2: the two keys then share the weight; negative
    ones saturate on the other side."""
    H, G, D, V, T = 1, 1, 32, 16, 40
    q, k = torch.zeros(T, H, D, dtype=F64), torch.zeros(T, G, D, dtype=F64)
    v = torch.randn(T, G, V, generator=torch.Generator().manual_seed(2)).to(BF16).double()
    q[:, 0, 0] = 8.0
    k[3, 0, 0], k[20, 0, 0], k[30, 0, 0] = 7.5, 75.0, -75.0
    capped, free = R.capped_attention_core(q, k, v, 1.0, 2.0), R.capped_attention_core(q, k, v, 1.0, None)
    assert rel(free[-1, 0], v[20, 0]) < 1e-9 and rel(capped[-1, 0], v[20, 0]) > 0.1
    for cap, want in ((2.0, capped), (None, free)):
        for t_new in (T, 1):
            assert rel(run_attention(q, k, v, 1.0, cap, dtype, kernel, t_new=t_new), want[T - t_new:]) < (2e-5 if kernel == "valu" else 1.5e-2)


# ---- mixers alone -----------------------------------------------------------------------------------------------------------------------
def operator_alone(cls, orig, tensors, width, dtype, spec_names, run, T=40):
    """An operator outside a model: h random, whole, in portions and one token at a time, against `run(P, h)`."""
    from ktransformers_amd.models.custom_cache import KHybridCache
    from ktransformers_amd.util.loader import DictLoader
    op = cls("m", DictLoader({f"m.{k}": v for k, v in tensors.items()}), SimpleNamespace(compute_dtype=dtype), orig, DEV, DEV)
    op.load()
    h = torch.randn(T, width, generator=torch.Generator().manual_seed(5)).to(dtype)
    want = run(R.as_double({f"m.{k}": v for k, v in tensors.items()}), h.double())
    assert set(op.state_spec()) <= set(spec_names)
    for cut in ([T], [1] * T, [T - 9, 2, 2, 5], [3, T - 3], [2] * (T // 2)):
        cache = KHybridCache([op.state_spec()], 256, max_requests=2, page_size=8, dtype=dtype, device=DEV)
        got, at = [], 0
        for n in cut:
            got.append(op(h[at:at + n].to(DEV), batch_of(cache, [("r", n)]), cache, 0))
            at += n
        assert rows_rel(torch.cat(got), want) < (3e-4 if dtype == F32 else 5e-2), cut[:4]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("heads,dim,vdim,tau,rank", [(3, 8, 12, 4.0, 6), (2, 32, 32, 16.0, 1), (1, 5, 7, 1.0, 40), (4, 64, 16, 8.0, 3), (1, 1, 1, 2.0, 1)])
def test_gated_linear_attention_on_its_own(dtype, heads, dim, vdim, tau, rank):
    from ktransformers_amd.operators.gated_linear import KGatedLinearAttention
    W = 24
    layer = R.parallel_layer(r_heads=heads, r_dim=dim, r_vdim=vdim, tau=tau, rank=rank, mlp=None)
    P = R.random_checkpoint(R.make_config([layer], width=W), 3)
    t = {k[len("l0.mix.right."):]: v for k, v in P.items() if k.startswith("l0.mix.right.")}
    orig = torch.nn.Module()
    for k, v in dict(heads=heads, dim=dim, vdim=vdim, tau=tau, eps=1e-4, width=W).items():
        setattr(orig, k, v)
    operator_alone(KGatedLinearAttention, orig, t, W, dtype, ("decay",),
                   lambda Q, h: R.gated_linear_attention(Q, "m.", layer["mixer"]["right"], h, 1e-4))


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("kw", [dict(), dict(heads=3, kv_heads=1, dim=10, vdim=6, conv=2, rot_dims=10, softcap=0.7), dict(heads=4, kv_heads=4, dim=32, vdim=16, conv=4, rot_dims=4),
                                dict(heads=2, kv_heads=1, dim=64, vdim=48, conv=1, rot_dims=0, softcap=None)])
def test_gated_capped_attention_on_its_own(dtype, kw):
    from ktransformers_amd.models.modeling_dunusun import DunusunAttention
    from ktransformers_amd.operators.window_attention import KWindowGQAttention
    W = 24
    layer = R.parallel_layer(mlp=None, **kw)
    P = R.random_checkpoint(R.make_config([layer], width=W), 3)
    t = {k[len("l0.mix.left."):]: v for k, v in P.items() if k.startswith("l0.mix.left.")}
    orig = DunusunAttention(SimpleNamespace(width=W, eps=1e-4), layer["mixer"]["left"])
    operator_alone(KWindowGQAttention, orig, t, W, dtype, ("kv", "conv"), lambda Q, h: R.gated_capped_attention(Q, "m.", layer["mixer"]["left"], h))


def mixer_alone(layer, dtype, seed, T=40, width=32, **kw):
    """The layer's mixer through the model: logits of a one-layer model whole, token by token and in portions, against the statement."""
    layer = dict(layer, mlp=None)
    cfg = R.make_config([layer], width=width)
    model, cache, P = build(cfg, seed, dtype, page_size=8, **kw)
    toks = tokens_of(cfg, T, seed)
    want = R.forward(P, cfg, toks)
    eng = engine_of(model, cache)
    tol = 3e-4 if dtype == F32 else 5e-2
    for sizes in ([T], [1] * T, [T - 9, 2, 2, 5], [3, T - 3], [2] * (T // 2) + [1] * (T % 2)):
        assert rows_rel(steps(eng, "a", toks, sizes), want) < tol, sizes
    return model


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("layer", [
    R.parallel_layer(),
    R.parallel_layer(heads=3, kv_heads=1, dim=10, vdim=6, conv=2, rot_dims=10, base=77.0, scale=0.4, softcap=1.5, r_heads=5, r_dim=3, r_vdim=7, tau=1.0, rank=1),
    R.parallel_layer(heads=4, kv_heads=1, dim=32, vdim=80, conv=4, rot_dims=32, r_heads=2, r_dim=32, r_vdim=64, tau=16.0, left_scale=1.4, right_scale=0.3, rank=33),
    R.parallel_layer(heads=2, kv_heads=2, dim=64, vdim=32, conv=1, rot_dims=0, softcap=None, r_heads=1, r_dim=64, r_vdim=96, left_scale=-0.5),
    R.parallel_layer(heads=1, kv_heads=1, dim=2, vdim=1, conv=9, rot_dims=2, r_heads=1, r_dim=1, r_vdim=1, rank=1),
    R.parallel_layer(heads=6, kv_heads=3, dim=12, vdim=20, conv=5, rot_dims=6, r_heads=4, r_dim=20, r_vdim=6),
], ids=["plain", "odd", "mfma", "bare", "ones", "taps-5"])
def test_parallel_layer(layer, dtype):
    model = mixer_alone(layer, dtype, 3)
    assert type(model.l0.mix).__name__ == "KScaledParallelMixer"


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("layer", [
    R.ssd_layer(),
    R.ssd_layer(heads=5, vdim=7, state=9, groups=1, conv=2, norm_groups=5),
    R.ssd_layer(heads=6, vdim=64, state=32, groups=3, conv=4, norm_groups=1),
    R.ssd_layer(heads=4, vdim=16, state=128, groups=4, conv=1, norm_groups=2),
    R.ssd_layer(heads=1, vdim=1, state=1, groups=1, conv=6, norm_groups=1),
    R.ssd_layer(heads=3, vdim=6, state=5, groups=3, conv=3, norm_groups=9),
], ids=["plain", "odd", "wide", "one-tap", "ones", "groups-across-heads"])
def test_state_space_layer(layer, dtype):
    model = mixer_alone(layer, dtype, 4)
    assert type(model.l0.mix).__name__ == "KStateSpaceDualMixer"


@pytest.mark.parametrize("mistake", ["mix transposed", "taps reversed", "no cap", "halves rotated", "decay not rooted", "scales swapped"])
def test_a_mistaken_statement_must_not_agree(mistake, monkeypatch):
    """The comparison sees each mechanism: the statement with one mistake in it disagrees with the framework."""
    cfg = R.make_config([R.parallel_layer(softcap=1.0, rot_dims=8), R.ssd_layer(mlp=None)])
    P = R.random_checkpoint(cfg, 5)
    model, cache, Pd = build(cfg, 5, F32, page_size=8, P=P)
    toks = tokens_of(cfg, 30, 1)
    got = steps(engine_of(model, cache), "a", toks, [30])
    assert rows_rel(got, R.forward(Pd, cfg, toks)) < 3e-4
    if mistake == "mix transposed":
        Pd = {k: (v.T.contiguous() if k.endswith(".mix") and v.dim() == 2 else v) for k, v in Pd.items()}
    elif mistake == "taps reversed":
        Pd = {k: (v.flip(1) if ".conv" in k and v.dim() == 2 else v) for k, v in Pd.items()}
    elif mistake == "no cap":
        cfg["layers"][0]["mixer"]["left"]["softcap"] = None
    elif mistake == "halves rotated":
        def halves(v, pos, base, dims):
            idx = torch.tensor([i // 2 + (i % 2) * (dims // 2) for i in range(dims)])
            w = v.clone()
            w[..., :dims] = v[..., idx]
            w = ROT(w, pos, base, dims)
            out = v.clone()
            out[..., idx] = w[..., :dims]
            return out
        ROT = R.rotate_pairs
        monkeypatch.setattr(R, "rotate_pairs", halves)
    elif mistake == "decay not rooted":
        cfg["layers"][0]["mixer"]["right"]["tau"] = 1.0
    else:
        m = cfg["layers"][0]["mixer"]
        m["left_scale"], m["right_scale"] = m["right_scale"], m["left_scale"]
    assert rows_rel(got, R.forward(Pd, cfg, toks)) > 1e-2


# ---- the model ------------------------------------------------------------------------------------------------------------------
CONFIGS = {
    # both layer kinds, a repeated block, a layer without feed-forward
    "mixed": lambda: R.make_config([R.parallel_layer(), R.ssd_layer(), R.parallel_layer(heads=2, kv_heads=2, conv=2, rot_dims=4, mlp=None), R.ssd_layer(mlp=None)],
                                   streams=3, loop={"start": 1, "stop": 3, "times": 2}),
    # the scan first, odd sizes everywhere, a layer repeated thrice
    "odd": lambda: R.make_config([R.ssd_layer(heads=5, vdim=7, state=9, groups=5, conv=3, norm_groups=7, mlp=R.dense_mlp(7)),
                                  R.parallel_layer(heads=3, kv_heads=1, dim=10, vdim=6, conv=5, rot_dims=6, base=77.0, scale=0.7, softcap=2.5, r_heads=5, r_dim=3,
                                                   r_vdim=7, tau=3.0, left_scale=1.2, right_scale=0.4, rank=5, mlp=R.dense_mlp(3))],
                                 width=29, vocab=53, eps=1e-3, streams=5, logit_softcap=3.0, loop={"start": 0, "stop": 1, "times": 3}),
    # sizes the matrix-core kernels take, prompts longer than a chunk of the scan
    "wide": lambda: R.make_config([R.parallel_layer(heads=8, kv_heads=2, dim=32, vdim=48, conv=4, rot_dims=32, r_heads=4, r_dim=32, r_vdim=64, tau=16.0, rank=16,
                                                    mlp=R.dense_mlp(256)),
                                   R.ssd_layer(heads=4, vdim=64, state=32, groups=2, norm_groups=2, mlp=R.dense_mlp(136)),
                                   R.parallel_layer(heads=4, kv_heads=4, dim=64, vdim=16, conv=3, rot_dims=16, r_heads=2, r_dim=64, r_vdim=32)],
                                  width=128, vocab=97, streams=4, loop={"start": 0, "stop": 2, "times": 2}),
    # everything optional left out: one stream, no loop, no caps, no rotation, no feed-forward
    "bare": lambda: R.make_config([R.parallel_layer(conv=1, rot_dims=0, softcap=None, mlp=None), R.ssd_layer(conv=1, mlp=None)], streams=1, logit_softcap=None),
    # sizes that are 1
    "ones": lambda: R.make_config([R.parallel_layer(heads=1, kv_heads=1, dim=2, vdim=1, conv=1, rot_dims=2, r_heads=1, r_dim=1, r_vdim=1, rank=1, tau=1.0,
                                                    mlp=R.dense_mlp(1)),
                                   R.ssd_layer(heads=1, vdim=1, state=1, groups=1, conv=1, norm_groups=1, mlp=R.dense_mlp(1))], width=3, vocab=5, streams=2),
}


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_model_whole_decoded_and_in_portions(name, dtype):
    cfg = CONFIGS[name]()
    model, cache, P = build(cfg, 7, dtype, page_size=16)
    T = 61 if name != "wide" else 150
    toks = tokens_of(cfg, T, 9)
    want, layers = R.forward(P, cfg, toks, return_layers=True)
    b = batch_of(cache, [("L", T)])
    lg, trail = model(torch.tensor(toks, dtype=torch.int32, device=DEV), None, cache, batch=b, return_layers=True)
    cache.release("L")
    tol = TOL[dtype]
    assert trail.shape[0] == layers.shape[0] == len(model.config.runs)
    for i in range(layers.shape[0]):
        assert rel(trail[i], layers[i]) < (tol if dtype == F32 else 4e-2), i
    lim = limits(P, cfg, toks, want, dtype)
    assert float(lim.median()) < 0.2
    assert held(lg, want, lim) < 1
    eng = engine_of(model, cache)
    for sizes in ([T], [T - 20] + [1] * 20, [2] * (T // 2) + [1] * (T % 2), [7, 33, 2, T - 45, 3], [1] * T):
        assert held(steps(eng, "a", toks, sizes), want, lim) < 1, sizes


@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_unequal_batches_and_reused_pages_and_slots(name, dtype):
    """Requests of different lengths in one batch, decoded together, against each alone; then the same through pages and slots that were
    freed in another order and still hold the earlier requests' rows and state."""
    cfg = CONFIGS[name]()
    model, cache, P = build(cfg, 12, dtype, max_tokens=512, max_requests=4, page_size=8)
    eng = engine_of(model, cache)
    lens = {"a": 1, "b": 37, "c": 18, "d": 70}
    n_dec = 14
    toks = {r: tokens_of(cfg, n + n_dec, 40 + i) for i, (r, n) in enumerate(lens.items())}
    want = {r: R.forward(P, cfg, t) for r, t in toks.items()}
    lim = {r: limits(P, cfg, t, want[r], dtype) for r, t in toks.items()}
    for order in (list(lens), ["c", "d", "a", "b"]):
        got = {r: [] for r in order}
        lg = eng.step([{"id": r, "tokens": toks[r][:lens[r]], "want": list(range(lens[r]))} for r in order])
        at = 0
        for r in order:
            got[r].append(lg[at:at + lens[r]])
            at += lens[r]
        live = list(order)
        for k in range(n_dec):
            if k == 5:
                live = live[1:]                      # a shorter request ends earlier
                cache.release(order[0])
            lg = eng.step([{"id": r, "tokens": [toks[r][lens[r] + k]], "want": [0]} for r in live])
            for i, r in enumerate(live):
                got[r].append(lg[i:i + 1])
        for r in order:
            g_ = torch.cat(got[r])
            assert held(g_, want[r][:g_.shape[0]], lim[r][:g_.shape[0]]) < 1, (order, r)
        for r in reversed(live):
            cache.release(r)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_mixed_steps_of_portions_and_single_tokens(dtype):
    """One step holds a prompt's first portion, a later portion of another and a decoded token of a third."""
    cfg = CONFIGS["mixed"]()
    model, cache, P = build(cfg, 13, dtype, page_size=8)
    eng = engine_of(model, cache)
    toks = {r: tokens_of(cfg, n, 60 + i) for i, (r, n) in enumerate((("a", 40), ("b", 33), ("c", 21)))}
    want = {r: R.forward(P, cfg, t) for r, t in toks.items()}
    lim = {r: limits(P, cfg, t, want[r], dtype) for r, t in toks.items()}
    plan = [[("a", 20)], [("b", 3), ("a", 1)], [("a", 1), ("c", 17), ("b", 9)], [("c", 1), ("b", 2), ("a", 16)], [("b", 19), ("c", 3), ("a", 2)]]
    at, got = {r: 0 for r in toks}, {r: [] for r in toks}
    for step in plan:
        lg = eng.step([{"id": r, "tokens": toks[r][at[r]:at[r] + n], "want": list(range(n))} for r, n in step])
        i = 0
        for r, n in step:
            got[r].append(lg[i:i + n])
            i, at[r] = i + n, at[r] + n
    for r, t in toks.items():
        assert at[r] == len(t) and held(torch.cat(got[r]), want[r], lim[r]) < 1, r


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_long_decoding_across_pages_and_chunks(dtype):
    cfg = CONFIGS["mixed"]()
    model, cache, P = build(cfg, 14, dtype, page_size=8)
    toks = tokens_of(cfg, 9 + 150, 3)
    want = R.forward(P, cfg, toks)
    assert held(steps(engine_of(model, cache), "a", toks, [9] + [1] * 150), want, limits(P, cfg, toks, want, dtype, draws=2)) < 1


@pytest.mark.parametrize("layer", [R.parallel_layer(tau=64.0, mlp=None), R.ssd_layer(mlp=None)], ids=["parallel", "scan"])
def test_a_changed_first_token_reaches_the_last_logits(layer):
    """Nothing is windowed: a change of ONE token — the first, one at a page border, one a chunk back — must move the last logits as the
    statement says, also when the last tokens are decoded one by one."""
    cfg = R.make_config([layer])
    P = R.random_checkpoint(cfg, 15)
    for k in P:
        if k.endswith("A_log"):
            P[k] = torch.full_like(P[k], -6.0)                  # a slow decay: the far token is still there
    model, cache, Pd = build(cfg, 15, F32, page_size=8, P=P)
    eng = engine_of(model, cache)
    T = 90
    base = tokens_of(cfg, T, 1)
    ref0, got0 = R.forward(Pd, cfg, base)[-1], steps(eng, "a", base, [T - 2, 1, 1])[-1].double().cpu()
    for pos in (0, 1, 7, 8, 63, 64, T - 3, T - 1):
        alt = list(base)
        alt[pos] = (alt[pos] + 1) % cfg["vocab"]
        dref = R.forward(Pd, cfg, alt)[-1] - ref0
        dgot = steps(eng, "b", alt, [T - 2, 1, 1])[-1].double().cpu() - got0
        assert float(dref.abs().max()) > 1e-5, pos
        assert rel(dgot, dref) < 5e-2 or float((dgot - dref).abs().max()) < 2e-5, pos


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_cache_outgrows_its_first_size(dtype):
    cfg = CONFIGS["mixed"]()
    model, cache, P = build(cfg, 17, dtype, max_tokens=16, max_requests=1, page_size=8)
    toks = {"a": tokens_of(cfg, 70, 1), "b": tokens_of(cfg, 33, 2)}
    eng = engine_of(model, cache)
    lg = eng.step([{"id": r, "tokens": t[:-4], "want": [len(t) - 5]} for r, t in toks.items()])
    rows = {r: [lg[i:i + 1]] for i, r in enumerate(toks)}
    for k in range(4, 0, -1):
        lg = eng.step([{"id": r, "tokens": [t[-k]], "want": [0]} for r, t in toks.items()])
        for i, r in enumerate(toks):
            rows[r].append(lg[i:i + 1])
    for r, t in toks.items():
        want = R.forward(P, cfg, t)
        assert held(torch.cat(rows[r]), want[-5:], limits(P, cfg, t, want, dtype)[-5:]) < 1


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_greedy_generation_through_both_loops(dtype):
    """util.generate.prefill_and_generate (one request, chunked prefill, the decode step replayed from a captured HIP graph) and
    BatchEngine.generate (a batch of unequal prompts) against the plain statement's greedy continuation."""
    from ktransformers_amd.models.custom_cache import KHybridCache
    from ktransformers_amd.models.modeling_dunusun import dunusun_layer_specs
    from ktransformers_amd.util.generate import prefill_and_generate
    cfg = CONFIGS["mixed"]()
    model, cache, P = build(cfg, 16, dtype, page_size=16)
    prompts = {"p": tokens_of(cfg, 19, 7), "q": tokens_of(cfg, 5, 8)}
    n_new = 12
    out = engine_of(model, cache).generate(prompts, max_new_tokens=n_new)
    for rid, prompt in prompts.items():
        assert len(out[rid]) == n_new
        lg = R.forward(P, cfg, prompt + out[rid])
        for k, tok in enumerate(out[rid]):      # teacher-forced on the framework's own tokens: the argmax wherever its margin is clear
            row = lg[len(prompt) - 1 + k]
            top2 = row.topk(2).values
            if float(top2[0] - top2[1]) > (1e-3 if dtype == F32 else 0.25):
                assert tok == int(row.argmax()), (rid, k)
    for use_graph in (False, True):
        c1 = KHybridCache(dunusun_layer_specs(model.config), 256, max_requests=1, page_size=16, dtype=dtype, device=DEV)
        ids = torch.tensor([prompts["p"]], dtype=torch.int64, device=DEV)
        toks = prefill_and_generate(model, ids, c1, max_new_tokens=n_new, use_cuda_graph=use_graph, chunk_size=8).tolist()
        if dtype == F32:
            assert toks == out["p"], (use_graph, toks, out["p"])
        else:                                   # (portions round differently: equal until a margin within rounding)
            lg = R.forward(P, cfg, prompts["p"] + toks)
            for k, tok in enumerate(toks):
                top2 = lg[len(prompts["p"]) - 1 + k].topk(2).values
                if float(top2[0] - top2[1]) > 0.25:
                    assert tok == int(lg[len(prompts["p"]) - 1 + k].argmax()), (use_graph, k)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_captured_decode_steps_equal_eager_ones(dtype):
    """Decode steps of a batch replayed from a captured HIP graph, with eager work (another request's prompt) and a change of the
    batch between replays: every replay against the eager engine's logits and against the plain statement."""
    cfg = CONFIGS["wide"]()
    model, cache, P = build(cfg, 21, dtype, page_size=16)
    _, cache2, _ = build(cfg, 21, dtype, page_size=16)
    eager, graphed = engine_of(model, cache2), engine_of(model, cache, use_graph=True)
    reqs = {"a": tokens_of(cfg, 30, 1), "b": tokens_of(cfg, 9, 2)}
    cont = {r: tokens_of(cfg, 12, 30 + i) for i, r in enumerate(reqs)}
    ref = {r: R.forward(P, cfg, reqs[r] + cont[r]) for r in reqs}
    lim = {r: limits(P, cfg, reqs[r] + cont[r], ref[r], dtype) for r in reqs}
    for eng in (eager, graphed):
        eng.step([{"id": r, "tokens": t, "want": []} for r, t in reqs.items()])
    live = list(reqs)
    for k in range(12):
        if k == 4:      # eager work between replays: a third request's prompt through the same cache
            for eng in (eager, graphed):
                eng.step([{"id": "z", "tokens": tokens_of(cfg, 21, 77), "want": [20]}], ["z"])
        if k == 8:
            live = ["a"]
        entries = [{"id": r, "tokens": [cont[r][k]], "want": [0]} for r in live]
        e, g_ = eager.step(entries), graphed.step(entries)
        for i, r in enumerate(live):
            at = slice(len(reqs[r]) + k, len(reqs[r]) + k + 1)
            assert held(g_[i:i + 1], ref[r][at], lim[r][at]) < 1, (k, r)
            # (a captured step cuts the keys into more ranges than an eager one: equal up to rounding)
            assert held(g_[i:i + 1], e[i:i + 1], lim[r][at] if dtype == BF16 else 1e-5) < 1, (k, r)
