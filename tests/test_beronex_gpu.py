"""Beronex on the GPU against the plain CPU statement of the design (oracle/beronex_ref.py, fp64): every mechanism alone through its
kernels and operator, then the model through the framework's registry, cache manager, step function and generation loops — whole
prompts, token-by-token decoding, portions, unequal batches, reused pages and slots, far keys, keys at page borders and window edges, odd
sizes.  Small random configurations; fp32 runs are held to rounding, bf16 runs to bf16 rounding."""
import math
from types import SimpleNamespace

import pytest
import torch

from oracle import beronex_ref as R

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF16, F64 = torch.float32, torch.bfloat16, torch.float64
TOL = {F32: 3e-4, BF16: 6e-2}


def rel(got, ref):
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    return float((got - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


def row_errors(got, ref):
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    return (got - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt().clamp_min(1e-30)


def rows_rel(got, ref):
    return float(row_errors(got, ref).max())


def held(got, ref, lim):
    """Largest ratio of a row's relative error to its limit (an infinite limit: a row that is not held)."""
    return float((row_errors(got, ref) / lim).max())


CLOSE_CALL = 0.12      # router scores nearer than this may fall the other way in bf16


def limits(P, cfg, toks, ref, dtype, draws=3):
    """What a row of logits may be off by: fp32 TOL; bf16 TOL, or four times what random relative noise of bf16's unit roundoff on the weights
    moves this row in the plain statement.  A bf16 row whose routing was a close call somewhere is not held (a fraction that stays small)."""
    lim = torch.full((len(toks),), TOL[dtype], dtype=F64)
    if dtype == F32:
        return lim
    g = torch.Generator().manual_seed(99)
    for _ in range(draws):
        noisy = {k: (v.double() * (1 + torch.randn(v.shape, generator=g, dtype=F64) * 2.0 ** -9) if v.dim() == 2 else v) for k, v in P.items()}
        lim = torch.maximum(lim, 4 * row_errors(R.forward(noisy, cfg, toks), ref))
    gaps = R.forward(P, cfg, toks, return_gaps=True)[1]
    lim[gaps < CLOSE_CALL] = float("inf")
    return lim


def build(cfg, seed, dtype, max_tokens=2048, max_requests=8, page_size=16, P=None):
    from ktransformers_amd.models import load_model
    from ktransformers_amd.models.custom_cache import KHybridCache
    from ktransformers_amd.models.modeling_beronex import beronex_layer_specs
    from ktransformers_amd.util.loader import DictLoader
    P = R.random_checkpoint(cfg, seed) if P is None else P
    model, config, _ = load_model(cfg, dtype=dtype, device=DEV, loader=DictLoader(P))
    cache = KHybridCache(beronex_layer_specs(config), max_tokens, max_requests=max_requests, page_size=page_size, dtype=dtype, device=DEV)
    return model, cache, R.as_double(P)


def tokens_of(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def engine_of(model, cache, **kw):
    from ktransformers_amd.util.batch_engine import BatchEngine
    return BatchEngine(model, cache, **kw)


def steps(eng, rid, toks, sizes):
    """Feed toks in portions of the given sizes; logits of every position."""
    got, at = [], 0
    for n in sizes:
        last = at + n == len(toks)
        got.append(eng.step([{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}], [rid] if last else []))
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


# ---- norms and the residual update --------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("W", [4, 37, 48, 1024, 1028, 2048, 2052, 4096, 4100, 1, 6])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_rms_post_norm_joins_the_residual_and_norms_it_again(W, dtype):
    """x += rms(y + gathered expert rows) w, and the next pre-norm from the same launch; rows held in registers and in LDS, one row and
    several, strided and unaligned y; the last norm's row gather through the plain form."""
    from ktransformers_amd._native_hyb import gated_norm_add
    from ktransformers_amd._native_seq import rms_combine
    g = torch.Generator().manual_seed(W)
    eps, neps = 1e-2, 3e-3
    for T, top in ((1, 1), (5, 3), (3, 9), (2, 0)):
        x, y, w, nw = (torch.randn(*s, generator=g) for s in ((T, W), (T, W + 8), (W,), (W,)))
        er, pos, tw = torch.randn(max(T * top, 1), W, generator=g), torch.randperm(max(T * top, 1), generator=g).int(), torch.rand(T, max(top, 1), generator=g)
        for off in (0, 4, 3):                                   # (column slices: a row stride, and for 3 no 16-byte alignment)
            for use_y in ((True, False) if top else (True,)):
                z = y[:, off:off + W].double() if use_y else torch.zeros(T, W, dtype=F64)
                if top:
                    z = z + (er.double()[pos.long()].view(T, top, W) * tw.double().unsqueeze(-1)).sum(1)
                want = x.double() + R.rms_norm(z, w.double(), eps)
                kw = dict(expert_rows=f32d(er), pair_pos=pos.to(DEV), topk_w=f32d(tw)) if top else {}
                xr = f32d(x)
                x2, h = gated_norm_add(xr, f32d(w), None, eps, y=f32d(y)[:, off:off + W] if use_y else None, next_norm=(f32d(nw), None, neps, dtype),
                                       rms=True, **kw)
                assert x2 is xr and h.dtype == dtype and rel(xr, want) < 1e-6
                assert rel(h, R.rms_norm(want, nw.double(), neps)) < (2e-6 if dtype == F32 else 4e-3)
                xr = f32d(x)
                assert gated_norm_add(xr, f32d(w), None, eps, y=f32d(y)[:, off:off + W] if use_y else None, rms=True, **kw) is xr and rel(xr, want) < 1e-6
        rows = torch.tensor([T - 1, 0], dtype=torch.int32, device=DEV)
        assert rel(rms_combine(f32d(x), f32d(w), eps, rows=rows, out_dtype=dtype), R.rms_norm(x.double()[[T - 1, 0]], w.double(), eps)) < (2e-6 if dtype == F32 else 4e-3)


def test_rms_norm_keeps_eps_inside_the_root():
    from ktransformers_amd._native_hyb import gated_norm_add
    x = torch.zeros(1, 8, device=DEV)
    y = torch.full((1, 8), 1e-3, device=DEV)
    gated_norm_add(x, torch.ones(8, device=DEV), None, 1e-6, y=y, rms=True)
    assert abs(float(x[0, 0]) - 1e-3 / math.sqrt(2e-6)) < 1e-6


# ---- gated linear units ---------------------------------------------------------------------------------------------------------------
UNITS = [("gelu_tanh", None, 1.0, 0.0), ("swish", 1.5, 1.702, 1.0), ("swish", None, 1.0, 0.0), ("gelu_tanh", 0.8, 1.0, 0.5), ("swish", 0.3, 2.5, -0.25)]


def unit_ref(unit, gate, up):
    kind, limit, slope, shift = unit
    if limit is not None:
        gate, up = gate.clamp(max=limit), up.clamp(-limit, limit)
    return (R.gelu_tanh(gate) if kind == "gelu_tanh" else gate * torch.sigmoid(slope * gate)) * (up + shift)


@pytest.mark.parametrize("unit", UNITS)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_gated_unit_behind_a_product(unit, dtype):
    from ktransformers_amd._native_hyb import glu_clamp_rows
    from ktransformers_amd._native_seq import glu_act
    g = torch.Generator().manual_seed(3)
    for T, F in ((3, 37), (1, 40), (9, 2052), (5, 1)):
        gate, up = torch.randn(T, F, generator=g) * 2, torch.randn(T, F, generator=g) * 2
        want, tol = unit_ref(unit, gate.double(), up.double()), 2e-6 if dtype == F32 else 4e-3
        pairs = torch.stack([gate, up], dim=2).reshape(T, 2 * F)
        assert rel(glu_clamp_rows(f32d(pairs), glu_act(*unit), out_dtype=dtype, paired=True), want) < tol
        assert rel(glu_clamp_rows(f32d(torch.cat([gate, up], dim=1)), glu_act(*unit), out_dtype=dtype), want) < tol
        wide = f32d(torch.cat([torch.zeros(T, 3), pairs], dim=1))[:, 3:]         # no 16-byte alignment
        assert rel(glu_clamp_rows(wide, glu_act(*unit), out_dtype=dtype, paired=True), want) < tol


@pytest.mark.parametrize("unit", UNITS[:3])
@pytest.mark.parametrize("M,F,K", [(1, 40, 64), (8, 37, 96), (16, 16, 32)])
def test_gated_unit_in_the_decode_products_launch(unit, M, F, K):
    from ktransformers_amd._native_seq import dense_gemv_glu, glu_act
    g = torch.Generator().manual_seed(M)
    a, gate, up = ((torch.randn(n, K, generator=g) * s).to(BF16) for n, s in ((M, 1), (F, 2 / math.sqrt(K)), (F, 2 / math.sqrt(K))))
    want = unit_ref(unit, a.double() @ gate.double().T, a.double() @ up.double().T)
    w = torch.stack([gate, up], dim=1).reshape(2 * F, K).contiguous().to(DEV)
    for dt, tol in ((F32, 2e-5), (BF16, 4e-3)):
        assert rel(dense_gemv_glu(a.to(DEV), w, glu_act(*unit), out_dtype=dt), want) < tol


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("E,top,T,F,K", [(5, 2, 3, 20, 32), (4, 3, 60, 36, 40), (3, 1, 400, 72, 64), (1, 1, 7, 5, 9), (6, 6, 20, 64, 96), (2, 1, 33, 130, 48)])
def test_gated_unit_in_the_epilogue_of_grouped_products(dtype, E, top, T, F, K):
    """Experts' gate and up rows alternate: streaming form, 64-row and 128-row tiles, aligned and odd sizes; an expert nobody chose."""
    from ktransformers_amd._native_hyb import expert_gemm, moe_plan
    from ktransformers_amd._native_seq import glu_act
    g = torch.Generator().manual_seed(T)
    unit = ("swish", 1.2, 1.702, 1.0)
    h = torch.randn(T, K, generator=g).to(dtype)
    gate, up = ((torch.randn(E, F, K, generator=g) * 2 / math.sqrt(K)).to(dtype) for _ in range(2))
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int()
    if E > 4:
        idx = torch.where(idx == 2, torch.full_like(idx, 3), idx)
    w = torch.stack([gate, up], dim=2).reshape(E, 2 * F, K).contiguous().to(DEV)
    for wide in ((False, True) if dtype == BF16 and T * top > 64 else (False,)):
        plan = moe_plan(idx.to(DEV), E, wide=wide)
        got = expert_gemm(h.to(DEV), w, plan, gather=True, out_dtype=dtype, unit=glu_act(*unit))
        assert tuple(got.shape) == (T * top, F)
        got = got[plan.pair_pos.long()].view(T, top, F)
        for k in range(top):
            e = idx[:, k].long()
            want = unit_ref(unit, torch.einsum("tk,tfk->tf", h.double(), gate.double()[e]), torch.einsum("tk,tfk->tf", h.double(), up.double()[e]))
            assert rel(got[:, k], want) < (2e-6 if dtype == F32 else 4e-3), (wide, k)


# ---- router -----------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("E,top,T", [(6, 2, 50), (3, 1, 7), (4, 4, 9), (70, 5, 300), (16, 3, 1), (130, 130, 5), (1, 1, 3)])
def test_router_with_a_bias_weighs_the_chosen_alone(E, top, T):
    from ktransformers_amd._native_swa import softmax_route, softmax_route_plan
    g = torch.Generator().manual_seed(E)
    z, b = torch.randn(T, E + 3, generator=g) * 2, torch.randn(E, generator=g) * 2
    ridx, rw = R.routed(z[:, :E].double() + b.double(), top)
    idx, w = softmax_route(f32d(z)[:, :E], top, 0.0, bias=f32d(b))
    assert torch.equal(idx.cpu().long(), ridx) and rel(w, rw) < 1e-6 and float((w.sum(1) - 1).abs().max()) < 1e-6
    if T <= 64:
        idx2, w2, plan = softmax_route_plan(f32d(z)[:, :E], top, 0.0, bias=f32d(b))
        assert torch.equal(idx, idx2) and torch.equal(w, w2) and int(plan.group_off[-1]) == T * top


def test_router_chooses_by_score_far_below_the_largest():
    """Scores 200 below the largest have no weight in fp32, yet their order still says which are chosen; the bias alone can decide."""
    from ktransformers_amd._native_swa import softmax_route
    z = torch.tensor([[0.0, -210.0, -205.0, -300.0, -207.0]])
    idx, w = softmax_route(f32d(z), 3, 0.0)
    assert idx.tolist() == [[0, 2, 4]] and float(w[0, 0]) == 1.0
    idx, w = softmax_route(f32d(torch.zeros(1, 4)), 2, 0.0, bias=f32d(torch.tensor([0.0, 1.0, -1.0, 2.0])))
    assert idx.tolist() == [[3, 1]] and rel(w[0], torch.softmax(torch.tensor([2.0, 1.0]), 0)) < 1e-6


# ---- rotations and preps ------------------------------------------------------------------------------------------------------------------
ROTS = [R.rot_of(8), R.rot_of(12, base=50.0, factor=3.0, original=40, fast=4.0, slow=0.5), R.rot_of(4, base=1e6, factor=20.0), R.rot_of(10, scaled=False),
        R.rot_of(2, base=7.0, original=7, fast=1.0, slow=1.0)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("rot", ROTS)
def test_window_attention_prep_scaled_rotation_then_unit_rms(rot, dtype):
    from ktransformers_amd._native_swa import swa_config, swa_prep
    from ktransformers_amd.models.custom_cache import KHybridCache
    from ktransformers_amd.operators.RoPE import turning_frequencies
    H, G, D, V, T, eps = 4, 2, 13, 7, 90, 1e-2
    g = torch.Generator().manual_seed(4)
    q, k, v = torch.randn(T, H, D, generator=g), torch.randn(T, G, D, generator=g), torch.randn(T, G, V, generator=g)
    wq, wk = (R.unit_rms(R.rotate(t.double(), rot, False), eps) for t in (q, k))
    freq, amp = turning_frequencies(rot["base"], rot["dims"], rot["scaling"])
    cache = KHybridCache([{"kv": (G, D, V)}], 256, max_requests=2, page_size=8, dtype=dtype, device=DEV)
    cfg = swa_config(H, G, D, V, rot["dims"], False, True, eps, 0.4, 9, 8, dtype, rot_scale=amp)
    proj = f32d(torch.cat([torch.zeros(T, 5), q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], dim=1))[:, 5:]
    batch_of(cache, [("pad", 11)])
    b = batch_of(cache, [("r", T)])
    got, vcs = swa_prep(cfg, proj, 0, H * D, (H + G) * D, freq.to(DEV), None, b.positions, b.cache_loc, cache.k_caches[0], cache.v_caches[0])
    assert vcs is None and rel(got.view(T, H, D), 0.4 * wq) < 2e-6
    tol = 2e-6 if dtype == F32 else 4e-3
    assert rel(cache.k_caches[0][b.cache_loc.long()], wk) < tol and rel(cache.v_caches[0][b.cache_loc.long()], v.double()) < tol
    # a layer that reads another's rows: the queries alone, nothing appended
    before = cache.k_caches[0].clone(), cache.v_caches[0].clone()
    got2, _ = swa_prep(cfg, proj[:, :H * D], 0, 0, 0, freq.to(DEV), None, b.positions, b.cache_loc, None, None)
    assert torch.equal(got, got2) and torch.equal(before[0], cache.k_caches[0]) and torch.equal(before[1], cache.v_caches[0])


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("rot", ROTS)
def test_latent_preps_scaled_half_rotation_and_the_query_latent(rot, dtype):
    from ktransformers_amd._native_hyb import latattn_config, latattn_latents, latattn_prep
    from ktransformers_amd.models.custom_cache import KHybridCache
    from ktransformers_amd.operators.RoPE import turning_frequencies
    H, D, Rd, L, Q, T, eps = 3, 6, 13, 21, 300, 70, 1e-2
    g = torch.Generator().manual_seed(5)
    cq, down, q = torch.randn(T, Q, generator=g), torch.randn(T, L + Rd, generator=g), torch.randn(T, H, D + Rd, generator=g)
    wq, wn = torch.randn(Q, generator=g), torch.randn(L, generator=g)
    freq, amp = turning_frequencies(rot["base"], rot["dims"], rot["scaling"])
    cache = KHybridCache([{"latent": L + Rd}], 256, max_requests=2, page_size=8, dtype=dtype, device=DEV)
    cfg = latattn_config(H, D, Rd, 5, L, rot["dims"], 1.0, 0, eps, 8, dtype, rot_half=True, rot_scale=amp)
    batch_of(cache, [("pad", 11)])
    b = batch_of(cache, [("r", T)])
    proj = f32d(torch.cat([torch.zeros(T, 3), cq, down], dim=1))
    tol = 2e-6 if dtype == F32 else 4e-3
    got = latattn_latents(cfg, proj, 3, Q, 3 + Q, f32d(wq), f32d(wn), freq.to(DEV), b.positions, b.cache_loc, cache.lat_caches[0], dtype)
    assert got.dtype == dtype and rel(got, R.rms_norm(cq.double(), wq.double(), eps)) < tol
    want_row = torch.cat([R.rms_norm(down[:, :L].double(), wn.double(), eps), R.rotate(down[:, L:].double().view(T, 1, Rd), rot, True)[:, 0]], dim=1)
    assert rel(cache.lat_caches[0][b.cache_loc.long()], want_row) < tol
    rows = cache.lat_caches[0].clone()
    # queries turned on their own, and both at once in the form without a query latent
    q_out = torch.zeros(T, H, L + Rd, device=DEV)
    qrows = f32d(torch.cat([q.reshape(T, -1), down], dim=1))
    latattn_prep(cfg, qrows, 0, 0, None, freq.to(DEV), b.positions, b.cache_loc, None, q_out)
    want_q = R.rotate(q[..., D:].double(), rot, True)
    assert rel(q_out[..., L:], want_q) < 2e-6 and torch.equal(rows, cache.lat_caches[0])
    cache.lat_caches[0].zero_()
    latattn_prep(cfg, qrows, 0, H * (D + Rd), f32d(wn), freq.to(DEV), b.positions, b.cache_loc, cache.lat_caches[0], q_out)
    assert rel(q_out[..., L:], want_q) < 2e-6 and rel(cache.lat_caches[0][b.cache_loc.long()], want_row) < tol


# ---- attention kernels --------------------------------------------------------------------------------------------------------------------
def run_attention(q, k, v, scale, window, dtype, kernel, nsplit=1, page_size=8, t_new=None, head_gate=None):
    """The attention kernels on keys and values written straight into paged caches; the last t_new positions are the queries."""
    from ktransformers_amd._native_swa import swa_config, swa_forward, swa_mfma, swa_mfma_eligible
    from ktransformers_amd.models.custom_cache import KHybridCache
    T, H, D = q.shape
    G, V = k.shape[1], v.shape[2]
    cache = KHybridCache([{"kv": (G, D, V)}], 4 * T + 64, max_requests=4, page_size=page_size, dtype=dtype, device=DEV)
    batch_of(cache, [("pad", page_size + 3)])                   # the request's pages do not start at row 0
    t_new = T if t_new is None else t_new
    if T > t_new:
        batch_of(cache, [("r", T - t_new)])
    b = batch_of(cache, [("r", t_new)])
    pages = cache.requests["r"]["pages"]
    loc = torch.tensor([pages[p // page_size] * page_size + p % page_size for p in range(T)], device=DEV)
    cache.k_caches[0].fill_(float("nan")), cache.v_caches[0].fill_(float("nan"))      # rows nobody wrote must not be read
    cache.k_caches[0][loc], cache.v_caches[0][loc] = k.to(DEV).to(dtype), v.to(DEV).to(dtype)
    cfg = swa_config(H, G, D, V, 0, False, False, 1e-6, 1.0, window or 0, page_size, dtype)
    qn = f32d((q * scale)[T - t_new:].reshape(t_new, H * D))
    assert kernel != "mfma" or swa_mfma_eligible(cfg)
    fn = swa_mfma if kernel == "mfma" else swa_forward
    return fn(cfg, qn, cache.k_caches[0], cache.v_caches[0], b, None, None, nsplit=nsplit, out_dtype=F32, head_gate=head_gate).view(t_new, H, V)


@pytest.mark.parametrize("kernel,dtype", [("valu", F32), ("valu", BF16), ("mfma", BF16)])
@pytest.mark.parametrize("H,G,D,V,T,window", [(4, 2, 40, 48, 90, 17), (3, 3, 8, 16, 70, 33), (6, 2, 72, 80, 140, 64), (2, 1, 104, 32, 75, 1), (4, 4, 56, 64, 130, None),
                                              (1, 1, 24, 16, 40, 200), (5, 1, 200, 128, 66, 31), (2, 2, 3, 5, 30, 4)])
@pytest.mark.parametrize("nsplit", [1, 3])
def test_window_attention_kernels(kernel, dtype, H, G, D, V, T, window, nsplit):
    """Head sizes that are not whole matrix-core steps (a multiple of 8 is filled up with zeros in the tile)."""
    if kernel == "mfma" and (D % 8 or V % 16):
        pytest.skip("sizes the matrix-core form does not take")
    g = torch.Generator().manual_seed(T)
    q, k, v = (torch.randn(T, n, d, generator=g).to(dtype).double() for n, d in ((H, D), (G, D), (G, V)))
    scale = 2.0 ** round(math.log2(D ** -0.5))                 # (exact in bf16: the kernels take q already scaled)
    want = R.softmax_attention(q, k, v, scale, window)
    for t_new in (T, 1, 2, 5):
        got = run_attention(q, k, v, scale, window, dtype, kernel, nsplit=nsplit, t_new=t_new)
        assert rel(got, want[T - t_new:]) < (2e-5 if kernel == "valu" else 1.5e-2), t_new


@pytest.mark.parametrize("kernel,dtype", [("valu", F32), ("mfma", BF16)])
@pytest.mark.parametrize("t_new", [None, 1, 2])
@pytest.mark.parametrize("window", [24, 25, 64])
def test_one_boosted_key_at_the_windows_edge(kernel, dtype, t_new, window):
    """ONE key with a score far above the rest: just inside the window it takes all the weight, just outside none; also at page and tile
    borders, at the first position and behind the query."""
    H, G, D, V, T, ps = 2, 1, 40, 16, 103, 8
    g = torch.Generator().manual_seed(11)
    base_q, base_k = torch.randn(T, H, D, generator=g) * 0.05, torch.randn(T, G, D, generator=g) * 0.05
    v = torch.randn(T, G, V, generator=g).to(BF16).double()
    i = T - 1
    for j in sorted({i - window + 1, i - window, i - window - 1, i, i - 1, 0, 95, 96, 88, 87, i - window + 2}):
        q, k = base_q.clone(), base_k.clone()
        q[:, :, 37], k[:, 0, 37] = 0.0, 0.0
        q[i, :, 37], k[j, 0, 37] = 6.0, 6.0                    # score 36 against ~0 elsewhere
        q, k = q.to(BF16).double(), k.to(BF16).double()
        want = R.softmax_attention(q, k, v, 1.0, window)
        seen = i - j < window
        assert (float((want[i, 0] - v[j, 0]).abs().max()) < 1e-6) == seen, j
        n = T if t_new is None else t_new
        got = run_attention(q, k, v, 1.0, window, dtype, kernel, page_size=ps, t_new=n)
        assert rel(got, want[T - n:]) < (2e-5 if kernel == "valu" else 1.5e-2), j
        assert (float((got[-1, 0].double().cpu() - v[j, 0]).abs().max()) < 2e-2) == seen, j
    q, k = base_q.clone(), base_k.clone()
    q[i - 1, :, 37], k[i, 0, 37] = 6.0, 6.0                    # the boosted key lies behind the query: it must not be seen
    got = run_attention(q.to(BF16).double(), k.to(BF16).double(), v, 1.0, window, dtype, kernel, page_size=ps, t_new=T if t_new is None else 2)
    assert float((got[-2, 0].double().cpu() - v[i, 0]).abs().max()) > 0.3


# ---- the scan with activations and constant decays ------------------------------------------------------------------------------------
def run_scan(q, k, v, decay, cut, chunk_len, garbage=3.0):
    """A longer neighbour and the sequence in one batch, in portions `cut`; constant decays, silu inside the scan."""
    from ktransformers_amd._native_gla import decay_scan
    from ktransformers_amd.models.custom_cache import KHybridCache
    T, H, V = v.shape
    D = k.shape[2]
    cache = KHybridCache([{"decay": (H, D, V)}], 4096, max_requests=4, page_size=8, dtype=F32, device=DEV)
    cache.S[0].fill_(garbage)
    rows = f32d(torch.cat([t.reshape(T, -1) for t in (q, k, v)], dim=1))
    dec = f32d(decay.view(1, H))
    got, at = [], 0
    for n in cut:
        other = n + 3 if at + n + 3 <= T else n
        bt = batch_of(cache, [("x", other), ("r", n)])
        p = rows[torch.tensor(list(range(other)) + list(range(at, at + n)), device=DEV)]
        o = decay_scan(p[:, :H * D], p[:, H * D:2 * H * D], p[:, 2 * H * D:], dec.expand(other + n, H), bt, cache.S[0], chunk_len=chunk_len, qkv_silu=True)
        got.append(o[other:])
        at += n
    assert at == T
    untouched = [s for s in range(cache.max_requests) if s not in (cache.requests["x"]["slot"], cache.requests["r"]["slot"])]
    assert float((cache.S[0][untouched] - garbage).abs().max()) == 0.0
    return torch.cat(got).view(T, H, V), cache.S[0][cache.requests["r"]["slot"]]


@pytest.mark.parametrize("H,D,V", [(3, 8, 12), (4, 32, 64), (2, 64, 32), (2, 128, 128), (1, 256, 70), (2, 100, 65), (1, 300, 16), (2, 1, 1), (3, 17, 33), (1, 512, 130),
                                   (1, 33, 200), (5, 2, 3)])
def test_lightning_scan_whole_portions_and_chunks(H, D, V):
    g = torch.Generator().manual_seed(D + V)
    T = 75
    q, k, v = (torch.randn(T, H, d, generator=g) * 1.5 for d in (D, D, V))
    decay = torch.tensor([[1.0, 0.93, 0.0, 0.999, 0.3][(h + D) % 5] for h in range(H)])
    want = torch.zeros(T, H, V, dtype=F64)
    for h in range(H):
        want[:, h] = R.decayed_scan(*(R.silu(t[:, h].double()) for t in (q, k, v)), float(decay[h]))
    final = None
    for cut, chunk in (([T], 0), ([T], 8), ([T], 64), ([T], 5), ([1] * T, 64), ([40, 2, 1, 2, 30], 16), ([2] * 37 + [1], 64), ([64, 11], 64), ([9, 66], 32),
                       ([5] * 15, 64), ([17, 16, 15, 27], 64), ([8, 9, 58], 64)):
        got, S = run_scan(q, k, v, decay, cut, chunk)
        assert rel(got, want) < 5e-6, (cut[:4], chunk)
        assert rows_rel(got.reshape(T, -1), want.reshape(T, -1)) < 5e-5, (cut[:4], chunk)
        final = S if final is None else final
        assert rel(S, final) < 5e-6


def test_lightning_scan_remembers_one_far_token():
    """A decay of 1: the pair written at position j is read back at the last position however many chunks lie between; a decay of 0 keeps
    only the current token's."""
    T, H, D, V = 200, 2, 16, 8
    v, k, q = torch.zeros(T, H, V), torch.zeros(T, H, D), torch.zeros(T, H, D)
    q[-1, :, 3] = 20.0                                          # silu(20) = 20
    for j in (0, 15, 16, 63, 64, 127, 128, 198, 199):
        kk, vv = k.clone(), v.clone()
        kk[j, :, 3] = 20.0
        vv[j] = torch.randn(H, V, generator=torch.Generator().manual_seed(j)).abs() * 3 + 1
        for chunk in (16, 64, 128, 0):
            got, _ = run_scan(q, kk, vv, torch.tensor([1.0, 0.0]), [T] if chunk else [T - 2, 1, 1], chunk)
            want = 400.0 * R.silu(vv[j].double())
            assert rel(got[-1, 0], want[0]) < 1e-6, (j, chunk)
            assert (float(got[-1, 1].abs().max()) == 0.0) == (j < T - 1), (j, chunk)


# ---- gates --------------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("kernel,dtype", [("valu", F32), ("valu", BF16), ("mfma", BF16)])
@pytest.mark.parametrize("nsplit", [1, 3])
def test_one_gate_per_head_inside_the_attention(kernel, dtype, nsplit):
    H, G, D, V, T, window = 6, 2, 40, 48, 70, 21
    g = torch.Generator().manual_seed(3)
    q, k, v = (torch.randn(T, n, d, generator=g).to(dtype).double() for n, d in ((H, D), (G, D), (G, V)))
    gate = torch.randn(T, H + 7, generator=g) * 3               # (a column slice: strided rows)
    want = R.softmax_attention(q, k, v, 0.125, window) * torch.sigmoid(gate[:, 4:4 + H].double()).view(T, H, 1)
    for t_new in (T, 1, 2):
        got = run_attention(q, k, v, 0.125, window, dtype, kernel, nsplit=nsplit, t_new=t_new, head_gate=f32d(gate[T - t_new:])[:, 4:4 + H])
        assert rel(got, want[T - t_new:]) < (2e-5 if kernel == "valu" else 1.5e-2), t_new
    for i in (0, T - 1):                                        # a gate that is shut is that token's and that head's alone
        shut = torch.zeros(T, H)
        shut[i, 4] = -200.0
        got = run_attention(q, k, v, 0.125, window, dtype, kernel, nsplit=nsplit, head_gate=f32d(shut)).cpu()
        assert float(got[i, 4].abs().max()) == 0.0 and int((got.abs().amax(dim=2) == 0).sum()) == 1


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T", [1, 3, 70])
def test_gate_and_norm_over_all_heads(dtype, T):
    """Norm groups as wide as all heads together: aligned pieces held in registers, rows in LDS beyond that, odd sizes, strided gates."""
    from ktransformers_amd._native_gla import gate_seg, gate_segments
    g = torch.Generator().manual_seed(T)
    tol = 2e-6 if dtype == F32 else 4e-3
    for n, odt in ((96, BF16), (21, F32), (2048, F32), (2048, BF16), (5, F32), (1170, F32), (1168, F32), (4096, F32), (4104, BF16), (512, F32), (520, BF16)):
        for off in (4, 3):
            o, gate, w = torch.randn(T, n, generator=g).to(odt), torch.randn(T, n + 8, generator=g), torch.randn(n, generator=g)
            od, gd = o.to(DEV), f32d(gate)[:, off:off + n]
            z = gate[:, off:off + n].double()
            got = gate_segments([gate_seg(od, gd, "sigmoid", norm=(f32d(w), n, 1e-2))], T, DEV, out_dtype=dtype)
            assert got.dtype == dtype and rel(got, R.rms_norm(o.double(), w.double(), 1e-2) * torch.sigmoid(z)) < tol, (n, off)
            got = gate_segments([gate_seg(od, gd, "silu", norm=(f32d(w), n, 1e-2), gate_first=True, scale=0.7)], T, DEV, out_dtype=dtype)
            assert rel(got, 0.7 * R.rms_norm(o.double() * R.silu(z), w.double(), 1e-2)) < tol, (n, off)
            got = gate_segments([gate_seg(od, gd, "sigmoid")], T, DEV, out_dtype=dtype)
            assert rel(got, o.double() * torch.sigmoid(z)) < tol, (n, off)


# ---- mixers and feed-forwards alone ---------------------------------------------------------------------------------------------------
def operator_of(cls, orig, P, prefix, dtype):
    from ktransformers_amd.util.loader import DictLoader
    op = cls("m", DictLoader({"m." + k[len(prefix):]: v for k, v in P.items() if k.startswith(prefix)}), SimpleNamespace(compute_dtype=dtype), orig, DEV, DEV)
    op.load()
    return op


def mixer_alone(layer, dtype, T=40, W=24):
    """The layer's mixer outside a model: h random, whole, in portions and one token at a time, against the statement."""
    from ktransformers_amd.models import modeling_beronex as M
    from ktransformers_amd.models.custom_cache import KHybridCache
    from ktransformers_amd.operators.latent_window_attention import KLatentWindowAttention
    from ktransformers_amd.operators.lightning import KLightningAttention
    from ktransformers_amd.operators.window_attention import KWindowGQAttention
    eps = 1e-3
    ns, c = SimpleNamespace(width=W, eps=eps), layer["mixer"]
    P = R.random_checkpoint(R.make_config([dict(layer, mlp=None)], width=W), 3)
    cls, skel, ref = {"attention": (KWindowGQAttention, M.BeronexAttention, lambda Q, h: R.window_attention(Q, "l0.mix.", c, h, eps, {})[0]),
                      "latent_attention": (KLatentWindowAttention, M.BeronexLatentAttention, lambda Q, h: R.latent_attention(Q, "l0.mix.", c, h, eps)),
                      "lightning": (KLightningAttention, M.BeronexLightning, lambda Q, h: R.lightning_attention(Q, "l0.mix.", c, h, eps))}[layer["type"]]
    op = operator_of(cls, skel(ns, c), P, "l0.mix.", dtype)
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(5)).to(dtype)
    want = ref(R.as_double(P), h.double())
    for cut in ([T], [1] * T, [T - 9, 2, 2, 5], [3, T - 3], [2] * (T // 2)):
        cache = KHybridCache([op.state_spec()], 256, max_requests=2, page_size=8, dtype=dtype, device=DEV)
        for t in cache.state_tensors():
            t.fill_(5.0)                                        # a slot's old contents do not matter
        got, at = [], 0
        for n in cut:
            y = op(h[at:at + n].to(DEV), batch_of(cache, [("r", n)]), cache, 0)
            got.append(y[0] if isinstance(y, tuple) else y)
            at += n
        assert rows_rel(torch.cat(got), want) < (3e-4 if dtype == F32 else 6e-2), cut[:4]
    return op


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("layer", [
    R.lightning_layer(), R.lightning_layer(heads=5, dim=3, vdim=7), R.lightning_layer(heads=2, dim=64, vdim=32, decay=[1.0, 0.7]), R.lightning_layer(heads=1, dim=1, vdim=1, decay=[0.9]),
    R.lightning_layer(heads=4, dim=130, vdim=16), R.lightning_layer(heads=2, dim=8, vdim=300),
    R.latent_layer(), R.latent_layer(heads=5, dim=3, rot_dim=6, vdim=7, q_rank=5, kv_rank=9, rot=R.rot_of(6, base=20.0, original=16)),
    R.latent_layer(heads=4, dim=32, rot_dim=16, vdim=32, q_rank=40, kv_rank=64, rot=R.rot_of(16)), R.latent_layer(heads=1, dim=1, rot_dim=2, vdim=1, q_rank=1, kv_rank=1, rot=R.rot_of(2)),
    R.latent_layer(heads=2, dim=16, rot_dim=64, vdim=8, q_rank=16, kv_rank=128, scale=0.3, rot=R.rot_of(64)), R.latent_layer(rot=R.rot_of(8, scaled=False)),
    R.attention_layer(), R.attention_layer(heads=3, kv_heads=1, dim=10, vdim=6, window=5, rot=R.rot_of(10, base=20.0, original=16)),
    R.attention_layer(heads=8, kv_heads=2, dim=40, vdim=32, window=17, rot=R.rot_of(40)), R.attention_layer(heads=2, kv_heads=2, dim=64, vdim=48, window=1, rot=R.rot_of(16)),
    R.attention_layer(heads=1, kv_heads=1, dim=2, vdim=1, window=2, rot=R.rot_of(2)), R.attention_layer(window=None), R.attention_layer(rot=R.rot_of(12, scaled=False), window=1000),
], ids=lambda L: f"{L['type']}-{L['mixer']['heads']}x{L['mixer']['dim']}x{L['mixer']['vdim']}")
def test_mixer_on_its_own(layer, dtype):
    mixer_alone(layer, dtype)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T", [1, 7, 30, 500])
@pytest.mark.parametrize("experts,top,ff,W", [(6, 2, 20, 32), (3, 3, 7, 9), (1, 1, 5, 24), (12, 5, 64, 64)])
def test_mixture_on_its_own(experts, top, ff, W, T, dtype):
    from ktransformers_amd.models.modeling_beronex import BeronexMoE
    from ktransformers_amd.operators.softmax_moe import KSoftmaxRoutedMoE
    c = R.moe_mlp(experts, top, ff, limit=0.9)
    P = R.random_checkpoint(R.make_config([R.lightning_layer(mlp=c)], width=W), 3)
    op = operator_of(KSoftmaxRoutedMoE, BeronexMoE(SimpleNamespace(width=W), c), P, "l0.mlp.", dtype)
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(T)).to(dtype)
    rows, pos, idx, wts, _, _ = op(h.to(DEV))
    got = (rows.double()[pos.long()].view(T, top, W) * wts.double().unsqueeze(-1)).sum(1)
    Pd = R.as_double(P)
    want = R.mixture(Pd, "l0.mlp.", c, h.double())
    z = torch.sort(R.router_scores(Pd, "l0.mlp.", h.double()), dim=-1, descending=True).values
    clear = (z[:, top - 1] - z[:, min(top, experts - 1)] > 1e-4) if top < experts else torch.ones(T, dtype=torch.bool)
    assert rows_rel(got.cpu()[clear], want[clear]) < (2e-5 if dtype == F32 else 3e-2)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T", [1, 16, 17, 200])
@pytest.mark.parametrize("ff,W", [(40, 32), (7, 9), (256, 64), (1, 3)])
def test_dense_feed_forward_on_its_own(ff, W, T, dtype):
    from ktransformers_amd.models.modeling_beronex import BeronexMLP
    from ktransformers_amd.operators.mlp import KClampedGLUMLP
    c = R.dense_mlp(ff)
    P = R.random_checkpoint(R.make_config([R.lightning_layer(mlp=c)], width=W), 3)
    op = operator_of(KClampedGLUMLP, BeronexMLP(SimpleNamespace(width=W), c), P, "l0.mlp.", dtype)
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(T)).to(dtype)
    want = R.dense_feed_forward(R.as_double(P), "l0.mlp.", h.double())
    assert rel(op(h.to(DEV)), want) < (1e-5 if dtype == F32 else 2e-2)


# ---- the comparison sees each mechanism -------------------------------------------------------------------------------------------------
MISTAKES = {
    "window one longer": lambda c, mp: c["layers"][0]["mixer"]["mask"].update(size=c["layers"][0]["mixer"]["mask"]["size"] + 1),
    "own window of a sharing layer": lambda c, mp: c["layers"][2]["mixer"].update(mask=c["layers"][0]["mixer"]["mask"]),
    "own scale of a sharing layer": lambda c, mp: c["layers"][2]["mixer"].update(scale=c["layers"][0]["mixer"]["scale"]),
    "no scaling of frequencies": lambda c, mp: c["layers"][0]["mixer"]["rot"].update(scaling=None),
    "ramp between other pairs": lambda c, mp: c["layers"][3]["mixer"]["rot"]["scaling"].update(fast=2.0),
    "layouts of pairs": lambda c, mp: mp.setattr(R, "rotate", lambda v, rot, half, f=R.rotate: f(v, rot, not half)),
    "amplitude left out": lambda c, mp: mp.setattr(R, "yarn", lambda *a, f=R.yarn: (f(*a)[0], 1.0)),
    "decays in reverse": lambda c, mp: c["layers"][1]["mixer"]["decay"].reverse(),
    "expert bound": lambda c, mp: c["layers"][1]["mlp"]["expert"].update(limit=4.0),
    "router weights over all": lambda c, mp: mp.setattr(R, "routed", lambda z, top: (torch.sort(z, -1, True).indices[:, :top], torch.softmax(z, -1).sort(-1, True).values[:, :top])),
    "gelu for silu": lambda c, mp: mp.setattr(R, "gelu_tanh", R.silu),
    "scale of the embedding": lambda c, mp: c["embedding"].update(scale=1.0),
    "eps": lambda c, mp: c["norm"].update(eps=0.0),
    "latent scale": lambda c, mp: c["layers"][3]["mixer"].update(scale=c["layers"][3]["mixer"]["scale"] * 1.2),
}


def mistake_config():
    return R.make_config([R.attention_layer(window=6), R.lightning_layer(mlp=R.moe_mlp()),
                          R.attention_layer(heads=6, window=17, scale=0.2, kv_from=0, mlp=R.moe_mlp(top=3, limit=0.7)), R.latent_layer()], eps=0.02, embed_scale=0.7)


@pytest.mark.parametrize("mistake", list(MISTAKES))
def test_a_mistaken_statement_must_not_agree(mistake, monkeypatch):
    cfg = mistake_config()
    P = R.random_checkpoint(cfg, 5)
    model, cache, Pd = build(cfg, 5, F32, page_size=8, P=P)
    toks = tokens_of(cfg, 40, 1)
    got = steps(engine_of(model, cache), "a", toks, [40])
    assert rows_rel(got, R.forward(Pd, cfg, toks)) < 3e-4
    wrong = mistake_config()
    MISTAKES[mistake](wrong, monkeypatch)
    assert rows_rel(got, R.forward(Pd, wrong, toks)) > 3e-3


# ---- the model ------------------------------------------------------------------------------------------------------------------
CONFIGS = {
    # every kind of layer, shared keys with another window, layers without a feed-forward, both feed-forwards
    "mixed": lambda: R.make_config([R.attention_layer(), R.lightning_layer(mlp=R.moe_mlp()), R.attention_layer(heads=6, window=20, scale=0.3, kv_from=0, mlp=None),
                                    R.latent_layer(mlp=R.moe_mlp(experts=5, top=3, ff=9, limit=0.8)), R.attention_layer(window=3, kv_from=0, mlp=R.moe_mlp(4, 1))]),
    # odd sizes everywhere, a latent layer first
    "odd": lambda: R.make_config([R.latent_layer(heads=5, dim=3, rot_dim=6, vdim=7, q_rank=11, kv_rank=9, rot=R.rot_of(6, base=20.0, original=16), mlp=R.moe_mlp(7, 4, 5, 2.5)),
                                  R.attention_layer(heads=3, kv_heads=1, dim=7, vdim=5, window=13, scale=0.9, rot=R.rot_of(6, base=77.0, factor=2.0), mlp=R.dense_mlp(7)),
                                  R.lightning_layer(heads=5, dim=3, vdim=7, mlp=None),
                                  R.attention_layer(heads=2, kv_heads=1, dim=7, vdim=5, window=4, rot=R.rot_of(6, base=77.0, factor=2.0), kv_from=1)], width=29, vocab=53, eps=1e-3,
                                 embed_scale=7.0),
    # sizes the matrix-core kernels take, prompts longer than a chunk of the scan and than a window
    "wide": lambda: R.make_config([R.lightning_layer(heads=4, dim=32, vdim=64, mlp=R.dense_mlp(256)),
                                   R.attention_layer(heads=8, kv_heads=2, dim=40, vdim=48, window=50, rot=R.rot_of(40), mlp=R.moe_mlp(8, 3, 64, 1.0)),
                                   R.latent_layer(heads=4, dim=32, rot_dim=16, vdim=32, q_rank=96, kv_rank=64, rot=R.rot_of(16), mlp=R.dense_mlp(136)),
                                   R.attention_layer(heads=4, kv_heads=2, dim=40, vdim=48, window=33, rot=R.rot_of(40), kv_from=1)], width=128, vocab=97),
    # sizes that are 1
    "ones": lambda: R.make_config([R.lightning_layer(heads=1, dim=1, vdim=1, decay=[0.8], mlp=R.moe_mlp(1, 1, 1, 1.0)),
                                   R.attention_layer(heads=1, kv_heads=1, dim=2, vdim=1, window=1, rot=R.rot_of(2), mlp=R.dense_mlp(1)),
                                   R.latent_layer(heads=1, dim=1, rot_dim=2, vdim=1, q_rank=1, kv_rank=1, rot=R.rot_of(2), mlp=None)], width=3, vocab=5, embed_scale=1.0, eps=0.05),
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
    lim = limits(P, cfg, toks, want, dtype)
    ok = torch.isfinite(lim)
    assert float(ok.double().mean()) > 0.4 and float(lim[ok].median()) < 0.2
    assert trail.shape[0] == layers.shape[0] == len(cfg["layers"])
    for i in range(layers.shape[0]):
        assert rel(trail[i].cpu()[ok], layers[i][ok]) < (TOL[dtype] if dtype == F32 else 4e-2), i
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
def test_long_decoding_across_pages_windows_and_chunks(dtype):
    cfg = CONFIGS["mixed"]()
    model, cache, P = build(cfg, 14, dtype, page_size=8)
    toks = tokens_of(cfg, 9 + 150, 3)
    want = R.forward(P, cfg, toks)
    assert held(steps(engine_of(model, cache), "a", toks, [9] + [1] * 150), want, limits(P, cfg, toks, want, dtype, draws=2)) < 1


@pytest.mark.parametrize("kind", ["attention", "shared", "latent", "lightning"])
def test_which_changed_token_reaches_the_last_logits(kind):
    """A change of ONE token must move the last logits exactly when the statement says so: for a window attention one just inside its window
    and none outside — also through a layer that shares the keys under a wider window —, for the others any, the first included; the last
    tokens decoded one by one."""
    win = 11
    layers = {"attention": [R.attention_layer(window=win)], "latent": [R.latent_layer()], "lightning": [R.lightning_layer(decay=[1.0, 0.99, 0.98])],
              "shared": [R.attention_layer(window=1), R.attention_layer(window=win, kv_from=0)]}[kind]
    cfg = R.make_config([dict(L, mlp=None) for L in layers])
    model, cache, Pd = build(cfg, 15, F32, page_size=8)
    eng = engine_of(model, cache)
    T = 90
    base = tokens_of(cfg, T, 1)
    ref0, got0 = R.forward(Pd, cfg, base)[-1], steps(eng, "a", base, [T - 2, 1, 1])[-1].double().cpu()
    for pos in (0, 1, 7, 8, 63, 64, T - win - 1, T - win, T - win + 1, T - 3, T - 2):
        alt = list(base)
        alt[pos] = (alt[pos] + 1) % cfg["vocab"]
        dref = R.forward(Pd, cfg, alt)[-1] - ref0
        seen = kind in ("latent", "lightning") or T - 1 - pos < win
        assert (float(dref.abs().max()) > 1e-6) == seen, pos
        for cut in ([T], [T - 2, 1, 1], [T - 20, 2, 18]):
            dgot = steps(eng, "b", alt, cut)[-1].double().cpu() - got0
            assert rel(dgot, dref) < 5e-2 or float((dgot - dref).abs().max()) < 2e-5, (pos, cut)


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
    from ktransformers_amd.models.modeling_beronex import beronex_layer_specs
    from ktransformers_amd.util.generate import prefill_and_generate
    cfg = CONFIGS["mixed"]()
    model, cache, P = build(cfg, 16, dtype, page_size=16)
    prompts = {"p": tokens_of(cfg, 19, 7), "q": tokens_of(cfg, 5, 8)}
    n_new = 12

    def follows(prompt, new):       # teacher-forced on the framework's own tokens: the argmax wherever its margin (and the routing) is clear
        lg, gaps = R.forward(P, cfg, prompt + new, return_gaps=True)
        for k, tok in enumerate(new):
            at = len(prompt) - 1 + k
            top2 = lg[at].topk(2).values
            if float(top2[0] - top2[1]) > (1e-3 if dtype == F32 else 0.3) and (dtype == F32 or float(gaps[at]) > CLOSE_CALL):
                assert tok == int(lg[at].argmax()), k

    out = engine_of(model, cache).generate(prompts, max_new_tokens=n_new)
    for rid, prompt in prompts.items():
        assert len(out[rid]) == n_new
        follows(prompt, out[rid])
    for use_graph in (False, True):
        c1 = KHybridCache(beronex_layer_specs(model.config), 256, max_requests=1, page_size=16, dtype=dtype, device=DEV)
        ids = torch.tensor([prompts["p"]], dtype=torch.int64, device=DEV)
        toks = prefill_and_generate(model, ids, c1, max_new_tokens=n_new, use_cuda_graph=use_graph, chunk_size=8).tolist()
        if dtype == F32:
            assert toks == out["p"], (use_graph, toks, out["p"])
        else:
            follows(prompts["p"], toks)


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
