"""Host side of the Beronex family: the plain statement's own invariants (oracle/beronex_ref.py), the config reader, the registry entry,
rule injection, the rotation's frequencies and what the cache manager is asked to keep.  No GPU."""
import math
import os

import pytest
import torch

from oracle import beronex_ref as R

D64 = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, dtype=D64, generator=torch.Generator().manual_seed(seed))


def test_statement_rotation_layouts_and_amplitude():
    v = rnd(5, 2, 7, seed=4)
    plain = {"base": 100.0, "dims": 4, "scaling": None}
    for half in (False, True):
        r = R.rotate(v, plain, half)
        assert torch.equal(r[..., 4:], v[..., 4:]) and torch.allclose(r[0], v[0]) and torch.allclose(r.norm(dim=-1), v.norm(dim=-1))
        a, b = (0, 2) if half else (0, 1)       # position 1 turns the first pair by angle 1
        assert torch.allclose(r[1, :, a], v[1, :, a] * math.cos(1.0) - v[1, :, b] * math.sin(1.0))
    scaled = dict(plain, scaling={"factor": 4.0, "original": 64, "fast": 4.0, "slow": 1.0})
    amp = 0.1 * math.log(4.0) + 1.0
    assert torch.allclose(R.rotate(v, scaled, True)[0, :, :4], v[0, :, :4] * amp) and torch.equal(R.rotate(v, scaled, True)[..., 4:], v[..., 4:])
    assert torch.equal(R.rotate(v, None, True), v)


def test_statement_frequencies_keep_the_fast_pairs_and_divide_the_slow_ones():
    freq, amp = R.yarn(10000.0, 32, {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0})
    turns = [4096 * 10000.0 ** (-2.0 * i / 32) / (2 * math.pi) for i in range(16)]
    for i, f in enumerate(freq):
        f0 = 10000.0 ** (-2.0 * i / 32)
        assert f0 / 8 * (1 - 1e-12) <= f <= f0 * (1 + 1e-12)
        if turns[i] > 64:
            assert f == f0
        if turns[i] < 0.5:
            assert abs(f - f0 / 8) < 1e-15
    assert any(10000.0 ** (-2.0 * i / 32) / 8 < f * 0.999 < 10000.0 ** (-2.0 * i / 32) * 0.998 for i, f in enumerate(freq))


@pytest.mark.parametrize("base,dims,scaling", [(10000.0, 64, {"factor": 4.0, "original": 512, "fast": 32.0, "slow": 1.0}), (77.0, 6, {"factor": 2.0, "original": 20, "fast": 2.0, "slow": 2.0}),
                                               (1e6, 2, {"factor": 16.0, "original": 100, "fast": 1.0, "slow": 0.01}), (500.0, 10, None), (3.0, 8, {"factor": 9.0, "original": 7, "fast": 9.0, "slow": 0.5}),
                                               (1e4, 0, None)])
def test_products_frequencies_equal_the_statements(base, dims, scaling):
    from ktransformers_amd.operators.RoPE import turning_frequencies
    freq, amp = turning_frequencies(base, dims, scaling)
    want, wamp = R.yarn(base, dims, scaling) if dims else ([], 1.0)
    assert freq.dtype == D64 and freq.numel() == dims // 2 and abs(amp - wamp) < 1e-15
    assert all(abs(float(f) - w) <= 1e-14 * abs(w) for f, w in zip(freq, want))


def test_statement_scan_window_and_router():
    q, k, v = rnd(6, 3, seed=1), rnd(6, 3, seed=2), rnd(6, 4, seed=3)
    o = R.decayed_scan(q, k, v, 0.8)
    for t in range(6):
        want = sum((0.8 ** (t - i) * (q[t] * k[i]).sum()) * v[i] for i in range(t + 1))
        assert torch.allclose(o[t], want, atol=1e-12)
    q, k, v = rnd(9, 2, 3, seed=1), rnd(9, 1, 3, seed=2), rnd(9, 1, 4, seed=3)
    w1 = R.softmax_attention(q, k, v, 1.0, 1)
    assert torch.allclose(w1, v.expand(9, 2, 4))                    # a window of one token: its own value
    assert torch.allclose(R.softmax_attention(q, k, v, 1.0, 9), R.softmax_attention(q, k, v, 1.0)) and not torch.allclose(
        R.softmax_attention(q, k, v, 1.0, 8), R.softmax_attention(q, k, v, 1.0))
    idx, w = R.routed(torch.tensor([[0.0, 3.0, 1.0, 3.0]], dtype=D64), 2)
    assert idx.tolist() == [[1, 3]] and torch.allclose(w, torch.full((1, 2), 0.5, dtype=D64))
    assert torch.allclose(R.gelu_tanh(rnd(50)), torch.nn.functional.gelu(rnd(50), approximate="tanh"))
    P = {"e.gate": torch.eye(2, dtype=D64), "e.up": torch.eye(2, dtype=D64), "e.down": torch.eye(2, dtype=D64)}
    y = R.bounded_expert(P, "e.", 2.0, torch.tensor([[5.0, -5.0]], dtype=D64))      # the gate is bounded from above only
    s = lambda z: 1 / (1 + math.exp(-1.702 * z))
    assert torch.allclose(y, torch.tensor([[2 * s(2) * 3, -5 * s(-5) * -1]], dtype=D64))


def test_statement_is_causal_windowed_and_remembers():
    def moved(layers, pos):
        cfg = R.make_config([dict(L, mlp=None) for L in layers])
        P = R.as_double(R.random_checkpoint(cfg, 3))
        toks = torch.randint(0, cfg["vocab"], (24,), generator=torch.Generator().manual_seed(0)).tolist()
        alt = list(toks)
        alt[pos] = (alt[pos] + 1) % cfg["vocab"]
        return (R.forward(P, cfg, alt) - R.forward(P, cfg, toks)).abs().amax(dim=1)
    for L in (R.latent_layer(), R.lightning_layer(decay=[1.0, 0.9, 0.99])):
        d = moved([L], 5)
        assert float(d[:5].sum()) == 0.0 and bool((d[5:] > 0).all())
    d = moved([R.attention_layer(window=7)], 5)
    assert float(d[:5].sum()) == 0.0 and bool((d[5:12] > 0).all()) and float(d[12:].sum()) == 0.0
    d = moved([R.attention_layer(window=1), R.attention_layer(window=7, kv_from=0)], 5)      # shared keys, the layer's own window
    assert float(d[:5].sum()) == 0.0 and bool((d[5:12] > 0).all()) and float(d[12:].sum()) == 0.0


def test_config_reader_registry_and_cache_specs():
    from ktransformers_amd.models import MODEL_REGISTRY, architecture_of
    from ktransformers_amd.models.modeling_beronex import beronex_layer_specs, make_beronex_config

    def raw():
        return R.make_config([R.attention_layer(heads=6, kv_heads=3, dim=10, vdim=8), R.lightning_layer(heads=5, dim=7, vdim=9, mlp=R.moe_mlp()),
                              R.attention_layer(heads=3, kv_heads=3, dim=10, vdim=8, window=99, kv_from=0, mlp=None), R.latent_layer(kv_rank=11, rot_dim=8)],
                             width=24, eps=1e-3, embed_scale=2.5)
    cfg = make_beronex_config(raw(), torch.float32)
    assert (cfg.width, cfg.eps, cfg.embed_scale, cfg.num_hidden_layers) == (24, 1e-3, 2.5, 4) and cfg.compute_dtype == torch.float32
    assert beronex_layer_specs(cfg) == [{"kv": (3, 10, 8)}, {"decay": (5, 7, 9)}, {}, {"latent": 19}]
    assert architecture_of(raw()) == "Beronex" and torch.float32 in MODEL_REGISTRY["Beronex"].dtypes
    mix = lambda c, i: c["layers"][i]["mixer"]
    for breakit, match in ((lambda c: c["layers"][0].update(type="serial"), "layer type"),
                           (lambda c: mix(c, 0).update(kv_heads=4), "multiple"),
                           (lambda c: mix(c, 0)["rot"].update(dims=3), "even"),
                           (lambda c: mix(c, 0)["rot"].update(dims=12), "at most"),
                           (lambda c: mix(c, 3)["rot"].update(dims=10), "at most"),
                           (lambda c: mix(c, 1).update(decay=[0.5] * 4), "decay"),
                           (lambda c: mix(c, 1).update(decay=[1.5] * 5), "decay"),
                           (lambda c: mix(c, 2).update(kv_from=1), "kv_from"),
                           (lambda c: mix(c, 2).update(kv_from=2), "kv_from"),
                           (lambda c: mix(c, 2).update(vdim=9), "kv_from"),
                           (lambda c: mix(c, 2)["rot"].update(base=9.0), "kv_from"),
                           (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "top"),
                           (lambda c: c.update(architecture="Other"), "architecture"),
                           (lambda c: c["layers"][0].update(mlp={"kind": "wide"}), "feed-forward")):
        bad = raw()
        breakit(bad)
        with pytest.raises(ValueError, match=match):
            make_beronex_config(bad)


def test_rules_replace_every_arithmetic_leaf():
    from ktransformers_amd.models import RULES_DIR
    from ktransformers_amd.models.modeling_beronex import BeronexForCausalLM, make_beronex_config
    from ktransformers_amd.models.modeling_deepseek import _Leaf
    from ktransformers_amd.optimize.optimize import gen_optimize_config, inject, load_rules
    from ktransformers_amd.util.loader import DictLoader
    raw = R.make_config([R.attention_layer(window=9, mlp=R.moe_mlp(limit=1.25)), R.lightning_layer(mlp=None), R.latent_layer(), R.attention_layer(window=5, kv_from=0)])
    cfg = make_beronex_config(raw)
    with torch.device("meta"):
        model = BeronexForCausalLM(cfg)
    plan = {}
    gen_optimize_config(model, plan, load_rules(os.path.join(RULES_DIR, "Beronex.yaml")))
    inject(model, plan, cfg, DictLoader(R.random_checkpoint(raw, 0)))
    kinds = {n: type(m).__name__ for n, m in model.named_modules() if type(m).__name__.startswith("K")}
    assert kinds["l0.mix"] == kinds["l3.mix"] == "KWindowGQAttention" and kinds["l1.mix"] == "KLightningAttention" and kinds["l2.mix"] == "KLatentWindowAttention"
    assert kinds["l0.mlp"] == "KSoftmaxRoutedMoE" and kinds["l2.mlp"] == "KClampedGLUMLP" and model.l1.mlp is None and "l1.norm2" not in kinds
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l1.norm1b"} <= set(kinds)
    left = [n for n, m in model.named_modules() if isinstance(m, _Leaf)]
    assert all("orig_module" in n for n in left)          # every leaf that is left sits behind its operator
    a, s, lat = model.l0.mix, model.l3.mix, model.l2.mix
    assert (a.window, s.window, a.kv_from, s.kv_from, a.gated, a.gate_columns) == (9, 5, None, 0, "per_head", 4) and a.qk_norm and a.rot_scaling["factor"] == 6.0
    assert a.state_spec() == {"kv": (2, 12, 10)} and s.state_spec() == {} and s.in_weight_names() == [("qkv", 48), ("g", 4)]
    assert lat.state_spec() == {"latent": 28} and (lat.q_rank, lat.rot_half, lat.has_sink, lat.window) == (18, True, False, 0) and lat.rot_scaling["factor"] == 4.0
    assert model.l1.mix.state_spec() == {"decay": (3, 8, 12)} and len(model.l1.mix.decay) == 3
    assert model.l0.mlp.glu == (1.25, 1.702, 1.0) and model.l0.mlp.router_bias and model.l0.mlp.sum_eps == 0.0
    assert model.l2.mlp.activation == "gelu_tanh" and model.l2.mlp.limit is None and model.l2.mlp.up_shift == 0.0


def test_cache_manager_gives_a_sharing_layer_nothing_of_its_own():
    from ktransformers_amd.models.custom_cache import KHybridCache
    c = KHybridCache([{"kv": (2, 4, 6)}, {}, {"decay": (3, 5, 7)}, {"latent": 9}], max_tokens=64, max_requests=2, page_size=8, dtype=torch.bfloat16, device="cpu")
    assert c.k_caches[0].shape[1:] == (2, 4) and c.v_caches[0].shape[1:] == (2, 6) and c.k_caches[1] is None and c.v_caches[1] is None and c.S[1] is None
    assert c.S[2].shape == (2, 3, 5, 7) and c.lat_caches[3].shape[1] == 9 and len(c.state_tensors()) == 1
