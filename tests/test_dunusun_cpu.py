"""Host side of the Dunusun family: the plain statement's own invariants (oracle/dunusun_ref.py), the config reader, the registry entry,
rule injection and what the cache manager is asked to keep.  No GPU."""
import os

import pytest
import torch

from oracle import dunusun_ref as R

D64 = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, dtype=D64, generator=torch.Generator().manual_seed(seed))


def test_statement_convolution_and_rotation():
    u, w, b = rnd(7, 3, seed=1), rnd(3, 4, seed=2), rnd(3, seed=3)
    y = R.causal_conv(u, w, b)
    for t in range(7):
        for c in range(3):
            want = b[c] + sum(w[c, j] * (u[t - 3 + j, c] if t - 3 + j >= 0 else 0.0) for j in range(4))
            assert abs(float(y[t, c] - want)) < 1e-12
    assert torch.equal(R.causal_conv(u, torch.ones(3, 1, dtype=D64)), u)
    v = rnd(5, 2, 6, seed=4)
    r = R.rotate_pairs(v, torch.arange(5), 100.0, 4)
    assert torch.equal(r[..., 4:], v[..., 4:]) and torch.allclose(r[0], v[0])
    assert torch.allclose(r[..., :4].norm(dim=-1), v[..., :4].norm(dim=-1))
    # pairs are neighbours: entry 0 of position 1 mixes with entry 1 by angle 1
    assert torch.allclose(r[1, :, 0], v[1, :, 0] * torch.cos(torch.tensor(1.0, dtype=D64)) - v[1, :, 1] * torch.sin(torch.tensor(1.0, dtype=D64)))


def test_statement_scan_and_hyper_connections():
    q, k, v = rnd(6, 3, seed=1), rnd(6, 3, seed=2), rnd(6, 4, seed=3)
    a = torch.sigmoid(rnd(6, 3, seed=4))
    o = R.decayed_outer_scan(q, k, v, a)
    # closed form: o_t = sum_{i <= t} (q_t . prod_{i < j <= t} a_j . k_i) v_i
    for t in range(6):
        want = sum(((q[t] * a[i + 1:t + 1].prod(dim=0) * k[i]).sum()) * v[i] for i in range(t + 1))
        assert torch.allclose(o[t], want, atol=1e-12)
    X, y, mix, out = rnd(3, 2, 5, seed=5), rnd(2, 5, seed=6), rnd(3, 3, seed=7), rnd(3, seed=8)
    Z = R.hyper_write(X, y, mix, out)
    assert torch.allclose(Z, torch.einsum("stw,sj->jtw", X, mix) + out.view(3, 1, 1) * y)
    # one stream with weights 1 is the plain residual sum
    one = torch.ones(1, dtype=D64)
    assert torch.allclose(R.hyper_write(X[:1], y, one.view(1, 1), one)[0], X[0] + y) and torch.equal(R.hyper_read(X[:1], one), X[0])
    assert R.run_order(6, {"start": 1, "stop": 3, "times": 3}) == [0, 1, 2, 1, 2, 1, 2, 3, 4, 5] and R.run_order(2, None) == [0, 1]


@pytest.mark.parametrize("layer", [R.parallel_layer(), R.ssd_layer()])
def test_statement_is_causal_and_remembers(layer):
    """A position's logits depend on earlier tokens only, and on all of them (nothing is windowed)."""
    cfg = R.make_config([layer])
    P = R.as_double(R.random_checkpoint(cfg, 3))
    toks = torch.randint(0, cfg["vocab"], (24,), generator=torch.Generator().manual_seed(0)).tolist()
    base = R.forward(P, cfg, toks)
    for pos in (23, 10, 0):
        alt = list(toks)
        alt[pos] = (alt[pos] + 1) % cfg["vocab"]
        d = (R.forward(P, cfg, alt) - base).abs().amax(dim=1)
        assert float(d[:pos].sum()) == 0.0 and float(d[pos]) > 0 and float(d[-1]) > 0


def test_statement_soft_caps():
    assert float(R.soft_cap(torch.tensor(1e6, dtype=D64), 5.0)) == 5.0 and abs(float(R.soft_cap(torch.tensor(1e-3, dtype=D64), 5.0)) - 1e-3) < 1e-9
    z = rnd(4)
    assert R.soft_cap(z, None) is z
    cfg = R.make_config([R.ssd_layer()], logit_softcap=0.5)
    P = R.as_double(R.random_checkpoint(cfg, 1))
    assert float(R.forward(P, cfg, [1, 2, 3]).abs().max()) < 0.5


def test_config_reader_registry_and_cache_specs():
    from ktransformers_amd.models import MODEL_REGISTRY, architecture_of
    from ktransformers_amd.models.modeling_dunusun import dunusun_layer_specs, make_dunusun_config

    def raw():
        return R.make_config([R.parallel_layer(heads=6, kv_heads=3, dim=10, vdim=8, conv=4, r_heads=5, r_dim=7, r_vdim=9),
                              R.ssd_layer(heads=6, vdim=10, state=5, groups=3, conv=2, norm_groups=4),
                              R.parallel_layer(conv=1, rot_dims=0, softcap=None, mlp=None), R.ssd_layer(conv=1)],
                             width=24, eps=1e-3, streams=5, loop={"start": 1, "stop": 3, "times": 2})
    cfg = make_dunusun_config(raw(), torch.float32)
    assert (cfg.width, cfg.eps, cfg.streams, cfg.logit_softcap, cfg.num_hidden_layers) == (24, 1e-3, 5, 8.0, 4) and cfg.compute_dtype == torch.float32
    assert cfg.runs == [0, 1, 2, 1, 2, 3]
    specs = dunusun_layer_specs(cfg)
    assert specs[0] == {"kv": (3, 10, 8), "conv": (6 * 10 + 3 * 18, 4), "decay": (5, 7, 9)}
    assert specs[1] == specs[3] == {"decay": (6, 5, 10), "conv": (60 + 2 * 3 * 5, 2)} and specs[2] == specs[4]
    assert specs[5]["conv"][1] == 1 and len(specs) == 6
    assert architecture_of(raw()) == "Dunusun" and torch.float32 in MODEL_REGISTRY["Dunusun"].dtypes
    for breakit, match in ((lambda c: c["layers"][0].update(type="serial"), "layer type"),
                           (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "multiple"),
                           (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=3), "even"),
                           (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=12), "at most"),
                           (lambda c: c["layers"][1]["mixer"].update(groups=4), "groups"),
                           (lambda c: c["layers"][1]["mixer"].update(norm_groups=7), "norm_groups"),
                           (lambda c: c.update(loop={"start": 2, "stop": 5, "times": 1}), "loop"),
                           (lambda c: c.update(streams=0), "streams"),
                           (lambda c: c.update(architecture="Other"), "architecture"),
                           (lambda c: c["layers"][0].update(mlp={"kind": "moe"}), "feed-forward")):
        bad = raw()
        breakit(bad)
        with pytest.raises(ValueError, match=match):
            make_dunusun_config(bad)


def test_rules_replace_every_arithmetic_leaf():
    from ktransformers_amd.models import RULES_DIR
    from ktransformers_amd.models.modeling_deepseek import _Leaf
    from ktransformers_amd.models.modeling_dunusun import DunusunForCausalLM, make_dunusun_config
    from ktransformers_amd.optimize.optimize import gen_optimize_config, inject, load_rules
    from ktransformers_amd.util.loader import DictLoader
    raw = R.make_config([R.parallel_layer(), R.ssd_layer(mlp=None), R.parallel_layer(conv=1)])
    cfg = make_dunusun_config(raw)
    with torch.device("meta"):
        model = DunusunForCausalLM(cfg)
    plan = {}
    gen_optimize_config(model, plan, load_rules(os.path.join(RULES_DIR, "Dunusun.yaml")))
    inject(model, plan, cfg, DictLoader(R.random_checkpoint(raw, 0)))
    kinds = {n: type(m).__name__ for n, m in model.named_modules() if type(m).__name__.startswith("K")}
    assert kinds["l0.mix"] == kinds["l2.mix"] == "KScaledParallelMixer" and kinds["l1.mix"] == "KStateSpaceDualMixer"
    assert type(model.l0.mix.left).__name__ == "KWindowGQAttention" and type(model.l0.mix.right).__name__ == "KGatedLinearAttention"
    assert kinds["l0.mlp"] == "KDenseMLP" and model.l0.mlp.activation == "relu_sq" and model.l1.mlp is None and "l1.norm2" not in kinds
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.hc1", "l0.hc2", "l1.hc1"} <= set(kinds) and "l1.hc2" not in kinds
    left = [n for n, m in model.named_modules() if isinstance(m, _Leaf)]
    assert all("orig_module" in n for n in left)          # every leaf that is left sits behind its operator
    a = model.l0.mix.left
    assert a.softcap == 5.0 and a.gated and a.conv_taps == 3 and a.rot_dims == 8 and a.conv_form and a.window == 0
    assert a.state_spec() == {"kv": (2, 16, 24), "conv": (4 * 16 + 2 * 40, 3)} and model.l0.mix.right.state_spec() == {"decay": (3, 8, 12)}
    assert model.l1.mix.state_spec() == {"decay": (4, 8, 12), "conv": (48 + 32, 4)} and model.head.soft_cap == 8.0


def test_cache_manager_serves_decaying_states():
    from ktransformers_amd.models.custom_cache import KHybridCache
    c = KHybridCache([{"kv": (2, 4, 6), "conv": (20, 4), "decay": (3, 5, 7)}, {"decay": (2, 3, 4), "conv": (9, 1)}], max_tokens=64, max_requests=2,
                     page_size=8, dtype=torch.bfloat16, device="cpu")
    assert c.S[0].shape == (2, 3, 5, 7) and c.S[0].dtype == torch.float32 and c.S[1].shape == (2, 2, 3, 4) and c.conv[1] is None
    assert len(c.state_tensors()) == 3
    c.S[0].fill_(2.0)
    c.admit("a"), c.admit("b"), c.admit("x")          # more requests than slots: the states grow, the old ones keep their contents
    assert c.S[0].shape[0] == c.max_requests >= 3 and float(c.S[0][:2].min()) == 2.0
    with pytest.raises(ValueError, match="one recurrent state"):
        KHybridCache([{"decay": (1, 1, 1), "delta": (1, 1, 1)}], max_tokens=8, device="cpu")


def test_padded_rows_keeps_the_weights_and_adds_zero_rows():
    from ktransformers_amd.operators.linear import padded_rows
    a, b = rnd(3, 4), rnd(6, 4, seed=1)
    p = padded_rows([a, b])
    assert p.shape == (16, 4) and torch.equal(p[:3], a) and torch.equal(p[3:9], b) and float(p[9:].abs().max()) == 0.0
    assert padded_rows([rnd(8, 4)]).shape == (8, 4)
