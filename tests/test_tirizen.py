"""Tirizen without a GPU: configuration, defaults, refusals, tensor names, which run uses which cache entry; the plain
implementation pinned by closed forms and invariants, one mechanism at a time."""
import math

import pytest
import torch

import plain_tirizen as plain
import tiny_tirizen as tt

F64 = torch.float64


def _cfg(raw):
    import cpmcu_amd
    arch = cpmcu_amd.get_architecture(raw["architecture"])
    return arch, arch.config_class.from_dict(raw)


def _rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, dtype=F64, generator=torch.Generator().manual_seed(seed)) * scale


# ---------------------------------------------------------------------------
# configuration and model
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("raw", [tt.tiny_a(), tt.tiny_b(), tt.tiny_c(), tt.tiny_d(), tt.medium()])
def test_configuration_reads_back(raw):
    arch, cfg = _cfg(raw)
    assert arch.config_class.from_dict(cfg.to_dict()) == cfg
    assert arch.config_class.from_dict(tt.with_defaults(raw)) == cfg
    assert cfg.vocabulary_size == raw["vocab"] and len(cfg.layers) == len(raw["layers"])
    assert cfg.longest_sequence == raw["max_positions"]


def test_defaults_of_absent_keys():
    _, cfg = _cfg(tt.tiny_d())
    assert (cfg.streams, cfg.residual_mult, cfg.logit_scale, cfg.embedding_scale) == (1, 1.0, 1.0, 1.0)
    a, g = cfg.layers[0].mixer, cfg.layers[1].mixer
    assert a.kv_heads == a.heads == 2 and a.vdim == a.dim == 16 and a.temp is None and a.kv_from is None
    assert g.vdim == g.dim == 16 and cfg.layers[1].mlp is None


@pytest.mark.parametrize("change, word", [
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda r: r["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda r: r["layers"][0]["mixer"]["q_temp"].update(every=0), "every"),
    (lambda r: r["layers"][0]["mixer"].update(dim=0), "sizes"),
    (lambda r: r["layers"][1]["mixer"].pop("tau"), "tau"),
    (lambda r: r["layers"][1]["mixer"].update(tau=0), "tau"),
    (lambda r: r["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda r: r["layers"][2]["mixer"].update(kv_from=2), "kv_from"),
    (lambda r: r["layers"][2]["mixer"].update(kv_from=3), "kv_from"),
    (lambda r: r["layers"][4]["mixer"].update(kv_from=2), "kv_from"),
    (lambda r: r["layers"][2]["mixer"].update(kv_from=-1), "kv_from"),
    (lambda r: r["layers"][4]["mixer"].update(kv_from=0), "other sizes"),
    (lambda r: r["layers"][0]["mlp"]["router"].update(top=7), "top"),
    (lambda r: r["layers"][0]["mlp"].update(kind="gated"), "kind"),
    (lambda r: r["layers"][0]["mlp"].pop("expert"), "expert"),
    (lambda r: r["layers"][1]["mlp"].update(ff=0), "sizes"),
    (lambda r: r["layers"][0].update(type="mamba2"), "type"),
    (lambda r: r.update(streams=0), "streams"),
    (lambda r: r.update(max_positions=0), "max_positions"),
    (lambda r: r.pop("max_positions"), "max_positions"),
    (lambda r: r.update(layers=[]), "layers"),
    (lambda r: r.pop("norm"), "norm"),
])
def test_refusals(change, word):
    from cpmcu_amd import ConfigError
    raw = tt.tiny_a()
    change(raw)
    with pytest.raises(ConfigError, match=word):
        _cfg(raw)


def test_tensor_names_and_cache_needs():
    arch, cfg = _cfg(tt.tiny_a())
    model = arch.build_model(cfg, None, {"l1.mix.a1": (5, 96)})
    specs = {s.name: tuple(s.shape) for s in model.all_weight_specs()}
    assert specs["embed"] == (203, 96) and specs["pos"] == (1500, 96) and specs["final.norm"] == (96,) and "head" not in specs
    assert specs["l0.mix.q"] == (144, 96) and specs["l0.mix.k"] == (72, 96) and specs["l0.mix.v"] == (120, 96)
    assert specs["l0.mix.q.norm"] == (144,) and specs["l0.mix.k.norm"] == (72,) and specs["l0.mix.g"] == (6, 96)
    assert specs["l1.mix.a1"] == (5, 96) and specs["l1.mix.a2"] == (60, 5) and specs["l1.mix.a2.b"] == (60,)
    assert specs["l1.mix.norm"] == (36,) and specs["l1.mix.g"] == (108, 96) and specs["l1.mlp.up"] == (112, 96)
    assert sorted(n for n in specs if n.startswith("l2.mix.")) == ["l2.mix.g", "l2.mix.o", "l2.mix.q", "l2.mix.q.norm"]
    assert specs["l0.mlp.router"] == (6, 96) and specs["l0.mlp.router.b"] == (6,) and specs["l0.mlp.e5.up"] == (40, 96)
    assert "l0.mlp.e0.gate" not in specs and "l0.mlp.e6.up" not in specs
    assert specs["l0.hc2.mix"] == (3, 3) and specs["l3.hc1.in"] == (3,) and "l3.hc2.in" not in specs and "l3.norm2" not in specs
    # a layer that reads another's keys has no cache entry of its own
    assert cfg.layer_runs() == [(0, True), (1, True), (0, False), (2, True), (2, False)]
    needs = model.cache_needs()
    assert len(needs) == 3 and dict(needs[0].streams)["v"].width == 3 * 48 and dict(needs[2].streams)["k"].width == 32
    assert needs[1].streams == () and dict(needs[1].state)["memory"].shape == (3, 36, 20)
    assert arch.ignore_tensor(cfg, "l3.norm2") and arch.ignore_tensor(cfg, "l3.hc2.mix") and not arch.ignore_tensor(cfg, "l2.norm2")


def test_a_borrowing_mixer_has_nothing_to_write():
    from cpmcu_amd.parts import MIXERS
    kw = dict(hidden_size=16, num_heads=2, num_kv_heads=1, key_dim=8, value_dim=8, position=None, scale=1.0)
    names = {"q": "q", "q_norm": "qn", "out": "o"}
    with pytest.raises(ValueError, match="borrows"):
        MIXERS.build("attention", names=dict(names, k="k"), borrows=True, norm_rows=True, **kw)
    with pytest.raises(ValueError, match="whole"):
        MIXERS.build("attention", names=dict(names, k="k", v="v"), norm_rows=True, **kw)
    with pytest.raises(ValueError, match="whole"):
        MIXERS.build("attention", names=dict(names, k="k", v="v", k_norm="kn", temp="t"), norm_rows=True, **kw)
    with pytest.raises(ValueError, match="temperature"):
        MIXERS.build("attention", names={"q": "q", "k": "k", "v": "v", "out": "o"}, query_temp=(0.1, 0), **kw)
    m = MIXERS.build("attention", names=names, borrows=True, norm_rows=True, **kw)
    with pytest.raises(ValueError, match="write"):
        m.forward(torch.zeros(1, 16), None, None, True)


def test_feed_forwards_and_routers_refuse():
    from cpmcu_amd.parts import FEED_FORWARDS
    with pytest.raises(ValueError, match="clamped_swish"):
        FEED_FORWARDS.build("plain", up_name="u", down_name="d", hidden_size=8, intermediate_size=8, activation="clamped_swish")
    kw = dict(names={"router": "r", "expert": "{e}{part}"}, hidden_size=8, expert_size=8, experts=2, top=1)
    with pytest.raises(ValueError, match="normalised"):
        FEED_FORWARDS.build("routed_experts", score="logit", normalize=False, **kw)
    with pytest.raises(ValueError, match="relu_squared"):
        FEED_FORWARDS.build("routed_experts", activation="relu_squared", **kw)
    with pytest.raises(ValueError, match="shared"):
        FEED_FORWARDS.build("routed_experts", gated=False, activation="relu_squared", shared_size=8, **kw)


def test_cuts_of_a_long_walk():
    from cpmcu_amd import ops
    if not torch.cuda.is_available():
        ops_units = ops.compute_units
        ops.compute_units = lambda: 256
    try:
        assert ops.gla_segments([100], 4, 64) == (1, 0)
        for lens, heads, dv in (([2048], 16, 128), ([300, 2000, 5], 2, 32), ([129], 1, 16), ([700] * 9, 3, 40)):
            n, seg = ops.gla_segments(lens, heads, dv)
            assert n == 1 or (seg % ops.GLA_SEGMENT == 0 and n * seg >= max(lens) > (n - 1) * seg)
            assert len(lens) * n <= max(ops.gla_segment_rows(2048, heads, dv), len(lens))
        assert ops.gla_segments([2048], 16, 128)[0] > 4 and ops.gla_segments([2048] * 64, 16, 128) == (1, 0)
    finally:
        if not torch.cuda.is_available():
            ops.compute_units = ops_units


# ---------------------------------------------------------------------------
# the plain implementation
# ---------------------------------------------------------------------------
def test_plain_recurrence_is_a_decayed_sum():
    """o_t = sum_s (q_t . prod_{s < r <= t} a_r . k_s) v_s, the token's own write undecayed."""
    q, k, v = _rand(6, 2, 3, seed=1), _rand(6, 2, 3, seed=2), _rand(6, 2, 4, seed=3)
    a = torch.sigmoid(_rand(6, 2, 3, seed=4))
    got = plain.recurrence(q, k, v, a)
    for t in range(6):
        want = torch.zeros(2, 4, dtype=F64)
        for s in range(t + 1):
            w = torch.ones(2, 3, dtype=F64)
            for r in range(s + 1, t + 1):
                w = w * a[r]
            want += (q[t] * w * k[s]).sum(-1, keepdim=True) * v[s]
        assert torch.allclose(got[t], want)


def test_plain_decay_far_out():
    W = {"a1": torch.eye(1, dtype=F64), "a2": torch.ones(1, 1, dtype=F64), "a2.b": torch.zeros(1, dtype=F64)}
    z = torch.tensor([[-2000.0], [-30.0], [0.0], [40.0]], dtype=F64)
    a = plain.channel_decay(z, W, "", 16.0)
    assert bool(torch.isfinite(a).all()) and abs(float(a[1, 0]) - math.exp(-30.0 / 16)) < 1e-12
    assert abs(float(a[2, 0]) - 0.5 ** (1 / 16)) < 1e-12 and float(a[3, 0]) == pytest.approx(1.0, abs=1e-12)


def test_plain_temperature():
    t = plain.temperature(200, {"coef": 0.5, "every": 64})
    assert float(t[62]) == 1.0 and float(t[63]) == float(t[126]) == 1 + 0.5 * math.log(2.0) and float(t[127]) == 1 + 0.5 * math.log(3.0)
    assert torch.equal(plain.temperature(3, None), torch.ones(3, dtype=F64))


def test_plain_streams():
    X, y = _rand(3, 2, 4, seed=5), _rand(2, 4, seed=6)
    mix, out = _rand(3, 3, seed=7), _rand(3, seed=8)
    got = plain.join_streams(X, y, mix, out, 0.5)
    for t in range(3):
        assert torch.allclose(got[t], sum(mix[s, t] * X[s] for s in range(3)) + 0.5 * out[t] * y)


def test_plain_router_weighs_the_chosen_only():
    W = {"router": torch.eye(3, dtype=F64), "router.b": torch.tensor([0.0, 0.0, 4.0], dtype=F64)}
    idx, w = plain.route(torch.tensor([[2.0, 1.0, -1.0]], dtype=F64), W, "", 2)
    assert idx.tolist() == [[2, 0]] and torch.allclose(w, torch.softmax(torch.tensor([[3.0, 2.0]], dtype=F64), -1))


def test_plain_norm_is_over_the_whole_projection():
    """Keys of one head far larger than the other's: each head keeps its share of the row's root mean square."""
    W = {"k": torch.diag(torch.tensor([100.0, 100.0, 1.0, 1.0], dtype=F64)), "v": torch.eye(4, dtype=F64),
         "k.norm": torch.ones(4, dtype=F64)}
    k, v = plain.keys_and_values(torch.ones(1, 4, dtype=F64), W, "", {"kv_heads": 2, "dim": 2, "vdim": 2}, 0.0)
    assert float(k[0, 0, 0] / k[0, 1, 0]) == pytest.approx(100.0) and float((k ** 2).mean()) == pytest.approx(1.0)
    assert torch.equal(v.flatten(), torch.ones(4, dtype=F64))


@pytest.mark.parametrize("raw", [tt.tiny_a(), tt.tiny_b()])
def test_plain_model_is_causal(raw):
    from cpmcu_amd.weights import random_tensors
    w = random_tensors(_cfg(raw)[1], 5, 0.08, 0.1)
    raw = tt.with_defaults(raw)
    a, b = [3, 1, 4, 1, 5, 9, 2, 6], [3, 1, 4, 1, 5, 8, 7, 0]
    la, lb = plain.forward(raw, w, a), plain.forward(raw, w, b)
    assert torch.allclose(la[:5], lb[:5], atol=1e-10) and not torch.allclose(la[5], lb[5], atol=1e-3)
