"""Pemalorn without a GPU: configuration, defaults, refusals, tensor names, the order of the runs and what each asks of
the cache; the plain implementation pinned by closed forms and invariants, one mechanism at a time."""
import math

import pytest
import torch

import plain_pemalorn as plain
import tiny_pemalorn as tp

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
@pytest.mark.parametrize("raw", [tp.tiny_s(), tp.tiny_t(), tp.tiny_u(), tp.tiny_v(), tp.medium_n()])
def test_configuration_reads_back(raw):
    arch, cfg = _cfg(raw)
    assert arch.config_class.from_dict(cfg.to_dict()) == cfg
    assert cfg.vocabulary_size == raw["vocab"] and len(cfg.layers) == len(raw["layers"])


def test_defaults_of_absent_keys():
    _, cfg = _cfg(tp.tiny_v())
    assert cfg.taps == 0 and cfg.token_dim == 0 and cfg.loop is None
    assert cfg.layers[0].mixer.window is None and cfg.layers[0].mixer.rot.scaling is None and cfg.layers[1].mlp is None
    raw = tp.tiny_t()
    del raw["layers"][0]["mixer"]["kv_heads"], raw["layers"][0]["mixer"]["vdim"], raw["layers"][1]["mixer"]["rot"]["dims"]
    cfg = _cfg(raw)[1]
    m = cfg.layers[0].mixer
    assert m.kv_heads == m.heads == 3 and m.vdim == m.dim == 20 and m.rot.dims == 0
    assert cfg.layers[1].mixer.rot.dims == 4 and cfg.layers[0].mlp.identity == 0


@pytest.mark.parametrize("change, word", [
    (lambda r: r["layers"][1]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=7), "dims"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=26), "rot.dims"),
    (lambda r: r["layers"][1]["mixer"].update(vdim=13), "vdim"),
    (lambda r: r["layers"][1]["mixer"].pop("rot"), "rot"),
    (lambda r: r["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(scaling={"factor": 2.0, "original": 8, "fast": 2.0, "slow": 1.0}), "scaling"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=6), "rot_dim"),
    (lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "scaling"),
    (lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda r: r["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda r: r["layers"][0]["mlp"]["router"].update(top=10), "top"),
    (lambda r: r["layers"][0]["mlp"]["router"].update(identity=-1), "identity"),
    (lambda r: r["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda r: r["layers"][0]["mlp"].pop("expert"), "expert"),
    (lambda r: r["layers"][0].update(type="mamba2"), "type"),
    (lambda r: r["loop"].update(stop=6), "loop"),
    (lambda r: r["loop"].update(start=3), "loop"),
    (lambda r: r["loop"].update(times=0), "times"),
    (lambda r: r["canon"].update(taps=0), "taps"),
    (lambda r: r["token_side"].update(dim=0), "token_side"),
    (lambda r: r.update(layers=[]), "layers"),
    (lambda r: r.pop("norm"), "norm"),
])
def test_refusals(change, word):
    from cpmcu_amd import ConfigError
    raw = tp.tiny_s()
    change(raw)
    with pytest.raises(ConfigError, match=word):
        _cfg(raw)


def test_order_of_the_runs():
    runs = lambda raw: list(_cfg(raw)[1].layer_runs())
    assert runs(tp.tiny_s()) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None), (4, None)]
    assert runs(tp.tiny_t()) == [(0, None), (1, None), (2, 0)]
    assert runs(tp.tiny_u()) == [(0, t) if i == 0 else (i, None) for t in range(3) for i in range(3)]
    assert runs(tp.tiny_v()) == [(0, None), (1, None)]


def test_tensor_names_and_cache_needs():
    arch, cfg = _cfg(tp.tiny_s())
    model = arch.build_model(cfg)
    specs = {s.name: tuple(s.shape) for s in model.all_weight_specs()}
    assert specs["embed"] == (211, 96) and specs["side.embed"] == (211, 60) and specs["final.norm"] == (96,)
    assert specs["loop.in"] == (96, 192) and specs["loop.step"] == (2, 96)
    assert specs["l0.mix.dq"] == (48, 96) and specs["l0.mix.uq"] == (3 * 32, 48) and specs["l0.mix.dkv"] == (64, 96)
    assert specs["l0.mix.uk"] == (3 * 24, 56) and specs["l0.mix.uv"] == (3 * 40, 56) and specs["l0.mix.g"] == (120, 96)
    assert specs["l0.mix.dq.norm"] == (48,) and specs["l0.mix.dkv.norm"] == (56,) and specs["l0.mix.sink"] == (3,)
    assert specs["l0.mlp.router"] == (9, 96) and specs["l0.mlp.correction"] == (9,)
    assert specs["l0.mlp.e5.down"] == (96, 40) and "l0.mlp.e6.down" not in specs
    assert specs["l0.canon1"] == (96, 3) and specs["l0.canon2"] == (96, 3) and "l2.canon1" in specs and "l2.canon2" not in specs
    assert specs["l4.side.gate"] == (12, 96) and specs["l4.side.proj"] == (96, 12) and specs["l4.side.norm"] == (96,)
    assert specs["l1.mix.v"] == (2 * 40, 96) and specs["l1.mix.g"] == (6, 96) and specs["l1.mix.temp"] == (6,)
    assert not any(n.startswith("l2.mlp") for n in specs)
    needs = model.cache_needs()
    # a looped layer has an entry, convolution state included, for every pass
    assert len(needs) == 7 and needs[1] == needs[3] and needs[2] == needs[4]
    assert needs[0].window == 20 and needs[2].window == 70 and needs[1].window is None and needs[6].window is None
    assert all(dict(n.state)["input_conv"].shape == (2, 96) for n in needs)
    assert dict(needs[0].streams)["k"].width == 64 and dict(needs[1].streams)["v"].width == 2 * 48
    assert {r.begins_pass for r in model.schedule} == {None, 0, 1}
    plain_needs = _cfg(tp.tiny_v())[0].build_model(_cfg(tp.tiny_v())[1]).cache_needs()
    assert all(n.state == () for n in plain_needs)


def test_the_table_and_the_loop_are_the_models_own():
    arch, cfg = _cfg(tp.tiny_s())
    model = arch.build_model(cfg)
    names = [s.name for s in model.all_weight_specs()]
    assert names.count("side.embed") == 1 and names.count("loop.in") == 1
    assert [b.token_input.offset for b in model.layers] == [0, 12, 24, 36, 48]
    from cpmcu_amd.models import DecoderModel, Run
    with pytest.raises(ValueError, match="pass"):
        DecoderModel(cfg, model.embedding, model.layers, model.final_norm, model.head, [Run(0, 0, True, 0)])


# ---------------------------------------------------------------------------
# the plain implementation
# ---------------------------------------------------------------------------
def test_plain_rotated_values_depend_on_distance_only():
    """One key takes all the weight: a head's output is that key's value turned by the distance to the query, back."""
    v = _rand(9, 1, 6, seed=1)
    turned = plain.turn_values(v, 50.0, 1.0)
    back = lambda p: plain.turn(torch.stack([turned[2]] * 9), plain.frequencies({"dims": 6, "base": 50.0})[0], 1.0, "halves", -1.0)[p]
    assert torch.allclose(back(2), v[2])
    for d in (1, 4):
        ahead = plain.turn(torch.stack([v[2]] * 9), plain.frequencies({"dims": 6, "base": 50.0})[0], 1.0, "halves", -1.0)[d]
        assert torch.allclose(back(2 + d), ahead)


def test_plain_pairs_of_both_layouts():
    x = torch.zeros(3, 1, 6, dtype=F64)
    x[:, 0, 0] = 1.0
    f = torch.tensor([math.pi / 2, 0.1], dtype=F64)
    half, inter = plain.turn(x, f, 1.0, "halves"), plain.turn(x, f, 1.0, "interleaved")
    assert torch.allclose(half[1, 0], torch.tensor([0, 0, 1, 0, 0, 0], dtype=F64), atol=1e-12)
    assert torch.allclose(inter[1, 0], torch.tensor([0, 1, 0, 0, 0, 0], dtype=F64), atol=1e-12)
    assert torch.allclose(plain.turn(half, f, 1.0, "halves", -1.0), x)


def test_plain_stretch_limits():
    rot = {"dims": 32, "base": 10000.0, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    f, mag = plain.frequencies(rot)
    g, one = plain.frequencies({"dims": 32, "base": 10000.0})
    assert one == 1.0 and abs(mag - (0.1 * math.log(8.0) + 1)) < 1e-12
    assert abs(float(f[0] / g[0]) - 1) < 1e-12 and abs(float(f[-1] / g[-1]) - 1 / 8.0) < 1e-12
    assert bool((f[:-1] >= f[1:]).all())


def test_plain_sink_takes_its_share():
    s = torch.zeros(4, 4, dtype=F64)
    w = plain.sink_softmax(s, plain.visible(4), torch.tensor(math.log(3.0), dtype=F64))
    assert torch.allclose(w.sum(-1), torch.tensor([1 / 4, 2 / 5, 3 / 6, 4 / 7], dtype=F64))
    big = plain.sink_softmax(s, plain.visible(4), torch.tensor(800.0, dtype=F64))
    assert bool(torch.isfinite(big).all()) and float(big.max()) < 1e-300


def test_plain_window():
    m = plain.visible(6, 3)
    assert m.sum(-1).tolist() == [1, 2, 3, 3, 3, 3] and bool(m[5, 3]) and not bool(m[5, 2])
    assert torch.equal(plain.visible(5, 5), plain.visible(5))


def test_plain_convolution_sees_the_past_only():
    w = _rand(4, 3, seed=2)
    u = torch.zeros(6, 4, dtype=F64)
    u[2] = 1.0
    y = plain.causal_conv(u, w)
    assert torch.equal(y[:2], torch.zeros(2, 4, dtype=F64)) and torch.equal(y[5], torch.zeros(4, dtype=F64))
    assert torch.equal(y[2], w[:, 2]) and torch.equal(y[3], w[:, 1]) and torch.equal(y[4], w[:, 0])


def test_plain_identity_experts_give_the_input_back():
    W = {"router": torch.zeros(5, 4, dtype=F64), "correction": torch.tensor([-1.0, -1, 0.0, 0, 0], dtype=F64)}
    h = _rand(3, 4, seed=3)
    out = plain.experts(h, W, "", {"router": {"experts": 2, "identity": 3, "top": 3}})
    assert torch.allclose(out, h * 3 / 5)              # three of five equal scores, as they are
    idx, w = plain.route(h, W, "", {"top": 2})
    assert idx.tolist() == [[2, 3]] * 3 and torch.allclose(w, torch.full((3, 2), 0.2, dtype=F64))


def test_plain_correction_enters_the_choice_only():
    W = {"router": torch.eye(3, dtype=F64), "correction": torch.tensor([0.0, 0.0, 5.0], dtype=F64)}
    h = torch.tensor([[2.0, 1.0, 0.0]], dtype=F64)
    idx, w = plain.route(h, W, "", {"top": 2})
    s = torch.softmax(h, -1)
    assert idx.tolist() == [[2, 0]] and torch.allclose(w, s[:, [2, 0]])


def test_plain_latent_attention_equals_expanded_keys():
    """With one head and a sink that takes nothing the result is ordinary attention over keys [Wuk c | r]."""
    m = {"heads": 1, "dim": 4, "rot_dim": 2, "vdim": 3, "q_rank": 5, "kv_rank": 6, "scale": 0.7, "rot": {"base": 9.0, "dims": 2}}
    shapes = {"dq": (5, 8), "uq": (6, 5), "dkv": (8, 8), "uk": (4, 6), "uv": (3, 6), "g": (3, 8), "o": (8, 3)}
    W = {k: _rand(*s, seed=i) for i, (k, s) in enumerate(shapes.items())}
    W.update({"dq.norm": torch.ones(5, dtype=F64), "dkv.norm": torch.ones(6, dtype=F64), "sink": torch.tensor([-1e9], dtype=F64)})
    h = _rand(7, 8, seed=20)
    got = plain.latent_attention(h, W, "", m, 1e-6)
    c = plain.rms((h @ W["dkv"].T)[:, :6], 1e-6)
    k = torch.cat([c @ W["uk"].T, plain.rotate((h @ W["dkv"].T)[:, None, 6:], m["rot"], "interleaved")[:, 0]], 1)
    q = plain.rms(h @ W["dq"].T, 1e-6) @ W["uq"].T
    q = torch.cat([q[:, :4], plain.rotate(q[:, None, 4:], m["rot"], "interleaved")[:, 0]], 1)
    s = (q @ k.T * 0.7).masked_fill(~plain.visible(7), -math.inf)
    want = (torch.softmax(s, -1) @ (c @ W["uv"].T) * torch.sigmoid(h @ W["g"].T)) @ W["o"].T
    assert torch.allclose(got, want)


def test_plain_model_is_causal():
    raw = tp.tiny_s()
    from cpmcu_amd.weights import random_tensors
    w = random_tensors(_cfg(raw)[1], 5, 0.08, 0.1)
    a, b = [3, 1, 4, 1, 5, 9, 2, 6], [3, 1, 4, 1, 5, 8, 7, 0]
    la, lb = plain.forward(raw, w, a), plain.forward(raw, w, b)
    assert torch.allclose(la[:5], lb[:5], atol=1e-10) and not torch.allclose(la[5], lb[5], atol=1e-3)
