"""Tirizen models drawn at random (GPU): sizes, head counts, the order of the layers, who reads whose keys, streams,
temperatures, decays, constants and seeds differ from draw to draw and from every tiny model of the other tests; each is
stepped whole, with a decoded tail and in an unequal batch by both engines against the plain implementation."""
import random

import pytest

import schedules
import tiny
import tiny_tirizen as tt
from test_tirizen_gpu import Reference, check, read

pytestmark = pytest.mark.gpu


def _mixer(rng, i, layers):
    if rng.random() < 0.45:
        return "gla", {"heads": rng.choice([1, 2, 3, 5]), "dim": rng.choice([8, 12, 20, 32, 40, 64, 96, 136]),
                       "vdim": rng.choice([6, 8, 16, 24, 40, 64, 96]), "tau": rng.choice([1.0, 2.5, 8.0, 16.0, 30.0])}
    owners = [j for j, l in enumerate(layers) if l["type"] == "attention" and "kv_from" not in l["mixer"]]
    scale = round(rng.uniform(0.05, 0.5), 3)
    if owners and rng.random() < 0.6:
        j = rng.choice(owners)
        m = dict(layers[j]["mixer"], scale=scale, kv_from=j)
        m.pop("q_temp", None)
    else:
        kv, group = rng.choice([1, 2, 3]), rng.choice([1, 2, 4, 17])
        m = {"heads": kv * group, "kv_heads": kv, "dim": rng.choice([8, 16, 20, 24, 32, 48, 64]),
             "vdim": rng.choice([6, 8, 16, 24, 40, 64, 96]), "scale": scale}
    if rng.random() < 0.8:
        m["q_temp"] = {"coef": round(rng.uniform(-0.2, 0.8), 2), "every": rng.choice([1, 7, 32, 64, 100])}
    return "attention", m


def _mlp(rng):
    r = rng.random()
    if r < 0.2:
        return None
    if r < 0.45:
        return {"kind": "dense", "ff": rng.choice([20, 64, 96, 200])}
    experts = rng.choice([1, 2, 5, 8, 24])
    return {"kind": "moe", "expert": {"ff": rng.choice([8, 20, 32, 64])}, "router": {"experts": experts, "top": rng.randint(1, min(experts, 5))}}


def draw(seed):
    rng = random.Random(seed)
    layers = []
    for i in range(rng.randint(3, 6)):
        kind, m = _mixer(rng, i, layers)
        layers.append({"type": kind, "mixer": m, "mlp": _mlp(rng)})
    return {"architecture": "Tirizen", "vocab": rng.randint(50, 300), "width": rng.choice([64, 72, 96, 100, 128, 160]),
            "norm": {"eps": rng.choice([1e-5, 1e-6])}, "embedding": {"scale": rng.choice([1.0, 6.0, 11.5])},
            "max_positions": rng.choice([256, 300, 1000]), "residual_mult": rng.choice([0.3, 0.75, 1.0]),
            "streams": rng.choice([1, 2, 3, 4, 6, 8]), "logit_scale": rng.choice([0.2, 1.0, 1.5]), "layers": layers}


@pytest.mark.parametrize("seed", [31, 32, 33, 34, 35, 36, 37, 38])
def test_a_drawn_model(seed, tmp_path):
    from cpmcu_amd import Engine, EngineOptions
    raw = draw(seed)
    d = str(tmp_path / "model")
    tt.write_model(raw, d, seed)
    cfg, w = read(d)
    reqs = {"a": tiny.random_tokens(150, raw["vocab"], seed), "b": tiny.random_tokens(37, raw["vocab"], seed + 100),
            "c": tiny.random_tokens(2, raw["vocab"], seed + 200)}
    refs = {r: Reference(cfg, w, t, conditioning=True) for r, t in reqs.items()}
    for dtype in ("float32", "bfloat16"):
        eng = Engine.from_dir(d, EngineOptions(dtype=dtype, max_tokens=512, max_slots=3, max_seq_len=256, hip_graph=True))
        check(schedules.whole(eng, reqs), refs, dtype, f"draw {seed} whole")
        check(schedules.tail(eng, {"a": reqs["a"]}, 110), {"a": refs["a"]}, dtype, f"draw {seed} tail")
        got = schedules.batched(eng, reqs, {"a": 70, "b": 36, "c": 1}, [("b", "a", "c")])
        check(got, refs, dtype, f"draw {seed} batched")
        eng.cache.check()
        assert not eng.cache.live
