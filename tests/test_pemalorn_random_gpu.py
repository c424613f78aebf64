"""Pemalorn models drawn at random (GPU): sizes, head counts, the order of the layers, the loop, windows, taps, ranks,
constants and seeds differ from draw to draw and from every tiny model of the other tests; each is stepped whole, with
a decoded tail and in an unequal batch by both engines against the plain implementation."""
import random

import pytest

import schedules
import tiny
import tiny_pemalorn as tp
from test_pemalorn_gpu import Reference, check

pytestmark = pytest.mark.gpu


def _mixer(rng, kind):
    scale = round(rng.uniform(0.05, 0.5), 3)
    base = rng.choice([50.0, 1000.0, 500000.0])
    if kind == "attention":
        kv, group, dim = rng.choice([1, 2, 3]), rng.choice([1, 2, 4, 17]), rng.choice([8, 16, 24, 32, 48, 64])
        return {"heads": kv * group, "kv_heads": kv, "dim": dim, "vdim": rng.choice([6, 8, 16, 24, 40, 64, 96]), "scale": scale,
                "rot": {"base": base, "dims": rng.choice([2, dim // 2 // 2 * 2, dim])}}
    rot = rng.choice([2, 4, 8, 16, 24])
    m = {"heads": rng.choice([1, 2, 3, 5, 16, 18]), "dim": rng.choice([8, 16, 24, 40]), "rot_dim": rot,
         "vdim": rng.choice([8, 16, 24, 40, 72]), "q_rank": rng.choice([8, 24, 33, 64]), "kv_rank": rng.choice([8, 16, 40, 64, 136]),
         "scale": scale, "rot": {"base": base, "dims": rot}}
    if rng.random() < 0.7:
        m["rot"]["scaling"] = {"factor": rng.choice([2.0, 4.0, 16.0]), "original": rng.choice([16, 64, 512]),
                               "fast": rng.choice([4.0, 32.0]), "slow": rng.choice([0.5, 1.0])}
    size = rng.choice([None, 1, 2, 5, 17, 63, 64, 65, 100])
    if size:
        m["mask"] = {"size": size}
    return m


def _mlp(rng):
    if rng.random() < 0.2:
        return None
    experts, identity = rng.choice([1, 2, 5, 8, 12]), rng.choice([0, 1, 3, 8])
    router = {"experts": experts, "top": rng.randint(1, min(experts + identity, 5))}
    if identity:
        router["identity"] = identity
    return {"kind": "moe", "expert": {"ff": rng.choice([8, 20, 32, 64])}, "router": router}


def draw(seed):
    rng = random.Random(seed)
    n = rng.randint(2, 4)
    raw = {"architecture": "Pemalorn", "vocab": rng.randint(50, 300), "width": rng.choice([64, 72, 96, 100, 128, 160]),
           "norm": {"eps": rng.choice([1e-5, 1e-6])}, "layers": [], "canon": {"taps": rng.choice([1, 2, 3, 4, 6])},
           "token_side": {"dim": rng.choice([1, 8, 13, 24, 40])}}
    for _ in range(n):
        kind = rng.choice(["attention", "latent_attention"])
        raw["layers"].append({"type": kind, "mixer": _mixer(rng, kind), "mlp": _mlp(rng)})
    if rng.random() < 0.8:
        a = rng.randrange(n)
        raw["loop"] = {"start": a, "stop": rng.randint(a + 1, n), "times": rng.choice([1, 2, 3])}
    return raw


@pytest.mark.parametrize("seed", [21, 22, 23, 24, 25, 26, 27, 28])
def test_a_drawn_model(seed, tmp_path):
    from cpmcu_amd import Engine, EngineOptions
    raw = draw(seed)
    d = str(tmp_path / "model")
    tp.write_model(raw, d, seed)
    cfg, w = tiny.read_model(d)
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
