"""The Tirizen engine against the plain implementation (GPU): whole prompts, prefill against token-by-token decoding,
portions of several sizes down to two tokens, unequal batches against each request alone, slots and pages that are used
again, long decoding, the first tokens of a sequence, the residual streams after every layer, and greedy generation
through the package's own entry point, scheduler, replay program and command line."""
import json
import os
import subprocess
import sys

import pytest
import torch

import plain_tirizen as plain
import schedules
import tiny
import tiny_tirizen as tt

pytestmark = pytest.mark.gpu

# pages of 64; temperatures that grow every 1, 20, 33 and 64 tokens
LENS = {"a": 13, "b": 171, "c": 85, "d": 41, "e": 1, "f": 2}
PROMPT = {"a": 5, "b": 130, "c": 64, "d": 39, "e": 1, "f": 1}
BATCHES = [("a", "b", "c"), ("d", "e", "f"), ("c", "a"), ("f", "b", "d")]
CONFIGS = (("A", tt.tiny_a, 501), ("B", tt.tiny_b, 503), ("C", tt.tiny_c, 509), ("D", tt.tiny_d, 521))
NAMES = [c[0] for c in CONFIGS]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, raw, seed in CONFIGS:
        raw = raw()
        d = str(tmp_path_factory.mktemp(f"tirizen_{name}"))
        tt.write_model(raw, d, seed)
        cfg, w = read(d)
        reqs = {r: tiny.random_tokens(n, raw["vocab"], 5700 + i) for i, (r, n) in enumerate(LENS.items())}
        out[name] = (d, cfg, w, reqs, {r: Reference(cfg, w, t, conditioning=True) for r, t in reqs.items()})
    return out


def read(d):
    cfg, w = tiny.read_model(d)
    return tt.with_defaults(cfg), w


def deviation(got, ref):
    """A position's deviation as the bfloat16 checks measure it: root mean square of the logits' difference (its mean
    taken off) against the spread of the request's logits."""
    d = got - ref
    return (d - d.mean(1, keepdim=True)).pow(2).mean(1).sqrt() / ref.std()


CLOSE_CALL = 0.15       # bfloat16's rounding of a router's input moves a logit of a few units by a few hundredths


class Reference:
    """The plain implementation's logits of a request, which of its positions chose their experts by a margin that
    bfloat16's rounding can overturn, and (``conditioning``) how far every position's logits move, in float64, when every
    matrix is disturbed by relative noise of bfloat16's size (2^-9); a margin that this noise moves by a quarter of itself is
    a close call as well."""

    def __init__(self, cfg, w, tokens, conditioning=False):
        margins = []
        self.logits = plain.forward(cfg, w, tokens, margins=margins).float()
        self.close = torch.zeros(len(tokens), dtype=torch.bool)
        for m in margins:
            self.close |= m < CLOSE_CALL
        self.moved = torch.zeros(len(tokens))
        if conditioning:
            for seed in (1, 2, 3):
                g = torch.Generator().manual_seed(seed)
                noisy = {k: w[k].double() * (1 + torch.randn(w[k].shape, generator=g, dtype=torch.float64) * 2.0 ** -9)
                         if w[k].dim() == 2 else w[k] for k in sorted(w)}
                disturbed = []
                moved = deviation(plain.forward(cfg, noisy, tokens, margins=disturbed).float(), self.logits)
                self.moved = torch.maximum(self.moved, moved)
                for m, d in zip(margins, disturbed):
                    self.close |= m < 4.0 * (m - d).abs()

    def rows(self, rows):
        out = Reference.__new__(Reference)
        out.logits, out.close, out.moved = self.logits[rows], self.close[rows], self.moved[rows]
        return out


_engines = {}


def engine_for(models, name, dtype, **kw):
    from cpmcu_amd import Engine, EngineOptions
    key = (name, dtype, tuple(sorted(kw.items())))
    if key not in _engines:
        opts = dict(dtype=dtype, max_tokens=1024, max_slots=3, max_seq_len=256)
        opts.update(kw)
        _engines[key] = Engine.from_dir(models[name][0], EngineOptions(**opts))
    return _engines[key]


def check(got, refs, dtype, what):
    """float32 (the sharp comparison): rounding of float sums, at every position.  bfloat16: a position's deviation is
    0.08 at most (plus six times what noise of bfloat16's size does to it in float64) and 0.04 in the median.  A
    position whose choice of experts was a close call may have gone to other experts and is not held to a bound; one
    position in fifty (or one) behind such a position, which reads its keys, values and state, is held to 0.5 only."""
    for r, ref in refs.items():
        if dtype == "float32":
            err = (got[r] - ref.logits).abs().max(dim=1).values
            bad = (err > 2e-4 * max(1.0, float(ref.logits.abs().max()))).nonzero().flatten()
            assert bad.numel() == 0, (f"{what}: request {r}: first wrong position {int(bad[0])} of {ref.logits.shape[0]} "
                                      f"(error {float(err[bad[0]]):.3g})")
            continue
        err, close, moved = deviation(got[r], ref.logits), ref.close, ref.moved
        over = ((err > 0.08 + 6.0 * moved) & ~close).nonzero().flatten()
        n = err.numel()
        allowed = max(1, n // 50) if (bool(close.any()) and over.numel() and int(over[0]) > int(close.nonzero()[0])) else 0
        clear = (err - 6.0 * moved)[~close]
        assert over.numel() <= allowed and (clear.numel() == 0 or float(clear.max()) <= 0.5) and float(err.median()) <= 0.04 + float(moved.median()), \
            (f"{what}: request {r}: {over.numel()} of {n} positions over 0.08 whose choice of experts was clear (first "
             f"{int(over[0]) if over.numel() else -1}, worst {float(err.max()):.3g}, median {float(err.median()):.3g}, "
             f"moved {float(moved.median()):.3g}; close calls at {close.nonzero().flatten().tolist()[:12]})")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(models, name, dtype):
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, dtype)
    check(schedules.whole(eng, reqs), refs, dtype, "whole")
    eng.cache.check()
    assert not eng.cache.live


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_prefill_then_token_by_token(models, name, dtype):
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, dtype)
    check(schedules.tail(eng, reqs, 45), refs, dtype, "tail-45")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_unequal_batches_and_slots_used_again(models, name, dtype):
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, dtype)
    for part in (BATCHES[:2], BATCHES[2:]):
        used = {r for b in part for r in b}
        got = schedules.batched(eng, {r: reqs[r] for r in used}, PROMPT, part)
        check(got, {r: refs[r] for r in used}, dtype, "batched")
    eng.cache.check()
    assert not eng.cache.live


@pytest.mark.parametrize("step", [2, 7, 33, 64])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_portions(models, name, dtype, step):
    """Forward passes of at most `step` tokens: a prompt is cut into portions, and a batch's sequences are split across
    passes (some of which then bring one token a sequence)."""
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, dtype, max_step_tokens=step)
    some = {r: reqs[r] for r in ("b", "d", "f")}
    check(schedules.whole(eng, some), {r: refs[r] for r in some}, dtype, f"portions of {step}")
    got = schedules.batched(eng, {r: reqs[r] for r in ("c", "a", "d")}, PROMPT, [("c", "a", "d")])
    check(got, {r: refs[r] for r in ("c", "a", "d")}, dtype, f"batch in portions of {step}")
    eng.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_long_decoding_from_the_first_token(models, name, dtype):
    """One token, then 170 more one by one (captured graphs), over two page edges and every step of the temperatures; the
    recurrent state is carried all the way."""
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, dtype, hip_graph=True)
    got = schedules.tail(eng, {"b": reqs["b"]}, len(reqs["b"]) - 1)
    check(got, {"b": refs["b"]}, dtype, "decoding from the first token")
    eng.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_steps_equal_eager_steps(models, dtype):
    """A captured decode step, replayed with other steps and prompts of the engine between the replays, gives what the
    eager step gives."""
    from cpmcu_amd import StepEntry
    _, cfg, w, reqs, refs = models["A"]
    eager, graph = engine_for(models, "A", dtype), engine_for(models, "A", dtype, hip_graph=True)
    slots = [(e.acquire(), e.acquire()) for e in (eager, graph)]
    for e, (s, t) in zip((eager, graph), slots):
        e.step([StepEntry(s, reqs["c"][:30], []), StepEntry(t, reqs["a"][:5], [])])
    for i in range(8):
        out = [e.step([StepEntry(s, [reqs["c"][30 + i]], [0]), StepEntry(t, [reqs["a"][5 + i]], [0])]).cpu()
               for e, (s, t) in zip((eager, graph), slots)]
        assert torch.equal(out[0], out[1]), f"replay {i}"
        extra = graph.acquire()
        graph.step([StepEntry(extra, reqs["d"][:3 + i], [])])
        graph.release(extra)
    for e, st in zip((eager, graph), slots):
        for s in st:
            e.release(s)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C"])
def test_a_request_does_not_depend_on_its_neighbours_or_its_pages(models, name, dtype):
    from cpmcu_amd import StepEntry
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, dtype)
    alone = schedules.whole(eng, {"c": reqs["c"]})["c"]
    s = [eng.acquire() for _ in range(3)]
    lg = eng.step([StepEntry(s[0], reqs["b"], []), StepEntry(s[1], reqs["c"], list(range(LENS["c"]))),
                   StepEntry(s[2], reqs["a"], [0])]).cpu()
    for x in (s[1], s[0], s[2]):
        eng.release(x)
    again = schedules.whole(eng, {"c": reqs["c"]})["c"]
    assert torch.equal(again, alone)
    if dtype == "float32":
        assert float((lg[:LENS["c"]] - alone).abs().max()) <= 5e-5 * max(1.0, float(alone.abs().max()))
    else:
        ref = refs["c"].rows(slice(None))
        ref.logits = alone
        check({"c": lg[:LENS["c"]]}, {"c": ref}, dtype, "in a batch against alone")


@pytest.mark.parametrize("name", ["A", "C"])
def test_a_freed_slot_starts_from_nothing(models, name):
    """float32: a slot that held a long request is given to a short one: its recurrent state starts at zero again, so the
    logits equal those before to the bit."""
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, "float32", max_slots=1)
    first = schedules.tail(eng, {"d": reqs["d"]}, 10)["d"]
    schedules.tail(eng, {"b": reqs["b"]}, 3)
    assert torch.equal(schedules.tail(eng, {"d": reqs["d"]}, 10)["d"], first)
    check({"d": first}, {"d": refs["d"]}, "float32", "one slot")


@pytest.mark.parametrize("name", NAMES)
def test_residual_streams_after_every_layer(models, name):
    """float32: the sum of the streams after every layer equals the plain implementation's.  A layer leaves its last
    result pending, so the streams are put together here from what the block left."""
    from cpmcu_amd import StepEntry
    _, cfg, w, reqs, refs = models[name]
    eng = engine_for(models, name, "float32")
    _, res = plain.forward(cfg, w, reqs["d"], return_layers=True)
    seen = []
    blocks = eng.model.layers
    originals = [b.forward for b in blocks]

    def spy(i):
        def f(stream, ctx, cache, writes_cache=True):
            originals[i](stream, ctx, cache, writes_cache)
            p = stream.take_pending()
            y, bias = p.pieces()
            y = y.double().sum(0) if y.dim() == 3 else y.double()
            assert bias is None
            seen.append(plain.join_streams(stream.x.double(), y, p.mix.double(), p.out.double(), p.scale).sum(0).cpu())
        return f
    try:
        for i, b in enumerate(blocks):
            b.forward = spy(i)
        s = eng.acquire()
        eng.step([StepEntry(s, reqs["d"], [0])])
        eng.release(s)
    finally:
        for b, o in zip(blocks, originals):
            b.forward = o
    assert len(seen) == len(res) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(seen, res)):
        err = float((a - b).abs().max())
        assert err < 2e-5 * max(1.0, float(b.abs().max())), f"residual after layer {i}: {err:.3g}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rank", [1, 5, 48])
def test_ranks_come_from_the_checkpoint(models, tmp_path, dtype, rank):
    """No configuration key holds the rank of a decay's product; a stored second norm of a layer without a feed-forward is
    read past."""
    from cpmcu_amd import Engine, EngineOptions
    from safetensors.torch import save_file
    _, cfg, w, reqs, _ = models["D"]
    g = torch.Generator().manual_seed(rank)
    w = dict(w)
    w["l1.mix.a1"] = (torch.randn(rank, 48, generator=g) * 0.3).bfloat16()
    w["l1.mix.a2"] = (torch.randn(32, rank, generator=g) * 0.3).bfloat16()
    w["l1.norm2"] = w["l1.norm1"].clone()
    with open(tmp_path / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    eng = Engine.from_dir(str(tmp_path), EngineOptions(dtype=dtype, max_tokens=512, max_slots=2))
    some = {r: reqs[r] for r in ("c", "f")}
    check(schedules.tail(eng, some, 20), {r: Reference(cfg, w, t, conditioning=True) for r, t in some.items()}, dtype, f"rank {rank}")
    from cpmcu_amd.weights.loader import load_tensors
    given = load_tensors(str(tmp_path), eng.model.all_weight_specs(), ignore=lambda n: n == "l1.norm2")
    again = Engine.from_tensors(eng.config, given, EngineOptions(dtype=dtype, max_tokens=512, max_slots=2))
    assert again.model.layers[1].mixer.rank == rank


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kinds", ["g", "a", "gg", "aa"])
def test_models_of_one_kind_of_layer(tmp_path, dtype, kinds):
    """No layer with pages, or none with a state; in the last one the second layer has no keys of its own and no layer a
    feed-forward."""
    from cpmcu_amd import Engine, EngineOptions
    raw = dict(tt.tiny_d(), streams=4, residual_mult=0.5)
    att = {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 12, "scale": 0.3, "q_temp": {"coef": 0.5, "every": 16}}
    layers = [{"type": "gla", "mixer": {"heads": 3, "dim": 24, "vdim": 20, "tau": 6.0}, "mlp": {"kind": "dense", "ff": 56}} if k == "g"
              else {"type": "attention", "mixer": dict(att, **({"kv_from": 0} if i else {})), "mlp": None} for i, k in enumerate(kinds)]
    raw["layers"] = layers
    d = str(tmp_path / "m")
    tt.write_model(raw, d, 541)
    cfg, w = read(d)
    reqs = {"a": tiny.random_tokens(140, raw["vocab"], 6200), "b": tiny.random_tokens(66, raw["vocab"], 6201), "c": tiny.random_tokens(1, raw["vocab"], 6202)}
    refs = {r: Reference(cfg, w, t, conditioning=True) for r, t in reqs.items()}
    eng = Engine.from_dir(d, EngineOptions(dtype=dtype, max_tokens=512, max_slots=3, hip_graph=True))
    assert eng.cache.has_state == ("g" in kinds)
    check(schedules.tail(eng, reqs, 70), refs, dtype, kinds)
    check(schedules.batched(eng, reqs, {"a": 100, "b": 60, "c": 1}, [("b", "a", "c")]), refs, dtype, kinds + " batched")
    eng.cache.check()
    assert not eng.cache.live


def test_sequences_longer_than_the_position_table_are_refused(models):
    from cpmcu_amd import Engine, EngineOptions, StepEntry
    d, cfg, w, reqs, _ = models["D"]
    with pytest.raises(ValueError, match="positions"):
        Engine.from_dir(d, EngineOptions(dtype="float32", max_tokens=512, max_seq_len=257))
    eng = Engine.from_dir(d, EngineOptions(dtype="float32", max_tokens=512, max_slots=2))
    s = eng.acquire()
    with pytest.raises(ValueError, match="longest"):
        eng.step([StepEntry(s, [1] * 257, [])])
    toks = tiny.random_tokens(256, cfg["vocab"], 5800)
    got = eng.step([StepEntry(s, toks, list(range(256)))]).cpu()
    eng.release(s)
    check({"full": got}, {"full": Reference(cfg, w, toks)}, "float32", "the whole table")


def _greedy(cfg, w, prompt, n):
    toks = list(prompt)
    out = []
    for _ in range(n):
        nxt = int(plain.forward(cfg, w, toks)[-1].argmax())
        out.append(nxt)
        toks.append(nxt)
    return out


def test_greedy_generation_through_the_entry_point(models):
    from cpmcu_amd.llm import LLM
    d, cfg, w, reqs, refs = models["B"]
    prompt = reqs["a"][:9]
    want = _greedy(cfg, w, prompt, 20)
    llm = LLM(d, dtype="float32", max_tokens=256)
    llm.init_storage()
    llm.load_from_hf()
    tokens, _, _ = llm.generate(torch.tensor(prompt, dtype=torch.int32), 20)
    assert tokens == want


def test_generation_loop_with_unequal_requests(models):
    """The scheduler's own loop: several prompts of unequal length in batches, greedy, against the plain
    implementation's tokens (float32); three slots, so slots and pages are used again."""
    from cpmcu_amd.engine.generate import generate
    d, cfg, w, reqs, refs = models["A"]
    eng = engine_for(models, "A", "float32", hip_graph=True)
    prompts = [reqs["a"][:7], reqs["c"][:50], reqs["d"][:3], reqs["b"][:90]]
    out = generate(eng, prompts, 12)
    for p, o in zip(prompts, out):
        assert list(o.tokens) == _greedy(cfg, w, p, 12)
    eng.cache.check()
    assert not eng.cache.live


def test_replay_program_with_a_tight_token_budget(models, tmp_path):
    """bin/trace_run as a user runs it (float32): an unequal batch, then decoding together with early leavers, with
    --max-tokens the bare sum of the requests' tokens; then a request that takes freed slots and pages."""
    import numpy as np
    d, cfg, w, reqs, refs = models["A"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    names = ["b", "c", "a", "f"]
    prompt = {"b": 160, "c": 66, "a": 2, "f": 1}
    steps = [{"step": 0, "entries": [{"id": r, "tokens": reqs[r][:prompt[r]], "want": [0, prompt[r] - 1]} for r in names],
              "end": []}]
    fed = dict(prompt)
    n = 1
    while any(fed[r] < LENS[r] for r in names):
        live = [r for r in names if fed[r] < LENS[r]]
        steps.append({"step": n, "entries": [{"id": r, "tokens": [reqs[r][fed[r]]], "want": [0]} for r in live],
                      "end": [r for r in live if fed[r] + 1 == LENS[r]]})
        for r in live:
            fed[r] += 1
        n += 1
    steps.append({"step": n, "entries": [{"id": "again", "tokens": reqs["d"], "want": [LENS["d"] - 1]}], "end": ["again"]})
    out = tmp_path / "out"
    budget = sum(LENS[r] for r in names)
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d, "--dtype", "float32",
                           "--out", str(out), "--max-tokens", str(budget)],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.split("\n") if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    V = cfg["vocab"]
    tol = lambda r: 2e-4 * max(1.0, float(refs[r].logits.abs().max()))
    at = dict(prompt)
    for s in steps[:-1]:
        rows, bound = [], 0.0
        for e in s["entries"]:
            base = 0 if s["step"] == 0 else at[e["id"]]
            rows += [refs[e["id"]].logits[base + wpos] for wpos in e["want"]]
            bound = max(bound, tol(e["id"]))
        if s["step"] > 0:
            for e in s["entries"]:
                at[e["id"]] += 1
        got = torch.from_numpy(np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(len(rows), V))
        assert float((got - torch.stack(rows)).abs().max()) < bound, f"step {s['step']}"
    got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(1, V))
    assert float((got[0] - refs["d"].logits[-1]).abs().max()) < tol("d")


def test_command_line(models, tmp_path):
    """The command line on a Tirizen folder (greedy tokens equal the plain implementation's, the timers name the kernel
    classes), and in random-weights mode from a config.json alone."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

    def run_cli(*args):
        env = dict(os.environ, PYTHONPATH=root)
        return subprocess.run([sys.executable, "-m", "cpmcu_amd.cli", *args], capture_output=True, text=True,
                              timeout=600, env=env)
    d, cfg, w, reqs, refs = models["A"]
    prompts = [reqs["a"][:6], reqs["c"][:45]]
    ids = tmp_path / "ids.txt"
    ids.write_text("\n".join(" ".join(map(str, p)) for p in prompts) + "\n")
    p = run_cli("--model-path", d, "--dtype", "float32", "--prompt-ids", str(ids), "--num-generate", "6",
                "--ignore-eos", "true", "--max-tokens", "512", "--use_stream", "false", "--perf")
    assert p.returncode == 0, p.stderr[-1500:]
    assert "prefill_linattn_prepare" in p.stdout and "decode_linattn_scan" in p.stdout and "decode_moe_route" in p.stdout
    lines = [l for l in p.stdout.splitlines() if l.startswith("[")]
    assert [[int(t) for t in l.split(") ")[1].split()] for l in lines] == [_greedy(cfg, w, pr, 6) for pr in prompts]
    cfgp = tmp_path / "config.json"
    cfgp.write_text(json.dumps(tt.tiny_b()))
    out = tmp_path / "model"
    p = run_cli("--random-weights", "--config", str(cfgp), "--seed", "3", "--model-path", str(out), "--prompt-lens", "70,5",
                "--num-generate", "3", "--max-tokens", "512")
    assert p.returncode == 0, p.stderr[-1500:]
    assert sorted(os.listdir(out)) == ["config.json", "model.safetensors"]
    assert len([l for l in p.stdout.splitlines() if l.startswith("[")]) == 2


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C"])
def test_a_long_sequence(models, name, dtype):
    """1,300 tokens (21 pages): the prompt in passes of 512 tokens (the recurrence in segments), then 40 tokens one by
    one; the attention still reads the first token."""
    from cpmcu_amd import StepEntry
    _, cfg, w, reqs, refs = models[name]
    toks = tiny.random_tokens(1300, cfg["vocab"], 5900)
    ref = Reference(cfg, w, toks, conditioning=True)
    eng = engine_for(models, name, dtype, max_tokens=2048, max_seq_len=1408, max_step_tokens=512)
    s = eng.acquire()
    want = list(range(0, 1260, 97)) + [1259]
    got = [eng.step([StepEntry(s, toks[:1260], want)]).cpu()]
    for i in range(1260, 1300):
        got.append(eng.step([StepEntry(s, toks[i:i + 1], [0])]).cpu())
    eng.release(s)
    check({"long": torch.cat(got)}, {"long": ref.rows(want + list(range(1260, 1300)))}, dtype, "a long sequence")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes_of_a_real_models_kind(dtype, tmp_path):
    """Width 1,024, heads of 128: a prompt of 330 tokens (the library's products, attention and experts on the matrix
    cores, the recurrence in segments), then 24 tokens one by one through captured graphs (strip and skinny products), and
    a batch of three unequal requests."""
    from cpmcu_amd import Engine, EngineOptions
    raw = tt.medium()
    d = str(tmp_path / "m")
    tt.write_model(raw, d, 533, std=0.03)
    cfg, w = read(d)
    reqs = {"a": tiny.random_tokens(354, raw["vocab"], 6100), "b": tiny.random_tokens(70, raw["vocab"], 6101),
            "c": tiny.random_tokens(9, raw["vocab"], 6102)}
    refs = {r: Reference(cfg, w, t, conditioning=(dtype == "bfloat16")) for r, t in reqs.items()}
    eng = Engine.from_dir(d, EngineOptions(dtype=dtype, max_tokens=1024, max_slots=3, max_seq_len=512, hip_graph=True))
    check(schedules.tail(eng, {"a": reqs["a"]}, 24), {"a": refs["a"]}, dtype, "prompt of 330, then 24 tokens")
    got = schedules.batched(eng, reqs, {"a": 300, "b": 66, "c": 2}, [("c", "a", "b")])
    check(got, refs, dtype, "batch of three")
    eng.cache.check()
    assert not eng.cache.live
