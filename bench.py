#!/usr/bin/env python3
"""Benchmark: decode tokens/s of a MiniCPM4-8B-shaped model with random weights on one MI355X.

python bench.py --gpus 1 --steps K --warmup W   prints ONE JSON line.  A step is one decode step
of the whole batch, the next token chosen by argmax included (default: batch 8 at context 4,096,
all 32 layers of the 8B shape).  The same line carries the prefill of 2,048 tokens, the decode
step's memory roofline against the published peak and against what a plain read kernel and a
large library product reach on this GPU, and decode at batch 1 and 64.  Before anything is timed,
one decode step from the captured graph is compared with the same step run eagerly.  Weights are
random (N(0, 0.02)), token ids uniform, the cache of the decode runs is filled with noise (what
filled it is not timed): nothing is downloaded.  The engine runs on one GPU only: for --gpus > 1
it says so and exits with 2.
"""
import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0          # MI355X HBM3E, published
PEAK_FLOPS = {"bf16": 2.5e15, "fp32": 157.3e12}


def config_8b(layers=None):
    import torch
    g = torch.Generator().manual_seed(1234)
    fac = lambda: [float(x) for x in (1.0 + 3.0 * torch.rand(64, generator=g, dtype=torch.float64))]
    return {
        "architectures": ["MiniCPMForCausalLM"], "model_type": "minicpm",
        "num_hidden_layers": layers or 32, "hidden_size": 4096, "num_attention_heads": 32, "num_key_value_heads": 2,
        "head_dim": 128, "intermediate_size": 16384, "vocab_size": 73448, "rms_norm_eps": 1e-6, "rope_theta": 10000.0,
        "max_position_embeddings": 32768,
        "rope_scaling": {"rope_type": "longrope", "short_factor": fac(), "long_factor": fac(),
                         "original_max_position_embeddings": 32768},
        "scale_emb": 12, "dim_model_base": 256, "scale_depth": 1.4, "tie_word_embeddings": False,
        "hidden_act": "silu", "torch_dtype": "bfloat16",
    }


def config_small():
    """The MiniCPM4-0.5B shape (tied embeddings)."""
    import torch
    g = torch.Generator().manual_seed(4321)
    fac = lambda: [float(x) for x in (1.0 + 3.0 * torch.rand(32, generator=g, dtype=torch.float64))]
    return {
        "architectures": ["MiniCPMForCausalLM"], "model_type": "minicpm",
        "num_hidden_layers": 24, "hidden_size": 1024, "num_attention_heads": 16, "num_key_value_heads": 2,
        "head_dim": 64, "intermediate_size": 4096, "vocab_size": 73448, "rms_norm_eps": 1e-6, "rope_theta": 10000.0,
        "max_position_embeddings": 32768,
        "rope_scaling": {"rope_type": "longrope", "short_factor": fac(), "long_factor": fac(),
                         "original_max_position_embeddings": 32768},
        "scale_emb": 12, "dim_model_base": 256, "scale_depth": 1.4, "tie_word_embeddings": True,
        "hidden_act": "silu", "torch_dtype": "bfloat16",
    }


SPARSE_32K = {"kernel_size": 32, "kernel_stride": 16, "block_size": 64, "init_blocks": 1, "topk": 64,
              "window_size": 2048, "dense_len": 8192}


def weight_bytes_per_step(cfg, esize):
    """Bytes of weights a decode step reads once: every layer's matrices and norms, final norm, lm_head."""
    H, I, V, L = cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size, cfg.num_hidden_layers
    qkv = (cfg.num_attention_heads + 2 * cfg.num_key_value_heads) * cfg.head_dim * H
    o = H * cfg.num_attention_heads * cfg.head_dim
    per_layer = (qkv + o + 3 * H * I) * esize + 2 * H * 4
    return L * per_layer + V * H * esize + H * 4


def kv_bytes_per_token(cfg, esize):
    return cfg.num_hidden_layers * 2 * cfg.num_key_value_heads * cfg.head_dim * esize


def prefill_flops(cfg, n):
    H, I, V, L = cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size, cfg.num_hidden_layers
    nh, nkv, hd = cfg.num_attention_heads, cfg.num_key_value_heads, cfg.head_dim
    lin = L * ((nh + 2 * nkv) * hd * H + H * nh * hd + 3 * H * I)
    attn = L * nh * hd * 2 * (n * (n + 1) // 2) * 2          # q.k and p.v over the causal half
    return 2 * n * lin + attn + 2 * V * H


def batch_prefill_flops(cfg, lens):
    """Prompts of several lengths in one step: the products once a token, causal attention a prompt, one head row each."""
    H, I, V, L = cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size, cfg.num_hidden_layers
    nh, nkv, hd = cfg.num_attention_heads, cfg.num_key_value_heads, cfg.head_dim
    lin = L * ((nh + 2 * nkv) * hd * H + H * nh * hd + 3 * H * I)
    attn = sum(L * nh * hd * 2 * (n * (n + 1) // 2) * 2 for n in lens)
    return 2 * sum(lens) * lin + attn + 2 * len(lens) * V * H


def sparse_keys_read(sc, context):
    """Keys a query at the end of `context` tokens attends to under InfLLM-v2: all of them up to dense_len, else
    the chosen blocks and the window."""
    if context <= sc["dense_len"]:
        return context
    return min(context, (sc["topk"] + sc["window_size"] // sc["block_size"]) * sc["block_size"])


def sparse_decode_bytes(cfg, sc, esize, batch, context):
    """What a decode step with block selection has to read: every weight once, and per sequence the attended
    keys and values and the compressed keys that the selection scores."""
    ck = cfg.num_hidden_layers * (context // sc["kernel_stride"]) * cfg.num_key_value_heads * cfg.head_dim * esize
    return weight_bytes_per_step(cfg, esize) + batch * (sparse_keys_read(sc, context) * kv_bytes_per_token(cfg, esize) + ck)


def sparse_prefill_flops(cfg, sc, n):
    """A prompt of n tokens with block selection: products, attention over the keys each query attends to (causal
    up to dense_len), the selection's scores over the compressed keys, one head row."""
    H, I, V, L = cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size, cfg.num_hidden_layers
    nh, nkv, hd = cfg.num_attention_heads, cfg.num_key_value_heads, cfg.head_dim
    lin = L * ((nh + 2 * nkv) * hd * H + H * nh * hd + 3 * H * I)
    dense = min(n, sc["dense_len"])
    keys = dense * (dense + 1) // 2 + sum(sparse_keys_read(sc, p + 1) for p in range(dense, n))
    scores = sum(p // sc["kernel_stride"] for p in range(dense, n))
    return 2 * n * lin + L * nh * hd * 2 * 2 * keys + L * nh * hd * 2 * scores + 2 * V * H


def calibrate_read(dev):
    """GB/s of a kernel that only reads, over 4 GiB (far beyond the caches)."""
    import torch
    from cpmcu_amd import ops
    buf = torch.empty(1 << 30, dtype=torch.int32, device=dev).random_()
    out = torch.zeros(8192, dtype=torch.int32, device=dev)
    best = 0.0
    for _ in range(4):
        torch.cuda.synchronize()
        t = time.perf_counter()
        ops.read_bandwidth(buf, out)
        torch.cuda.synchronize()
        best = max(best, buf.numel() * 4 / (time.perf_counter() - t) / 1e9)
    return best


def timer_table(eng, run, title):
    """The timers by kernel class (average ms a call) for `run()` with the engine's timers switched on; steps
    then run eagerly, so the figures are of the kernels with their launches, not of the graph."""
    from cpmcu_amd.utils.perf import PerfTimers
    import torch
    before = eng.perf
    eng.perf = PerfTimers(enabled=True)
    try:
        run()
        torch.cuda.synchronize()
        rows = eng.perf.summary()
    finally:
        eng.perf = before
    print(f"[bench] timers, {title}:", file=sys.stderr)
    for label, kind, count, total, avg in sorted(rows, key=lambda r: -r[3]):
        print(f"[bench]   {label:<28}{count:>7} calls{total:>11.3f} ms{avg * 1e3:>10.1f} us each", file=sys.stderr)
    return {label: round(avg, 5) for label, kind, count, total, avg in rows}


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=4096)
    ap.add_argument("--layers", type=int, default=None, help="fewer layers than the model's 32 (named in config)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--prefill-tokens", type=int, default=2048)
    ap.add_argument("--no-points", action="store_true", help="skip decode at batch 1 and 64")
    ap.add_argument("--no-prefill", action="store_true")
    ap.add_argument("--hip-graph", type=int, default=1)
    ap.add_argument("--no-rehearse", action="store_true",
                    help="build the engine without its rehearsal passes (a profile then holds the benchmark's own "
                         "kernels only; the workspace grows during the warm-up steps instead)")
    ap.add_argument("--perf", action="store_true",
                    help="after the timed runs, a few eager steps with the engine's timers on: average ms by kernel "
                         "class (products / attention / selection / norms / head) on stderr and under 'timers'")
    ap.add_argument("--scenario", default="headline", choices=["headline", "small_batch64", "sparse32k", "duvulix", "gumodra", "sagedra", "nelutar", "pemalorn", "tirizen"],
                    help="headline: the 8B shape at batch 8, context 4,096 (the default line); "
                         "small_batch64: the 0.5B shape, 64 unequal prompts through the generation loop; sparse32k: "
                         "the 8B shape with InfLLM-v2 at 32k context; duvulix: four Duvulix layers of a real model's "
                         "sizes (latent attention, chunked attention, Mamba-2, a layer that reads the first one's "
                         "latent cache) beside four MiniCPM4-8B layers of equal width: decode and prefill of both; gumodra: "
                         "four Gumodra layers of a real model's sizes (windowed attention with a sink, mLSTM, dense and "
                         "routed feed-forwards) beside the four Duvulix layers; sagedra: four Sagedra layers of a real model's sizes "
                         "(differential attention, windowed attention beside a gated delta rule, four residual streams) "
                         "beside the four Gumodra layers; nelutar: four Nelutar layers of a real model's sizes (capped windowed "
                         "attention beside linear attention, windowed attention beside a delta rule with a decay a key "
                         "channel, retention, routed experts, a layer that runs twice) beside the four Sagedra layers; pemalorn: four Pemalorn layer "
                         "runs of a real model's sizes (latent attention under a window, attention with rotated values "
                         "twice, routed and identity experts, input convolutions, a token table) beside the four Duvulix "
                         "and the four Gumodra layers; tirizen: four Tirizen layers of a real model's sizes (gated linear "
                         "attention, attention with norms over whole projections, a layer that reads another's keys, "
                         "feed-forwards and experts without a gate, four residual streams) beside the four Nelutar and "
                         "the four Sagedra layers")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported (no multi-GPU path exists)")
        sys.exit(2)

    import torch
    import cpmcu_amd
    from cpmcu_amd import Engine, EngineOptions, StepEntry
    from cpmcu_amd.config import MiniCPMConfig
    from cpmcu_amd.weights import random_tensors

    dev = "cuda:0"
    if args.scenario != "headline":
        other_scenarios(args, dev)
        return
    raw = config_8b(args.layers)
    cfg = MiniCPMConfig.from_dict(raw)
    esize = 2 if args.dtype == "bfloat16" else 4
    t0 = time.time()
    tensors = random_tensors(cfg, seed=0, device=dev)
    max_b = max(args.batch, 1 if args.no_points else 64)
    per_seq = -(-(args.context + args.steps + args.warmup + 64) // 64) * 64
    eng = Engine.from_tensors(cfg, tensors, EngineOptions(
        dtype=args.dtype, max_tokens=max(max_b * per_seq, args.prefill_tokens + 64), max_slots=max_b,
        max_step_tokens=max(args.prefill_tokens, 2048), device=dev, hip_graph=bool(args.hip_graph), rehearse=not args.no_rehearse))
    del tensors
    torch.cuda.synchronize()
    print(f"[bench] model ready in {time.time() - t0:.1f} s: {cfg.num_hidden_layers} layers, "
          f"{weight_bytes_per_step(cfg, esize) / 1e9:.2f} GB of weights a step", file=sys.stderr, flush=True)
    g = torch.Generator().manual_seed(7)
    rand_ids = lambda n: [int(t) for t in torch.randint(0, cfg.vocab_size, (n,), generator=g)]

    def fill_context(batch, context):
        """Slots that hold `context - 1` tokens of random keys and values: the state a decode step at that
        context length starts from (the timed steps do all of their own work; what filled the cache is not timed)."""
        slots = [eng.acquire() for _ in range(batch)]
        for s in slots:
            eng.cache.extend(s, context - 1)
        eng.cache.sync()
        for grp in eng.cache.groups:
            for st in grp.storage.values():
                for t in st.values():
                    t.normal_(0.0, 0.5)
        return slots

    from cpmcu_amd import ops
    next_tok = torch.zeros(64, dtype=torch.int32, device=dev)

    def decode_run(batch, context, steps, warmup):
        """Seconds for `steps` decode steps of `batch` sequences at `context`: each step runs the model on one
        token a sequence and chooses the next by argmax (on the device; the tokens fed are fixed beforehand so
        that every run does the same work)."""
        slots = fill_context(batch, context)
        toks = [rand_ids(batch) for _ in range(steps + warmup)]
        for i in range(warmup):
            ops.argmax(eng.step([StepEntry(s, [toks[i][j]], [0]) for j, s in enumerate(slots)]), next_tok[:batch])
        torch.cuda.synchronize()
        t = time.perf_counter()
        for i in range(warmup, warmup + steps):
            ops.argmax(eng.step([StepEntry(s, [toks[i][j]], [0]) for j, s in enumerate(slots)]), next_tok[:batch])
        torch.cuda.synchronize()
        dt = time.perf_counter() - t
        for s in slots:
            eng.release(s)
        return dt

    def graph_check(batch, context):
        """One decode step replayed from the captured graph against the same step run eagerly (the cache is
        wound back one token in between): finite and equal up to the order of float sums."""
        if not args.hip_graph:
            return None
        slots = fill_context(batch, context)
        ids = rand_ids(batch)
        entries = [StepEntry(s, [ids[j]], [0]) for j, s in enumerate(slots)]
        eng.options.hip_graph = False
        eager = eng.step(entries).clone()
        eng.options.hip_graph = True
        outs = []
        for _ in range(2):                   # the first captures, the second replays
            for s in slots:
                eng.cache.truncate(s, context - 1)
            outs.append(eng.step(entries).clone())
        for s in slots:
            eng.release(s)
        if not bool(torch.isfinite(eager).all()):
            raise SystemExit("bench.py: the decode step's logits are not finite")
        scale = float(eager.abs().max())
        err = max(float((o - eager).abs().max()) for o in outs)
        if err > 1e-3 * scale:
            raise SystemExit(f"bench.py: a decode step from the captured graph differs from the eager step by {err:.3g} "
                             f"(logits up to {scale:.3g})")
        return err / scale

    def calibrate():
        """What this GPU gives a kernel that only reads (GB/s) and the library's product of two large bf16
        matrices (FLOP/s): the ceilings that memory-bound and matrix-bound work can be held against besides
        the published peaks."""
        best = calibrate_read(dev)
        a = torch.randn(8192, 8192, device=dev, dtype=torch.bfloat16)
        b = torch.randn(8192, 8192, device=dev, dtype=torch.bfloat16)
        c = torch.empty_like(a)
        flops = 0.0
        for _ in range(4):
            torch.cuda.synchronize()
            t = time.perf_counter()
            for _ in range(4):
                torch.mm(a, b.t(), out=c)
            torch.cuda.synchronize()
            flops = max(flops, 4 * 2 * 8192 ** 3 / (time.perf_counter() - t))
        return best, flops

    def step_bytes(batch, context, steps):
        return weight_bytes_per_step(cfg, esize) + batch * (context + steps // 2) * kv_bytes_per_token(cfg, esize)

    read_gbs, mm_flops = calibrate()
    graph_err = graph_check(args.batch, args.context)
    dt = decode_run(args.batch, args.context, args.steps, args.warmup)
    ms_step = dt / args.steps * 1e3
    value = args.batch * args.steps / dt
    achieved = step_bytes(args.batch, args.context, args.steps) / (ms_step * 1e-3) / 1e9
    rec = {
        "metric": f"MiniCPM4-8B decode tok/s @ batch {args.batch}, context {args.context} "
                  f"({'bf16' if args.dtype == 'bfloat16' else 'fp32'}, random weights)",
        "value": round(value, 2), "unit": "tokens/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(ms_step, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic",
        "config": {"model": "MiniCPM4-8B shape, random weights N(0,0.02)", "layers": cfg.num_hidden_layers,
                   "layers_full_model": 32, "hidden": cfg.hidden_size, "heads": cfg.num_attention_heads,
                   "kv_heads": cfg.num_key_value_heads, "head_dim": cfg.head_dim,
                   "intermediate": cfg.intermediate_size, "vocab": cfg.vocab_size, "global_batch": args.batch,
                   "seq_len": args.context, "prefill_tokens": args.prefill_tokens, "parallelism": "1gpu",
                   "page_size": 64, "hip_graph": bool(args.hip_graph), "sampling": "argmax inside the timed step",
                   "cache_fill": "noise (not timed)"},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                     "frac": round(achieved / HBM_PEAK_GBS, 4), "read_kernel": round(read_gbs, 1),
                     "frac_of_read_kernel": round(achieved / read_gbs, 4)},
    }
    if graph_err is not None:
        rec["graph_check"] = {"max_rel_diff_to_eager": float(f"{graph_err:.3g}")}
    if not args.no_prefill:
        n = args.prefill_tokens
        times = []
        for it in range(3):
            s = eng.acquire()
            ids = rand_ids(n)
            torch.cuda.synchronize()
            t = time.perf_counter()
            eng.step([StepEntry(s, ids, [n - 1])])
            torch.cuda.synchronize()
            times.append(time.perf_counter() - t)
            eng.release(s)
        pt = min(times[1:])
        peak = PEAK_FLOPS["bf16" if args.dtype == "bfloat16" else "fp32"]
        rec["prefill"] = {"value": round(n / pt, 1), "tokens": n, "ms": round(pt * 1e3, 3),
                          "frac": round(prefill_flops(cfg, n) / pt / peak, 4),
                          "library_product": round(mm_flops / 1e12, 1), "library_product_unit": "TFLOP/s",
                          "frac_of_library_product": round(prefill_flops(cfg, n) / pt / mm_flops, 4)}
    if not args.no_points:
        pts = {}
        for b in (1, 64):
            st = max(args.steps // 2, 8)
            d = decode_run(b, args.context, st, max(args.warmup // 2, 3))
            gbs = step_bytes(b, args.context, st) / (d / st) / 1e9
            pts[f"decode_b{b}"] = round(b * st / d, 2)
            pts[f"decode_b{b}_ms"] = round(d / st * 1e3, 4)
            pts[f"decode_b{b}_frac"] = round(gbs / HBM_PEAK_GBS, 4)
        rec["points"] = pts
    if args.perf:
        def few_steps():
            slots = fill_context(args.batch, args.context)
            for _ in range(4):
                eng.step([StepEntry(s, [1], [0]) for s in slots])
            for s in slots:
                eng.release(s)
            if not args.no_prefill:
                s = eng.acquire()
                eng.step([StepEntry(s, rand_ids(args.prefill_tokens), [args.prefill_tokens - 1])])
                eng.release(s)
        rec["timers"] = timer_table(eng, few_steps, f"batch {args.batch}, context {args.context}")
    print(json.dumps(rec), flush=True)


def config_duvulix():
    """Four layers of sizes that resemble a real model's: width 4,096; latent attention with 32 heads of 128 + 64
    features over a latent of 512; attention with 32 heads on 8 kv heads of 128, chunks of 2,048 tokens, YaRN;
    Mamba-2 with 128 heads of 64, state 128, 8 groups; PolyNorm feed-forwards of 16,384."""
    latent = {"heads": 32, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5,
              "rot": {"base": 500000.0, "dims": 64}}
    mlp = {"kind": "dense", "ff": 16384}
    return {
        "architecture": "Duvulix", "vocab": 73448, "width": 4096, "norm": {"eps": 1e-6},
        "layers": [
            {"type": "latent_attention", "mixer": dict(latent), "mlp": mlp},
            {"type": "attention", "mixer": {"heads": 32, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                                            "rot": {"base": 500000.0, "dims": 128,
                                                    "scaling": {"factor": 8.0, "original": 8192, "fast": 32.0, "slow": 1.0}},
                                            "mask": {"size": 2048}}, "mlp": mlp},
            {"type": "mamba2", "mixer": {"heads": 128, "vdim": 64, "state": 128, "groups": 8, "conv": 4,
                                         "norm_groups": 8}, "mlp": mlp},
            {"type": "latent_attention", "mixer": dict(latent, kv_from=0), "mlp": mlp},
        ],
    }


def duvulix_step_bytes(raw, esize, batch, context):
    """Bytes a decode step must move: every matrix once (the embedding's rows aside), and per sequence what its
    mixers read: the latent cache once per layer that reads it, the keys and values of the query's chunk, the
    recurrent state read and written."""
    W = raw["width"]
    weights = raw["vocab"] * W
    per_seq = 0
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "latent_attention":
            weights += m["heads"] * (m["dim"] + m["rot_dim"]) * W + m["heads"] * W + m["heads"] * m["vdim"] * W
            weights += m["heads"] * (m["dim"] + m["vdim"]) * m["kv_rank"]
            if m.get("kv_from") is None:
                weights += (m["kv_rank"] + m["rot_dim"]) * W
            per_seq += context * (2 * m["kv_rank"] + m["rot_dim"]) * esize
        elif layer["type"] == "attention":
            weights += (m["heads"] * (m["dim"] + m["vdim"]) + m["kv_heads"] * (m["dim"] + m["vdim"])) * W
            seen = context if not m.get("mask") else (context - 1) % m["mask"]["size"] + 1
            per_seq += seen * m["kv_heads"] * (m["dim"] + m["vdim"]) * esize
        else:
            inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
            weights += (2 * inner + 2 * gn + m["heads"]) * W + inner * W
            per_seq += 2 * 4 * (m["heads"] * m["vdim"] * m["state"] + (m["conv"] - 1) * (inner + 2 * gn))
        if layer.get("mlp"):
            weights += 2 * layer["mlp"]["ff"] * W
    return weights * esize + batch * per_seq, weights


def config_gumodra():
    """Four layers of sizes that resemble a real model's: width 4,096; attention with 32 heads on 8 kv heads of 128
    (the keys double as values), 64 rotated features, a window of 2,048 tokens that keeps the first 128, a sink a
    head; an mLSTM of 8 heads with keys of 256 and values of 512; SiLU-gated feed-forwards of 11,008; mixtures of 64
    experts of 1,408 in 8 groups (4 kept), 6 a token, with a shared expert of 2,816."""
    attn = {"heads": 32, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
            "rot": {"base": 500000.0, "dims": 64}, "mask": {"size": 2048, "keep_first": 128}}
    dense = {"kind": "dense", "ff": 11008}
    moe = {"kind": "moe", "expert": {"ff": 1408}, "router": {"experts": 64, "top": 6, "groups": {"count": 8, "keep": 4}},
           "shared": {"ff": 2816}}
    return {
        "architecture": "Gumodra", "vocab": 73448, "width": 4096, "norm": {"eps": 1e-6}, "embedding": {"scale": 12.0},
        "layers": [
            {"type": "attention", "mixer": dict(attn), "mlp": dense},
            {"type": "attention", "mixer": dict(attn), "mlp": moe},
            {"type": "mlstm", "mixer": {"heads": 8, "dim": 256, "vdim": 512, "gate_cap": 15.0}, "mlp": dense},
            {"type": "attention", "mixer": dict(attn), "mlp": moe},
        ],
    }


def gumodra_step_bytes(raw, esize, batch, context):
    """Bytes a decode step must move: every matrix that the step reads once (of a mixture: the router, the shared
    expert, and an expert for every (token, choice) pair, at most all of them), and per sequence what its mixers
    read: keys and values of the window and of the kept first tokens, the recurrent state read and written."""
    W = raw["width"]
    weights = raw["vocab"] * W
    per_seq = 0
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "attention":
            weights += (2 * m["heads"] * m["dim"] + m["kv_heads"] * m["dim"]) * W
            mask = m.get("mask")
            seen = context if not mask else min(context, mask["size"] + mask.get("keep_first", 0))
            per_seq += seen * m["kv_heads"] * 2 * m["dim"] * esize
        else:
            hk, hv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            weights += (2 * hk + 3 * hv + 2 * m["heads"]) * W
            per_seq += 2 * 4 * (m["heads"] * m["dim"] * m["vdim"] + hk + m["heads"])
        mlp = layer.get("mlp")
        weights += W * W * (2 if mlp else 1)                       # the gates of the two results
        if mlp and mlp["kind"] == "dense":
            weights += 3 * mlp["ff"] * W
        elif mlp:
            r = mlp["router"]
            weights += r["experts"] * W + (3 * mlp["shared"]["ff"] * W + W if mlp.get("shared") else 0)
            weights += min(max(batch, 1) * r["top"], r["experts"]) * 3 * mlp["expert"]["ff"] * W
    return weights * esize + batch * per_seq, weights


def gumodra_prefill_params(raw):
    """Matrix elements a prompt token is multiplied with (of a mixture: the chosen experts only)."""
    W = raw["width"]
    total = raw["vocab"] * W
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "attention":
            total += (2 * m["heads"] * m["dim"] + m["kv_heads"] * m["dim"]) * W
        else:
            total += (2 * m["heads"] * m["dim"] + 3 * m["heads"] * m["vdim"] + 2 * m["heads"]) * W
        mlp = layer.get("mlp")
        total += W * W * (2 if mlp else 1)
        if mlp and mlp["kind"] == "dense":
            total += 3 * mlp["ff"] * W
        elif mlp:
            total += mlp["router"]["experts"] * W + (3 * mlp["shared"]["ff"] * W if mlp.get("shared") else 0)
            total += mlp["router"]["top"] * 3 * mlp["expert"]["ff"] * W
    return total


def config_sagedra():
    """Four layers of sizes that resemble a real model's: width 4,096 in 4 residual streams; differential attention
    with 16 heads of two maps each on 4 key heads of 128 and values of 256, 4 convolution taps and a query
    temperature; pairs of a sliding-window attention (32 heads on 8 kv heads of 128, all features rotated with
    stretched frequencies, a window of 2,048, an output gate) beside a gated delta rule (32 heads on 16 key heads,
    128 by 128, 4 taps); GELU-gated feed-forwards of 11,008; a logit cap."""
    diff = {"heads": 16, "kv_heads": 4, "dim": 128, "vdim": 256, "scale": 128 ** -0.5, "diff": 0.35, "conv": 4,
            "q_temp": {"coef": 0.1, "every": 1024}}
    pair = {"left": {"heads": 32, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 1.0,
                     "rot": {"base": 500000.0, "dims": 128,
                             "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}},
                     "mask": {"size": 2048}},
            "right": {"heads": 32, "kv_heads": 16, "dim": 128, "vdim": 128, "conv": 4}}
    dense = {"kind": "dense", "ff": 11008}
    return {
        "architecture": "Sagedra", "vocab": 73448, "width": 4096, "norm": {"eps": 1e-6}, "embedding": {"scale": 64.0},
        "streams": 4, "logit_softcap": 50.0,
        "layers": [
            {"type": "attention", "mixer": dict(diff), "mlp": dense},
            {"type": "parallel", "mixer": dict(pair), "mlp": dense},
            {"type": "attention", "mixer": dict(diff), "mlp": dense},
            {"type": "parallel", "mixer": dict(pair), "mlp": dense},
        ],
    }


def sagedra_step_bytes(raw, esize, batch, context):
    """Bytes a decode step must move: every matrix once, and per sequence what its mixers read: keys of both maps
    and the values of all cached tokens (differential attention), keys and values of the window, the delta rule's
    state read and written, the convolutions' last inputs."""
    W = raw["width"]
    weights = raw["vocab"] * W
    per_seq = 0
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "attention":
            qk, v = 2 * m["dim"], m["vdim"]
            weights += (m["heads"] * (qk + v) + m["kv_heads"] * (qk + v)) * W
            per_seq += context * m["kv_heads"] * (qk + v) * esize
            per_seq += 2 * 4 * (m.get("conv", 1) - 1) * (m["heads"] * qk + m["kv_heads"] * (qk + v))
        else:
            a, d = m["left"], m["right"]
            weights += (a["heads"] * (a["dim"] + 2 * a["vdim"]) + a["kv_heads"] * (a["dim"] + a["vdim"])) * W
            seen = context if not a.get("mask") else min(context, a["mask"]["size"])
            per_seq += seen * a["kv_heads"] * (a["dim"] + a["vdim"]) * esize
            hk, hv = d["kv_heads"] * d["dim"], d["heads"] * d["vdim"]
            weights += (2 * hk + 3 * hv + 2 * d["heads"]) * W
            per_seq += 2 * 4 * (d["heads"] * d["dim"] * d["vdim"] + (d["conv"] - 1) * (2 * hk + hv))
        if layer.get("mlp"):
            weights += 3 * layer["mlp"]["ff"] * W
    return weights * esize + batch * per_seq, weights


def config_nelutar():
    """Four layers of sizes that resemble a real model's: width 4,096, a bigram table of 100,003 buckets; a pair of
    capped windowed attention (32 heads on 8 kv heads of 128, 64 rotated features, 4 convolution taps, a window of
    2,048) beside linear attention of 32 heads of 128 by 128 with fixed decays, and a SiLU-gated feed-forward of
    11,008; a pair of windowed attention beside a delta rule with a decay a key channel (32 heads on 16 key heads,
    128 by 128, 4 taps, decay and gate through products of rank 512) with 64 experts of 1,408 in 8 groups (4 kept),
    6 a token, and a shared expert of 2,816; retention of 32 heads of 128 by 128 with the same experts; and the
    second layer's weights once more."""
    left = {"heads": 32, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": 2048}}
    decays = [1.0 - 2.0 ** (-5.0 - 3.0 * h / 31.0) for h in range(32)]
    dense = {"kind": "dense", "ff": 11008}
    moe = {"kind": "moe", "expert": {"ff": 1408, "limit": 7.0},
           "router": {"experts": 64, "top": 6, "scale": 2.0, "groups": {"count": 8, "keep": 4}},
           "shared": {"ff": 2816, "limit": 7.0}}
    pair = {"left": dict(left, rot={"base": 500000.0, "dims": 128}),
            "right": {"heads": 32, "kv_heads": 16, "dim": 128, "vdim": 128, "conv": 4}}
    return {
        "architecture": "Nelutar", "vocab": 73448, "width": 4096, "norm": {"eps": 1e-6},
        "embedding": {"bigram": {"buckets": 100003, "mul_prev": 36313, "mul_cur": 27191}},
        "layers": [
            {"type": "parallel_2", "mixer": {
                "left": dict(left, rot={"base": 10000.0, "dims": 64}, conv=4, softcap=30.0),
                "right": {"heads": 32, "dim": 128, "vdim": 128, "decay": decays}, "left_scale": 0.7, "right_scale": 0.4},
             "mlp": dense},
            {"type": "parallel", "mixer": pair, "mlp": moe},
            {"type": "retention", "mixer": {"heads": 32, "dim": 128, "vdim": 128, "decay": decays,
                                            "rot": {"base": 100000.0, "dims": 128}}, "mlp": moe},
            {"type": "parallel", "mixer": pair, "mlp": moe, "weights_of": 1},
        ],
    }


def nelutar_step_bytes(raw, esize, batch, context, prefill=False):
    """Bytes a decode step must move: every matrix that the step reads once (a layer that borrows weights reads them
    again; of a mixture: the router, the shared expert, and an expert for every (token, choice) pair, at most all of
    them), and per sequence what its mixers read: keys and values of the window, the recurrent states read and
    written, the convolutions' last inputs.  With ``prefill``: the matrix elements a prompt token is multiplied with
    (of a mixture: the chosen experts only)."""
    W = raw["width"]
    weights = raw["vocab"] * W
    per_seq = W * esize                                              # the bigram table's row
    for layer in raw["layers"]:
        m = layer["mixer"]

        def attention(a):
            nonlocal weights, per_seq
            weights += (2 * a["heads"] * a["dim"] + a["kv_heads"] * (a["dim"] + a["vdim"])) * W
            seen = context if not a.get("mask") else min(context, a["mask"]["size"])
            per_seq += seen * a["kv_heads"] * (a["dim"] + a["vdim"]) * esize
            if a.get("conv"):
                per_seq += 2 * 4 * (a["conv"] - 1) * (a["heads"] * a["dim"] + a["kv_heads"] * (a["dim"] + a["vdim"]))

        def decay_attention(d):
            nonlocal weights, per_seq
            weights += (2 * d["heads"] * d["dim"] + 3 * d["heads"] * d["vdim"]) * W
            per_seq += 2 * 4 * d["heads"] * d["dim"] * d["vdim"]

        if layer["type"] == "retention":
            decay_attention(m)
        else:
            attention(m["left"])
            if layer["type"] == "parallel_2":
                decay_attention(m["right"])
            else:
                d = m["right"]
                hk, hv = d["kv_heads"] * d["dim"], d["heads"] * d["vdim"]
                ra, rg = d["heads"] * d["dim"] // 8, hv // 8
                weights += (2 * hk + 2 * hv + d["heads"] + ra + rg) * W + ra * d["heads"] * d["dim"] + rg * hv
                per_seq += 2 * 4 * (d["heads"] * d["dim"] * d["vdim"] + (d["conv"] - 1) * (2 * hk + hv))
        mlp = layer.get("mlp")
        if mlp and mlp["kind"] == "dense":
            weights += 3 * mlp["ff"] * W
        elif mlp:
            r = mlp["router"]
            weights += r["experts"] * W + (3 * mlp["shared"]["ff"] * W if mlp.get("shared") else 0)
            pairs = r["top"] if prefill else min(max(batch, 1) * r["top"], r["experts"])
            weights += pairs * 3 * mlp["expert"]["ff"] * W
    return weights * esize + batch * per_seq, weights


def config_pemalorn():
    """Three layers, the second one twice (four layer runs), of sizes that resemble a real model's: width 4,096; latent
    attention with 32 heads of 128 + 64 features, a query latent of 1,536, a latent of 512 and a window of 2,048;
    attention with 32 heads on 8 kv heads of 128 with rotated values; 64 experts of 1,408 and 16 identity experts, 6 a
    token; 4 taps on what the sub-layers read; a token table of 256 numbers a layer."""
    latent = {"heads": 32, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": 1536, "kv_rank": 512, "scale": 192 ** -0.5,
              "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}},
              "mask": {"size": 2048}}
    attn = {"heads": 32, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "rot": {"base": 500000.0, "dims": 128}}
    moe = {"kind": "moe", "expert": {"ff": 1408}, "router": {"experts": 64, "identity": 16, "top": 6}}
    return {
        "architecture": "Pemalorn", "vocab": 73448, "width": 4096, "norm": {"eps": 1e-6}, "canon": {"taps": 4},
        "token_side": {"dim": 256}, "loop": {"start": 1, "stop": 2, "times": 2},
        "layers": [{"type": "latent_attention", "mixer": dict(latent), "mlp": moe},
                   {"type": "attention", "mixer": dict(attn), "mlp": moe},
                   {"type": "latent_attention", "mixer": dict(latent), "mlp": moe}],
    }


def pemalorn_step_bytes(raw, esize, batch, context, prefill=False):
    """Bytes a decode step must move: every matrix that the step reads once a layer run (of a mixture: the router, and
    an expert for every (token, choice) pair that is no identity expert, at most all of them), and per sequence what the
    mixers read (the latent cache of the window, keys and values), the convolutions' last inputs, the token table's
    row.  With ``prefill``: the matrix elements a prompt token is multiplied with (of a mixture: the chosen experts)."""
    W, side, taps = raw["width"], raw["token_side"]["dim"], raw["canon"]["taps"]
    weights = raw["vocab"] * W
    per_seq = 0
    loop = raw["loop"]
    for i, layer in enumerate(raw["layers"]):
        m = layer["mixer"]
        w = 2 * side * W
        s = side * esize + 2 * 4 * (taps - 1) * W
        if layer["type"] == "latent_attention":
            H, R, r = m["heads"], m["kv_rank"], m["rot_dim"]
            w += (m["q_rank"] + R + r + H * m["vdim"]) * W + H * (m["dim"] + r) * m["q_rank"]
            w += H * (m["dim"] + m["vdim"]) * R + H * m["vdim"] * W
            s += min(context, m["mask"]["size"]) * (2 * R + r) * esize
        else:
            w += (m["heads"] * (m["dim"] + m["vdim"]) + m["kv_heads"] * (m["dim"] + m["vdim"]) + m["heads"]) * W
            s += context * m["kv_heads"] * (m["dim"] + m["vdim"]) * esize
        r = layer["mlp"]["router"]
        real = r["experts"] / (r["experts"] + r["identity"])
        w += (r["experts"] + r["identity"]) * W
        pairs = r["top"] * real if prefill else min(max(batch, 1) * r["top"] * real, r["experts"])
        w += pairs * 3 * layer["mlp"]["expert"]["ff"] * W
        runs = loop["times"] if loop["start"] <= i < loop["stop"] else 1
        weights += runs * w
        per_seq += runs * s
    weights += loop["times"] * 2 * W * W
    return weights * esize + batch * per_seq, int(weights)


def config_tirizen():
    """Four layers of sizes that resemble a real model's: width 4,096 in 4 residual streams; gated linear attention of 32
    heads of 128 by 128 (decays of rank 16), attention with 32 heads on 8 kv heads of 128, and a layer of the same attention
    that reads the other's keys and values; a feed-forward of 16,512 without a gate (as many numbers as a gated one of
    11,008) and 64 experts of 2,112 (gated: 1,408), 6 a token."""
    gla = {"heads": 32, "dim": 128, "vdim": 128, "tau": 16.0}
    attn = {"heads": 32, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "q_temp": {"coef": 0.1, "every": 1024}}
    moe = {"kind": "moe", "expert": {"ff": 2112}, "router": {"experts": 64, "top": 6}}
    return {
        "architecture": "Tirizen", "vocab": 73448, "width": 4096, "norm": {"eps": 1e-6}, "embedding": {"scale": 64.0},
        "max_positions": 8192, "residual_mult": 0.7, "streams": 4, "logit_scale": 0.25,
        "layers": [
            {"type": "gla", "mixer": dict(gla), "mlp": {"kind": "dense", "ff": 16512}},
            {"type": "attention", "mixer": dict(attn), "mlp": moe},
            {"type": "gla", "mixer": dict(gla), "mlp": moe},
            {"type": "attention", "mixer": dict(attn, kv_from=1), "mlp": moe},
        ],
    }


def tirizen_step_bytes(raw, esize, batch, context, prefill=False):
    """Bytes a decode step must move: every matrix that the step reads once (of a mixture: the router, and an expert for
    every (token, choice) pair, at most all of them), and per sequence what the mixers read: keys and values (a layer that
    borrows them reads them again), the recurrent states read and written, the row of the position table.  With
    ``prefill``: the matrix elements a prompt token is multiplied with (of a mixture: the chosen experts only)."""
    W = raw["width"]
    weights = raw["vocab"] * W
    per_seq = W * esize
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "gla":
            hk, hv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            weights += (2 * hk + 3 * hv + 16) * W + 16 * hk
            per_seq += 2 * 4 * m["heads"] * m["dim"] * m["vdim"]
        else:
            weights += m["heads"] * (m["dim"] + m["vdim"] + 1) * W
            if m.get("kv_from") is None:
                weights += m["kv_heads"] * (m["dim"] + m["vdim"]) * W
            per_seq += context * m["kv_heads"] * (m["dim"] + m["vdim"]) * esize
        mlp = layer["mlp"]
        if mlp["kind"] == "dense":
            weights += 2 * mlp["ff"] * W
        else:
            r = mlp["router"]
            pairs = r["top"] if prefill else min(max(batch, 1) * r["top"], r["experts"])
            weights += r["experts"] * W + pairs * 2 * mlp["expert"]["ff"] * W
    return weights * esize + batch * per_seq, weights


def duvulix_scenario(args, dev):
    """Decode and prefill of the Duvulix layer shapes beside the MiniCPM4-8B layer shape (equal width, equal
    number of layers, random weights): one JSON line with both models' figures and their timers by kernel class."""
    layer_shapes_scenario(args, dev, "duvulix", "Duvulix", config_duvulix(), ("minicpm", config_8b(4)))


def gumodra_scenario(args, dev):
    """The same for the Gumodra layer shapes beside the Duvulix layer shapes (the package's other design of mixed
    attention and recurrent layers; equal width, vocabulary and number of layers)."""
    layer_shapes_scenario(args, dev, "gumodra", "Gumodra", config_gumodra(), ("duvulix", config_duvulix()))


def sagedra_scenario(args, dev):
    """The same for the Sagedra layer shapes beside the Gumodra layer shapes (the package's closest design: windowed
    attention beside a matrix-state recurrence; equal width, vocabulary and number of layers)."""
    layer_shapes_scenario(args, dev, "sagedra", "Sagedra", config_sagedra(), ("gumodra", config_gumodra()))


def nelutar_scenario(args, dev):
    """The same for the Nelutar layer shapes beside the Sagedra layer shapes (the package's closest design: windowed
    attention beside a gated delta rule, layers whose weights run more than once; equal width, vocabulary and number
    of layers)."""
    layer_shapes_scenario(args, dev, "nelutar", "Nelutar", config_nelutar(), ("sagedra", config_sagedra()))


def pemalorn_scenario(args, dev):
    """The same for the Pemalorn layer shapes beside the Duvulix (latent attention) and the Gumodra layer shapes
    (parallel layers with a softmax sink and routed experts): equal width, vocabulary and number of layer runs."""
    layer_shapes_scenario(args, dev, "pemalorn", "Pemalorn", config_pemalorn(), ("duvulix", config_duvulix()),
                          ("gumodra", config_gumodra()))


def tirizen_scenario(args, dev):
    """The same for the Tirizen layer shapes beside the Nelutar (linear attention with decays, routed experts) and the
    Sagedra layer shapes (a residual of four streams, a matrix-state recurrence): equal width, vocabulary, number of layers,
    and numbers a feed-forward."""
    layer_shapes_scenario(args, dev, "tirizen", "Tirizen", config_tirizen(), ("nelutar", config_nelutar()),
                          ("sagedra", config_sagedra()))


def layer_shapes_scenario(args, dev, first, title, first_raw, *others):
    import torch
    import cpmcu_amd
    from cpmcu_amd import Engine, EngineOptions, StepEntry, ops
    from cpmcu_amd.weights import random_tensors

    esize = 2 if args.dtype == "bfloat16" else 4
    batches = sorted({1, args.batch, 32})
    n_prefill = args.prefill_tokens
    g = torch.Generator().manual_seed(7)
    next_tok = torch.zeros(64, dtype=torch.int32, device=dev)
    read_gbs = calibrate_read(dev)
    out = {}
    for name, raw in ((first, first_raw),) + others:
        arch = cpmcu_amd.get_architecture(raw.get("architecture") or raw["architectures"][0])
        cfg = arch.config_class.from_dict(raw)
        per_seq = -(-(args.context + args.steps + args.warmup + 64) // 64) * 64
        eng = Engine.from_tensors(cfg, random_tensors(cfg, seed=0, device=dev), EngineOptions(
            dtype=args.dtype, max_tokens=max(max(batches) * per_seq, n_prefill + 64), max_slots=max(batches),
            max_seq_len=max(per_seq, n_prefill + 64), max_step_tokens=max(n_prefill, 2048), device=dev,
            hip_graph=bool(args.hip_graph), rehearse=not args.no_rehearse))
        rand_ids = lambda n: [int(t) for t in torch.randint(0, cfg.vocabulary_size, (n,), generator=g)]

        def filled(batch):
            slots = [eng.acquire() for _ in range(batch)]
            for s in slots:
                eng.cache.extend(s, args.context - 1)
            eng.cache.sync()
            for grp in eng.cache.groups:
                for st in list(grp.storage.values()) + list(grp.state.values()):
                    for t in st.values():
                        if t.is_floating_point():
                            t.normal_(0.0, 0.5)
            return slots

        def decode(batch, steps, warmup):
            slots = filled(batch)
            toks = [rand_ids(batch) for _ in range(steps + warmup)]
            for i in range(warmup):
                ops.argmax(eng.step([StepEntry(s, [toks[i][j]], [0]) for j, s in enumerate(slots)]), next_tok[:batch])
            torch.cuda.synchronize()
            t = time.perf_counter()
            for i in range(warmup, warmup + steps):
                ops.argmax(eng.step([StepEntry(s, [toks[i][j]], [0]) for j, s in enumerate(slots)]), next_tok[:batch])
            torch.cuda.synchronize()
            dt = time.perf_counter() - t
            for s in slots:
                eng.release(s)
            return dt

        def prefill():
            ids = rand_ids(n_prefill)
            best = None
            for _ in range(3):
                s = eng.acquire()
                torch.cuda.synchronize()
                t = time.perf_counter()
                ops.argmax(eng.step([StepEntry(s, ids, [n_prefill - 1])]), next_tok[:1])
                torch.cuda.synchronize()
                dt = time.perf_counter() - t
                eng.release(s)
                best = dt if best is None else min(best, dt)
            return best

        prefill_params = None
        if name == "duvulix":
            step_bytes = lambda b: duvulix_step_bytes(raw, esize, b, args.context)[0]
            params = duvulix_step_bytes(raw, esize, 0, 0)[1]
        elif name == "gumodra":
            step_bytes = lambda b: gumodra_step_bytes(raw, esize, b, args.context)[0]
            params = gumodra_step_bytes(raw, esize, args.batch, 0)[1]
            prefill_params = gumodra_prefill_params(raw)
        elif name == "sagedra":
            step_bytes = lambda b: sagedra_step_bytes(raw, esize, b, args.context)[0]
            params = sagedra_step_bytes(raw, esize, 0, 0)[1]
        elif name == "nelutar":
            step_bytes = lambda b: nelutar_step_bytes(raw, esize, b, args.context)[0]
            params = nelutar_step_bytes(raw, esize, args.batch, 0)[1]
            prefill_params = nelutar_step_bytes(raw, esize, 1, 0, prefill=True)[1]
        elif name == "pemalorn":
            step_bytes = lambda b: pemalorn_step_bytes(raw, esize, b, args.context)[0]
            params = pemalorn_step_bytes(raw, esize, args.batch, 0)[1]
            prefill_params = pemalorn_step_bytes(raw, esize, 1, 0, prefill=True)[1]
        elif name == "tirizen":
            step_bytes = lambda b: tirizen_step_bytes(raw, esize, b, args.context)[0]
            params = tirizen_step_bytes(raw, esize, args.batch, 0)[1]
            prefill_params = tirizen_step_bytes(raw, esize, 1, 0, prefill=True)[1]
        else:
            step_bytes = lambda b: weight_bytes_per_step(cfg, esize) + b * args.context * kv_bytes_per_token(cfg, esize)
            params = weight_bytes_per_step(cfg, esize) // esize
        rec = {"decode": {}, "weights_gb": round(params * esize / 1e9, 3)}
        for b in batches:
            dt = decode(b, args.steps, args.warmup)
            ms = dt / args.steps * 1e3
            gbs = step_bytes(b) / (ms * 1e-3) / 1e9
            rec["decode"][str(b)] = {"tokens_per_s": round(b * args.steps / dt, 1), "ms_per_step": round(ms, 4),
                                     "gb_per_step": round(step_bytes(b) / 1e9, 3), "frac_of_hbm_peak": round(gbs / HBM_PEAK_GBS, 4),
                                     "frac_of_read_kernel": round(gbs / read_gbs, 4)}
            print(f"[bench] {name}: decode batch {b} context {args.context}: {ms:.3f} ms a step, {gbs:.0f} GB/s", file=sys.stderr, flush=True)
        if not args.no_prefill:
            dt = prefill()
            flops = 2.0 * (prefill_params or params) * n_prefill
            rec["prefill"] = {"tokens": n_prefill, "ms": round(dt * 1e3, 3), "tokens_per_s": round(n_prefill / dt, 1),
                              "matrix_flops_frac_of_peak": round(flops / dt / PEAK_FLOPS["bf16" if esize == 2 else "fp32"], 4)}
            print(f"[bench] {name}: prefill of {n_prefill} tokens: {dt * 1e3:.2f} ms", file=sys.stderr, flush=True)
        if args.perf:
            slots = filled(args.batch)
            ids = rand_ids(args.batch)
            rec["timers_decode"] = timer_table(eng, lambda: [eng.step([StepEntry(s, [ids[j]], [0]) for j, s in enumerate(slots)])
                                                            for _ in range(8)], f"{name}, decode batch {args.batch}")
            for s in slots:
                eng.release(s)
            pid = rand_ids(n_prefill)

            def one_prompt():
                for _ in range(3):
                    s = eng.acquire()
                    eng.step([StepEntry(s, pid, [n_prefill - 1])])
                    eng.release(s)
            rec["timers_prefill"] = timer_table(eng, one_prompt, f"{name}, prefill of {n_prefill}")
        out[name] = rec
        del eng
        torch.cuda.empty_cache()
    d = out[first]["decode"][str(args.batch)]
    print(json.dumps({
        "metric": f"{title} layer shapes (4 layers, width 4096): decode tok/s at batch {args.batch}, context {args.context}",
        "value": d["tokens_per_s"], "unit": "tokens/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": d["ms_per_step"], "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if esize == 2 else "fp32", "data": "synthetic",
        "config": {"model": f"{title} layer shapes beside {' and '.join(o[0] for o in others)} layer shapes, 4 layers each, random weights",
                   "global_batch": args.batch, "seq_len": args.context, "parallelism": "1gpu",
                   "hip_graph": bool(args.hip_graph), first: first_raw},
        "read_kernel_gbs": round(read_gbs, 1), "models": out}))


def other_scenarios(args, dev):
    """The further workloads, each one JSON line of the same shape."""
    if args.scenario == "duvulix":
        duvulix_scenario(args, dev)
        return
    if args.scenario == "gumodra":
        gumodra_scenario(args, dev)
        return
    if args.scenario == "sagedra":
        sagedra_scenario(args, dev)
        return
    if args.scenario == "nelutar":
        nelutar_scenario(args, dev)
        return
    if args.scenario == "pemalorn":
        pemalorn_scenario(args, dev)
        return
    if args.scenario == "tirizen":
        tirizen_scenario(args, dev)
        return
    import torch
    from cpmcu_amd import Engine, EngineOptions, StepEntry
    from cpmcu_amd.config import MiniCPMConfig
    from cpmcu_amd.engine.generate import generate
    from cpmcu_amd.weights import random_tensors

    g = torch.Generator().manual_seed(11)
    if args.scenario == "small_batch64":
        cfg = MiniCPMConfig.from_dict(config_small())
        lens = [int(x) for x in torch.randint(128, 2049, (64,), generator=g)]
        new = 256
        eng = Engine.from_tensors(cfg, random_tensors(cfg, 0, device=dev), EngineOptions(
            dtype=args.dtype, max_tokens=sum(-(-(n + new) // 64) * 64 for n in lens), max_slots=64,
            max_step_tokens=8192, device=dev, hip_graph=bool(args.hip_graph), rehearse=not args.no_rehearse))
        prompts = [[int(t) for t in torch.randint(0, cfg.vocab_size, (n,), generator=g)] for n in lens]
        generate(eng, prompts[:4], 8)                                   # warm-up: kernels loaded, graphs of small batches
        outs = generate(eng, prompts, new)
        prefill_s = max(o.prefill_time for o in outs)
        decode_s = max(o.decode_time for o in outs)
        n_dec = sum(len(o.tokens) - 1 for o in outs)
        esize = 2 if args.dtype == "bfloat16" else 4
        ms_step = decode_s / (new - 1) * 1e3
        # a decode step reads every weight once and the live cache: all 64 sequences, half-way through their 256 tokens
        step_b = weight_bytes_per_step(cfg, esize) + sum(n + new // 2 for n in lens) * kv_bytes_per_token(cfg, esize)
        read_gbs = calibrate_read(dev)
        achieved = step_b / (ms_step * 1e-3) / 1e9
        peak = PEAK_FLOPS["bf16" if args.dtype == "bfloat16" else "fp32"]
        rec = {"metric": "MiniCPM4-0.5B shape, 64 unequal prompts (128..2048), 256 new tokens each: decode tok/s through "
                         "the generation loop", "value": round(n_dec / decode_s, 1), "unit": "tokens/s", "n_gpus": 1,
               "steps": new - 1, "warmup": 0, "ms_per_step": round(decode_s / (new - 1) * 1e3, 4),
               "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
               "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic",
               "config": {"model": "MiniCPM4-0.5B shape, random weights N(0,0.02)", "layers": 24, "hidden": 1024,
                          "heads": 16, "kv_heads": 2, "head_dim": 64, "intermediate": 4096, "vocab": 73448,
                          "global_batch": 64, "prompt_tokens": sum(lens), "new_tokens": new, "parallelism": "1gpu",
                          "hip_graph": bool(args.hip_graph)},
               "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                            "frac": round(achieved / HBM_PEAK_GBS, 4), "bytes_per_step": step_b,
                            "read_kernel": round(read_gbs, 1), "frac_of_read_kernel": round(achieved / read_gbs, 4)},
               "prefill": {"value": round(sum(lens) / prefill_s, 1), "tokens": sum(lens), "ms": round(prefill_s * 1e3, 2),
                           "frac": round(batch_prefill_flops(cfg, lens) / prefill_s / peak, 4)}}
        if args.perf:
            rec["timers"] = timer_table(eng, lambda: generate(eng, prompts[:64], 4), "64 unequal prompts, 4 tokens each")
        print(json.dumps(rec), flush=True)
        return
    raw = config_8b(args.layers)
    raw["sparse_config"] = dict(SPARSE_32K)
    cfg = MiniCPMConfig.from_dict(raw)
    n_prompt, new = 32000, 256
    esize = 2 if args.dtype == "bfloat16" else 4
    peak = PEAK_FLOPS["bf16" if args.dtype == "bfloat16" else "fp32"]
    read_gbs = calibrate_read(dev)
    eng = Engine.from_tensors(cfg, random_tensors(cfg, 0, device=dev), EngineOptions(
        dtype=args.dtype, max_tokens=4 * 32768, max_slots=4, max_step_tokens=2048, device=dev,
        hip_graph=bool(args.hip_graph), rehearse=not args.no_rehearse))
    rec = {"metric": "MiniCPM4-8B shape with InfLLM-v2 at 32k context: decode tok/s at batch 1 after a 32,000-token prefill",
           "unit": "tokens/s", "n_gpus": 1, "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
           "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic",
           "config": {"model": "MiniCPM4-8B shape + sparse_config, random weights", "layers": cfg.num_hidden_layers,
                      "layers_full_model": 32, "kernel_size": 32, "kernel_stride": 16, "block_size": 64, "topk": 64,
                      "window_size": 2048, "dense_len": 8192, "prompt_tokens": n_prompt, "new_tokens": new,
                      "parallelism": "1gpu", "hip_graph": bool(args.hip_graph)}, "points": {}}
    # warm-up: one whole prompt and a few decode steps (kernel libraries loaded, the weights' decode layouts made,
    # scratch grown to this context's sizes; none of that belongs to a step)
    s = eng.acquire()
    warm = [int(t) for t in torch.randint(0, cfg.vocab_size, (n_prompt + 4,), generator=g)]
    for a in range(0, n_prompt, 2048):
        eng.step([StepEntry(s, warm[a:min(a + 2048, n_prompt)], [])])
    for i in range(4):
        eng.step([StepEntry(s, [warm[n_prompt + i]], [0])])
    eng.release(s)
    for batch in (1, 4):
        slots = [eng.acquire() for _ in range(batch)]
        ids = [[int(t) for t in torch.randint(0, cfg.vocab_size, (n_prompt + new,), generator=g)] for _ in slots]
        torch.cuda.synchronize()
        t = time.perf_counter()
        for sl, tok in zip(slots, ids):
            for a in range(0, n_prompt, 2048):
                eng.step([StepEntry(sl, tok[a:min(a + 2048, n_prompt)], [])])
        torch.cuda.synchronize()
        pre = time.perf_counter() - t
        for i in range(8):
            eng.step([StepEntry(sl, [tok[n_prompt + i]], [0]) for sl, tok in zip(slots, ids)])
        torch.cuda.synchronize()
        t = time.perf_counter()
        for i in range(8, new):
            eng.step([StepEntry(sl, [tok[n_prompt + i]], [0]) for sl, tok in zip(slots, ids)])
        torch.cuda.synchronize()
        dec = time.perf_counter() - t
        for sl in slots:
            eng.release(sl)
        ms_step = dec / (new - 8) * 1e3
        step_b = sparse_decode_bytes(cfg, SPARSE_32K, esize, batch, n_prompt + new // 2)
        achieved = step_b / (ms_step * 1e-3) / 1e9
        if batch == 1:
            rec.update({"value": round((new - 8) / dec, 2), "steps": new - 8, "warmup": 8,
                        "ms_per_step": round(ms_step, 4),
                        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                                     "frac": round(achieved / HBM_PEAK_GBS, 4), "bytes_per_step": step_b,
                                     "read_kernel": round(read_gbs, 1),
                                     "frac_of_read_kernel": round(achieved / read_gbs, 4)},
                        "prefill": {"value": round(n_prompt / pre, 1), "tokens": n_prompt, "ms": round(pre * 1e3, 1),
                                    "frac": round(sparse_prefill_flops(cfg, SPARSE_32K, n_prompt) / (pre / batch) / peak, 4)}})
        rec["points"][f"decode_b{batch}"] = round(batch * (new - 8) / dec, 2)
        rec["points"][f"decode_b{batch}_ms"] = round(ms_step, 4)
        rec["points"][f"decode_b{batch}_frac"] = round(achieved / HBM_PEAK_GBS, 4)
    if args.perf:
        def few_steps():
            sl = eng.acquire()
            for a in range(0, n_prompt, 2048):
                eng.step([StepEntry(sl, warm[a:min(a + 2048, n_prompt)], [])])
            for i in range(4):
                eng.step([StepEntry(sl, [warm[n_prompt + i]], [0])])
            eng.release(sl)
        rec["timers"] = timer_table(eng, few_steps, "a 32,000-token prompt in chunks of 2,048 and 4 decode steps")
    print(json.dumps(rec), flush=True)


if __name__ == "__main__":
    main()
