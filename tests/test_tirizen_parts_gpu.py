"""Tirizen's mechanisms alone, through their kernel entry points, against the plain implementation (GPU): the embedding
with learned positions into several streams; decays a channel; the recurrence in portions, segments and slots, with one
key that stands out far back; its single-token step; whole-row norms, temperature and gates on the way into the cache and
keys that stand out at page borders; streams with a scaled branch; routers by the logits; experts and feed-forwards without
a gate."""
import math

import pytest
import torch

import plain_tirizen as plain

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64


def dev(t, dtype=None):
    return t.to(DEV, dtype) if dtype is not None else t.to(DEV)


def i32(x):
    return dev(torch.as_tensor(x, dtype=torch.int32))


def close(got, want, dtype, scale=None, what=""):
    want = want.to(F64)
    tol = (2e-5 if dtype == "float32" else 1.5e-2) * float(scale if scale is not None else want.abs().max())
    err = float((got.detach().cpu().to(F64) - want).abs().max())
    assert err <= tol, f"{what} error {err:.3g} > {tol:.3g}"


# ---------------------------------------------------------------------------
# embedding and streams
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, S", [(96, 1), (100, 3), (33, 5), (1030, 8)])
def test_embedding_with_positions_into_streams(dtype, H, S):
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(91)
    table, pos_table = torch.randn(31, H, generator=g).to(DT[dtype]), torch.randn(50, H, generator=g).to(DT[dtype])
    ids, pos = torch.randint(0, 31, (9,), generator=g), torch.randint(0, 50, (9,), generator=g)
    want = table.double()[ids] * 3.5 + pos_table.double()[pos]
    out = torch.empty(S, 9, H, device=DEV)
    ops.embed(dev(table), i32(ids.tolist()), out, 3.5, dev(pos_table), i32(pos.tolist()))
    for s in range(S):
        close(out[s], want, "float32")
    flat = torch.empty(9, H, device=DEV)
    ops.embed(dev(table), i32(ids.tolist()), flat, 3.5, dev(pos_table), i32(pos.tolist()))
    assert torch.equal(flat, out[0])
    ops.embed(dev(table), i32(ids.tolist()), flat, -2.0)
    close(flat, table.double()[ids] * -2.0, "float32")


@pytest.mark.parametrize("S, H, n", [(1, 96, 3), (3, 100, 2), (5, 33, 4), (4, 1024, 8), (8, 64, 600)])
def test_streams_with_a_scaled_branch(S, H, n):
    """Join and read of two sub-layers in a row, the branch as one tensor and as partial sums, and the last norm over
    chosen rows, which leaves the streams as they are."""
    from cpmcu_amd.parts import NORMS
    from cpmcu_amd.parts.base import Runtime, StreamsBranch, Workspace
    g = torch.Generator().manual_seed(92)
    rnd = lambda *s: torch.randn(*s, generator=g)
    X, w, m, eps = rnd(S, n, H), rnd(H), 0.37, 1e-5
    norm = NORMS.build("rms_norm", name="w", hidden_size=H, eps=eps)
    norm.bind({"w": dev(w)}, Runtime(torch.device(DEV), torch.float32, Workspace(DEV), 64))
    ctx = type("Ctx", (), {"ws": Workspace(DEV)})()
    x, Xw = dev(X.clone()), X.double()
    for form in (1, 4):
        y = rnd(form, n, H) if form > 1 else rnd(n, H)
        read, mix, out = rnd(S), rnd(S, S), rnd(S)
        Xw = plain.join_streams(Xw, y.double().sum(0) if form > 1 else y.double(), mix.double(), out.double(), m)
        got = norm.forward_streams(x, StreamsBranch(dev(y), dev(mix), dev(out), m), dev(read), ctx)
        close(x, Xw, "float32", what="streams")
        close(got, plain.rms(torch.einsum("s,snw->nw", read.double(), Xw), eps) * w.double(), "float32", scale=4 * float(w.abs().max()), what="normed")
    y, mix, out = rnd(n, H), rnd(S, S), rnd(S)
    before = x.clone()
    rows = torch.tensor([n - 1, 0])
    got = norm.forward_streams(x, StreamsBranch(dev(y), dev(mix), dev(out), m), None, ctx, rows=i32(rows.tolist()))
    end = plain.join_streams(Xw, y.double(), mix.double(), out.double(), m).sum(0)[rows]
    close(got, plain.rms(end, eps) * w.double(), "float32", scale=4 * float(w.abs().max()), what="last norm")
    assert torch.equal(x, before)


# ---------------------------------------------------------------------------
# gated linear attention
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n, R, C, tau", [(1, 1, 5, 12.0), (9, 12, 84, 6.0), (30, 70, 300, 1.0), (17, 130, 257, 3.5)])
def test_decays_a_channel(dtype, n, R, C, tau):
    """Among them decays next to zero and next to one, which keep their relative precision, and that of 1 - a."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(93)
    low = torch.randn(n, R + 7, generator=g).to(DT[dtype])
    up, b = torch.randn(C, R, generator=g) * R ** -0.5, torch.randn(C, generator=g) * 3
    b[0], b[1] = 60.0, -60.0
    out = torch.empty(n, C, device=DEV)
    ops.channel_decay(dev(low)[:, 3:3 + R], dev(up.t().contiguous()), dev(b), tau, out)
    z = low[:, 3:3 + R].double() @ up.double().T + b.double()
    want = torch.exp(torch.nn.functional.logsigmoid(z) / tau)
    rel = ((out.cpu().double() - want).abs() / want).max()
    assert float(rel) < 2e-5 * max(1.0, 60.0 / tau), float(rel)
    assert bool((out <= 1.0).all()) and bool((out > 0).all())


def _gla_inputs(T, H, dk, dv, dtype, g, R=5):
    """Rows [k | q | pad | v | gate | low] of T tokens, the decay's product, and the plain recurrence's operands.  A key at
    token 3 stands out, in channels whose decay stays next to one, and queries far behind it ask for it."""
    hk, hv = H * dk, H * dv
    rnd = lambda *s: torch.randn(*s, generator=g)
    k, q, v, gate, low = rnd(T, H, dk) * 0.3, rnd(T, H, dk) * 0.3, rnd(T, H, dv), rnd(T, hv), rnd(T, R)
    up, b = rnd(hk, R) * 0.5, rnd(hk)
    b.view(H, dk)[:, 0] = 14.0
    up.view(H, dk, R)[:, 0] = 0.0
    if T > 4:
        k[3, :, 0] = 6.0
        q[T // 2::7, :, 0] = 6.0
        q[T - 1, :, 0] = 6.0
    rows = torch.cat([k.reshape(T, hk), q.reshape(T, hk), rnd(T, 3), v.reshape(T, hv), gate, low], 1).to(DT[dtype])
    offs = {"k": 0, "q": hk, "v": 2 * hk + 3, "g": 2 * hk + 3 + hv, "low": 2 * hk + 3 + 2 * hv}
    d = rows.double()
    at = lambda o, w: d[:, offs[o]:offs[o] + w]
    a = torch.exp(torch.nn.functional.logsigmoid(at("low", R) @ up.double().T + b.double()) / 4.0)
    ops_ = (at("q", hk).reshape(T, H, dk), at("k", hk).reshape(T, H, dk), at("v", hv).reshape(T, H, dv), a.view(T, H, dk))
    return rows, offs, up, b, ops_, at("g", hv)


SHAPES = [(3, 44, 28), (3, 20, 36), (5, 13, 7), (1, 200, 1), (2, 128, 48), (1, 256, 33), (4, 8, 24), (2, 70, 130), (1, 64, 64), (2, 33, 16)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, dk, dv", SHAPES)
def test_recurrence_in_portions_segments_and_slots(dtype, H, dk, dv):
    """Two sequences in slots 3 and 1, in portions of unequal sizes down to one token, uncut and cut into segments (some
    empty, the last one short); other slots stay as they were."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(94)
    lens = {3: 333, 1: 70}
    seqs = {s: _gla_inputs(T, H, dk, dv, dtype, g) for s, T in lens.items()}
    qs = dk ** -0.5
    want = {s: plain.recurrence(x[4][0] * qs, *x[4][1:]) for s, x in seqs.items()}
    for segments, seg in ((1, 0), (2, 128), (5, 64), (3, 64)):
        state = torch.zeros(5, H, dv, dk, device=DEV)
        state[0] = 5.0
        cuts = {3: [0, 1, 3, 141, 333], 1: [0, 2, 60, 61, 70]}
        got = {s: [] for s in lens}
        for step in range(4):
            batch = [(s, cuts[s][step], cuts[s][step + 1]) for s in (3, 1)]
            longest = max(b - a for _, a, b in batch)
            n_seg, sl = (segments, seg) if segments * seg >= longest else (1, 0)
            cu = [0]
            for s, a, b in batch:
                cu.append(cu[-1] + b - a)
            rows = dev(torch.cat([seqs[s][0][a:b] for s, a, b in batch]))
            decay = dev(torch.cat([seqs[s][4][3][a:b].reshape(b - a, H * dk).float() for s, a, b in batch]))
            n = cu[-1]
            y = torch.full((n, H * dv), float("nan"), device=DEV)
            scratch = None
            if n_seg > 1:
                scratch = (torch.full((2 * n_seg, H, dv, dk), float("nan"), device=DEV), torch.full((2 * n_seg, H, dk), float("nan"), device=DEV),
                           torch.full((n, H * dk), float("nan"), device=DEV))
            o = seqs[3][1]
            ops.gla_scan(rows, o["q"], o["k"], o["v"], decay, state, y, i32(cu), i32([3, 1]), H, dk, dv, qs, n_seg, sl, scratch)
            for i, (s, a, b) in enumerate(batch):
                got[s].append(y[cu[i]:cu[i + 1]].cpu())
        for s, T in lens.items():
            close(torch.cat(got[s]), want[s].reshape(T, H * dv), "float32", what=f"segments {segments} slot {s}")
        assert bool((state[0] == 5.0).all()) and bool((state[2] == 0).all()) and bool((state[4] == 0).all())
        q, k, v, a = seqs[1][4]
        S = torch.zeros(H, dk, dv, dtype=F64)
        for t in range(lens[1]):
            S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        close(state[1], S.transpose(1, 2), "float32", what="state")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, dk, dv", SHAPES)
@pytest.mark.parametrize("act", ["silu", "sigmoid"])
def test_single_token_steps(dtype, H, dk, dv, act):
    """Decays, recurrence, norm a head and gate in one launch, forty steps of three sequences whose slots change places in
    the batch, the shortest ending early."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(95)
    T, eps, qs = 40, 1e-5, 0.3
    slots = [4, 0, 2]
    seqs = [_gla_inputs(T, H, dk, dv, dtype, g) for _ in slots]
    for s in seqs:                                   # one product for all
        for i in (2, 3):
            s[i].copy_(seqs[0][i])
    w = torch.rand(dv, generator=g) + 0.5
    o, up, b = seqs[0][1], seqs[0][2], seqs[0][3]
    R = up.shape[1]
    state = torch.zeros(5, H, dv, dk, device=DEV)
    state[1] = 7.0
    args = (dev(up.t().contiguous()), dev(b), 4.0, dev(w), eps)
    got = [[] for _ in slots]
    for t in range(T):
        order = [(t + i) % 3 for i in range(3)]
        order = [i for i in order if i != 1 or t < 25]
        rows = dev(torch.stack([seqs[i][0][t] for i in order]))
        out = torch.empty(len(order), H * dv, dtype=DT[dtype], device=DEV)
        ops.gla_step(rows, o["q"], o["k"], o["v"], o["g"], o["low"], *args, state, out, i32(list(range(len(order) + 1))),
                     i32([slots[i] for i in order]), H, dk, dv, qs, act)
        for j, i in enumerate(order):
            got[i].append(out[j].cpu())
    for i, s in enumerate(seqs):
        n = 25 if i == 1 else T
        low = s[0].double()[:, o["low"]:o["low"] + R]
        a = torch.exp(torch.nn.functional.logsigmoid(low @ up.double().T + b.double()) / 4.0).view(T, H, dk)
        y = plain.recurrence(s[4][0] * qs, s[4][1], s[4][2], a)
        y = (plain.rms(y, eps) * w.double()).reshape(T, H * dv)
        y = y * (plain.silu(s[5]) if act == "silu" else torch.sigmoid(s[5]))
        close(torch.stack(got[i]), y[:n], dtype, what=f"sequence {i}")
    assert bool((state[1] == 7.0).all()) and bool((state[3] == 0).all())


# ---------------------------------------------------------------------------
# attention
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", [(6, 2, 24, 40, 0), (1, 1, 32, 16, 32), (3, 3, 20, 10, 8), (8, 1, 12, 22, 0), (4, 2, 128, 128, 64), (17, 1, 16, 8, 2)])
@pytest.mark.parametrize("parts", [1, 3, 11])
def test_whole_row_norms_into_the_cache(dtype, shape, parts):
    """Norms over all heads (one head's queries and keys far larger than the others'), the temperature, the rotation
    behind them, the gates' copy; rows as one tensor or as partial sums; positions around the temperature's steps.  Without
    keys of its own the call leaves the cache as it was."""
    from cpmcu_amd import ops
    H, G, d, dv, rd = shape
    g = torch.Generator().manual_seed(96)
    T, page, eps, coef, every = 70, 64, 1e-5, 0.8, 33
    W = H * d + G * (d + dv) + H
    src = torch.randn(parts, T, W, generator=g)
    src[..., :d] *= 9.0
    src[..., H * d:H * d + d] *= 7.0
    src = src.to(DT[dtype]) if parts == 1 else src
    row = src.double().sum(0)
    qn, kn = torch.rand(H * d, generator=g) + 0.5, torch.rand(G * d, generator=g) + 0.5
    inv = (300.0 ** (-torch.arange(0, rd, 2, dtype=F64) / max(rd, 1))) if rd else None

    def turn(x):
        if not rd:
            return x
        ang = torch.arange(T, dtype=F64)[:, None, None] * inv
        a, b = x[..., :rd // 2], x[..., rd // 2:rd]
        return torch.cat([a * torch.cos(ang) - b * torch.sin(ang), b * torch.cos(ang) + a * torch.sin(ang), x[..., rd:]], -1)
    q = turn(((plain.rms(row[:, :H * d], eps) * qn.double()) * plain.temperature(T, {"coef": coef, "every": every})[:, None]).view(T, H, d))
    k = turn((plain.rms(row[:, H * d:H * d + G * d], eps) * kn.double()).view(T, G, d))
    v = row[:, H * d + G * d:H * d + G * (d + dv)].view(T, G, dv)
    pk, pv = -(-d // 16) * 16, -(-dv // 16) * 16
    table = torch.tensor([[0, 0], [2, 1]], dtype=torch.int32)
    kp = torch.zeros(3, page, G * pk, dtype=DT[dtype], device=DEV)
    vp = torch.zeros(3, page, G * pv, dtype=DT[dtype], device=DEV)
    pos, slot = i32(list(range(T))), i32([1] * T)
    q_out = torch.empty(T, H * d, dtype=DT[dtype], device=DEV)
    gates = torch.empty(T, H, dtype=DT[dtype], device=DEV)
    rows = dev(src[0] if parts == 1 else src)
    kw = dict(temp_coef=coef, temp_every=every, gate_col=W - H, gate_out=gates)
    freq = dev(inv.float()) if rd else None
    ops.qkv_row_norm_store(rows, q_out, H, G, d, dv, rd, pos, slot, freq, 1.0, kp, vp, dev(table), page, dev(qn), dev(kn), eps, **kw)
    close(q_out, q.reshape(T, H * d), dtype, what="queries")
    close(gates, row[:, W - H:], dtype, what="gates")
    # the keys and values as the attention reads them: one query a key that only this key answers
    sure = torch.zeros(T, H, d, dtype=F64)
    for t in range(T):
        for h in range(H):
            sure[t, h] = k[t, h // (H // G)]
    got = torch.empty(T, H * dv, dtype=DT[dtype], device=DEV)
    qq = dev(sure.reshape(T, H * d).to(DT[dtype]))
    ops.attention_general(qq, got, H, G, d, dv, 0.5, kp, vp, dev(table), page, pos, slot)
    kd, vd = (k.to(DT[dtype]).double(), v.to(DT[dtype]).double())
    want = plain.causal_attention(sure.to(DT[dtype]).double(), kd, vd, 0.5)
    close(got, want.reshape(T, H * dv), dtype, scale=2 * float(want.abs().max()), what="attention over what was stored")
    before = kp.clone(), vp.clone()
    if parts == 1:
        borrowed = dev(torch.cat([src[0][:, :H * d], src[0][:, W - H:]], 1))
    else:
        borrowed = dev(torch.cat([src[..., :H * d], src[..., W - H:]], -1).contiguous())
    q2, g2 = torch.empty_like(q_out), torch.empty_like(gates)
    ops.qkv_row_norm_store(borrowed, q2, H, G, d, dv, rd, pos, slot, freq, 1.0, None, None, None, page, dev(qn), None, eps, write_kv=False,
                           temp_coef=coef, temp_every=every, gate_col=H * d, gate_out=g2)
    close(q2, q.reshape(T, H * d), dtype, what="queries without keys")
    assert torch.equal(g2, gates) and torch.equal(kp, before[0]) and torch.equal(vp, before[1])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, G, d, dv", [(6, 2, 24, 40), (4, 4, 80, 80), (8, 1, 128, 128)])
def test_far_keys_and_gated_heads(dtype, H, G, d, dv):
    """Over pages in disorder, whole prompts and single tokens (whole and split keys): for chosen queries one key's score
    stands far above the rest, at position 0, at both sides of page borders, far back, among hundreds alike; each head
    times its gate."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(97)
    T, page, scale = 700, 64, 0.4
    q, k, v = torch.randn(T, H, d, generator=g) * 0.3, torch.randn(T, G, d, generator=g) * 0.3, torch.randn(T, G, dv, generator=g)
    gate = torch.randn(T, H, generator=g)
    for i, (qp, kp_) in enumerate({1: 0, 63: 63, 64: 63, 65: 64, 130: 0, 300: 236, 511: 1, 512: 448, 699: 0, 698: 640}.items()):
        q[qp, :, (3 * i) % d] = 9.0
        k[kp_, :, (3 * i) % d] = 9.0
    q, k, v, gate = (t.to(DT[dtype]) for t in (q, k, v, gate))
    want = (plain.causal_attention(q.double(), k.double(), v.double(), scale) * torch.sigmoid(gate.double())[:, :, None]).reshape(T, H * dv)
    row = dev(torch.cat([q.reshape(T, H * d), k.reshape(T, G * d), v.reshape(T, G * dv)], 1))
    table = torch.zeros(2, 11, dtype=torch.int32)
    table[1] = torch.tensor([3, 0, 4, 1, 9, 10, 2, 8, 7, 5, 6])
    pk, pv = -(-d // 16) * 16, -(-dv // 16) * 16
    kp, vp = (torch.zeros(11, page, G * p, dtype=DT[dtype], device=DEV) for p in (pk, pv))
    pos, slot = i32(list(range(T))), i32([1] * T)
    q_out = torch.empty(T, H * d, dtype=DT[dtype], device=DEV)
    ops.qkv_rotate_store(row, q_out, H, G, d, dv, 0, pos, slot, None, 1.0, kp, vp, dev(table), page)

    class Ctx:
        pass
    for a, b in ((0, T), (699, 700), (698, 699), (512, 513), (64, 65)):
        ctx = Ctx()
        from cpmcu_amd.parts.base import Workspace
        ctx.max_pos, ctx.single_token, ctx.ws, ctx.extras, ctx.q_lens = b - 1, b - a == 1, Workspace(DEV), {}, [b - a]
        ctx.positions, ctx.tok_slot, ctx.kv_lens, ctx.n_seqs, ctx.n_tokens = pos[a:b], slot[a:b], [b], 1, b - a
        ctx.cu_q, ctx.seq_slot, ctx.seq_len = i32([0, b - a]), i32([1]), i32([b])
        heads = torch.empty(b - a, H * dv, device=DEV)
        fin = ops.HeadFinish(torch.empty(b - a, H * dv, dtype=DT[dtype], device=DEV), None, dev(gate)[a:b].contiguous(), False)
        done = ops.attention_any(q_out[a:b], heads, H, G, d, dv, scale, kp, vp, dev(table), page, ctx, finish=fin)
        if not done:
            ops.head_output(heads, fin.out, H, dv, ctx.positions, None, fin.gate)
        close(fin.out, want[a:b], dtype, scale=float(want.abs().max()), what=f"rows {a}..{b}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_temperature_with_norms_a_head(dtype):
    """The other kernel between projection and cache takes the temperature as well."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(98)
    T, H, d = 90, 3, 16
    x = torch.randn(T, H * d, generator=g).to(DT[dtype])
    scales = torch.rand(H, generator=g) + 0.5
    out = torch.empty(T, H * d, dtype=DT[dtype], device=DEV)
    ops.qkv_norm_rotate_store(dev(x), out, H, 1, d, d, 0, i32(list(range(T))), i32([0] * T), None, 1.0, None, None, None, 64, write_kv=False,
                              q_scale=dev(scales), temp_coef=0.6, temp_every=20)
    want = x.double().view(T, H, d) * scales.double()[:, None] * plain.temperature(T, {"coef": 0.6, "every": 20})[:, None, None]
    close(out, want.reshape(T, H * d), dtype)


# ---------------------------------------------------------------------------
# feed-forwards
@pytest.mark.parametrize("n, K, N", [(1, 96, 112), (5, 64, 33), (16, 1024, 300), (64, 200, 64), (17, 4096, 128)])
@pytest.mark.parametrize("act", ["relu_squared", "silu", "gelu_tanh"])
def test_product_with_a_nonlinearity(n, K, N, act):
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(99)
    x, w = torch.randn(n, K, generator=g).bfloat16(), (torch.randn(N, K, generator=g) * K ** -0.5).bfloat16()
    z = x.double() @ w.double().T
    f = {"relu_squared": plain.squared_relu, "silu": plain.silu,
         "gelu_tanh": lambda u: 0.5 * u * (1 + torch.tanh(math.sqrt(2 / math.pi) * (u + 0.044715 * u ** 3)))}[act]
    for weight in (dev(w), ops.TiledWeight(dev(w))):
        out = torch.empty(n, N, dtype=torch.bfloat16, device=DEV)
        ops.gemm_skinny(dev(x), weight, out, mode="act", activation=act)
        close(out, f(z), "bfloat16")
    for dtype in ("float32", "bfloat16"):
        t = z.to(DT[dtype])
        got = dev(t)
        ops.activate(got, act)
        close(got, f(t.double()), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("score", ["logit", "softmax", "sigmoid"])
@pytest.mark.parametrize("n, H, E, top", [(3, 96, 6, 3), (1, 100, 11, 2), (9, 64, 64, 6), (70, 96, 8, 8), (5, 33, 1, 1), (4, 64, 300, 4)])
def test_router_with_a_bias(dtype, score, n, H, E, top):
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(100)
    h = torch.randn(n, H, generator=g).to(DT[dtype])
    W = {"router": torch.randn(E, H, generator=g) * 2 * H ** -0.5, "router.b": torch.randn(E, generator=g) * 2}
    z = h.double() @ W["router"].double().T + W["router.b"].double()
    idx, wts = torch.empty(n, top, dtype=torch.int32, device=DEV), torch.empty(n, top, device=DEV)
    ops.moe_route(dev(h), dev(W["router"]), None, None, 1, 1, top, idx, wts, score=score, bias=dev(W["router.b"]))
    order, w_logit = plain.route(h.double(), {k: v.double() for k, v in W.items()}, "", top)
    assert torch.equal(idx.cpu().long(), order)
    s = torch.softmax(z, -1) if score == "softmax" else torch.sigmoid(z)
    want = w_logit if score == "logit" else s.gather(1, order) / s.gather(1, order).sum(-1, keepdim=True)
    close(wts, want, "float32", scale=1.0)
    # logits far below zero and far apart
    big = W["router.b"] * 100 - 500
    ops.moe_route(dev(h), dev(W["router"]), None, None, 1, 1, top, idx, wts, score="logit", bias=dev(big))
    order, w_logit = plain.route(h.double(), {"router": W["router"].double(), "router.b": big.double()}, "", top)
    assert torch.equal(idx.cpu().long(), order) and bool(torch.isfinite(wts).all())
    close(wts, w_logit, "float32", scale=10.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n, H, F, E, top", [(3, 96, 40, 6, 3), (1, 100, 20, 2, 1), (9, 64, 16, 64, 6), (130, 64, 24, 4, 2), (200, 128, 264, 3, 3),
                                             (70, 96, 30, 8, 8), (5, 512, 256, 12, 1), (600, 192, 72, 12, 3)])
def test_experts_without_a_gate(dtype, n, H, F, E, top):
    """The products for few tokens and, bfloat16, the grouped ones."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(101)
    W = {"router": torch.randn(E, H, generator=g) * 3 * H ** -0.5, "router.b": torch.randn(E, generator=g)}
    for e in range(E):
        for part, shape in (("up", (F, H)), ("down", (H, F))):
            W[f"e{e}.{part}"] = torch.randn(*shape, generator=g) * shape[1] ** -0.5
    W = {k: v.bfloat16() for k, v in W.items()}
    h = torch.randn(n, H, generator=g).to(DT[dtype])
    W64 = {k: v.double() for k, v in W.items()}
    idx, wts = plain.route(h.double(), W64, "", top)
    want = plain.experts(h.double(), W64, "", {"router": {"experts": E, "top": top}})
    idx, wts, hd = i32(idx), dev(wts.float()), dev(h)
    up, dn = (dev(torch.stack([W[f"e{e}.{p}"] for e in range(E)]), DT[dtype]) for p in ("up", "down"))
    act, out = torch.empty(n, top, F, dtype=DT[dtype], device=DEV), torch.empty(n, H, device=DEV)
    ops.moe_up(hd, up, idx, act, "relu_squared")
    ops.moe_down(act, dn, idx, wts, out, h=hd)
    close(out, want, dtype, what="few tokens")
    tiles = ops.moe_tiles(n, top, E)
    if ops.moe_experts_mfma_ok(hd, F, tiles):
        out2, y = torch.empty(n, H, device=DEV), torch.empty(n, top, H, dtype=torch.bfloat16, device=DEV)
        act2 = torch.full((n, top, F), float("nan"), dtype=torch.bfloat16, device=DEV)
        ops.moe_experts_mfma(hd, up, dn, idx, wts, out2, act2, y, torch.empty(tiles * ops.MOE_TILE, dtype=torch.int32, device=DEV),
                             torch.empty(tiles, dtype=torch.int32, device=DEV), torch.empty(1, dtype=torch.int32, device=DEV),
                             activation="relu_squared", gated=False)
        close(out2, want, dtype, what="grouped")
        close(act2, act.double().cpu(), dtype, what="grouped act")


def test_refusals():
    from cpmcu_amd import ops
    from cpmcu_amd.parts import Runtime, TokenEmbedding, Workspace
    z = lambda *s: torch.zeros(*s, device=DEV)
    zi = lambda *s: torch.zeros(*s, dtype=torch.int32, device=DEV)
    with pytest.raises(ops.KernelError, match="tau"):
        ops.channel_decay(z(2, 3), z(3, 4), z(4), 0.0, z(2, 4))
    with pytest.raises(ops.KernelError, match="at most 256"):
        ops.gla_scan(z(2, 900), 0, 300, 600, z(2, 300), z(1, 1, 300, 300), z(2, 300), zi(2), zi(1), 1, 300, 300, 1.0)
    with pytest.raises(ops.KernelError, match="columns"):
        ops.gla_scan(z(2, 20), 0, 8, 16, z(2, 8), z(1, 1, 8, 8), z(2, 8), zi(2), zi(1), 1, 8, 8, 1.0)
    with pytest.raises(ops.KernelError, match="columns"):
        ops.gla_step(z(1, 32), 0, 8, 16, 24, 32, z(2, 8), z(8), 1.0, z(8), 1e-5, z(1, 1, 8, 8), z(1, 8), zi(2), zi(1), 1, 8, 8, 1.0)
    with pytest.raises(ops.KernelError, match="gates"):
        ops.qkv_row_norm_store(z(2, 16), z(2, 16), 2, 1, 8, 8, 0, zi(2), None, None, 1.0, None, None, None, 64, z(16), None, 1e-5,
                               write_kv=False, gate_col=16, gate_out=z(2, 2))
    with pytest.raises(ops.KernelError, match="LDS"):
        ops.qkv_row_norm_store(z(1, 16384), z(1, 16384), 128, 1, 128, 128, 0, zi(1), None, None, 1.0, None, None, None, 64, z(16384), None,
                               1e-5, write_kv=False)
    with pytest.raises(ops.KernelError, match="clamped_swish"):
        ops.activate(z(8), "clamped_swish")
    with pytest.raises(ops.KernelError, match="normalised"):
        ops.moe_route(z(1, 8), z(2, 8), None, None, 1, 1, 1, zi(1, 1), z(1, 1), score="logit", normalize=False)
    e = TokenEmbedding("e", 4, 8, positions=("p", 100))
    with pytest.raises(ValueError, match="positions"):
        e.bind({"e": z(4, 8), "p": z(100, 8)}, Runtime(torch.device(DEV), torch.float32, Workspace(DEV), 101))
