"""Pemalorn's mechanisms alone, through their kernel entry points, against the plain implementation (GPU): the row
kernel that adds a branch (plain, normed, or in the residual's place), norms and convolves; the short convolutions in
portions and slots; the sum of two results and its copy for a product; the token table's gated lookup; rotated values
written, attended to and turned back, with one key made to stand out far back and at page borders; latent rows under a
window and a sink, with keys just inside and just outside the window; the product over heads with a gate a feature; the
router with identity experts, in every product that can run the experts."""
import math

import pytest
import torch

import plain_pemalorn as plain

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
# rows
@pytest.mark.parametrize("odt", ["float32", "bfloat16"])
@pytest.mark.parametrize("bdt", ["float32", "bfloat16"])
@pytest.mark.parametrize("n, H", [(3, 96), (1, 100), (5, 33), (2, 1030), (1, 5003), (7, 4096), (520, 256), (2, 8192), (600, 2052)])
def test_rows_added_normed_and_replaced(n, H, bdt, odt):
    """A branch as one tensor and as partial sums, with a bias, with a norm of its own, in the residual's place, absent;
    no norm, layer norm and RMS norm behind it; chosen rows only; rows of a wider tensor as output.  Widths for every
    way the kernel holds a row."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(71)
    rnd = lambda *s: torch.randn(*s, generator=g)
    x0, w, yw, bias = rnd(n, H) * 2 + 0.7, rnd(H) + 1, rnd(H), rnd(H)
    eps = 1e-5
    norms = {None: lambda t: t, "layer": lambda t: plain.layer_norm(t, w.double(), eps), "rms": lambda t: plain.rms(t, eps) * w.double()}
    parts = [rnd(n, H).to(DT[bdt]), rnd(3, n, H).to(DT[bdt])]
    for i, (norm, form) in enumerate([("layer", "normed"), ("layer", "replace"), (None, "normed"), ("rms", "bias"), ("layer", None),
                                      (None, "replace"), ("layer", "scaled")]):
        y = parts[i % 2]
        total = y.double().sum(0) if y.dim() == 3 else y.double()
        kw = {} if form is None else dict(branch=dev(y))
        x = x0.double()
        if form == "normed":
            kw.update(branch_norm=dev(yw), branch_eps=3e-4)
            x = x + plain.rms(total, 3e-4) * yw.double()
        elif form == "replace":
            kw.update(branch_bias=dev(bias), replace=True)
            x = total + bias.double()
        elif form == "bias":
            kw.update(branch_bias=dev(bias))
            x = x + total + bias.double()
        elif form == "scaled":
            kw.update(branch_scale=-0.3)
            x = x - 0.3 * total
        want = norms[norm](x)
        xg = dev(x0.clone())
        wide = torch.full((n, 2 * H), 9.0, dtype=DT[odt], device=DEV)
        out = wide[:, H:]                                  # columns of a wider tensor
        ops.norm_rows(xg, out, norm, dev(w) if norm else None, eps, **kw)
        close(out, want, odt, what=f"{norm} {form}")
        assert bool((wide[:, :H] == 9.0).all())
        close(xg, x, "float32", what="residual")
        rows = torch.tensor([n - 1, 0])
        xr = dev(x0.clone())
        picked = torch.empty(2, H, dtype=DT[odt], device=DEV)
        ops.norm_rows(xr, picked, norm, dev(w) if norm else None, eps, rows=i32(rows.tolist()), **kw)
        close(picked, want[rows], odt, what=f"{norm} {form} chosen rows")
        assert torch.equal(xr.cpu(), x0)
    xg = dev(x0.clone())
    ops.norm_rows(xg, None, None, branch=dev(parts[0]), branch_bias=dev(bias), replace=True)
    close(xg, parts[0].double() + bias.double(), "float32", what="replaced alone")


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 7])
@pytest.mark.parametrize("H", [96, 100, 51, 1032])
@pytest.mark.parametrize("idt, odt", [("float32", "float32"), ("float32", "bfloat16"), ("bfloat16", "bfloat16")])
def test_input_convolutions_in_portions_and_slots(taps, H, idt, odt):
    """Two sequences in slots 3 and 1, in portions of unequal sizes down to one token (shorter than what the filters
    remember); two filters over the same rows, and one alone; other slots stay as they were; a step that does not write
    leaves the slots as they were."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(72)
    lens = {3: 43, 1: 12}
    ws = [torch.randn(H, taps, generator=g) for _ in range(2)]
    rows = {s: torch.randn(L, H, generator=g).to(DT[idt]) for s, L in lens.items()}
    state = torch.zeros(4, max(taps - 1, 1), H, device=DEV)
    state[0] = 5.0
    state = state[:, :taps - 1].contiguous() if taps > 1 else None
    wd = [dev(w.t().contiguous()) for w in ws]
    cuts = {3: [0, 1, 3, 12, 42, 43], 1: [0, 2, 12]}
    got = {s: ([], []) for s in lens}

    def run(batch, n_convs=2, write=True):
        cu = [0]
        for s, a, b in batch:
            cu.append(cu[-1] + b - a)
        h = dev(torch.cat([rows[s][a:b] for s, a, b in batch]))
        outs = [torch.empty(cu[-1], H, dtype=DT[odt], device=DEV) for _ in range(n_convs)]
        ops.conv_rows(h, wd[:n_convs], state, outs, i32(cu), i32([s for s, _, _ in batch]), max(b - a for _, a, b in batch), write)
        return [[o[cu[i]:cu[i + 1]].cpu() for i in range(len(batch))] for o in outs]
    for step in range(5):
        batch = [(s, cuts[s][step], cuts[s][step + 1]) for s in (3, 1) if step + 1 < len(cuts[s])]
        before = state.clone() if state is not None else None
        probe = run(batch, 1, write=False)
        if state is not None:
            assert torch.equal(state, before)
        outs = run(batch)
        for i, (s, _, _) in enumerate(batch):
            assert torch.equal(probe[0][i], outs[0][i])
            for k in range(2):
                got[s][k].append(outs[k][i])
    for s, L in lens.items():
        for k in range(2):
            want = rows[s].double() + plain.causal_conv(rows[s].double(), ws[k].double())
            close(torch.cat(got[s][k]), want, odt, what=f"slot {s} filter {k}")
        if taps > 1:
            close(state[s], rows[s][-(taps - 1):].double(), "float32")
    if taps > 1:
        assert bool((state[0] == 5.0).all()) and bool((state[2] == 0).all())


@pytest.mark.parametrize("taps", [1, 2, 4, 6])
@pytest.mark.parametrize("H", [64, 100, 33, 4096])
@pytest.mark.parametrize("odt", ["float32", "bfloat16"])
def test_norm_and_convolutions_of_single_tokens_in_one_launch(taps, H, odt):
    """Steps of one token a sequence: branch, norm and both convolutions at once, fifteen steps from the sequences'
    start with slots in another order every step, against norm and convolution of the whole rows."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(73)
    T, eps = 15, 1e-5
    ws = [torch.randn(H, taps, generator=g) for _ in range(2)]
    w, yw = torch.randn(H, generator=g), torch.randn(H, generator=g)
    x, y = torch.randn(2, T, H, generator=g) * 3, torch.randn(2, T, H, generator=g)
    state = torch.zeros(3, taps - 1, H, device=DEV) if taps > 1 else None
    slot = [2, 0]
    for t in range(T):
        order = [0, 1] if t % 2 else [1, 0]
        xg, yg = dev(x[order, t].contiguous()), dev(y[order, t].contiguous())
        outs = [torch.empty(2, H, dtype=DT[odt], device=DEV) for _ in range(2)]
        ops.norm_rows(xg, outs[0], "layer", dev(w), eps, branch=yg, branch_norm=dev(yw), branch_eps=eps,
                      convs=[dev(c.t().contiguous()) for c in ws], conv_state=state, slots=i32([slot[s] for s in order]), out2=outs[1])
        for i, s in enumerate(order):
            full = x[s, :t + 1].double() + plain.rms(y[s, :t + 1].double(), eps) * yw.double()
            h = plain.layer_norm(full, w.double(), eps)
            for k in range(2):
                close(outs[k][i], (h + plain.causal_conv(h, ws[k].double()))[t], odt, scale=float(h.abs().max()) * taps, what=f"step {t} filter {k}")
    if taps > 1:
        assert bool((state[1] == 0).all())


@pytest.mark.parametrize("n, H, dts", [(3, 96, ("float32", "float32", "bfloat16")), (5, 33, ("bfloat16", "float32", "float32")),
                                       (300, 256, ("bfloat16", "bfloat16", "bfloat16")), (2, 100, ("float32", "bfloat16", "float32"))])
def test_sum_of_two_results_into_the_residual(n, H, dts):
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(74)
    x0 = torch.randn(n, H, generator=g)
    a = torch.randn(*((4, n, H) if dts[0] == "float32" else (n, H)), generator=g).to(DT[dts[0]])
    f = torch.randn(n, H, generator=g).to(DT[dts[1]])
    ab, fb = torch.randn(H, generator=g), torch.randn(H, generator=g)
    total = lambda t: t.double().sum(0) if t.dim() == 3 else t.double()
    for with_f, biased, copied in ((True, True, True), (False, True, True), (True, False, False), (None, False, True)):
        want = x0.double()
        if with_f is not None:
            want = want + total(a) + (ab.double() if biased else 0)
        if with_f:
            want = want + total(f) + (fb.double() if biased else 0)
        x = dev(x0.clone())
        wide = torch.zeros(n, 2 * H, dtype=DT[dts[2]], device=DEV)
        ops.add_rows(x, dev(a) if with_f is not None else None, dev(ab) if biased else None, dev(f) if with_f else None,
                     dev(fb) if (biased and with_f) else None, wide[:, :H] if copied else None)
        close(x, want, "float32")
        close(wide, torch.cat([want if copied else want * 0, want * 0], 1), dts[2], scale=float(want.abs().max()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("D, off, parts", [(12, 24, 1), (1, 3, 2), (128, 0, 5), (13, 39, 1)])
def test_gated_lookup_of_the_token_table(dtype, D, off, parts):
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(75)
    n, V = 9, 31
    table = torch.randn(V, off + D + 7, generator=g).to(DT[dtype])
    ids = torch.randint(0, V, (n,), generator=g)
    z = torch.randn(*((parts, n, D) if parts > 1 else (n, D)), generator=g) * 2
    if parts == 1:
        z = z.to(DT[dtype])
    zz = z.double().sum(0) if parts > 1 else z.double()
    out = torch.empty(n, D, dtype=DT[dtype], device=DEV)
    ops.gated_lookup(dev(z), dev(table), off, i32(ids.tolist()), out)
    close(out, plain.gelu_tanh(zz) * table.double()[ids][:, off:off + D], dtype)


@pytest.mark.parametrize("n, K, D, off", [(1, 96, 12, 24), (8, 4096, 256, 256), (16, 1000, 40, 3), (5, 64, 1, 0), (3, 200, 17, 5)])
def test_product_and_lookup_in_one_launch(n, K, D, off):
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(81)
    x, w = torch.randn(n, K, generator=g).bfloat16(), (torch.randn(D, K, generator=g) * K ** -0.5).bfloat16()
    table, ids = torch.randn(23, off + D + 2, generator=g).bfloat16(), torch.randint(0, 23, (n,), generator=g)
    out = torch.empty(n, D, dtype=torch.bfloat16, device=DEV)
    ops.lookup_strip(dev(x), ops.TiledWeight(dev(w)), dev(table), off, i32(ids.tolist()), out)
    close(out, plain.gelu_tanh(x.double() @ w.double().T) * table.double()[ids][:, off:off + D], "bfloat16")
    with pytest.raises(ops.KernelError, match="tokens"):
        ops.lookup_strip(torch.zeros(17, K, dtype=torch.bfloat16, device=DEV), ops.TiledWeight(dev(w)), dev(table), off,
                         torch.zeros(17, dtype=torch.int32, device=DEV), torch.empty(17, D, dtype=torch.bfloat16, device=DEV))


# ---------------------------------------------------------------------------
# rotated values, a number a head on the scores, a sink and a gate a head
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", [(6, 2, 24, 40, 8), (1, 1, 32, 16, 32), (3, 3, 20, 10, 0), (5, 1, 12, 22, 6), (4, 2, 128, 128, 64),
                                   (4, 1, 16, 64, 16), (17, 1, 16, 8, 2), (2, 1, 64, 160, 64)])
def test_rotated_values_through_the_cache(dtype, shape):
    """Whole prompts and single tokens (whole and split keys) over pages in disorder.  For chosen queries one key's score
    stands far above the rest: at position 0, one page back, at both sides of a page border, far back; the output is
    then that key's value turned by the distance between the two positions, which is wrong if either rotation is.
    Other queries see hundreds of keys alike."""
    from cpmcu_amd import ops
    H, G, d, dv, rd = shape
    g = torch.Generator().manual_seed(76)
    T, page, base, scale = 700, 64, 300.0, 0.4
    q, k = torch.randn(T, H, d, generator=g) * 0.3, torch.randn(T, G, d, generator=g) * 0.3
    v = torch.randn(T, G, dv, generator=g)
    temp, sink = 0.5 + torch.rand(H, generator=g), torch.randn(H, generator=g)
    rot = {"base": base, "dims": rd}
    gate = torch.randn(T, H, generator=g)
    for i, (qp, kp_) in enumerate({1: 0, 63: 63, 64: 63, 65: 64, 130: 0, 300: 236, 511: 1, 512: 448, 699: 0, 698: 640}.items()):
        # equal vectors at the positions themselves, undone for the rotation: the score after it is the largest
        u = torch.zeros(d)
        u[(rd + 3 * i) % d if rd < d else (3 * i) % d] = 9.0
        back = lambda pos: plain.turn(torch.stack([u] * T)[:, None].double(), plain.frequencies(rot)[0], 1.0, "halves", -1.0)[pos, 0].float() if rd else u
        q[qp], k[kp_] = back(qp), back(kp_)
    q, k, v, gate = (t.to(DT[dtype]) for t in (q, k, v, gate))
    qr, kr = plain.rotate(q.double(), rot, "halves"), plain.rotate(k.double(), rot, "halves")
    vr = plain.turn_values(v.double(), base, 1.0)
    # what the kernel stores (scores of 30 would magnify the rounding of queries and keys to bfloat16)
    qt, kr, vr = ((t.to(DT[dtype]).double() for t in (qr * temp.double()[:, None], kr, vr)))
    outs = []
    for h in range(H):
        wts = plain.sink_softmax(qt[:, h] @ kr[:, h // (H // G)].T * scale, plain.visible(T), sink[h].double())
        outs.append(wts @ vr[:, h // (H // G)])
    want = (plain.turn_values(torch.stack(outs, 1), base, -1.0) * torch.sigmoid(gate.double())[:, :, None]).reshape(T, H * dv)
    row = dev(torch.cat([q.reshape(T, H * d), k.reshape(T, G * d), v.reshape(T, G * dv), gate], 1))
    table = torch.zeros(2, 11, dtype=torch.int32)
    table[1] = torch.tensor([3, 0, 4, 1, 9, 10, 2, 8, 7, 5, 6])
    pk, pv = -(-d // 16) * 16, -(-dv // 16) * 16
    kp = torch.zeros(11, page, G * pk, dtype=DT[dtype], device=DEV)
    vp = torch.zeros(11, page, G * pv, dtype=DT[dtype], device=DEV)
    pos, slot = i32(list(range(T))), i32([1] * T)
    freq = lambda n: dev((base ** (-torch.arange(0, n, 2, dtype=F64) / n)).float()) if n else None
    q_out = torch.empty(T, H * d, dtype=DT[dtype], device=DEV)
    ops.qkv_norm_rotate_store(row, q_out, H, G, d, dv, rd, pos, slot, freq(rd), 1.0, kp, vp, dev(table), page, q_scale=dev(temp),
                              v_inv_freq=freq(dv))
    close(q_out, qt.reshape(T, H * d), dtype, what="queries")
    gcol = row[:, H * d + G * (d + dv):]

    def finish(a, b, heads):
        out = torch.empty(b - a, H * dv, dtype=DT[dtype], device=DEV)
        ops.head_output(heads, out, H, dv, pos[a:b], freq(dv), gcol[a:b])
        return out
    heads = torch.empty(T, H * dv, dtype=DT[dtype], device=DEV)
    ops.attention_general(q_out, heads, H, G, d, dv, scale, kp, vp, dev(table), page, pos, slot, sink=dev(sink))
    close(finish(0, T, heads), want, dtype, what="plain kernel")
    if dtype != "bfloat16" or d % 8:
        return
    cases = [(0, T, 1, False), (699, 700, 1, False), (699, 700, 4, False), (511, 513, 3, False), (64, 66, 1, False)]
    if H // G <= 8:
        cases.append((0, T, 1, True))
    for a, b, splits, tiled in cases:
        heads = torch.empty(b - a, H * dv, device=DEV)
        po = torch.empty(b - a, H, splits, dv, device=DEV) if splits > 1 else None
        pm = torch.empty(b - a, H, splits, 2, device=DEV) if splits > 1 else None
        tiles, tpt = None, 1
        if tiled:
            tpt = ops.attention_general_tokens_per_tile(b - a, H, G, pv)
            tiles = ops.prefill_tiles([b - a], tpt, DEV)
        ops.attention_general_mfma(q_out[a:b], heads, H, G, d, dv, scale, kp, vp, dev(table), page, pos[a:b], slot[a:b], 0, splits,
                                   po, pm, tiles, tpt, sink=dev(sink))
        close(finish(a, b, heads), want[a:b], "bfloat16", scale=float(want.abs().max()), what=f"matrix cores rows {a}..{b} splits {splits} tiled {tiled}")
        if splits > 1:               # the merge of the shares turns back and gates on its way
            out = torch.empty(b - a, H * dv, dtype=torch.bfloat16, device=DEV)
            ops.attention_general_mfma(q_out[a:b], out, H, G, d, dv, scale, kp, vp, dev(table), page, pos[a:b], slot[a:b], 0, splits,
                                       po, pm, sink=dev(sink), v_inv_freq=freq(dv), head_gate=gcol[a:b])
            close(out, want[a:b], "bfloat16", scale=float(want.abs().max()), what=f"merge rows {a}..{b} splits {splits}")
            ops.attention_general_mfma(q_out[a:b], out, H, G, d, dv, scale, kp, vp, dev(table), page, pos[a:b], slot[a:b], 0, splits,
                                       po, pm, sink=dev(sink), head_gate=gcol[a:b])
            gated = heads.double().cpu().reshape(b - a, H, dv) * torch.sigmoid(gate[a:b].double())[:, :, None]
            close(out, gated.reshape(b - a, H * dv), "bfloat16", what="merge with the gate alone")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_heads_turned_back_and_gated(dtype):
    """head_output's forms: only turned, only gated, neighbouring pairs, float rows into a bfloat16 result."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(77)
    n, H, dv, base = 40, 3, 20, 90.0
    o, gate = torch.randn(n, H * dv, generator=g), torch.randn(n, H + 4, generator=g).to(DT[dtype])
    inv = (base ** (-torch.arange(0, dv, 2, dtype=F64) / dv)).float()
    for inter in (False, True):
        for turned in (False, True):
            for gated in (False, True):
                want = o.double().reshape(n, H, dv)
                if turned:
                    want = plain.turn(want, inv.double(), 1.0, "interleaved" if inter else "halves", -1.0)
                if gated:
                    want = want * torch.sigmoid(gate[:, 2:2 + H].double())[:, :, None]
                out = torch.empty(n, H * dv, dtype=DT[dtype], device=DEV)
                ops.head_output(dev(o), out, H, dv, i32(list(range(n))), dev(inv) if turned else None,
                                dev(gate)[:, 2:2 + H] if gated else None, interleaved=inter)
                close(out, want.reshape(n, H * dv), dtype, what=f"{inter} {turned} {gated}")


# ---------------------------------------------------------------------------
# latent rows
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", [(3, 24, 8, 56, 48, 20), (4, 20, 4, 36, 27, 33), (8, 16, 8, 32, 64, 64), (2, 16, 16, 64, 24, 1),
                                   (18, 8, 16, 136, 40, 70), (5, 128, 64, 512, 96, 100), (2, 32, 8, 64, 24, 0)])
def test_latent_rows_under_a_window_with_a_sink(dtype, shape):
    """The query latent's norm, the cache's rows (normed latent, rotated shared key part, neighbouring pairs, YaRN's
    magnitude) and the rotated query parts, each call with its own sources; then attention in the latent space.  For
    chosen queries one key stands far out: even queries' stands just outside the window and must not be seen, odd
    queries' is the oldest that is (at page borders, at position 0, far back)."""
    from cpmcu_amd import ops
    H, dim, rot, R, q_rank, window = shape
    g = torch.Generator().manual_seed(78)
    T, page, eps, scale = 300, 64, 1e-5, 0.05
    sc = {"base": 400.0, "dims": rot, "scaling": {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    f, mag = plain.frequencies(sc)
    proj = torch.randn(T, 3 + q_rank + R + rot + 5, generator=g)
    qsrc = torch.randn(T, 2 + H * (dim + rot), generator=g)
    qn, cn, sink = torch.rand(q_rank, generator=g) + 0.5, torch.rand(R, generator=g) + 0.5, torch.randn(H, generator=g)
    proj, qsrc = proj.to(DT[dtype]), qsrc.to(DT[dtype])
    c_in, r_in = proj[:, 3 + q_rank:3 + q_rank + R].double(), proj[:, 3 + q_rank + R:3 + q_rank + R + rot].double()
    c = plain.rms(c_in, eps) * cn.double()
    r = plain.turn(r_in[:, None], f, mag, "interleaved")[:, 0]
    q_rot = plain.turn(qsrc[:, 2:].double().reshape(T, H, dim + rot)[..., dim:], f, mag, "interleaved")
    q_lat = torch.randn(T, H, R, generator=g).to(DT[dtype])
    w = window or T
    for qp in (w - 1, w, 150, 151, 190, 191, 255, 256, 299):
        if 0 <= qp < T:
            kp_ = max(qp - w + 1, 0) if qp % 2 else max(qp - w, 0)
            q_lat[qp] = (c[kp_] * 40.0 / float(c[kp_].norm()) / scale / float(c[kp_].norm())).to(DT[dtype])    # a score of 40
    table = torch.zeros(2, 5, dtype=torch.int32)
    table[1] = torch.tensor([3, 0, 4, 1, 2])
    pk, pv = -(-(R + rot) // 16) * 16, -(-R // 16) * 16
    kpool = torch.zeros(5, page, pk, dtype=DT[dtype], device=DEV)
    vpool = torch.zeros(5, page, pv, dtype=DT[dtype], device=DEV)
    pos, slot, inv = i32(list(range(T))), i32([1] * T), dev(f.float())
    q = torch.empty(T, H, R + rot, dtype=DT[dtype], device=DEV)
    q[:, :, :R] = dev(q_lat)
    q2 = q.view(T, H * (R + rot))
    cq = torch.empty(T, q_rank, dtype=DT[dtype], device=DEV)
    pd = dev(proj)
    args = (q2, H, dim, rot, R, eps, pos, slot, inv, mag)
    ops.latent_store(*args, cq_src=pd[:, 3:3 + q_rank], cq_norm_w=dev(qn), cq_out=cq, down=pd[:, 3 + q_rank:3 + q_rank + R + rot],
                     norm_w=dev(cn), kpool=kpool, vpool=vpool, page_table=dev(table), page_size=page, interleaved=True)
    close(cq, plain.rms(proj[:, 3:3 + q_rank].double(), eps) * qn.double(), dtype, what="query latent")
    assert torch.equal(q[:, :, :R].cpu(), q_lat)
    ops.latent_store(*args, q_src=dev(qsrc)[:, 2:], interleaved=True)
    close(q[:, :, R:], q_rot, dtype, what="rotated query parts")
    assert torch.equal(q[:, :, :R].cpu(), q_lat)
    outs = []
    for h in range(H):
        s = (q_lat[:, h].double() @ c.T + q_rot[:, h] @ r.T) * scale
        outs.append(plain.sink_softmax(s, plain.visible(T, window or None), sink[h].double()) @ c)
    want = torch.stack(outs, 1).reshape(T, H * R)
    out = torch.empty(T, H * R, dtype=DT[dtype], device=DEV)
    ops.attention_general(q2, out, H, 1, R + rot, R, scale, kpool, vpool, dev(table), page, pos, slot, window=window, sink=dev(sink))
    close(out, want, dtype, scale=float(want.abs().max()) * (1 if dtype == "float32" else 2), what="plain kernel")
    if dtype != "bfloat16" or (R + rot) % 8:
        return
    cases = [(0, T, 1, False), (T - 1, T, 1, False), (T - 1, T, 3, False), (255, 257, 2, False), (150, 152, 1, False)]
    if H <= 8:
        cases.append((0, T, 1, True))
    for a, b, splits, tiled in cases:
        out = torch.empty(b - a, H * R, dtype=torch.bfloat16, device=DEV)
        po = torch.empty(b - a, H, splits, R, device=DEV) if splits > 1 else None
        pm = torch.empty(b - a, H, splits, 2, device=DEV) if splits > 1 else None
        tiles, tpt = None, 1
        if tiled:
            tpt = ops.attention_general_tokens_per_tile(b - a, H, 1, pv)
            tiles = ops.prefill_tiles([b - a], tpt, DEV)
        ops.attention_general_mfma(q2[a:b], out, H, 1, R + rot, R, scale, kpool, vpool, dev(table), page, pos[a:b], slot[a:b], 0,
                                   splits, po, pm, tiles, tpt, window=window, sink=dev(sink))
        close(out, want[a:b], "bfloat16", scale=float(want.abs().max()) * 2, what=f"matrix cores rows {a}..{b} splits {splits} tiled {tiled}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("M, H, N, K", [(3, 5, 24, 40), (70, 3, 12, 36), (17, 2, 128, 512), (1, 8, 40, 16), (300, 4, 65, 64)])
def test_product_over_heads_with_a_gate_a_feature(dtype, M, H, N, K):
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(79)
    x = torch.randn(M, H * K, generator=g).to(DT[dtype])
    w = (torch.randn(H, N, K, generator=g) * K ** -0.5).to(DT[dtype])
    gate = torch.randn(M, 3 + H * N, generator=g).to(DT[dtype])
    want = torch.einsum("mhk,hnk->mhn", x.double().reshape(M, H, K), w.double()).reshape(M, H * N) * torch.sigmoid(gate[:, 3:].double())
    for plain_kernel in (False, True):
        out = torch.empty(M, H * N, dtype=DT[dtype], device=DEV)
        ops.gemm_heads(dev(x), 0, K, dev(w), out, 0, N, gate=dev(gate)[:, 3:], plain=plain_kernel)
        close(out, want, dtype)


@pytest.mark.parametrize("dims, base, scaling", [(8, 500.0, (4.0, 64, 16.0, 1.0)), (24, 2e5, (3.0, 700, 20.0, 1.5)), (2, 20.0, (8.0, 32, 4.0, 1.0)),
                                                 (64, 10000.0, (40.0, 4096, 32.0, 1.0))])
def test_stretched_frequencies(dims, base, scaling):
    from cpmcu_amd.parts import POSITION_ENCODINGS, Runtime, Workspace
    pe = POSITION_ENCODINGS.build("yarn", head_dim=dims, theta=base, factor=scaling[0], original=scaling[1], fast=scaling[2], slow=scaling[3],
                                  pairs="interleaved")
    pe.bind({}, Runtime(torch.device(DEV), torch.float32, Workspace(DEV), 64))
    inv, mag = pe.rotary_params()
    f, m = plain.frequencies({"dims": dims, "base": base, "scaling": dict(zip(("factor", "original", "fast", "slow"), scaling))})
    assert pe.pairs == "interleaved" and abs(mag - m) < 1e-12
    assert float((inv.cpu().double() / f - 1).abs().max()) < 1e-6


# ---------------------------------------------------------------------------
# experts
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n, H, F, E, I, top", [(3, 96, 40, 6, 3, 3), (1, 100, 20, 2, 9, 3), (9, 64, 16, 64, 64, 6), (130, 64, 24, 4, 4, 2),
                                                (200, 128, 64, 1, 8, 5), (70, 96, 32, 8, 0, 8), (5, 512, 256, 12, 3, 1)])
def test_experts_and_identity_experts(dtype, n, H, F, E, I, top):
    """Softmax over experts and identity experts, a correction in the choice only, weights as the scores are; tokens all
    of whose choices are identity experts, and none; the products for few tokens and, bfloat16, the grouped ones."""
    from cpmcu_amd import ops
    g = torch.Generator().manual_seed(80)
    W = {"router": torch.randn(E + I, H, generator=g) * 3 * H ** -0.5, "correction": torch.randn(E + I, generator=g) * 0.05}
    for e in range(E):
        for part, shape in (("gate", (F, H)), ("up", (F, H)), ("down", (H, F))):
            W[f"e{e}.{part}"] = torch.randn(*shape, generator=g) * shape[1] ** -0.5
    W = {k: v.bfloat16() for k, v in W.items()}
    h = torch.randn(n, H, generator=g).to(DT[dtype])
    if n > 2 and I >= top:
        W["correction"][0] = 0.0
        h[1] = (W["router"][E:].float().sum(0) * 4).to(DT[dtype])        # identity experts take this token
    W64 = {k: v.double() for k, v in W.items()}
    mlp = {"router": {"experts": E, "identity": I, "top": top}, "expert": {"ff": F}}
    margins = []
    idx_want, w_want = plain.route(h.double(), W64, "", mlp["router"], margins)
    idx, wts = torch.empty(n, top, dtype=torch.int32, device=DEV), torch.empty(n, top, device=DEV)
    hd = dev(h)
    ops.moe_route(hd, dev(W["router"].float()), dev(W["correction"].float()), None, 1, 1, top, idx, wts, normalize=False)
    sure = margins[0] > 1e-4
    assert bool(sure.any()) and torch.equal(idx.cpu().long()[sure], idx_want[sure])
    close(wts[dev(sure)], w_want[sure], "float32", scale=1.0)
    # a choice that float rounding decides is taken as the kernel made it
    idx_c, w_c = idx.cpu().long(), wts.cpu().double()
    want = torch.zeros(n, H, dtype=F64)
    for e in range(E + I):
        t, k = (idx_c == e).nonzero(as_tuple=True)
        if t.numel():
            want[t] += w_c[t, k][:, None] * (plain.expert(h[t].double(), W64, f"e{e}.") if e < E else h[t].double())
    if bool(sure.all()):
        close(want, plain.experts(h.double(), W64, "", mlp), "float32")
    gu = dev(torch.stack([torch.cat([W[f"e{e}.gate"], W[f"e{e}.up"]]) for e in range(E)]), DT[dtype])
    dn = dev(torch.stack([W[f"e{e}.down"] for e in range(E)]), DT[dtype])
    act = torch.full((n, top, F), float("nan"), dtype=DT[dtype], device=DEV)      # identity pairs' rows are never read
    out = torch.empty(n, H, device=DEV)
    ops.moe_gated(hd, gu, idx, act)
    ops.moe_down(act, dn, idx, wts, out, h=hd)
    close(out, want, dtype, what="few tokens")
    # the router's products by the library, the choice from them
    if dtype == "bfloat16":
        rows = torch.cat([W["router"], torch.zeros(1, H, dtype=torch.bfloat16)])
        logits = torch.empty(n, E + I + 1, device=DEV)
        torch.mm(hd, dev(rows).t(), out_dtype=torch.float32, out=logits)
        idx3, wts3 = torch.empty_like(idx), torch.empty_like(wts)
        ops.moe_route(hd, dev(W["router"].float()), dev(W["correction"].float()), None, 1, 1, top, idx3, wts3, None, logits,
                      normalize=False, logits_ready=True)
        assert torch.equal(idx3.cpu().long()[sure], idx_want[sure])
        close(wts3[dev(sure)], w_want[sure], "float32", scale=1.0)

    def joined(run):
        """The same with the layer's sum ended there: another result (float parts, a bf16 tensor with a bias, none)."""
        for a, bias in ((torch.randn(5, n, H, generator=g), None), (torch.randn(n, H, generator=g).bfloat16(), torch.randn(H, generator=g)), (None, None)):
            x0 = torch.randn(n, H, generator=g)
            x, copy = dev(x0.clone()), torch.empty(n, H, dtype=DT[dtype], device=DEV)
            run(ops.Join(x, dev(a) if a is not None else None, dev(bias) if bias is not None else None, copy))
            total = x0.double() + want + (0 if a is None else (a.double().sum(0) if a.dim() == 3 else a.double())) + (0 if bias is None else bias.double())
            close(x, total, dtype, scale=float(want.abs().max()) if dtype == "bfloat16" else None, what="joined")
            close(copy, total, dtype, what="copy of the joined residual")
    joined(lambda j: ops.moe_down(act, dn, idx, wts, None, h=hd, join=j))
    tiles = ops.moe_tiles(n, top, E)
    if ops.moe_experts_mfma_ok(hd, F, tiles):
        out2 = torch.empty(n, H, device=DEV)
        y = torch.full((n, top, H), float("nan"), dtype=torch.bfloat16, device=DEV)
        act2 = torch.full((n, top, F), float("nan"), dtype=torch.bfloat16, device=DEV)
        ops.moe_experts_mfma(hd, gu, dn, idx, wts, out2, act2, y, torch.empty(tiles * ops.MOE_TILE, dtype=torch.int32, device=DEV),
                             torch.empty(tiles, dtype=torch.int32, device=DEV), torch.empty(1, dtype=torch.int32, device=DEV))
        close(out2, want, dtype, what="grouped")
        joined(lambda j: ops.moe_experts_mfma(hd, gu, dn, idx, wts, None, act2, y, torch.empty(tiles * ops.MOE_TILE, dtype=torch.int32, device=DEV),
                                              torch.empty(tiles, dtype=torch.int32, device=DEV), torch.empty(1, dtype=torch.int32, device=DEV), join=j))


def test_refusals():
    from cpmcu_amd import ops
    from cpmcu_amd.parts import FEED_FORWARDS, MIXERS, POSITION_ENCODINGS
    z = lambda *s: torch.zeros(*s, device=DEV)
    with pytest.raises(ops.KernelError, match="missing"):
        ops.norm_rows(z(2, 8), z(2, 8), None, replace=True)
    with pytest.raises(ops.KernelError, match="norm"):
        ops.norm_rows(z(2, 8), z(2, 8), "batch")
    with pytest.raises(ops.KernelError, match="table"):
        ops.gated_lookup(z(2, 8), z(5, 10), 3, torch.zeros(2, dtype=torch.int32, device=DEV), z(2, 8))
    with pytest.raises(ops.KernelError, match="even"):
        ops.head_output(z(2, 9), z(2, 9), 1, 9, torch.zeros(2, dtype=torch.int32, device=DEV), z(4))
    with pytest.raises(ops.KernelError, match="nothing"):
        ops.latent_store(None, 1, 8, 2, 8, 1e-5, torch.zeros(2, dtype=torch.int32, device=DEV), None, None, 1.0)
    names = {"q": "q", "k": "k", "v": "v", "out": "o", "gate": "g"}
    rope = POSITION_ENCODINGS.build("rope", head_dim=8, theta=10.0)
    with pytest.raises(ValueError, match="gate"):
        MIXERS.build("attention", names=names, hidden_size=16, num_heads=2, num_kv_heads=1, key_dim=8, value_dim=8, position=rope, scale=1.0,
                     value_position=rope)
    with pytest.raises(ValueError, match="even"):
        MIXERS.build("attention", names={k: v for k, v in names.items() if k != "gate"}, hidden_size=16, num_heads=2, num_kv_heads=1,
                     key_dim=8, value_dim=7, position=rope, scale=1.0, value_position=rope)
    with pytest.raises(ValueError, match="experts"):
        FEED_FORWARDS.build("routed_experts", names={"router": "r", "expert": "{e}{part}"}, hidden_size=8, expert_size=8, experts=2, top=4,
                            identity=1)
