"""Plain implementation of the Pemalorn design: whole sequences, no cache, float64, one function per mechanism.

It reads the raw config.json dictionary and the checkpoint's tensors by name and shares no code with the package:
every formula is restated here.  Positions count from 0; "rms" always has eps inside the root.

    embedding       x_t = x0_t = embed[tok_t]
    order           the layers in turn; with loop {start, stop, times} layers start..stop-1 run `times` times in a
                    row, and before each of those passes x <- Win [x | x0] + step[pass]
    layer           h = (x - mean) / sqrt(var + eps) * w;  h1 = h + conv1(h), h2 = h + conv2(h) (causal, a filter a
                    channel);  x += mixer(h1) + ff(h2)  (a layer may have no feed-forward);  then, with e = the layer's
                    columns of side.embed[tok], y = P (gelu_tanh(G x) * e),  x += y / rms(y) * w_side
    rotation        first `dims` features of a head; pairs (i, i + dims/2) ("halves") or (2i, 2i+1)
                    ("interleaved"): (u, v) -> m (u cos a - v sin a, v cos a + u sin a), a = p f_i,
                    f_i = base^(-2i/dims), blended and m = 0.1 ln(factor) + 1 with a stretch (YaRN), else m = 1
    attention       q, k, v = W h; q, k rotated (halves); v of key j rotated by j over the whole value (halves), the
                    head's sum turned back by the query's position; score q.k * scale * temp_h; causal; softmax
                    whose denominator also holds exp(sink_h); times sigmoid(Wg h)_h; Wo
    latent          q = Wuq (rms(Wdq h) * w), per head [plain | rotated (interleaved)]; Wdkv h = [c | r]: c = rms(c) *
                    w, r rotated, shared by the heads; key [Wuk c | r], value Wuv c; score * scale; window; softmax
                    with sink; heads side by side * sigmoid(Wg h); Wo
    feed-forward    router s = softmax(Wr h) over experts and identity experts; the `top` largest s + correction are
                    chosen; weights s (as they are); expert e: Wd (silu(Wg h) * (Wu h)); an identity expert: h
    output          logits = head . layer norm(x)
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u], 0)
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + pad[j:j + T] * w[:, j]
    return y


def frequencies(rot):
    """(f_i, magnitude) of a rotation of rot.dims features."""
    dims, base = int(rot["dims"]), float(rot["base"])
    i = torch.arange(dims // 2, dtype=F64)
    f = base ** (-2.0 * i / dims)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    at = lambda turns: dims * math.log(float(sc["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(at(float(sc["fast"]))), 0), min(math.ceil(at(float(sc["slow"]))), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return f / float(sc["factor"]) * ramp + f * (1.0 - ramp), 0.1 * math.log(float(sc["factor"])) + 1.0


def turn(x, f, mag, pairing, sign=1.0):
    """x [T, heads, dim]: its first 2 len(f) features rotated by sign * position * f."""
    dims, T = 2 * f.numel(), x.shape[0]
    ang = sign * torch.arange(T, dtype=F64)[:, None] * f
    c, s = (mag * torch.cos(ang))[:, None, :], (mag * torch.sin(ang))[:, None, :]
    a, b = (x[..., 0:dims:2], x[..., 1:dims:2]) if pairing == "interleaved" else (x[..., :dims // 2], x[..., dims // 2:dims])
    out = x.clone()
    if pairing == "interleaved":
        out[..., 0:dims:2], out[..., 1:dims:2] = a * c - b * s, b * c + a * s
    else:
        out[..., :dims // 2], out[..., dims // 2:dims] = a * c - b * s, b * c + a * s
    return out


def rotate(x, rot, pairing):
    if not rot or not rot.get("dims"):
        return x
    f, mag = frequencies(rot)
    return turn(x, f, mag, pairing)


def turn_values(v, base, sign):
    """All features of v [T, heads, vdim], halves layout, by sign * position * base^(-2m/vdim)."""
    f = float(base) ** (-2.0 * torch.arange(v.shape[-1] // 2, dtype=F64) / v.shape[-1])
    return turn(v, f, 1.0, "halves", sign)


def sink_softmax(scores, mask, sink):
    """scores [T, T] of one head -> weights; the denominator also holds exp(sink)."""
    s = scores.masked_fill(~mask, -math.inf)
    m = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def visible(T, size=None):
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & (d < size) if size else d >= 0


def attention(h, W, p, m, eps):
    T, H, G, d, dv = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rotate((h @ W[p + "q"].T).view(T, H, d), m["rot"], "halves")
    k = rotate((h @ W[p + "k"].T).view(T, G, d), m["rot"], "halves")
    v = turn_values((h @ W[p + "v"].T).view(T, G, dv), m["rot"]["base"], 1.0)
    mask, outs = visible(T), []
    for i in range(H):
        g = i // (H // G)
        w = sink_softmax(q[:, i] @ k[:, g].T * float(m["scale"]) * W[p + "temp"][i], mask, W[p + "sink"][i])
        outs.append(w @ v[:, g])
    o = turn_values(torch.stack(outs, 1), m["rot"]["base"], -1.0)
    o = o * torch.sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ W[p + "o"].T


def latent_attention(h, W, p, m, eps):
    T, H, d, r, dv, R = (h.shape[0], int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]))
    q = ((rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]) @ W[p + "uq"].T).view(T, H, d + r)
    down = h @ W[p + "dkv"].T
    c = rms(down[:, :R], eps) * W[p + "dkv.norm"]
    q_rot = rotate(q[..., d:], m["rot"], "interleaved")
    k_rot = rotate(down[:, None, R:], m["rot"], "interleaved")[:, 0]
    k, v = (c @ W[p + "uk"].T).view(T, H, d), (c @ W[p + "uv"].T).view(T, H, dv)
    mask, outs = visible(T, int(m["mask"]["size"]) if m.get("mask") else None), []
    for i in range(H):
        s = (q[:, i, :d] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * float(m["scale"])
        outs.append(sink_softmax(s, mask, W[p + "sink"][i]) @ v[:, i])
    return (torch.cat(outs, -1) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


MIXERS = {"attention": attention, "latent_attention": latent_attention}


def expert(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(h, W, p, r, margins=None):
    """(chosen experts [T, top], weights [T, top]).  ``margins`` (a list) receives, per token, how clear the choice
    was: the gap between the last choice score taken and the first one left, against the two scores' sum (rounding of
    the router's input moves a softmax score in proportion to itself)."""
    top = int(r["top"])
    s = torch.softmax(h @ W[p + "router"].T, -1)
    c = s + W[p + "correction"]
    ranked, order = c.sort(-1, descending=True)
    if margins is not None:
        if top < c.shape[1]:
            near = s.gather(1, order[:, top - 1:top + 1]).sum(-1)
            margins.append((ranked[:, top - 1] - ranked[:, top]) / near)
        else:
            margins.append(torch.full((h.shape[0],), math.inf, dtype=F64))
    idx = order[:, :top]
    return idx, s.gather(1, idx)


def experts(h, W, p, mlp, margins=None):
    r = mlp["router"]
    idx, w = route(h, W, p, r, margins)
    out = torch.zeros_like(h)
    for e in range(int(r["experts"]) + int(r.get("identity") or 0)):
        t, k = (idx == e).nonzero(as_tuple=True)
        if t.numel():
            y = expert(h[t], W, f"{p}e{e}.") if e < int(r["experts"]) else h[t]
            out[t] += w[t, k][:, None] * y
    return out


def token_input(x, tokens, W, i, dim, eps):
    """What layer i adds to the residual x for the tokens themselves."""
    p = f"l{i}.side."
    e = W["side.embed"][torch.as_tensor(tokens, dtype=torch.long)][:, i * dim:(i + 1) * dim]
    return rms((gelu_tanh(x @ W[p + "gate"].T) * e) @ W[p + "proj"].T, eps) * W[p + "norm"]


def forward(raw, tensors, tokens, return_layers=False, margins=None):
    """Logits [T, vocab] of one sequence (and the residual after every layer run).  ``margins`` (a list) receives one
    tensor [T] for every routed layer run: how clear each token's choice of experts was (route)."""
    W = {k: v.to(F64) for k, v in tensors.items()}
    eps = float(raw["norm"]["eps"])
    x0 = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x = x0.clone()
    loop, n, after = raw.get("loop"), len(raw["layers"]), []
    order = [(i, None) for i in range(n)]
    if loop:
        a, b = int(loop["start"]), int(loop["stop"])
        span = lambda t: [(i, t if i == a else None) for i in range(a, b)]
        order = order[:a] + [run for t in range(int(loop["times"])) for run in span(t)] + order[b:]
    for i, begins in order:
        layer, p = raw["layers"][i], f"l{i}."
        if begins is not None:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][begins]
        h = layer_norm(x, W[p + "norm1"], eps)
        mixed = lambda k: h + causal_conv(h, W[f"{p}canon{k}"]) if raw.get("canon") else h
        y = MIXERS[layer["type"]](mixed(1), W, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + experts(mixed(2), W, p + "mlp.", layer["mlp"], margins)
        x = x + y
        if raw.get("token_side"):
            x = x + token_input(x, tokens, W, i, int(raw["token_side"]["dim"]), eps)
        after.append(x)
    logits = layer_norm(x, W["final.norm"], eps) @ W["head"].T
    return (logits, torch.stack(after)) if return_layers else logits
