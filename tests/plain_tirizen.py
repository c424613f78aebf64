"""Plain implementation of the Tirizen design: whole sequences, no cache, float64, one function per mechanism.

It reads the raw config.json dictionary and the checkpoint's tensors by name and shares no code with the package:
every formula is restated here.  Positions count from 0; "rms" always has eps inside the root.

    embedding       e_t = embed[tok_t] * scale + pos[t]; the residual is S copies X_1..X_S of it
    layer           twice (mixer, then feed-forward, which a layer may lack), with numbers in[S], out[S], mix[S, S]:
                    u = sum_s in_s X_s;  y = sub(rms(u) * w);  X_t <- sum_s mix[s, t] X_s + m out_t y, all t at once
    gla             q = Wq h / sqrt(dim), k = Wk h, v = Wv h per head; decays a number a head and key channel,
                    a = sigmoid(Wa2 (Wa1 h) + b)^(1/tau); S <- diag(a) S + k v^T, o = S^T q; rms(o) * w a head, the
                    heads side by side * silu(Wg h), Wo
    attention       q, k each divided by the root mean square of its whole row and weighted; q * (1 + coef
                    ln(floor((p + 1) / every) + 1)); score q.k * scale; causal softmax; times sigmoid(Wg h)_head; Wo.
                    A layer may use an earlier layer's keys and values
    feed-forward    Wd relu(Wu h)^2; or a mixture: z = Wr h + b, the `top` largest z are chosen, weights their softmax
                    among themselves
    output          logits = embed . (rms(X_1 + .. + X_S) * w) * logit_scale
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def squared_relu(z):
    return torch.clamp(z, min=0.0) ** 2


def embedding(raw, W, tokens):
    return W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(raw["embedding"]["scale"]) + W["pos"][:len(tokens)]


def join_streams(X, y, mix, out, m):
    """X [S, T, width] -> the streams after a sub-layer's result y [T, width]."""
    return torch.einsum("st,snw->tnw", mix, X) + m * out[:, None, None] * y[None]


def channel_decay(h, W, p, tau):
    """[T, heads * dim], in the logarithm first: sigmoid(z)^(1/tau)."""
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def recurrence(q, k, v, a):
    """q, k, a [T, heads, dim], v [T, heads, vdim] -> o [T, heads, vdim]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def gla(h, W, p, m, eps, kv=None):
    T, H, d, dv = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ W[p + "q"].T).view(T, H, d) * d ** -0.5
    k, v = (h @ W[p + "k"].T).view(T, H, d), (h @ W[p + "v"].T).view(T, H, dv)
    a = channel_decay(h, W, p, float(m["tau"])).view(T, H, d)
    o = rms(recurrence(q, k, v, a), eps) * W[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def temperature(T, temp):
    p = torch.arange(T, dtype=F64)
    if not temp:
        return torch.ones(T, dtype=F64)
    return 1.0 + float(temp["coef"]) * torch.log(torch.floor((p + 1) / int(temp["every"])) + 1.0)


def keys_and_values(h, W, p, m, eps):
    T, G = h.shape[0], int(m["kv_heads"])
    k = rms(h @ W[p + "k"].T, eps) * W[p + "k.norm"]
    return k.view(T, G, int(m["dim"])), (h @ W[p + "v"].T).view(T, G, int(m["vdim"]))


def causal_attention(q, k, v, scale):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    mask, outs = torch.tril(torch.ones(T, T, dtype=torch.bool)), []
    for i in range(H):
        s = (q[:, i] @ k[:, i // (H // G)].T * scale).masked_fill(~mask, -math.inf)
        outs.append(torch.softmax(s, -1) @ v[:, i // (H // G)])
    return torch.stack(outs, 1)


def attention(h, W, p, m, eps, kv=None):
    T, H, d, dv = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"]) * temperature(T, m.get("q_temp"))[:, None]
    k, v = kv if kv is not None else keys_and_values(h, W, p, m, eps)
    o = causal_attention(q.view(T, H, d), k, v, float(m["scale"])) * torch.sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ W[p + "o"].T


MIXERS = {"attention": attention, "gla": gla}


def expert(h, W, p):
    return squared_relu(h @ W[p + "up"].T) @ W[p + "down"].T


def route(h, W, p, top, margins=None):
    """(chosen experts [T, top], weights [T, top]).  ``margins`` (a list) receives, per token, the gap between the last
    logit taken and the first one left."""
    z = h @ W[p + "router"].T + W[p + "router.b"]
    ranked, order = z.sort(-1, descending=True)
    if margins is not None:
        margins.append(ranked[:, top - 1] - ranked[:, top] if top < z.shape[1] else torch.full((h.shape[0],), math.inf, dtype=F64))
    return order[:, :top], torch.softmax(ranked[:, :top], -1)


def experts(h, W, p, mlp, margins=None):
    idx, w = route(h, W, p, int(mlp["router"]["top"]), margins)
    out = torch.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        t, k = (idx == e).nonzero(as_tuple=True)
        if t.numel():
            out[t] += w[t, k][:, None] * expert(h[t], W, f"{p}e{e}.")
    return out


def feed_forward(h, W, p, mlp, margins=None):
    return expert(h, W, p) if mlp["kind"] == "dense" else experts(h, W, p, mlp, margins)


def forward(raw, tensors, tokens, return_layers=False, margins=None):
    """Logits [T, vocab] of one sequence (and the sum of the streams after every layer)."""
    W = {k: v.to(F64) for k, v in tensors.items()}
    eps, m = float(raw["norm"]["eps"]), float(raw["residual_mult"])
    X = torch.stack([embedding(raw, W, tokens)] * int(raw["streams"]))
    kept, after = {}, []
    for i, layer in enumerate(raw["layers"]):
        p, mixer = f"l{i}.", layer["mixer"]
        numbers = lambda q: tuple(W[f"{p}hc{q}.{t}"] for t in ("in", "mix", "out"))
        read, mix, out = numbers(1)
        h = rms(torch.einsum("s,snw->nw", read, X), eps) * W[p + "norm1"]
        kv = None
        if layer["type"] == "attention":
            j = mixer.get("kv_from")
            kept[i] = kv = keys_and_values(h, W, p + "mix.", mixer, eps) if j is None else kept[int(j)]
        X = join_streams(X, MIXERS[layer["type"]](h, W, p + "mix.", mixer, eps, kv), mix, out, m)
        if layer.get("mlp") is not None:
            read, mix, out = numbers(2)
            h = rms(torch.einsum("s,snw->nw", read, X), eps) * W[p + "norm2"]
            X = join_streams(X, feed_forward(h, W, p + "mlp.", layer["mlp"], margins), mix, out, m)
        after.append(X.sum(0))
    logits = (rms(X.sum(0), eps) * W["final.norm"]) @ W["embed"].T * float(raw["logit_scale"])
    return (logits, torch.stack(after)) if return_layers else logits
