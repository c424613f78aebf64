"""Pemalorn: which parts, with which numbers.

A decoder of parallel layers: one layer norm (a weight, no bias) a layer; mixer and mixture of experts each read its
rows through a short causal convolution of their own, h + conv(h), and both results join the residual; then an input of
the token itself, columns of a table gated by a projection of the residual, projected back and RMS-normed, joins it.
A span of layers may run several times with the same weights and a cache entry a run; every pass over it begins with
x <- W [x | embedding] + step[pass].  Mixers:

* ``attention``: grouped-query attention whose values are rotated by their positions and turned back by the query's
  (pairs half a rotation apart, as for q and k), a number a head on the scores, a softmax sink, an output gate a head.
* ``latent_attention``: queries from a normed latent, keys and values from one cached latent a token and one rotated
  key part (neighbouring pairs, frequencies stretched by YaRN), a sliding window, a softmax sink, an output gate a
  feature.

Feed-forward: routed SiLU-gated experts and identity experts; softmax scores, a correction that enters the choice only,
weights as the scores are.

Checkpoint tensors: ``embed``, ``head``, ``final.norm``, ``loop.in|step``, ``side.embed`` and per layer i
``l<i>.norm1``, ``l<i>.canon1|canon2``, ``l<i>.side.gate|proj|norm``, ``l<i>.mlp.router|correction|e<j>.gate|up|down``
and ``l<i>.mix.*``: attention q, k, v, g, o, temp, sink; latent_attention dq, dq.norm, uq, dkv, dkv.norm, uk, uv, g, o,
sink.
"""
from __future__ import annotations

from ..config.pemalorn import ARCHITECTURE, PemalornConfig
from ..parts import (BLOCKS, FEED_FORWARDS, MIXERS, NORMS, POSITION_ENCODINGS, InputConvolution, LMHead, LoopInput,
                     TokenEmbedding, TokenInput, TokenTable)
from ..registry import Architecture, register_architecture
from .decoder import DecoderModel, Run


def _rotation(rot, pairs: str):
    if not rot.dims:
        return None
    if rot.scaling is not None:
        factor, original, fast, slow = rot.scaling
        return POSITION_ENCODINGS.build("yarn", head_dim=rot.dims, theta=rot.base, factor=factor, original=original, fast=fast,
                                        slow=slow, pairs=pairs)
    return POSITION_ENCODINGS.build("rope", head_dim=rot.dims, theta=rot.base, pairs=pairs)


def _mixer(cfg: PemalornConfig, i: int):
    layer, p = cfg.layers[i], f"l{i}.mix."
    m = layer.mixer
    if layer.type == "latent_attention":
        names = {"q_down": p + "dq", "q_norm": p + "dq.norm", "q_up": p + "uq", "down": p + "dkv", "down_norm": p + "dkv.norm",
                 "up_k": p + "uk", "up_v": p + "uv", "gate": p + "g", "out": p + "o", "sink": p + "sink"}
        return MIXERS.build("latent_attention", names=names, hidden_size=cfg.width, num_heads=m.heads, key_dim=m.dim,
                            rot_dim=m.rot_dim, value_dim=m.vdim, kv_rank=m.kv_rank, position=_rotation(m.rot, "interleaved"),
                            scale=m.scale, eps=cfg.eps, q_rank=m.q_rank, mask_window=m.window, gate_features=True)
    names = {"q": p + "q", "k": p + "k", "v": p + "v", "head_gate": p + "g", "out": p + "o", "temp": p + "temp",
             "sink": p + "sink"}
    return MIXERS.build("attention", names=names, hidden_size=cfg.width, num_heads=m.heads, num_kv_heads=m.kv_heads,
                        key_dim=m.dim, value_dim=m.vdim, position=_rotation(m.rot, "halves"), scale=m.scale,
                        value_position=POSITION_ENCODINGS.build("rope", head_dim=m.vdim, theta=m.rot.base))


def _feed_forward(cfg: PemalornConfig, i: int):
    ff, p = cfg.layers[i].mlp, f"l{i}.mlp."
    if ff is None:
        return None
    names = {"router": p + "router", "correction": p + "correction", "expert": p + "e{e}.{part}"}
    return FEED_FORWARDS.build("routed_experts", names=names, hidden_size=cfg.width, expert_size=ff.ff, experts=ff.experts,
                               top=ff.top, normalize=False, identity=ff.identity)


def build(cfg: PemalornConfig) -> DecoderModel:
    norm = lambda name: NORMS.build("layer_norm", name=name, hidden_size=cfg.width, eps=cfg.eps)
    table = TokenTable("side.embed", cfg.vocab, len(cfg.layers) * cfg.token_dim) if cfg.token_dim else None
    layers = []
    for i in range(len(cfg.layers)):
        p = f"l{i}."
        ff = _feed_forward(cfg, i)
        conv = side = None
        if cfg.taps:
            conv = InputConvolution([p + "canon1"] + ([p + "canon2"] if ff is not None else []), cfg.width, cfg.taps)
        if table is not None:
            side = TokenInput(table, i * cfg.token_dim, cfg.token_dim, cfg.width, gate_name=p + "side.gate",
                              proj_name=p + "side.proj", norm_name=p + "side.norm", eps=cfg.eps)
        layers.append(BLOCKS.build("parallel", norm=norm(p + "norm1"), mixer=_mixer(cfg, i), feed_forward=ff,
                                   hidden_size=cfg.width, input_conv=conv, token_input=side))
    # every run of a layer, also a repeated one, has a cache entry of its own
    schedule = [Run(layer, entry, True, begins) for entry, (layer, begins) in enumerate(cfg.layer_runs())]
    loop = LoopInput("loop.in", "loop.step", cfg.width, cfg.loop[2]) if cfg.loop is not None else None
    return DecoderModel(cfg, TokenEmbedding("embed", cfg.vocab, cfg.width, 1.0), layers, norm("final.norm"),
                        LMHead("head", cfg.vocab, cfg.width, 1.0), schedule, loop_input=loop,
                        shared=[table] if table is not None else [])


def _ignore(cfg: PemalornConfig, name: str) -> bool:
    """A layer without a feed-forward has no second convolution: a checkpoint that stores one all the same is read
    without it."""
    return any(layer.mlp is None and name == f"l{i}.canon2" for i, layer in enumerate(cfg.layers))


register_architecture(Architecture(name=ARCHITECTURE, config_class=PemalornConfig, build=build, ignore_tensor=_ignore))
