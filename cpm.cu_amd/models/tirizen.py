"""Tirizen: which parts, with which numbers.

A decoder of pre-norm layers (RMS norms) whose residual is several streams (hyper-connections: every sub-layer reads a
weighted sum of the streams, and its result, times a number of the configuration, joins all of them through a mixing
matrix).  The embedding is multiplied by a number and a learned vector a position is added; the head is the embedding
table without that number, its logits multiplied by another.  Mixers:

* ``attention``: grouped-query attention without rotation; all query heads of a token are divided by one root mean
  square, as are all its key heads; a query temperature that grows with the position; a sigmoid gate a head.  A layer
  with ``kv_from`` has no keys and values: its runs read the cache entry of the layer it names.
* ``gla``: gated linear attention, whose decay is a number a head and key channel from a low-rank product.

Feed-forwards have no gate, down(relu(up h)^2): dense, or a mixture of such experts whose router has a bias, chooses by
the logits and weighs by the softmax of the chosen ones.

Checkpoint tensors: ``embed``, ``pos``, ``final.norm``, and per layer i ``l<i>.norm1|norm2``, ``l<i>.hc1|hc2.in|out|mix``,
``l<i>.mlp.up|down`` or ``l<i>.mlp.router|router.b|e<j>.up|down``, and ``l<i>.mix.*``: attention q, q.norm, g, o and, with
keys and values of its own, k, k.norm, v; gla q, k, v, g, o, norm, a1, a2, a2.b.
"""
from __future__ import annotations

from ..config.tirizen import ARCHITECTURE, TirizenConfig
from ..parts import BLOCKS, FEED_FORWARDS, MIXERS, NORMS, LMHead, TokenEmbedding
from ..registry import Architecture, register_architecture
from .decoder import DecoderModel, Run

DEFAULT_DECAY_RANK = 16


def _mixer(cfg: TirizenConfig, i: int, ranks):
    layer, p = cfg.layers[i], f"l{i}.mix."
    m = layer.mixer
    if layer.type == "gla":
        names = {"q": p + "q", "k": p + "k", "v": p + "v", "gate": p + "g", "out": p + "o", "norm": p + "norm",
                 "decay_down": p + "a1", "decay_up": p + "a2", "decay_bias": p + "a2.b"}
        return MIXERS.build("gated_linear_attention", names=names, hidden_size=cfg.width, heads=m.heads, key_dim=m.dim,
                            value_dim=m.vdim, decay_rank=ranks.get(i, DEFAULT_DECAY_RANK), tau=m.tau, eps=cfg.eps)
    names = {"q": p + "q", "q_norm": p + "q.norm", "head_gate": p + "g", "out": p + "o"}
    if m.kv_from is None:
        names.update({"k": p + "k", "k_norm": p + "k.norm", "v": p + "v"})
    return MIXERS.build("attention", names=names, hidden_size=cfg.width, num_heads=m.heads, num_kv_heads=m.kv_heads,
                        key_dim=m.dim, value_dim=m.vdim, position=None, scale=m.scale, norm_eps=cfg.eps, norm_rows=True,
                        query_temp=m.temp, borrows=m.kv_from is not None)


def _feed_forward(cfg: TirizenConfig, i: int):
    ff, p = cfg.layers[i].mlp, f"l{i}.mlp."
    if ff is None:
        return None
    if ff.kind == "dense":
        return FEED_FORWARDS.build("plain", up_name=p + "up", down_name=p + "down", hidden_size=cfg.width,
                                   intermediate_size=ff.ff, activation="relu_squared")
    names = {"router": p + "router", "router_bias": p + "router.b", "expert": p + "e{e}.{part}"}
    return FEED_FORWARDS.build("routed_experts", names=names, hidden_size=cfg.width, expert_size=ff.ff, experts=ff.experts,
                               top=ff.top, score="logit", gated=False, activation="relu_squared")


def build(cfg: TirizenConfig, ranks=None) -> DecoderModel:
    """``ranks``: {layer: rank of its decay's product} of the ``gla`` layers, read from the checkpoint's tensor shapes (no
    configuration key holds them); a random-weights model takes DEFAULT_DECAY_RANK."""
    norm = lambda name: NORMS.build("rms_norm", name=name, hidden_size=cfg.width, eps=cfg.eps)
    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        ff = _feed_forward(cfg, i)
        hc = [tuple(f"{p}hc{q}.{t}" for t in ("in", "out", "mix")) for q in ((1, 2) if ff is not None else (1,))]
        layers.append(BLOCKS.build("hyper_connections", mixer_norm=norm(p + "norm1"), mixer=_mixer(cfg, i, ranks or {}),
                                   streams=cfg.streams, names=hc, ff_norm=norm(p + "norm2") if ff is not None else None,
                                   feed_forward=ff, residual_scale=cfg.residual_mult))
    schedule = [Run(i, entry, writes) for i, (entry, writes) in enumerate(cfg.layer_runs())]
    embedding = TokenEmbedding("embed", cfg.vocab, cfg.width, cfg.embedding_scale, positions=("pos", cfg.max_positions))
    head = LMHead("embed", cfg.vocab, cfg.width, cfg.logit_scale, tied_to=embedding)
    return DecoderModel(cfg, embedding, layers, norm("final.norm"), head, schedule, streams=cfg.streams)


def _checkpoint_options(cfg: TirizenConfig, tensors) -> dict:
    """The rank of a decay's low-rank product stands in no configuration key: the checkpoint's shapes give it.
    ``tensors``: names (with shapes where the loader knows them)."""
    shapes = tensors if isinstance(tensors, dict) else {}
    ranks = {i: int(shapes[f"l{i}.mix.a1"][0]) for i, layer in enumerate(cfg.layers)
             if layer.type == "gla" and f"l{i}.mix.a1" in shapes}
    return {"ranks": ranks} if ranks else {}


def _ignore(cfg: TirizenConfig, name: str) -> bool:
    """A layer without a feed-forward has no second norm and no second set of stream numbers: a checkpoint that stores
    them all the same is read without them."""
    return any(layer.mlp is None and (name == f"l{i}.norm2" or name.startswith(f"l{i}.hc2."))
               for i, layer in enumerate(cfg.layers))


register_architecture(Architecture(name=ARCHITECTURE, config_class=TirizenConfig, build=build, options={"ranks": None},
                                   checkpoint_options=_checkpoint_options, ignore_tensor=_ignore))
