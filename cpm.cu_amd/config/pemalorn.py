"""Typed configuration of Pemalorn (config.json with ``"architecture": "Pemalorn"``).

A list of parallel layers (one layer norm; short convolutions on what mixer and feed-forward read; an input of the
token itself afterwards), each with a mixer of its own kind and sizes and an optional mixture of experts; a span of
the layers may run several times in a row, every pass beginning with a product of residual and embedding:

    {"architecture": "Pemalorn", "vocab": V, "width": W, "norm": {"eps": e}, "canon": {"taps": n} (optional),
     "token_side": {"dim": d} (optional), "loop": {"start": a, "stop": b, "times": n} (optional),
     "layers": [{"type": "attention" | "latent_attention", "mixer": {...}, "mlp": {...} | null}, ...]}

mixer of ``attention``: {heads, kv_heads, dim, vdim, scale, rot {base, dims}}; rot.base also turns the values.
mixer of ``latent_attention``: {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot {base, dims, optional scaling
{factor, original, fast, slow}}, optional mask {size}}.
mlp: {"kind": "moe", "expert": {ff}, "router": {experts, top, optional identity}}.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .base import ConfigError, ModelConfig, field_from, require

ARCHITECTURE = "Pemalorn"
MIXER_KINDS = ("attention", "latent_attention")


def _object(raw: Dict[str, Any], key: str, where: str, needed: bool = False) -> Optional[Dict[str, Any]]:
    v = raw.get(key)
    if v is None:
        require(not needed, f"{where}: '{key}' must be an object")
        return None
    require(isinstance(v, dict), f"{where}: '{key}' must be an object")
    return v


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int                                                     # 0: no rotation of queries and keys
    scaling: Optional[Tuple[float, float, float, float]] = None   # YaRN: (factor, original, fast, slow)

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str, dims: Optional[int] = None):
        rot = _object(raw, "rot", where, True)
        r = where + " rot"
        scaling = _object(rot, "scaling", r)
        s = lambda k: field_from(scaling, k, float, where=r + " scaling")
        c = cls(field_from(rot, "base", float, where=r), field_from(rot, "dims", int, *(() if dims is None else (dims,)), where=r),
                (s("factor"), s("original"), s("fast"), s("slow")) if scaling is not None else None)
        require(c.dims >= 0 and c.dims % 2 == 0, f"{r}: dims ({c.dims}) must be even")
        require(c.base > 1.0, f"{r}: base must exceed 1")
        require(c.scaling is None or min(c.scaling) > 0, f"{r} scaling: its numbers must be positive")
        return c

    def to_dict(self):
        d: Dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            d["scaling"] = dict(zip(("factor", "original", "fast", "slow"), self.scaling))
        return d


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Rotation

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str):
        g = lambda k, *d: field_from(raw, k, int, *d, where=where)
        heads, dim = g("heads"), g("dim")
        c = cls(heads, g("kv_heads", heads), dim, g("vdim", dim), field_from(raw, "scale", float, where=where),
                Rotation.from_dict(raw, where))
        require(min(c.heads, c.kv_heads, c.dim, c.vdim) > 0, f"{where}: sizes must be positive")
        require(c.heads % c.kv_heads == 0, f"{where}: heads ({c.heads}) must be a multiple of kv_heads ({c.kv_heads})")
        require(c.rot.dims <= c.dim, f"{where}: rot.dims ({c.rot.dims}) must be at most dim ({c.dim})")
        require(c.vdim % 2 == 0, f"{where}: vdim ({c.vdim}) must be even, the values are rotated")
        require(c.rot.scaling is None, f"{where} rot: scaling belongs to latent_attention")
        return c

    def to_dict(self):
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
                "rot": self.rot.to_dict()}


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: Rotation
    window: Optional[int] = None          # None: every earlier token is seen

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str):
        g = lambda k: field_from(raw, k, int, where=where)
        mask = _object(raw, "mask", where)
        c = cls(g("heads"), g("dim"), g("rot_dim"), g("vdim"), g("q_rank"), g("kv_rank"),
                field_from(raw, "scale", float, where=where), Rotation.from_dict(raw, where, g("rot_dim")),
                field_from(mask, "size", int, None, where=where + " mask") if mask is not None else None)
        require(min(c.heads, c.dim, c.vdim, c.q_rank, c.kv_rank) > 0, f"{where}: sizes must be positive")
        require(c.rot.dims == c.rot_dim, f"{where}: rot.dims ({c.rot.dims}) must equal rot_dim ({c.rot_dim})")
        require(c.window is None or c.window > 0, f"{where}: mask.size must be positive")
        return c

    def to_dict(self):
        d: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim,
                             "q_rank": self.q_rank, "kv_rank": self.kv_rank, "scale": self.scale, "rot": self.rot.to_dict()}
        if self.window is not None:
            d["mask"] = {"size": self.window}
        return d


@dataclass(frozen=True)
class ExpertsConfig:
    ff: int                               # width of one expert
    experts: int
    top: int
    identity: int = 0                     # identity experts behind the experts

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str):
        require(isinstance(raw, dict), f"{where}: must be an object or null")
        kind = field_from(raw, "kind", str, "moe", where=where)
        if kind != "moe":
            raise ConfigError(f"{where}: kind '{kind}' is not supported (supported: moe)")
        expert, router = _object(raw, "expert", where, True), _object(raw, "router", where, True)
        r = lambda k, *d: field_from(router, k, int, *d, where=where + " router")
        c = cls(field_from(expert, "ff", int, where=where + " expert"), r("experts"), r("top"), r("identity", 0))
        require(c.ff > 0 and c.experts > 0, f"{where}: sizes must be positive")
        require(c.identity >= 0, f"{where} router: identity must not be negative")
        require(0 < c.top <= c.experts + c.identity,
                f"{where} router: top ({c.top}) must lie in 1..experts + identity ({c.experts + c.identity})")
        return c

    def to_dict(self):
        router = {"experts": self.experts, "top": self.top}
        if self.identity:
            router["identity"] = self.identity
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": router}


_MIXER_CONFIGS = {"attention": AttentionConfig, "latent_attention": LatentAttentionConfig}


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: Any
    mlp: Optional[ExpertsConfig]          # None: the layer has no feed-forward

    @classmethod
    def from_dict(cls, raw: Any, i: int):
        where = f"config.json layers[{i}]"
        require(isinstance(raw, dict), f"{where}: must be an object")
        kind = field_from(raw, "type", str, where=where)
        if kind not in _MIXER_CONFIGS:
            raise ConfigError(f"{where}: type '{kind}' is not supported (supported: {', '.join(MIXER_KINDS)})")
        mixer = _MIXER_CONFIGS[kind].from_dict(_object(raw, "mixer", where, True), where + " mixer")
        mlp = raw.get("mlp")
        return cls(kind, mixer, ExpertsConfig.from_dict(mlp, where + " mlp") if mlp is not None else None)

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None}


@dataclass(frozen=True)
class PemalornConfig(ModelConfig):
    vocab: int = 0
    width: int = 0
    eps: float = 1e-5
    taps: int = 0                                     # of the convolutions on the sub-layers' inputs; 0: none
    token_dim: int = 0                                # numbers a token and layer of the token table; 0: none
    loop: Optional[Tuple[int, int, int]] = None       # (start, stop, times): layers start..stop-1 run `times` times
    layers: Tuple[LayerConfig, ...] = ()

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "PemalornConfig":
        vocab, width = field_from(raw, "vocab", int), field_from(raw, "width", int)
        require(vocab > 0 and width > 0, "config.json: vocab and width must be positive")
        norm = _object(raw, "norm", "config.json", True)
        eps = field_from(norm, "eps", float, where="config.json norm")
        require(eps >= 0, "config.json norm: eps must not be negative")
        canon, side = _object(raw, "canon", "config.json"), _object(raw, "token_side", "config.json")
        taps = field_from(canon, "taps", int, where="config.json canon") if canon is not None else 0
        require(taps >= (1 if canon is not None else 0), "config.json canon: taps must be at least 1")
        token_dim = field_from(side, "dim", int, where="config.json token_side") if side is not None else 0
        require(token_dim >= (1 if side is not None else 0), "config.json token_side: dim must be at least 1")
        layers = raw.get("layers")
        require(isinstance(layers, list) and len(layers) > 0, "config.json: 'layers' must be a non-empty list")
        loop_raw, loop = _object(raw, "loop", "config.json"), None
        if loop_raw is not None:
            l = lambda k: field_from(loop_raw, k, int, where="config.json loop")
            loop = (l("start"), l("stop"), l("times"))
            require(0 <= loop[0] < loop[1] <= len(layers), f"config.json loop: start {loop[0]} and stop {loop[1]} "
                    f"must name a span of the {len(layers)} layers")
            require(loop[2] >= 1, "config.json loop: times must be at least 1")
        return cls(ARCHITECTURE, vocab, width, eps, taps, token_dim, loop,
                   tuple(LayerConfig.from_dict(l, i) for i, l in enumerate(layers)))

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                             "norm": {"eps": self.eps}, "layers": [l.to_dict() for l in self.layers]}
        if self.taps:
            d["canon"] = {"taps": self.taps}
        if self.token_dim:
            d["token_side"] = {"dim": self.token_dim}
        if self.loop is not None:
            d["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return d

    def layer_runs(self) -> Tuple[Tuple[int, Optional[int]], ...]:
        """The layers in the order they run, each with the number of the pass it begins (None: it begins none)."""
        n = len(self.layers)
        if self.loop is None:
            return tuple((i, None) for i in range(n))
        start, stop, times = self.loop
        runs = [(i, None) for i in range(start)]
        for t in range(times):
            runs += [(i, t if i == start else None) for i in range(start, stop)]
        return tuple(runs + [(i, None) for i in range(stop, n)])

    @property
    def vocabulary_size(self) -> int:
        return self.vocab
