"""Typed configuration of Tirizen (config.json with ``"architecture": "Tirizen"``).

A list of pre-norm layers over a residual of several streams, each with a mixer of its own kind and sizes and an optional
feed-forward:

    {"architecture": "Tirizen", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s},
     "max_positions": P, "residual_mult": m, "streams": S, "logit_scale": c,
     "layers": [{"type": "attention" | "gla", "mixer": {...}, "mlp": {...} | null}, ...]}

mixer of ``attention``: {heads, kv_heads, dim, vdim, scale, optional q_temp {coef, every}, optional kv_from}; kv_from
names the earlier attention layer whose keys and values this one reads.
mixer of ``gla``: {heads, dim, vdim, tau}.
mlp: {"kind": "dense", ff} or {"kind": "moe", "expert": {ff}, "router": {experts, top}}.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from .base import ConfigError, ModelConfig, field_from, require

ARCHITECTURE = "Tirizen"
MIXER_KINDS = ("attention", "gla")


def _object(raw: Dict[str, Any], key: str, where: str, needed: bool = False) -> Optional[Dict[str, Any]]:
    v = raw.get(key)
    if v is None:
        require(not needed, f"{where}: '{key}' must be an object")
        return None
    require(isinstance(v, dict), f"{where}: '{key}' must be an object")
    return v


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temp: Optional[Tuple[float, int]] = None      # query temperature: (coef, every)
    kv_from: Optional[int] = None                 # the layer whose keys and values are read; None: its own

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str):
        g = lambda k, *d: field_from(raw, k, int, *d, where=where)
        heads, dim = g("heads"), g("dim")
        t = _object(raw, "q_temp", where)
        temp = None
        if t is not None:
            temp = (field_from(t, "coef", float, where=where + " q_temp"), field_from(t, "every", int, where=where + " q_temp"))
            require(temp[1] > 0, f"{where} q_temp: every must be positive")
        c = cls(heads, g("kv_heads", heads), dim, g("vdim", dim), field_from(raw, "scale", float, where=where), temp,
                g("kv_from", None))
        require(min(c.heads, c.kv_heads, c.dim, c.vdim) > 0, f"{where}: sizes must be positive")
        require(c.heads % c.kv_heads == 0, f"{where}: heads ({c.heads}) must be a multiple of kv_heads ({c.kv_heads})")
        return c

    def to_dict(self):
        d: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
                             "scale": self.scale}
        if self.temp is not None:
            d["q_temp"] = {"coef": self.temp[0], "every": self.temp[1]}
        if self.kv_from is not None:
            d["kv_from"] = self.kv_from
        return d


@dataclass(frozen=True)
class GLAConfig:
    heads: int
    dim: int
    vdim: int
    tau: float

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], where: str):
        g = lambda k, *d: field_from(raw, k, int, *d, where=where)
        dim = g("dim")
        c = cls(g("heads"), dim, g("vdim", dim), field_from(raw, "tau", float, where=where))
        require(min(c.heads, c.dim, c.vdim) > 0, f"{where}: sizes must be positive")
        require(c.tau > 0, f"{where}: tau must be positive")
        return c

    def to_dict(self):
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}


@dataclass(frozen=True)
class FeedForwardConfig:
    kind: str                             # 'dense' or 'moe'
    ff: int                               # width of the layer, or of one expert
    experts: int = 0
    top: int = 0

    @classmethod
    def from_dict(cls, raw: Any, where: str):
        require(isinstance(raw, dict), f"{where}: must be an object or null")
        kind = field_from(raw, "kind", str, where=where)
        if kind == "dense":
            c = cls(kind, field_from(raw, "ff", int, where=where))
        elif kind == "moe":
            expert, router = _object(raw, "expert", where, True), _object(raw, "router", where, True)
            r = lambda k: field_from(router, k, int, where=where + " router")
            c = cls(kind, field_from(expert, "ff", int, where=where + " expert"), r("experts"), r("top"))
            require(0 < c.top <= c.experts, f"{where} router: top ({c.top}) must lie in 1..experts ({c.experts})")
        else:
            raise ConfigError(f"{where}: kind '{kind}' is not supported (supported: dense, moe)")
        require(c.ff > 0, f"{where}: sizes must be positive")
        return c

    def to_dict(self):
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}


_MIXER_CONFIGS = {"attention": AttentionConfig, "gla": GLAConfig}


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: Any
    mlp: Optional[FeedForwardConfig]      # None: the layer has no feed-forward

    @classmethod
    def from_dict(cls, raw: Any, i: int):
        where = f"config.json layers[{i}]"
        require(isinstance(raw, dict), f"{where}: must be an object")
        kind = field_from(raw, "type", str, where=where)
        if kind not in _MIXER_CONFIGS:
            raise ConfigError(f"{where}: type '{kind}' is not supported (supported: {', '.join(MIXER_KINDS)})")
        mixer = _MIXER_CONFIGS[kind].from_dict(_object(raw, "mixer", where, True), where + " mixer")
        mlp = raw.get("mlp")
        return cls(kind, mixer, FeedForwardConfig.from_dict(mlp, where + " mlp") if mlp is not None else None)

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None}


@dataclass(frozen=True)
class TirizenConfig(ModelConfig):
    vocab: int = 0
    width: int = 0
    eps: float = 1e-6
    embedding_scale: float = 1.0
    max_positions: int = 0
    residual_mult: float = 1.0
    streams: int = 1
    logit_scale: float = 1.0
    layers: Tuple[LayerConfig, ...] = ()

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "TirizenConfig":
        vocab, width, positions = (field_from(raw, k, int) for k in ("vocab", "width", "max_positions"))
        require(vocab > 0 and width > 0 and positions > 0, "config.json: vocab, width and max_positions must be positive")
        norm = _object(raw, "norm", "config.json", True)
        eps = field_from(norm, "eps", float, where="config.json norm")
        require(eps >= 0, "config.json norm: eps must not be negative")
        emb = _object(raw, "embedding", "config.json") or {}
        streams = field_from(raw, "streams", int, 1)
        require(streams >= 1, f"config.json: streams ({streams}) must be at least 1")
        layers = raw.get("layers")
        require(isinstance(layers, list) and len(layers) > 0, "config.json: 'layers' must be a non-empty list")
        c = cls(ARCHITECTURE, vocab, width, eps, field_from(emb, "scale", float, 1.0, where="config.json embedding"), positions,
                field_from(raw, "residual_mult", float, 1.0), streams, field_from(raw, "logit_scale", float, 1.0),
                tuple(LayerConfig.from_dict(l, i) for i, l in enumerate(layers)))
        for i, layer in enumerate(c.layers):
            j = layer.mixer.kv_from if layer.type == "attention" else None
            if j is None:
                continue
            where = f"config.json layers[{i}] mixer"
            require(0 <= j < i and c.layers[j].type == "attention" and c.layers[j].mixer.kv_from is None,
                    f"{where}: kv_from ({j}) must name an earlier attention layer with keys and values of its own")
            o, m = c.layers[j].mixer, layer.mixer
            require((o.kv_heads, o.dim, o.vdim) == (m.kv_heads, m.dim, m.vdim),
                    f"{where}: kv_from ({j}) has keys and values of other sizes")
        return c

    def to_dict(self) -> Dict[str, Any]:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
                "embedding": {"scale": self.embedding_scale}, "max_positions": self.max_positions,
                "residual_mult": self.residual_mult, "streams": self.streams, "logit_scale": self.logit_scale,
                "layers": [l.to_dict() for l in self.layers]}

    def layer_runs(self) -> List[Tuple[int, bool]]:
        """(cache entry, whether the layer writes it) of every layer: a layer that reads another's keys and values has no
        entry of its own."""
        runs: List[Tuple[int, bool]] = []
        entries = 0
        for layer in self.layers:
            j = layer.mixer.kv_from if layer.type == "attention" else None
            if j is None:
                runs.append((entries, True))
                entries += 1
            else:
                runs.append((runs[j][0], False))
        return runs

    @property
    def vocabulary_size(self) -> int:
        return self.vocab

    @property
    def longest_sequence(self) -> Optional[int]:
        return self.max_positions
