"""Typed configuration of the Gerorax decoder.

config.json of this design is nested: ``layers`` lists every layer with its ``type`` (``attention``), the mixer's sizes
and constants (``mixer``) and its feed-forward (``mlp``: ``kind`` ``dense`` or ``moe``; null for a layer without one);
``loop`` names a run of layers that is gone through several times; ``embedding.scale`` multiplies the embedding's rows
and ``residual_mult`` what every sublayer adds to the stream; ``norm.eps``, ``vocab`` and ``width`` stand at the top, and
``architecture`` names the design.  Every layer may have sizes of its own.  The design has no largest position;
``max_positions`` (not a key of the design) bounds a request's length for the engine and defaults to 2^20.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, Optional, Tuple, Union

from .base import ConfigError, ModelConfig, as_float, as_int, as_positive_int, key, optional, parse_fields
from .duduvik import ClampedExpert, ScaledEmbedding
from .morulix import LayerLoop, _eps, _obj


def as_count(v: Any) -> int:
    v = as_int(v)
    if v < 0:
        raise ValueError(f"expected an integer that is not negative, got {v}")
    return v


@dataclasses.dataclass(frozen=True)
class KeepingWindow:
    """A token sees the last ``size`` keys, its own among them, and its request's first ``keep_first``."""
    size: int = key(convert=as_positive_int)
    keep_first: int = key(default=0, convert=as_count)

    @classmethod
    def from_json(cls, obj, where="mask"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        return {"keep_first": self.keep_first, "size": self.size}


@dataclasses.dataclass(frozen=True)
class BiasedAttentionMixer:
    """Grouped attention with normed heads, scores biased by distance, a window that keeps first keys, and sinks."""
    kind = "attention"
    dim: int = key(convert=as_positive_int)
    heads: int = key(convert=as_positive_int)
    kv_heads: int = key(convert=as_positive_int)
    vdim: int = key(convert=as_positive_int)
    scale: float = key(convert=as_float)
    mask: Optional[KeepingWindow] = key(default=None, convert=optional(_obj(KeepingWindow, "mask")))

    @classmethod
    def from_json(cls, obj, where="mixer"):
        m = cls(**parse_fields(cls, obj, where))
        p = []
        if m.heads % m.kv_heads:
            p.append(f"heads {m.heads} is not a multiple of kv_heads {m.kv_heads}")
        if m.dim > 256 or m.vdim > 256:
            p.append("heads of more than 256 columns are not supported")
        if p:
            raise ConfigError(f"{where}: " + "; ".join(p))
        return m

    def to_dict(self):
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
                             "vdim": self.vdim}
        if self.mask is not None:
            d["mask"] = self.mask.to_dict()
        return d


MIXERS = {BiasedAttentionMixer.kind: BiasedAttentionMixer}


@dataclasses.dataclass(frozen=True)
class GeluFeedForward:
    """``down(gelu(gate(x)) * up(x))``, gelu in its tanh form."""
    kind = "dense"
    ff: int = key(convert=as_positive_int)

    @classmethod
    def from_json(cls, obj, where="mlp"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        return {"kind": "dense", "ff": self.ff}


@dataclasses.dataclass(frozen=True)
class ExpertGroups:
    """``count`` equal groups of neighbouring experts, of which the ``keep`` best can be chosen from."""
    count: int = key(convert=as_positive_int)
    keep: int = key(convert=as_positive_int)

    @classmethod
    def from_json(cls, obj, where="groups"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        return {"count": self.count, "keep": self.keep}


@dataclasses.dataclass(frozen=True)
class GroupedRouter:
    experts: int = key(convert=as_positive_int)
    top: int = key(convert=as_positive_int)
    groups: Optional[ExpertGroups] = key(default=None, convert=optional(_obj(ExpertGroups, "groups")))

    @classmethod
    def from_json(cls, obj, where="router"):
        r = cls(**parse_fields(cls, obj, where))
        if r.top > r.experts or r.experts > 1024:
            raise ConfigError(f"{where}: top {r.top} of {r.experts} experts (up to 1,024) is not possible")
        g = r.groups
        if g is not None and (r.experts % g.count or g.keep > g.count or g.keep * (r.experts // g.count) < r.top):
            raise ConfigError(f"{where}: {r.experts} experts in {g.count} equal groups, top {r.top} from the best {g.keep} "
                              f"of them, is not possible")
        return r

    def to_dict(self):
        d: Dict[str, Any] = {"experts": self.experts, "top": self.top}
        if self.groups is not None:
            d["groups"] = self.groups.to_dict()
        return d


@dataclasses.dataclass(frozen=True)
class GroupedExperts:
    kind = "moe"
    expert: ClampedExpert = key(convert=_obj(ClampedExpert, "expert"))
    router: GroupedRouter = key(convert=_obj(GroupedRouter, "router"))
    shared: Optional[ClampedExpert] = key(default=None, convert=optional(_obj(ClampedExpert, "shared")))

    @classmethod
    def from_json(cls, obj, where="mlp"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        d: Dict[str, Any] = {"kind": "moe", "expert": self.expert.to_dict(), "router": self.router.to_dict()}
        if self.shared is not None:
            d["shared"] = self.shared.to_dict()
        return d


FEED_FORWARDS = {c.kind: c for c in (GeluFeedForward, GroupedExperts)}


@dataclasses.dataclass(frozen=True)
class GeroraxLayer:
    type: str
    mixer: BiasedAttentionMixer
    mlp: Union[GeluFeedForward, GroupedExperts, None]

    @classmethod
    def from_json(cls, obj, where):
        if not isinstance(obj, dict) or "type" not in obj or "mixer" not in obj:
            raise ConfigError(f"{where}: a layer needs 'type' and 'mixer'")
        if obj["type"] not in MIXERS:
            raise ConfigError(f"{where}: layer type {obj['type']!r} is not supported (known: {', '.join(sorted(MIXERS))})")
        mlp = obj.get("mlp")
        if mlp is not None:
            if not isinstance(mlp, dict) or mlp.get("kind") not in FEED_FORWARDS:
                raise ConfigError(f"{where}.mlp: kind must be one of {', '.join(sorted(FEED_FORWARDS))}")
            mlp = FEED_FORWARDS[mlp["kind"]].from_json(mlp, where + ".mlp")
        return cls(obj["type"], MIXERS[obj["type"]].from_json(obj["mixer"], where + ".mixer"), mlp)

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None}


def _layers(v: Any) -> Tuple[GeroraxLayer, ...]:
    if not isinstance(v, list) or not v:
        raise ConfigError("layers: expected a list with at least one layer")
    return tuple(GeroraxLayer.from_json(x, f"layers[{i}]") for i, x in enumerate(v))


@dataclasses.dataclass(frozen=True)
class GeroraxConfig(ModelConfig):
    architectures = ("Gerorax",)

    layers: Tuple[GeroraxLayer, ...] = key(convert=_layers)
    norm_eps: float = key("norm", convert=_eps)
    vocab: int = key(convert=as_positive_int)
    width: int = key(convert=as_positive_int)
    embedding: ScaledEmbedding = key(default=ScaledEmbedding(), convert=_obj(ScaledEmbedding, "embedding"))
    residual_mult: float = key(default=1.0, convert=as_float)
    loop: Optional[LayerLoop] = key(default=None, convert=optional(_obj(LayerLoop, "loop")))
    max_positions: int = key(default=1 << 20, convert=as_positive_int)

    def validate(self, where: str) -> None:
        if self.loop is not None and not 0 <= self.loop.start < self.loop.stop <= len(self.layers):
            raise ConfigError(f"{where}: loop {self.loop.start}..{self.loop.stop} does not lie within the "
                              f"{len(self.layers)} layers")

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"architecture": "Gerorax", "embedding": self.embedding.to_dict(),
                             "layers": [l.to_dict() for l in self.layers], "norm": {"eps": self.norm_eps},
                             "residual_mult": self.residual_mult, "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            d["loop"] = self.loop.to_dict()
        if self.max_positions != 1 << 20:
            d["max_positions"] = self.max_positions
        return d
