"""Typed configuration of the Duduvik decoder.

config.json of this design is nested: ``layers`` lists every layer with its ``type`` (which mixer it has: ``gla``,
``retention`` or ``latent_attention``), the mixer's sizes and constants (``mixer``) and its feed-forward (``mlp``:
``kind`` ``dense`` or ``moe``; null for a layer without one); ``embedding.scale`` multiplies the embedding's rows;
``norm.eps``, ``vocab`` and ``width`` stand at the top, and ``architecture`` names the design.  Every layer may have
sizes of its own.  The design has no largest position (rotation angles are worked out from the position);
``max_positions`` (not a key of the design) bounds a request's length for the engine and defaults to 2^20.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, Optional, Tuple, Union

from .bafilorn import _decays
from .base import ConfigError, ModelConfig, as_float, as_int, as_positive_int, key, optional, parse_fields
from .morulix import WindowMask, _eps, _obj


def as_positive_float(v: Any) -> float:
    v = as_float(v)
    if not v > 0:
        raise ValueError(f"expected a positive number, got {v}")
    return v


@dataclasses.dataclass(frozen=True)
class HalfRotation:
    """Rotation of the first ``dims`` columns of a head (or of a head's rotated part), column i paired with column
    i + dims/2."""
    base: float = key(convert=as_positive_float)
    dims: int = key(convert=as_int)

    @classmethod
    def from_json(cls, obj, where="rot"):
        r = cls(**parse_fields(cls, obj, where))
        if r.dims < 0 or r.dims % 2:
            raise ConfigError(f"{where}: dims must be even and not negative")
        return r

    def to_dict(self):
        return {"base": self.base, "dims": self.dims}


@dataclasses.dataclass(frozen=True)
class GatedLinearMixer:
    """Linear attention with a decay per key channel and token."""
    kind = "gla"
    dim: int = key(convert=as_positive_int)
    heads: int = key(convert=as_positive_int)
    tau: float = key(convert=as_positive_float)
    vdim: int = key(convert=as_positive_int)
    #: inner size of the decays' low-rank map for random weights (not a key of the design: a checkpoint's tensors say)
    rank: Optional[int] = key(default=None, convert=optional(as_positive_int))

    @classmethod
    def from_json(cls, obj, where="mixer"):
        m = cls(**parse_fields(cls, obj, where))
        if m.dim > 256:
            raise ConfigError(f"{where}: dim beyond 256 is not supported")
        return m

    def to_dict(self):
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "tau": self.tau, "vdim": self.vdim}
        if self.rank is not None:
            d["rank"] = self.rank
        return d


@dataclasses.dataclass(frozen=True)
class RetentionMixer:
    """Linear attention with a fixed decay per head and rotated queries and keys."""
    kind = "retention"
    decay: Tuple[float, ...] = key(convert=_decays)
    dim: int = key(convert=as_positive_int)
    heads: int = key(convert=as_positive_int)
    vdim: int = key(convert=as_positive_int)
    rot: Optional[HalfRotation] = key(default=None, convert=optional(_obj(HalfRotation, "rot")))

    @classmethod
    def from_json(cls, obj, where="mixer"):
        m = cls(**parse_fields(cls, obj, where))
        p = []
        if len(m.decay) != m.heads:
            p.append(f"{len(m.decay)} decays for {m.heads} heads")
        if m.dim > 256:
            p.append("dim beyond 256 is not supported")
        if m.rot is not None and m.rot.dims > m.dim:
            p.append(f"dim {m.dim} cannot hold the {m.rot.dims} rotated columns")
        if p:
            raise ConfigError(f"{where}: " + "; ".join(p))
        return m

    def to_dict(self):
        d: Dict[str, Any] = {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclasses.dataclass(frozen=True)
class WindowedLatentMixer:
    """Attention over a cached latent with a rotated key part shared by the heads, queries through a latent of their own,
    and a window."""
    kind = "latent_attention"
    dim: int = key(convert=as_positive_int)
    heads: int = key(convert=as_positive_int)
    kv_rank: int = key(convert=as_positive_int)
    q_rank: int = key(convert=as_positive_int)
    rot_dim: int = key(convert=as_int)
    vdim: int = key(convert=as_positive_int)
    scale: float = key(convert=as_float)
    mask: Optional[WindowMask] = key(default=None, convert=optional(_obj(WindowMask, "mask")))
    rot: Optional[HalfRotation] = key(default=None, convert=optional(_obj(HalfRotation, "rot")))

    @classmethod
    def from_json(cls, obj, where="mixer"):
        m = cls(**parse_fields(cls, obj, where))
        p = []
        if m.rot_dim < 0:
            p.append("rot_dim must not be negative")
        if m.rot is not None and m.rot.dims > m.rot_dim:
            p.append(f"rot_dim {m.rot_dim} cannot hold the {m.rot.dims} rotated columns")
        if m.kv_rank + m.rot_dim > 256:
            p.append(f"a cached key of {m.kv_rank + m.rot_dim} columns is more than the attention kernels' 256")
        if p:
            raise ConfigError(f"{where}: " + "; ".join(p))
        return m

    def to_dict(self):
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank,
                             "rot_dim": self.rot_dim, "vdim": self.vdim, "scale": self.scale}
        if self.mask is not None:
            d["mask"] = {"size": self.mask.size}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


MIXERS = {c.kind: c for c in (GatedLinearMixer, RetentionMixer, WindowedLatentMixer)}


@dataclasses.dataclass(frozen=True)
class DenseFeedForward:
    """``down(relu(gate(x)) * up(x))``."""
    kind = "dense"
    ff: int = key(convert=as_positive_int)

    @classmethod
    def from_json(cls, obj, where="mlp"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        return {"kind": "dense", "ff": self.ff}


@dataclasses.dataclass(frozen=True)
class ClampedExpert:
    """Columns of an expert and the bound of its gate and up values."""
    ff: int = key(convert=as_positive_int)
    limit: float = key(convert=as_positive_float)

    @classmethod
    def from_json(cls, obj, where="expert"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        return {"ff": self.ff, "limit": self.limit}


@dataclasses.dataclass(frozen=True)
class Router:
    experts: int = key(convert=as_positive_int)
    top: int = key(convert=as_positive_int)

    @classmethod
    def from_json(cls, obj, where="router"):
        r = cls(**parse_fields(cls, obj, where))
        if r.top > r.experts or r.experts > 1024:
            raise ConfigError(f"{where}: top {r.top} of {r.experts} experts (up to 1,024) is not possible")
        return r


@dataclasses.dataclass(frozen=True)
class ExpertsFeedForward:
    kind = "moe"
    expert: ClampedExpert = key(convert=_obj(ClampedExpert, "expert"))
    router: Router = key(convert=_obj(Router, "router"))
    shared: Optional[ClampedExpert] = key(default=None, convert=optional(_obj(ClampedExpert, "shared")))

    @classmethod
    def from_json(cls, obj, where="mlp"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        d: Dict[str, Any] = {"kind": "moe", "expert": self.expert.to_dict(),
                             "router": {"experts": self.router.experts, "top": self.router.top}}
        if self.shared is not None:
            d["shared"] = self.shared.to_dict()
        return d


FEED_FORWARDS = {c.kind: c for c in (DenseFeedForward, ExpertsFeedForward)}


@dataclasses.dataclass(frozen=True)
class DuduvikLayer:
    type: str
    mixer: Union[GatedLinearMixer, RetentionMixer, WindowedLatentMixer]
    mlp: Union[DenseFeedForward, ExpertsFeedForward, None]

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


@dataclasses.dataclass(frozen=True)
class ScaledEmbedding:
    scale: float = key(default=1.0, convert=as_float)

    @classmethod
    def from_json(cls, obj, where="embedding"):
        return cls(**parse_fields(cls, obj, where))

    def to_dict(self):
        return {"scale": self.scale}


def _layers(v: Any) -> Tuple[DuduvikLayer, ...]:
    if not isinstance(v, list) or not v:
        raise ConfigError("layers: expected a list with at least one layer")
    return tuple(DuduvikLayer.from_json(x, f"layers[{i}]") for i, x in enumerate(v))


@dataclasses.dataclass(frozen=True)
class DuduvikConfig(ModelConfig):
    architectures = ("Duduvik",)

    layers: Tuple[DuduvikLayer, ...] = key(convert=_layers)
    norm_eps: float = key("norm", convert=_eps)
    vocab: int = key(convert=as_positive_int)
    width: int = key(convert=as_positive_int)
    embedding: ScaledEmbedding = key(default=ScaledEmbedding(), convert=_obj(ScaledEmbedding, "embedding"))
    max_positions: int = key(default=1 << 20, convert=as_positive_int)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"architecture": "Duduvik", "embedding": self.embedding.to_dict(),
                             "layers": [l.to_dict() for l in self.layers], "norm": {"eps": self.norm_eps},
                             "vocab": self.vocab, "width": self.width}
        if self.max_positions != 1 << 20:
            d["max_positions"] = self.max_positions
        return d
