"""Position encodings.

``RotaryEncoding``: rotation of half-split pairs (i, i + hd/2) by angle position x inv_freq_i.  Inverse
frequencies are ``theta^(-2i/hd)`` (models/src/llama.rs:146-152), optionally rescaled by the llama3 rule
(models/src/llama.rs:163-186).  The table of cos and sin is built once, in float32, for every position below
``max_positions`` (models/src/llama.rs:189-199) and stays float32 whatever the activation dtype is; all layers
with equal parameters share it.  ``NoPosition`` encodes nothing.  ``DistanceBias`` rotates nothing and takes a multiple of
the distance off the scores.
"""
from __future__ import annotations

import math
from typing import Dict, Optional, Tuple

import torch

from ..kernels import ops
from .base import PositionEncoding, register_position

_TABLES: Dict[tuple, Tuple[torch.Tensor, torch.Tensor]] = {}


def rotary_inv_freq(head_size: int, theta: float, scaling: Optional[dict], precise: bool = False) -> torch.Tensor:
    """float32 inverse frequencies [head_size / 2]; ``scaling`` holds the llama3 constants or is None.  ``precise``:
    worked out in float64 and rounded once, where the default follows the reference's float32 steps."""
    if precise:
        return _inv_freq(head_size, theta, scaling, torch.float64).to(torch.float32)
    return _inv_freq(head_size, theta, scaling, torch.float32)


def _inv_freq(head_size: int, theta: float, scaling: Optional[dict], f32: torch.dtype) -> torch.Tensor:
    exps = torch.arange(0, head_size, 2, dtype=f32) / torch.tensor(float(head_size), dtype=f32)
    freq = 1.0 / torch.pow(torch.tensor(float(theta), dtype=f32), exps)
    if scaling is None:
        return freq
    orig = torch.tensor(float(scaling["original_max_position_embeddings"]), dtype=f32)
    factor = torch.tensor(float(scaling["factor"]), dtype=f32)
    low = torch.tensor(float(scaling["low_freq_factor"]), dtype=f32)
    high = torch.tensor(float(scaling["high_freq_factor"]), dtype=f32)
    wavelen = torch.tensor(2.0, dtype=f32) * torch.tensor(math.pi, dtype=f32) / freq
    smooth = (orig / wavelen - low) / (high - low)
    mid = (1.0 - smooth) * freq / factor + smooth * freq
    return torch.where(wavelen < orig / high, freq, torch.where(wavelen > orig / low, freq / factor, mid))


class RotaryEncoding(PositionEncoding):
    def __init__(self, head_size: int, theta: float, max_positions: int, scaling: Optional[dict] = None,
                 rotary_dim: Optional[int] = None, precise: bool = False):
        self.precise = bool(precise)
        self.head_size, self.theta, self.max_positions = int(head_size), float(theta), int(max_positions)
        self.scaling = dict(scaling) if scaling else None
        self.rotary_dim = int(rotary_dim) if rotary_dim is not None else self.head_size
        if self.rotary_dim % 2 or not 0 < self.rotary_dim <= self.head_size:
            raise ValueError(f"rotary_dim {self.rotary_dim} must be even and at most the head size {self.head_size}")
        self.cos = self.sin = None

    def _key(self, device):
        sc = tuple(sorted(self.scaling.items())) if self.scaling else None
        return (self.rotary_dim, self.theta, self.max_positions, sc, str(device), self.precise)

    def graph_safe(self) -> bool:
        return True

    def prepare(self, device) -> None:
        key = self._key(device)
        if key not in _TABLES:
            inv = rotary_inv_freq(self.rotary_dim, self.theta, self.scaling, self.precise)
            ang = torch.arange(self.max_positions, dtype=torch.float32)[:, None] * inv[None, :]
            _TABLES[key] = (torch.cos(ang).to(device).contiguous(), torch.sin(ang).to(device).contiguous())
        self.cos, self.sin = _TABLES[key]

    def load(self, get, device, act_dtype) -> None:
        self.prepare(device)

    def rotary_tables(self):
        return self.cos, self.sin, self.rotary_dim

    def apply(self, q, k, positions) -> None:
        # q and k are rotated with the same kernel that mixers fuse with the cache write, without a cache
        t, nh, hd = q.shape
        nkv = k.shape[1]
        for x, heads in ((q, nh), (k, nkv)):
            ops.rope_cache_write(x.view(t, heads * hd), positions, self.cos, self.sin, self.rotary_dim, None, None,
                                 None, 1, heads, 0, hd)


class NoPosition(PositionEncoding):
    def __init__(self, **_):
        pass

    def graph_safe(self) -> bool:
        return True

    def apply(self, q, k, positions) -> None:
        return None


class DistanceBias(NoPosition):
    """The score of the key at j for the query at p loses ``slope_h (p - j)``, slope_h = 2^(-exponent (h + 1) / heads)
    for head h = 0 .. heads - 1."""

    def __init__(self, exponent: float = 8.0):
        self.exponent = float(exponent)

    def score_slopes(self, num_heads: int) -> torch.Tensor:
        h = torch.arange(1, num_heads + 1, dtype=torch.float64)
        return torch.pow(2.0, -self.exponent * h / num_heads).to(torch.float32)


def clear_tables() -> None:
    _TABLES.clear()


def rotation_frequencies(base: float, dims: int, scaling: Optional[dict] = None):
    """(float32 tensor [dims / 2] of base^(-2i / dims), worked out in double precision and rounded once; the factor on
    cosines and sines).  ``scaling`` = {factor, original, fast, slow} slows the long waves down: with
    where(t) = dims ln(original / (2 pi t)) / (2 ln base), lo = max(floor(where(fast)), 0), hi = min(ceil(where(slow)),
    dims - 1) and ramp_i = clamp((i - lo) / max(hi - lo, 0.001), 0, 1), pair i turns at
    f_i / factor * ramp_i + f_i (1 - ramp_i), and cosines and sines are multiplied by 0.1 ln(factor) + 1."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / max(dims, 1))
    mag = 1.0
    if scaling is not None:
        factor, original = float(scaling["factor"]), float(scaling["original"])

        def where(turns: float) -> float:
            return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

        lo = max(math.floor(where(float(scaling["fast"]))), 0)
        hi = min(math.ceil(where(float(scaling["slow"]))), dims - 1)
        ramp = torch.clamp((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
        f = f / factor * ramp + f * (1.0 - ramp)
        mag = 0.1 * math.log(factor) + 1.0
    return f.to(torch.float32), mag


register_position("rotary", RotaryEncoding)
register_position("none", NoPosition)
register_position("distance_bias", DistanceBias)
