"""Shared pieces of the Gerorax tests: small configurations that differ from each other in every size, and the plain
model's weights as numpy arrays."""
from __future__ import annotations

import os

import numpy as np
import torch


def attention(dim=24, heads=6, kv_heads=2, vdim=40, scale=0.2, window=13, keep=3):
    m = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale, "vdim": vdim}
    if window:
        m["mask"] = {"keep_first": keep, "size": window}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff=32, experts=6, top=2, groups=(3, 2), limit=1.5, shared=(48, 0.7)):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if groups:
        m["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def config(layers, width=64, vocab=97, eps=1e-5, scale=3.0, mult=0.7, loop=None):
    c = {"architecture": "Gerorax", "embedding": {"scale": scale},
         "layers": [{"type": "attention", "mixer": m, "mlp": f} for m, f in layers], "norm": {"eps": eps},
         "residual_mult": mult, "vocab": vocab, "width": width}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


# heads whose number is no power of two, values wider and narrower than keys, a window shorter than a page and one with more
# kept keys than a page holds, a layer without a window and without a feed-forward; a loop in the middle, run three times
GER_A = config([
    (attention(24, 6, 2, 40, 0.2, 13, 3), moe(32, 6, 2, (3, 2), 1.5, (48, 0.7))),
    (attention(16, 4, 4, 16, 0.3, 21, 18), dense(48)),
    (attention(40, 3, 1, 24, 0.15, None), None),
    (attention(16, 2, 1, 56, 0.25, 50, 33), moe(64, 8, 3, (4, 3), 0.8, (32, 2.0))),
], width=64, vocab=97, scale=3.0, mult=0.7, loop=(1, 3, 3))
# sizes the kernels like; the first layers looped twice; one group kept; every expert used in the last layer; no shared one
GER_B = config([
    (attention(64, 8, 4, 64, 0.125, 50, 5), moe(64, 12, 4, (2, 1), 1.0, (64, 1.0))),
    (attention(32, 8, 2, 32, 0.2, 32, 1), dense(96)),
    (attention(48, 4, 2, 80, 0.15, 17, 0), moe(32, 4, 4, None, 3.0, None)),
], width=128, vocab=211, eps=3e-6, scale=1.0, mult=1.0, loop=(0, 2, 2))
# sizes that are no multiple of anything; a window of one key; all groups kept; no loop; a number that shrinks the embedding
GER_C = config([
    (attention(10, 3, 3, 5, 0.4, 1, 2), dense(20)),
    (attention(7, 5, 1, 3, 0.5, 9, 0), moe(10, 6, 2, (3, 3), 0.5, (7, 0.25))),
    (attention(18, 2, 2, 33, 0.3, None), moe(12, 6, 1, (6, 1), 5.0, (20, 0.1))),
], width=40, vocab=50, scale=0.5, mult=1.3)
# one of everything: one head, a column, a window of one key beside the first, one expert, one pass of the loop
GER_D = config([
    (attention(2, 1, 1, 1, 1.0, 1, 1), moe(16, 1, 1, (1, 1), 1.0, (16, 1.0))),
    (attention(8, 1, 1, 8, 0.7, 2, 1), dense(16)),
], width=32, vocab=30, scale=2.0, mult=0.25, loop=(1, 2, 1))


def random_config(rng):
    """A configuration drawn from ``rng`` (a ``random.Random``): two to five layers, sizes that are and are not multiples
    of what the kernels like, every optional key present or absent."""
    layers = []
    for _ in range(rng.randint(2, 5)):
        r = rng.random()
        experts, top, groups = rng.choice([(4, 1, (2, 1)), (6, 3, (2, 1)), (8, 8, None), (16, 4, (4, 2)), (70, 6, (7, 3)),
                                           (12, 2, (12, 5))])
        mlp = None if r < 0.12 else dense(rng.choice([64, 100, 256])) if r < 0.5 else moe(
            rng.choice([16, 24, 64, 100]), experts, top, groups if rng.random() < 0.8 else None, rng.choice([0.5, 1.0, 7.0]),
            rng.choice([None, (32, 1.0), (60, 0.5), (128, 3.0)]))
        kv = rng.choice([1, 2, 3])
        m = attention(rng.choice([8, 12, 16, 32, 60, 64]), kv * rng.choice([1, 2, 3, 4]), kv,
                      rng.choice([8, 16, 20, 32, 50, 64]), rng.choice([0.1, 0.3]),
                      rng.choice([None, 1, 5, 16, 31, 64, 100, 150]), rng.choice([0, 1, 4, 16, 17, 40]))
        layers.append((m, mlp))
    n = len(layers)
    lo = rng.randint(0, n - 1)
    return config(layers, width=rng.choice([96, 128, 192, 256, 320]), vocab=rng.choice([50, 97, 300, 1000]),
                  eps=rng.choice([1e-6, 1e-5]), scale=rng.choice([1.0, 10.0, 0.5]), mult=rng.choice([1.0, 0.3, 0.8]),
                  loop=rng.choice([None, (lo, rng.randint(lo + 1, n), rng.randint(1, 3))]))


def numpy_weights(path: str):
    from safetensors.torch import load_file
    return {k: v.to(torch.float64).numpy() for k, v in load_file(os.path.join(path, "model.safetensors")).items()}


def as_numpy(w: dict, prefix: str = ""):
    """A dict of torch tensors as float64 numpy arrays, the names behind ``prefix``."""
    return {prefix + k: np.asarray(v.to(torch.float64)) for k, v in w.items()}
