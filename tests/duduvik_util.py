"""Shared pieces of the Duduvik tests: small configurations that differ from each other in every size, and the plain
model's weights as numpy arrays."""
from __future__ import annotations

import os

import numpy as np
import torch


def gla(heads=3, dim=24, vdim=40, tau=8.0, rank=None):
    m = {"dim": dim, "heads": heads, "tau": tau, "vdim": vdim}
    if rank is not None:
        m["rank"] = rank
    return m


def retention(heads=3, dim=16, vdim=24, base=100.0, rot_dims=None, decay=None):
    m = {"decay": list(decay) if decay is not None else [0.5 + 0.49 * (h + 1) / heads for h in range(heads)], "dim": dim,
         "heads": heads, "vdim": vdim}
    dims = dim if rot_dims is None else rot_dims
    if dims:
        m["rot"] = {"base": base, "dims": dims}
    return m


def latent(dim=16, heads=4, kv_rank=40, q_rank=24, rot_dim=8, vdim=24, scale=0.2, base=100.0, window=13):
    m = {"dim": dim, "heads": heads, "kv_rank": kv_rank, "q_rank": q_rank, "rot_dim": rot_dim, "vdim": vdim, "scale": scale}
    if rot_dim:
        m["rot"] = {"base": base, "dims": rot_dim}
    if window:
        m["mask"] = {"size": window}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff=32, experts=5, top=2, limit=1.5, shared=(48, 0.7)):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def config(layers, width=64, vocab=97, eps=1e-5, scale=3.0):
    return {"architecture": "Duduvik", "embedding": {"scale": scale},
            "layers": [{"type": k, "mixer": m, "mlp": f} for k, m, f in layers], "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


# all three mixers, both feed-forwards and none; experts whose shared expert has another width and another bound
DUD_A = config([
    ("retention", retention(heads=3, dim=16, vdim=24, base=100.0), moe(32, 5, 2, 1.5, (48, 0.7))),
    ("latent_attention", latent(window=13), dense(48)),
    ("gla", gla(heads=3, dim=24, vdim=40, tau=8.0, rank=6), None),
    ("gla", gla(heads=2, dim=40, vdim=16, tau=2.0, rank=20), moe(64, 7, 3, 0.8, (32, 2.0))),
], width=64, vocab=97, scale=3.0)
# sizes the kernels like; two windows (two groups of pages), one of them a page long; only half of the columns rotated; no
# factor on the embedding; every expert used
DUD_B = config([
    ("latent_attention", latent(dim=32, heads=2, kv_rank=64, q_rank=48, rot_dim=32, vdim=16, scale=0.15, base=500.0,
                                window=16), moe(64, 4, 4, 1.0, (64, 1.0))),
    ("gla", gla(heads=4, dim=64, vdim=128, tau=16.0, rank=16), dense(96)),
    ("retention", retention(heads=2, dim=64, vdim=64, base=3000.0, rot_dims=32, decay=[0.97, 0.999]), dense(64)),
    ("latent_attention", latent(dim=16, heads=8, kv_rank=32, q_rank=32, rot_dim=16, vdim=32, scale=0.2, base=50.0,
                                window=50), moe(32, 9, 1, 3.0, None)),
], width=128, vocab=211, eps=3e-6, scale=1.0)
# sizes that are no multiple of anything; one head; a decay of one and one of nothing; no rotation; no window; a power of
# one for the decays
DUD_C = config([
    ("retention", retention(heads=4, dim=10, vdim=5, rot_dims=0, decay=[1.0, 0.0, 0.3, 0.9]), dense(20)),
    ("gla", gla(heads=1, dim=7, vdim=3, tau=1.0, rank=3), moe(10, 3, 2, 0.5, (7, 0.25))),
    ("latent_attention", latent(dim=10, heads=3, kv_rank=20, q_rank=12, rot_dim=6, vdim=6, scale=0.4, base=30.0,
                                window=None), moe(12, 6, 1, 5.0, (20, 0.1))),
    ("retention", retention(heads=1, dim=18, vdim=33, base=20.0, rot_dims=6, decay=[0.8]), None),
], width=40, vocab=50, scale=0.5)
# one of everything: one head, one column, a window of one key, one expert
DUD_D = config([
    ("latent_attention", latent(dim=8, heads=1, kv_rank=16, q_rank=8, rot_dim=2, vdim=8, scale=1.0, base=2.0, window=1),
     moe(16, 1, 1, 1.0, (16, 1.0))),
    ("retention", retention(heads=1, dim=2, vdim=1, base=2.0, decay=[0.9]), dense(16)),
    ("gla", gla(heads=1, dim=1, vdim=1, tau=4.0, rank=1), dense(16)),
], width=32, vocab=30, scale=2.0)


def random_config(rng):
    """A configuration drawn from ``rng`` (a ``random.Random``): two to six layers of the three kinds in any order, sizes
    that are and are not multiples of what the kernels like, every optional key present or absent."""
    kinds = ["gla", "retention", "latent_attention"]
    order = [rng.choice(kinds) for _ in range(rng.randint(2, 4))]
    order += [k for k in kinds if k not in order and rng.random() < 0.7]
    layers = []
    for k in order:
        r = rng.random()
        mlp = None if r < 0.15 else dense(rng.choice([64, 100, 256])) if r < 0.5 else moe(
            rng.choice([16, 24, 64, 100]), *rng.choice([(4, 1), (6, 3), (8, 8), (16, 4), (70, 6)]), rng.choice([0.5, 1.0, 7.0]),
            rng.choice([None, (32, 1.0), (60, 0.5), (128, 3.0)]))
        if k == "gla":
            m = gla(rng.choice([1, 2, 4, 5]), rng.choice([8, 20, 32, 48, 64, 96, 128, 160]), rng.choice([8, 24, 33, 64, 100, 144]),
                    rng.choice([1.0, 4.0, 16.0, 20.0]), rng.choice([2, 8, 16, 21]))
        elif k == "retention":
            d, h = rng.choice([8, 16, 32, 48, 64, 100, 128]), rng.choice([1, 2, 4, 6])
            m = retention(h, d, rng.choice([8, 24, 33, 64, 128]), rng.choice([100.0, 1e4, 5e5]),
                          rng.choice([c for c in (0, 4, 8, 16, d) if c <= d]),
                          [1.0 - 2.0 ** -rng.uniform(1.0, 11.0) for _ in range(h)])
        else:
            rd = rng.choice([0, 2, 8, 16, 32])
            m = latent(rng.choice([8, 16, 24, 64]), rng.choice([1, 2, 3, 8]), rng.choice([16, 24, 48, 96, 128]),
                       rng.choice([8, 32, 64, 100]), rd, rng.choice([8, 16, 48, 64]), rng.choice([0.1, 0.2]),
                       rng.choice([100.0, 1e4, 5e4]), rng.choice([None, 2, 5, 16, 31, 64, 100]))
        layers.append((k, m, mlp))
    return config(layers, width=rng.choice([96, 128, 192, 256, 320]), vocab=rng.choice([50, 97, 300, 1000]),
                  eps=rng.choice([1e-6, 1e-5]), scale=rng.choice([1.0, 10.0, 0.5]))


def numpy_weights(path: str):
    from safetensors.torch import load_file
    return {k: v.to(torch.float64).numpy() for k, v in load_file(os.path.join(path, "model.safetensors")).items()}


def as_numpy(w: dict, prefix: str = ""):
    """A dict of torch tensors as float64 numpy arrays, the names behind ``prefix``."""
    return {prefix + k: np.asarray(v.to(torch.float64)) for k, v in w.items()}
