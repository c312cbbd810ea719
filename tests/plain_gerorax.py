"""A plain, slow Gerorax: one function per mechanism, numpy float64, whole sequences at once.

It shares no code with the engine.  ``cfg`` is the JSON object of a config.json, ``w`` a dict of float64 arrays by
checkpoint name.  Notation: h [T, width] is a sublayer's input, p the positions 0 .. T-1 of one sequence.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def norm(x, wt, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * wt


def sinusoid(p, width):
    """[T, width]: entries 2i and 2i + 1 are sine and cosine of p 10000^(-2i / width)."""
    out = np.zeros((len(p), width))
    for c in range(width):
        i = c // 2
        ang = np.asarray(p, dtype=np.float64) * 10000.0 ** (-2.0 * i / width)
        out[:, c] = np.sin(ang) if c % 2 == 0 else np.cos(ang)
    return out


def embed(tokens, p, w, cfg):
    return w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"] + sinusoid(p, cfg["width"])


# ---------------------------------------------------------------------------------------------------- attention

def slopes(heads):
    return np.array([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)])


def visible(p, mask):
    """[T, T] booleans: position i sees j <= i that is near (i - j < size) or among the first ``keep_first``."""
    i, j = np.asarray(p)[:, None], np.asarray(p)[None, :]
    seen = j <= i
    if mask:
        seen = seen & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return seen


def biased_softmax(q, k, v, p, scale, mask=None, sink=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]: scores (q . k) scale - slope_h (i - j) over the visible keys,
    a softmax whose denominator also holds exp(sink_h)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    seen = visible(p, mask)
    dist = np.asarray(p, dtype=np.float64)[:, None] - np.asarray(p, dtype=np.float64)[None, :]
    sl = slopes(H)
    for h in range(H):
        s = np.where(seen, q[:, h] @ k[:, h // per].T * scale - sl[h] * dist, -np.inf)
        top = s.max(axis=1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        e = np.exp(s - top)
        den = e.sum(axis=1, keepdims=True) + (np.exp(sink[h] - top) if sink is not None else 0.0)
        out[:, h] = (e / den) @ v[:, h // per]
    return out


def attention(h, p, w, pre, m, eps):
    H, G, d, dv, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q = norm((h @ w[pre + "q"].T).reshape(T, H, d), w[pre + "q.norm"], eps)
    k = norm((h @ w[pre + "k"].T).reshape(T, G, d), w[pre + "k.norm"], eps)
    v = (h @ w[pre + "v"].T).reshape(T, G, dv)
    o = biased_softmax(q, k, v, p, m["scale"], m.get("mask"), w[pre + "sink"])
    return o.reshape(T, H * dv) @ w[pre + "o"].T


# ---------------------------------------------------------------------------------------------------- feed-forwards

def dense(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def expert(h, w, pre, limit):
    """g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit); W_down (g sigmoid(1.702 g) (u + 1))."""
    g = np.minimum(h @ w[pre + "gate"].T, limit)
    u = np.clip(h @ w[pre + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def route(z, top, groups=None):
    """(chosen [T, top], their weights) from logits z [T, experts]: the softmax over all experts scores; with ``groups``
    only the experts of the ``keep`` groups whose best score is largest can be chosen."""
    e = np.exp(z - z.max(axis=1, keepdims=True))
    s = e / e.sum(axis=1, keepdims=True)
    can = np.ones_like(s, dtype=bool)
    if groups:
        size = z.shape[1] // groups["count"]
        best = s.reshape(len(s), groups["count"], size).max(axis=2)
        kept = np.argsort(-best, axis=1, kind="stable")[:, : groups["keep"]]
        can[:] = False
        for t in range(len(s)):
            for g in kept[t]:
                can[t, g * size: (g + 1) * size] = True
    ids = np.argsort(-np.where(can, s, -1.0), axis=1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, axis=1)


def moe(h, w, pre, m):
    ids, weights = route(h @ w[pre + "router"].T, m["router"]["top"], m["router"].get("groups"))
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(ids[t], weights[t]):
            out[t] += s * expert(h[t: t + 1], w, f"{pre}e{e}.", m["expert"]["limit"])[0]
    if m.get("shared"):
        out = out + expert(h, w, pre + "shared.", m["shared"]["limit"])
    return out


def feed_forward(h, w, pre, m):
    return dense(h, w, pre) if m["kind"] == "dense" else moe(h, w, pre, m)


# ---------------------------------------------------------------------------------------------------- the model

def layer(x, p, w, i, cfg):
    pre, eps, m, spec = f"l{i}.", cfg["norm"]["eps"], cfg["residual_mult"], cfg["layers"][i]
    y = attention(norm(x, w[pre + "norm1"], eps), p, w, pre + "mix.", spec["mixer"], eps)
    x = x + m * (w[pre + "ls1"] * norm(y, w[pre + "norm1b"], eps))
    if spec.get("mlp") is not None:
        y = feed_forward(norm(x, w[pre + "norm2"], eps), w, pre + "mlp.", spec["mlp"])
        x = x + m * (w[pre + "ls2"] * norm(y, w[pre + "norm2b"], eps))
    return x


def runs(cfg):
    """The layer runs in order: (layer, number of the pass that this layer begins or None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    body = list(range(loop["start"], loop["stop"]))
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == body[0] else None) for i in body]
    return out + [(i, None) for i in range(loop["stop"], n)]


def forward(tokens, w, cfg):
    """(logits [T, vocab], the stream after every layer run [runs, T, width]) for one whole sequence."""
    p = np.arange(len(tokens))
    x0 = embed(tokens, p, w, cfg)
    x, seen = x0, []
    for i, begins in runs(cfg):
        if begins is not None:
            if begins > 0:
                x = x + x0
            x = x + w["loop.step"][begins]
        x = layer(x, p, w, i, cfg)
        seen.append(x.copy())
    return norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T, np.stack(seen)
