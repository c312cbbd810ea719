"""A plain, slow Duduvik: one function per mechanism, numpy float64, whole sequences at once or token by token.

It shares no code with the engine.  ``cfg`` is the JSON object of a config.json, ``w`` a dict of float64 arrays by
checkpoint name.  Notation: h [T, width] is a sublayer's input, p the positions 0 .. T-1 of one sequence.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_one_plus(x, wt, eps):
    return unit_rms(x, eps) * (1.0 + wt)


def embed(tokens, w, cfg):
    return w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]


def rotate_half(x, p, rot):
    """x [T, heads, d]: column i < dims / 2 of every head paired with column i + dims / 2, turned by p base^(-2i / dims);
    columns from dims on stay."""
    if not rot or not rot["dims"]:
        return x.copy()
    half = rot["dims"] // 2
    freq = np.array([rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(half)])
    ang = np.asarray(p, dtype=np.float64)[:, None] * freq[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half: 2 * half]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * half:]], axis=-1)


# ---------------------------------------------------------------------------------------------------- recurrences

def decayed_sum(q, k, v, alpha, state=None):
    """Per head S <- diag(alpha) S + k v^T, o = S^T q; q, k, alpha [T, H, d], v [T, H, dv] -> (o [T, H, dv], S)."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2])) if state is None else np.array(state, dtype=np.float64)
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.sum(S * q[t][:, :, None], axis=1)
    return o, S


def gla_decay(h, w, pre, m):
    """alpha [T, H, d] = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)."""
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    return np.exp(-np.logaddexp(0.0, -z) / m["tau"]).reshape(h.shape[0], m["heads"], m["dim"])


def gla(h, w, pre, m, eps, state=None):
    """Gated linear attention.  Returns (output, state [H, d, dv])."""
    H, d, dv, T = m["heads"], m["dim"], m["vdim"], h.shape[0]
    q = (h @ w[pre + "q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w[pre + "k"].T).reshape(T, H, d)
    v = (h @ w[pre + "v"].T).reshape(T, H, dv)
    o, S = decayed_sum(q, k, v, gla_decay(h, w, pre, m), state)
    o = unit_rms(o, eps) * w[pre + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T, S


def retention(h, p, w, pre, m, eps, state=None):
    """Linear attention with a fixed decay per head and rotated q and k.  Returns (output, state [H, d, dv])."""
    H, d, dv, T = m["heads"], m["dim"], m["vdim"], h.shape[0]
    q = rotate_half((h @ w[pre + "q"].T).reshape(T, H, d), p, m.get("rot"))
    k = rotate_half((h @ w[pre + "k"].T).reshape(T, H, d), p, m.get("rot")) * d ** -0.5
    v = (h @ w[pre + "v"].T).reshape(T, H, dv)
    alpha = np.broadcast_to(np.asarray(m["decay"], dtype=np.float64)[None, :, None], (T, H, d))
    o, S = decayed_sum(q, k, v, alpha, state)
    return (unit_rms(o, eps).reshape(T, H * dv) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T, S


# ---------------------------------------------------------------------------------------------------- attention

def windowed_softmax(q, k, v, p, scale, window=None):
    """q [T, H, d], k [T, H, d], v [T, H, dv]; position i sees j with 0 <= i - j < window (every j <= i without one)."""
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[2]))
    dist = np.asarray(p)[:, None] - np.asarray(p)[None, :]
    seen = (dist >= 0) & (dist < window) if window else dist >= 0
    for hh in range(H):
        s = np.where(seen, (q[:, hh] @ k[:, hh].T) * scale, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, hh] = (e / e.sum(axis=1, keepdims=True)) @ v[:, hh]
    return out


def latent_attention(h, p, w, pre, m, eps):
    H, d, r, dv, kr, T = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], h.shape[0]
    cq = unit_rms(h @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]
    q = (cq @ w[pre + "uq"].T).reshape(T, H, d + r)
    low = h @ w[pre + "dkv"].T
    c = unit_rms(low[:, :kr], eps) * w[pre + "dkv.norm"]
    shared = rotate_half(low[:, kr:].reshape(T, 1, r), p, m.get("rot"))
    qq = np.concatenate([q[..., :d], rotate_half(q[..., d:], p, m.get("rot"))], axis=2)
    k = np.concatenate([(c @ w[pre + "uk"].T).reshape(T, H, d), np.repeat(shared, H, axis=1)], axis=2)
    v = (c @ w[pre + "uv"].T).reshape(T, H, dv)
    window = m["mask"]["size"] if m.get("mask") else None
    return windowed_softmax(qq, k, v, p, m["scale"], window).reshape(T, H * dv) @ w[pre + "o"].T


# ---------------------------------------------------------------------------------------------------- feed-forwards

def dense(h, w, pre):
    return (np.maximum(h @ w[pre + "gate"].T, 0.0) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def expert(h, w, pre, limit):
    """g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit); W_down (g sigmoid(1.702 g) (u + 1))."""
    g = np.minimum(h @ w[pre + "gate"].T, limit)
    u = np.clip(h @ w[pre + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def route(h, w, pre, top):
    """(chosen [T, top], their weights): the largest logits, softmax over the chosen ones."""
    z = h @ w[pre + "router"].T + w[pre + "router.b"]
    ids = np.argsort(-z, axis=1, kind="stable")[:, :top]
    zc = np.take_along_axis(z, ids, axis=1)
    e = np.exp(zc - zc.max(axis=1, keepdims=True))
    return ids, e / e.sum(axis=1, keepdims=True)


def moe(h, w, pre, m):
    ids, weights = route(h, w, pre, m["router"]["top"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(ids[t], weights[t]):
            out[t] += s * expert(h[t: t + 1], w, f"{pre}e{e}.", m["expert"]["limit"])[0]
    if m.get("shared"):
        out = out + expert(h, w, pre + "shared.", m["shared"]["limit"])
    return out


def feed_forward(h, w, pre, m):
    return dense(h, w, pre) if m["kind"] == "dense" else moe(h, w, pre, m)


def mixer(kind, h, p, w, pre, m, eps):
    if kind == "gla":
        return gla(h, w, pre, m, eps)[0]
    if kind == "retention":
        return retention(h, p, w, pre, m, eps)[0]
    if kind == "latent_attention":
        return latent_attention(h, p, w, pre, m, eps)
    raise ValueError(kind)


def forward(tokens, w, cfg):
    """(logits [T, vocab], the stream after every layer [layers, T, width]) for one whole sequence."""
    eps = cfg["norm"]["eps"]
    p = np.arange(len(tokens))
    x = embed(tokens, w, cfg)
    seen = []
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        y = mixer(layer["type"], norm_one_plus(x, w[pre + "norm1"], eps), p, w, pre + "mix.", layer["mixer"], eps)
        x = x + norm_one_plus(y, w[pre + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = feed_forward(norm_one_plus(x, w[pre + "norm2"], eps), w, pre + "mlp.", layer["mlp"])
            x = x + norm_one_plus(y, w[pre + "norm2b"], eps)
        seen.append(x.copy())
    return norm_one_plus(x, w["final.norm"], eps) @ w["embed"].T, np.stack(seen)
