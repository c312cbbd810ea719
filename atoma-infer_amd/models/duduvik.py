"""The Duduvik decoder put together from parts.

The embedding's rows are multiplied by a number; every layer is a sandwich block (a norm before and behind each
sublayer, weights stored around zero).  The mixer is, layer by layer, gated linear attention (``gla``: a decay per key
channel and token), retention (a fixed decay per head, rotated queries and keys) or attention over a cached latent with
a rotated key part and a window (``latent_attention``); the feed-forward a dense one gated by relu, or routed experts
with clamped gates (the softmax over the chosen logits weighs the experts' outputs) beside an expert that every token
uses.  The output head is the embedding table, without its factor.  Tensor names are the checkpoint's own: ``embed``,
``l<i>.norm1`` / ``norm1b`` / ``norm2`` / ``norm2b``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``.
"""
from __future__ import annotations

from ..config.duduvik import (DenseFeedForward, DuduvikConfig, ExpertsFeedForward, GatedLinearMixer, RetentionMixer,
                              WindowedLatentMixer)
from ..config.registry import register_architecture
from ..parts.base import make_part
from ..parts.embedding import OutputHead, TokenEmbedding
from .spec import ModelSpec

GATE_SLOPE = 1.702      # of the experts' gate, g sigmoid(slope g): fixed by the design


def _mixer(m, width: int, eps: float):
    if isinstance(m, GatedLinearMixer):
        return make_part("mixer", "decayed_linear_attention", width=width, heads=m.heads, dim=m.dim, vdim=m.vdim,
                         norm_eps=eps, tau=m.tau, rank=m.rank, q_scale=m.dim ** -0.5, norm_weight=True)
    if isinstance(m, RetentionMixer):
        return make_part("mixer", "decayed_linear_attention", width=width, heads=m.heads, dim=m.dim, vdim=m.vdim,
                         norm_eps=eps, decay=m.decay, rotary_base=m.rot.base if m.rot else 10000.0,
                         rotary_dim=m.rot.dims if m.rot else 0, k_scale=m.dim ** -0.5)
    if isinstance(m, WindowedLatentMixer):
        return make_part("mixer", "rotary_latent_attention", width=width, num_heads=m.heads, head_size=m.dim,
                         rotary_size=m.rot_dim, value_size=m.vdim, rank=m.kv_rank, q_rank=m.q_rank, scale=m.scale,
                         norm_eps=eps, rotary_base=m.rot.base if m.rot else 10000.0,
                         rotary_dim=m.rot.dims if m.rot else 0, interleaved=False, gated=False,
                         window=m.mask.size if m.mask else None)
    raise TypeError(f"no part for mixer {m!r}")


def _feed_forward(f, width: int):
    if f is None:
        return None
    if isinstance(f, DenseFeedForward):
        return make_part("feed_forward", "swiglu", width=width, intermediate=f.ff, names=("gate", "up", "down"),
                         activation="relu")
    if isinstance(f, ExpertsFeedForward):
        act = lambda e: ("clamped_sigmoid", e.limit, GATE_SLOPE)
        return make_part("feed_forward", "routed_experts", width=width, intermediate=f.expert.ff,
                         experts=f.router.experts, top=f.router.top, score="softmax_chosen", router_bias=True,
                         activation=act(f.expert), weigh="output", shared=f.shared.ff if f.shared else 0,
                         shared_activation=act(f.shared) if f.shared else None)
    raise TypeError(f"no part for feed-forward {f!r}")


def build_duduvik(cfg: DuduvikConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps
    norm = lambda name: make_part("norm", "rmsnorm", width=w, eps=eps, name=name, offset=1.0)
    layers = []
    for i, layer in enumerate(cfg.layers):
        ffn = _feed_forward(layer.mlp, w)
        norms = (norm("norm1"), norm("norm1b"), norm("norm2") if ffn else None, norm("norm2b") if ffn else None)
        layers.append((f"l{i}", make_part("block", "sandwich", norms=norms, mixer=_mixer(layer.mixer, w, eps),
                                          feed_forward=ffn)))
    # a layer without a feed-forward may still carry the two norms of one in its checkpoint
    ignorable = tuple(rf"l{i}\.norm2b?" for i, layer in enumerate(cfg.layers) if layer.mlp is None)
    embedding = TokenEmbedding(cfg.vocab, w, name="embed", scale=cfg.embedding.scale)
    return ModelSpec(width=w, vocab_size=cfg.vocab, max_positions=cfg.max_positions, embedding=("", embedding),
                     layers=layers, final_norm=("", norm("final.norm")),
                     head=("", OutputHead(w, cfg.vocab, tied_to=embedding)), ignorable=ignorable)


for _name in DuduvikConfig.architectures:
    register_architecture(_name, DuduvikConfig, build_duduvik, replace=True)
