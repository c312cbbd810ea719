"""The Gerorax decoder put together from parts.

The embedding's rows are multiplied by a number and joined by a sinusoid of the position; every layer is a sandwich block
(a norm before and behind each sublayer, the second one followed by a learned scale per column and a number that all
sublayers share).  The mixer is grouped attention whose heads are normed, whose scores lose a multiple of the distance
(a slope per head), and whose window keeps a request's first keys (``head_norm_attention``); the feed-forward a dense
one gated by gelu, or routed experts with clamped gates, chosen inside the best groups of them and weighed by the
softmax over all, beside an expert that every token uses.  A run of layers may be gone through several times with the
same weights, each pass with a cache of its own, begun by a learned vector and, from the second pass on, the embedding's
rows joining the stream (``loop``).  The output head is the embedding table, without its factor.  Tensor names are the
checkpoint's own: ``embed``, ``loop.step``, ``l<i>.norm1`` / ``norm1b`` / ``ls1`` / ``norm2`` / ``norm2b`` / ``ls2``,
``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``.
"""
from __future__ import annotations

from ..config.gerorax import GeluFeedForward, GeroraxConfig, GroupedExperts
from ..config.registry import register_architecture
from ..parts.base import make_part
from ..parts.embedding import OutputHead, TokenEmbedding
from .spec import LayerCall, ModelSpec

# fixed by the design
GATE_SLOPE = 1.702            # of the experts' gate, g sigmoid(slope g)
SINUSOID_BASE = 10000.0
BIAS_EXPONENT = 8.0           # head h's slope is 2^(-exponent (h + 1) / heads)


def _mixer(m, width: int, eps: float):
    return make_part("mixer", "head_norm_attention", width=width, num_heads=m.heads, num_kv_heads=m.kv_heads,
                     head_size=m.dim, value_size=m.vdim, scale=m.scale, norm_eps=eps,
                     position=make_part("position", "distance_bias", exponent=BIAS_EXPONENT),
                     window=m.mask.size if m.mask else None, keep_first=m.mask.keep_first if m.mask else 0)


def _feed_forward(f, width: int):
    if f is None:
        return None
    if isinstance(f, GeluFeedForward):
        return make_part("feed_forward", "swiglu", width=width, intermediate=f.ff, names=("gate", "up", "down"),
                         activation="gelu_tanh")
    if isinstance(f, GroupedExperts):
        act = lambda e: ("clamped_sigmoid", e.limit, GATE_SLOPE)
        g = f.router.groups
        return make_part("feed_forward", "routed_experts", width=width, intermediate=f.expert.ff,
                         experts=f.router.experts, top=f.router.top, score="softmax", activation=act(f.expert),
                         weigh="output", groups=(g.count, g.keep) if g else None,
                         shared=f.shared.ff if f.shared else 0, shared_activation=act(f.shared) if f.shared else None)
    raise TypeError(f"no part for feed-forward {f!r}")


def build_gerorax(cfg: GeroraxConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps
    before = lambda name: make_part("norm", "rmsnorm", width=w, eps=eps, name=name)
    behind = lambda name, gain: make_part("norm", "rmsnorm", width=w, eps=eps, name=name, gain=gain,
                                          factor=cfg.residual_mult)
    layers = []
    for i, layer in enumerate(cfg.layers):
        ffn = _feed_forward(layer.mlp, w)
        norms = (before("norm1"), behind("norm1b", "ls1"), before("norm2") if ffn else None,
                 behind("norm2b", "ls2") if ffn else None)
        layers.append((f"l{i}", make_part("block", "sandwich", norms=norms, mixer=_mixer(layer.mixer, w, eps),
                                          feed_forward=ffn)))
    # a layer without a feed-forward may still carry the tensors around one in its checkpoint
    ignorable = tuple(rf"l{i}\.(norm2b?|ls2)" for i, layer in enumerate(cfg.layers) if layer.mlp is None)
    n = len(layers)
    order = [LayerCall(i) for i in range(n)]
    if cfg.loop is not None:
        layers.append(("loop", make_part("block", "loop_step", width=w, times=cfg.loop.times)))
        lo, hi = cfg.loop.start, cfg.loop.stop
        order = [LayerCall(i) for i in range(lo)]
        for _ in range(cfg.loop.times):
            order += [LayerCall(n)] + [LayerCall(i) for i in range(lo, hi)]
        order += [LayerCall(i) for i in range(hi, n)]
    embedding = TokenEmbedding(cfg.vocab, w, name="embed", scale=cfg.embedding.scale, sinusoid_base=SINUSOID_BASE)
    return ModelSpec(width=w, vocab_size=cfg.vocab, max_positions=cfg.max_positions, embedding=("", embedding),
                     layers=layers, final_norm=("", before("final.norm")),
                     head=("", OutputHead(w, cfg.vocab, tied_to=embedding)), run_order=order, ignorable=ignorable)


for _name in GeroraxConfig.architectures:
    register_architecture(_name, GeroraxConfig, build_gerorax, replace=True)
