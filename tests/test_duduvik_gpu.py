"""Duduvik on the GPU against the plain implementation: every mechanism alone, then the whole model through the
runner's step function (portions, batches, pages and slots used again) and through the engine's own entry point."""
import json
import os
import types

import numpy as np
import pytest
import torch

import plain_duduvik as pd
from duduvik_util import (DUD_A, DUD_B, DUD_C, DUD_D, as_numpy, gla, latent, numpy_weights, random_config, retention)
from somesun_util import make_runner, plain_config, row_errors, run_schedule, tokens, write_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
# float32: the engine's sums run in another order than the plain model's float64 ones; bfloat16: activations are
# rounded to 8 bits about ten times a layer
TOL = {"float32": 3e-5, "bfloat16": 4e-2}
PART_TOL = {torch.float32: 2e-5, torch.bfloat16: 2.5e-2}
CONFIGS = {"A": DUD_A, "B": DUD_B, "C": DUD_C, "D": DUD_D}


def _lively(t):
    """Decays that are and are not near one, norms away from one, routers that decide clearly, gates that reach their
    bounds."""
    g = torch.Generator().manual_seed(5)
    for k in t:
        if k.endswith((".a1", ".a2")):
            t[k] = t[k] * 2
        elif k.endswith((".gate", ".up")):
            t[k] = t[k] * 8
        elif k.endswith(".router"):
            t[k] = t[k] + torch.randn(t[k].shape, generator=g)
        elif k.endswith("router.b"):
            t[k] = t[k] * 3


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("duduvik")
    return {n: write_model(str(root / n), c, 51 + i, _lively) for i, (n, c) in enumerate(CONFIGS.items())}


def oracle(path, toks):
    return torch.from_numpy(pd.forward(list(toks), numpy_weights(path), plain_config(path))[0]).float()


def sensitivity(path, toks, dtype, want):
    """Row errors of the plain model whose norms put out rounded values (to bfloat16, or by a few units in the last
    place of float32) against itself: what rounding alone does to these weights and tokens.  It differs a hundredfold
    between models of random weights: a norm behind a sublayer that puts out little, or a router's close call, makes
    much of a rounding."""
    rng, exact = np.random.default_rng(0), pd.norm_one_plus
    if dtype == "float32":
        rough = lambda x, wt, eps: exact(x, wt, eps) * (1.0 + 3e-7 * rng.standard_normal(x.shape))
    else:
        rough = lambda x, wt, eps: torch.from_numpy(exact(x, wt, eps)).to(torch.bfloat16).double().numpy()
    pd.norm_one_plus = rough
    try:
        return row_errors(oracle(path, toks), want)
    finally:
        pd.norm_one_plus = exact


def assert_logits(got, want, dtype, path, toks, what=""):
    """float32: every row within the tolerance, or within a few times what rounding alone does.  bfloat16: rounding now
    and then sends a token of random weights to another expert, whose row then differs by more: half of the rows within
    half of the tolerance and nine in ten within it (or a few times what rounding does), which no fault of a cache, a
    state or a mask passes."""
    e = row_errors(got, want)
    if float(e.max()) < TOL[dtype]:
        return
    sens = sensitivity(path, toks[: len(want)], dtype, want)
    if dtype == "float32":
        assert float(e.max()) < 5 * float(sens.max()), (what, float(e.max()), int(e.argmax()), float(sens.max()))
    else:
        for q, floor in ((0.5, TOL[dtype] / 2), (0.9, TOL[dtype])):
            at, ref = float(e.quantile(q)), float(sens.quantile(q))
            assert at < max(floor, 3 * ref), (what, q, at, ref)


def _ctx(starts, counts, slots):
    """What a part reads of a step, for entries of ``counts`` tokens at ``starts``, built by hand."""
    t = int(sum(counts))
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
    seq = [e for e, c in enumerate(counts) for _ in range(c)]
    pos = [s + j for s, c in zip(starts, counts) for j in range(c)]
    q_start = np.concatenate([[0], np.cumsum(counts)]).tolist()
    return types.SimpleNamespace(n_tokens=t, n_entries=len(counts), positions=i32(pos), token_seq=i32(seq),
                                 q_start=i32(q_start), state_slots=i32(slots), h_starts=np.asarray(starts, dtype=np.int32),
                                 h_counts=np.asarray(counts, dtype=np.int32), plans={}, scratch={}, decode_bucket=None)


def _load(part, weights, dtype):
    part.load(lambda name: weights[name].to(torch.bfloat16), torch.device(DEV), dtype)


def _drawn(part, tag, seed, boost=()):
    """Random tensors for a part as bfloat16 values held in float32; ``boost`` names tensors to make larger."""
    from atoma_infer_amd.weights.random_init import random_tensor
    w = {n: random_tensor(tag + n, ws, seed, torch.bfloat16, 0.1).float() for n, ws in part.weight_specs().items()}
    for n, f in boost:
        if n in w:
            w[n] = (w[n] * f).to(torch.bfloat16).float()
    return w


def _flat(y):
    if hasattr(y, "terms"):
        return sum(_flat(t) * s for t, s in y.terms)
    return (y.sum(0) if y.dim() == 3 else y).float().cpu()


def _rel(a, b):
    b = torch.as_tensor(b)
    return float((a.double() - b.double()).norm() / b.double().norm().clamp_min(1e-30))


def _inputs(lens, width, seed):
    g = torch.Generator().manual_seed(seed)
    return [torch.randn(c, width, generator=g).to(torch.bfloat16).float() for c in lens]


# ---- small kernels and the feed-forwards --------------------------------------------------------------------------

def test_the_embedding_is_multiplied_on_its_way_in_and_not_in_the_head():
    from atoma_infer_amd.kernels import ops
    from atoma_infer_amd.parts import OutputHead, TokenEmbedding
    from atoma_infer_amd.parts.base import make_part
    for dtype in (torch.float32, torch.bfloat16):
        emb = TokenEmbedding(50, 36, name="embed", scale=2.5)
        w = _drawn(emb, "e.", 2)
        _load(emb, w, dtype)
        head = OutputHead(36, 50, tied_to=emb)
        head.load(None, torch.device(DEV), dtype)
        toks = torch.tensor([3, 49, 0, 3, 60], dtype=torch.int32, device=DEV)
        want = w["embed"][[3, 49, 0, 3]] * 2.5
        x = emb.forward(toks).cpu()
        assert torch.equal(x[:4], want) and bool(x[4].isnan().all())
        norm = make_part("norm", "rmsnorm", width=36, eps=1e-5, name="n", offset=1.0)
        nw = _drawn(norm, "n.", 3)
        _load(norm, nw, dtype)
        x, begun = emb.forward(toks[:4], norm)
        assert torch.equal(x.cpu(), want)
        if dtype is torch.bfloat16:
            assert _rel(begun.tensor().float().cpu(), pd.norm_one_plus(want.double().numpy(), nw["n"].double().numpy(), 1e-5)) < 6e-3
        else:
            assert begun is None
        h = _inputs([3], 36, 1)[0]
        assert _rel(head.forward(h.to(DEV, dtype)).cpu(), h.double() @ w["embed"].double().T) < 1e-5
        assert torch.equal(ops.embed(toks[:1], emb.weight).cpu(), w["embed"][[3]])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width, ff", [(64, 48), (40, 20), (128, 96), (256, 512)])
def test_dense_feed_forwards_gated_by_relu_and_by_clamped_values(width, ff, dtype):
    from atoma_infer_amd.parts.base import make_part
    for act in ("relu", ("clamped_sigmoid", 0.6, 1.702)):
        part = make_part("feed_forward", "swiglu", width=width, intermediate=ff, names=("gate", "up", "down"), activation=act)
        w = _drawn(part, "f.", 3, boost=(("gate", 6), ("up", 6)))
        _load(part, w, dtype)
        for t in (1, 7, 70):
            h = _inputs([t], width, ff + t)[0]
            n = as_numpy(w, "m.")
            hn = h.double().numpy()
            want = pd.dense(hn, n, "m.") if act == "relu" else pd.expert(hn, n, "m.", 0.6)
            assert _rel(_flat(part.forward(h.to(DEV, dtype), None)), want) < PART_TOL[dtype], (act, t)
            if act != "relu":      # the bound bites, on both sides of the up value and above the gate
                gate, up = hn @ n["m.gate"].T, hn @ n["m.up"].T
                assert (gate > 0.6).any() and (up > 0.6).any() and (up < -0.6).any()


@pytest.mark.parametrize("experts, top", [(5, 2), (12, 4), (70, 6), (200, 130), (1, 1), (8, 8)])
def test_the_router_weighs_by_the_softmax_over_the_chosen_logits_alone(experts, top):
    from atoma_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(experts)
    t = 37
    z, b = torch.randn(t, experts, generator=g) * 3, torch.randn(experts, generator=g) * 4
    ids, wts = ops.route_topk(z.to(DEV), top, "softmax_chosen", bias=b.to(DEV))
    full = (z + b).double()
    order = torch.argsort(-full, dim=1, stable=True)[:, :top]
    assert torch.equal(ids.cpu().long(), order)
    want = torch.softmax(full.gather(1, order), dim=1)
    assert (wts.cpu().double() - want).abs().max() < 2e-6
    # without its bias the router chooses otherwise
    if 1 < top < experts:
        assert not torch.equal(ops.route_topk(z.to(DEV), top, "softmax_chosen")[0].cpu().long(), order)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width, ff, experts, top, limit, shared", [
    (64, 32, 5, 2, 1.5, (48, 0.7)), (128, 64, 12, 4, 0.5, (64, 0.5)), (40, 10, 3, 3, 0.8, None), (96, 96, 32, 6, 1.0, (20, 2.0)),
    (64, 16, 1, 1, 0.3, (16, 9.0))])
def test_clamped_experts_weighed_on_their_outputs_beside_a_shared_one(width, ff, experts, top, limit, shared, dtype):
    from atoma_infer_amd.parts.base import make_part
    act = lambda l: ("clamped_sigmoid", l, 1.702)
    part = make_part("feed_forward", "routed_experts", width=width, intermediate=ff, experts=experts, top=top,
                     score="softmax_chosen", router_bias=True, activation=act(limit), weigh="output",
                     shared=shared[0] if shared else 0, shared_activation=act(shared[1]) if shared else None)
    w = _drawn(part, "x.", 7, boost=[("router", 3), ("router.b", 4)] + [
        (f"{e}.{n}", 6) for e in ["shared"] + [f"e{i}" for i in range(experts)] for n in ("gate", "up")])
    _load(part, w, dtype)
    assert part.mfma == (dtype is torch.bfloat16 and width % 32 == 0 and ff % 32 == 0)
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    for t in (1, 9, 150):
        h = _inputs([t], width, ff + t)[0]
        got = _flat(part.forward(h.to(DEV, dtype), None))
        n = as_numpy(w, "m.")
        hn = h.double().numpy()
        want = torch.from_numpy(pd.moe(hn, n, "m.", m))
        z = np.sort(hn @ n["m.router"].T + n["m.router.b"], axis=1)[:, ::-1]
        clear = torch.from_numpy(z[:, top - 1] - z[:, top] > 1e-3) if top < experts else torch.ones(t, dtype=torch.bool)
        assert int(clear.sum()) > 0.8 * t
        assert _rel(got[clear], want[clear]) < PART_TOL[dtype], t


# ---- linear attention alone ---------------------------------------------------------------------------------------

def _la_case(kind, heads, dim, vdim, lens, seed, rank=5, tau=4.0, shift=1.0, rot=None, decay=None):
    """Projections of a step's entries with tensors of the mechanism, and what the plain recurrence makes of them:
    (proj, sizes, tensors, plain fn(entry, start, state) -> (y, state))."""
    from atoma_infer_amd.kernels import ops
    from atoma_infer_amd.parts.position import rotation_frequencies
    g = torch.Generator().manual_seed(seed)
    nq, nv, t = heads * dim, heads * vdim, sum(lens)
    ld = -(-(2 * nq + 2 * nv + rank) // 16) * 16
    proj = torch.randn(t, ld, generator=g)
    norm = None if kind == "retention" else 1.0 + 0.3 * torch.randn(vdim, generator=g)
    offs = (0, nq, 2 * nq, 2 * nq + nv)
    if kind == "gla":
        w2, b2 = torch.randn(nq, rank, generator=g), torch.randn(nq, generator=g) * 2 + shift
        ten = dict(w2=w2, b2=b2, norm=norm)
        sizes = ops.LinearAttentionSizes(heads, dim, vdim, offs, 1e-5, dim ** -0.5, 1.0, 0, (2 * nq + 2 * nv, rank), 1.0 / tau)
    else:
        decay = torch.tensor(decay if decay is not None else [1.0 - 0.5 ** (1 + 2 * h) for h in range(heads)])
        rot = dim // 2 * 2 if rot is None else rot
        ten = dict(decay=decay, freq=rotation_frequencies(100.0, rot)[0] if rot else None)
        sizes = ops.LinearAttentionSizes(heads, dim, vdim, offs, 1e-5, 1.0, dim ** -0.5, rot)
    starts = np.concatenate([[0], np.cumsum(lens)])

    def plain(e, p0, state):
        x = proj[starts[e]: starts[e + 1]].double().numpy()
        n = len(x)
        q, k = x[:, :nq].reshape(n, heads, dim), x[:, nq: 2 * nq].reshape(n, heads, dim)
        v, gt = x[:, 2 * nq: 2 * nq + nv].reshape(n, heads, vdim), x[:, 2 * nq + nv: 2 * nq + 2 * nv]
        if kind == "gla":
            z = x[:, 2 * nq + 2 * nv: 2 * nq + 2 * nv + rank] @ w2.double().numpy().T + b2.double().numpy()
            al = np.exp(-np.logaddexp(0.0, -z) / tau).reshape(n, heads, dim)
        else:
            al = np.broadcast_to(decay.double().numpy()[None, :, None], (n, heads, dim))
            r = {"base": 100.0, "dims": rot}
            q, k = pd.rotate_half(q, np.arange(p0, p0 + n), r), pd.rotate_half(k, np.arange(p0, p0 + n), r)
        o, s = pd.decayed_sum(q * sizes.q_scale, k * sizes.k_scale, v, al, state)
        o = pd.unit_rms(o, 1e-5) * (1.0 if norm is None else norm.double().numpy())
        return o.reshape(n, nv) * pd.silu(gt), s
    dev = {n: (None if x is None else x.to(DEV, torch.float32).contiguous()) for n, x in ten.items()}
    return proj, sizes, ops.LinearAttentionTensors(**dev), plain


LA_SIZES = [(3, 16, 24), (2, 64, 64), (1, 128, 128), (4, 48, 33), (1, 7, 3), (2, 96, 100), (1, 200, 17), (1, 256, 256),
            (2, 32, 512), (1, 1, 1)]


@pytest.mark.parametrize("kind", ["gla", "retention"])
@pytest.mark.parametrize("heads, dim, vdim", LA_SIZES)
def test_linear_attention_token_by_token_and_in_chunks_against_the_plain_recurrence(heads, dim, vdim, kind):
    """Entries of one token to hundreds side by side, from states that are not zero; entries on both sides of the length
    from which chunks are used, and lengths on both sides of a chunk's edge.  The chunked kernels split their float32
    operands in two, so their states agree to 16 bits, far closer than bfloat16 rounding."""
    from atoma_infer_amd.kernels import ops
    lens, starts, slots = [1, 70, 3, 64, 39, 129, 200, 40], [0, 5, 100, 7, 0, 33, 0, 1000], [4, 0, 7, 1, 2, 6, 3, 8]
    proj, sizes, ten, plain = _la_case(kind, heads, dim, vdim, lens, heads * 1000 + dim)
    g = torch.Generator().manual_seed(1)
    state = torch.randn(10, heads, vdim, dim, generator=g)
    want = [plain(e, starts[e], state[slots[e]].permute(0, 2, 1).double().numpy()) for e in range(len(lens))]
    ctx = _ctx(starts, lens, slots)
    for chunked, dtype in ((0, torch.float32), (0, torch.bfloat16), (40, torch.bfloat16)):
        st = state.reshape(10, -1).to(DEV).contiguous()
        arr, meta = ops.linear_attention_plan(lens, chunked)
        plan = (torch.from_numpy(arr).to(DEV), meta)
        y = ops.linear_attention(proj.to(DEV), sizes, ten, ctx.positions, ctx.q_start, ctx.state_slots, st, dtype, plan,
                                 chunked).float().cpu()
        st = st.cpu().reshape(state.shape)
        o = 0
        for e, n in enumerate(lens):
            err, serr = _rel(y[o: o + n], want[e][0]), _rel(st[slots[e]].permute(0, 2, 1), want[e][1])
            # (the float32 angle of a position p is off by up to p 2^-24; one number alone may cancel)
            angle = 0.0 if kind == "gla" else 3e-8 * (starts[e] + n)
            exact = not chunked or n < 40
            assert err < (1e-5 + angle if dtype is torch.float32 else 4e-3), (chunked, e, err)
            assert serr < (3e-6 if exact else 3e-5) * (10 if dim == 1 else 1) + angle, (chunked, e, serr)
            o += n
        assert torch.equal(st[[5, 9]], state[[5, 9]])          # slots of no entry


@pytest.mark.parametrize("shift, tau", [(-60.0, 1.0), (0.0, 1.0), (40.0, 16.0)])
def test_decays_of_any_strength_neither_overflow_nor_lose_the_state(shift, tau):
    """Decays of e^-60 a token, of about a half, and of one to eight digits, in chunks: products of decays only, so
    nothing is divided by what has underflowed."""
    from atoma_infer_amd.kernels import ops
    lens = [300]
    proj, sizes, ten, plain = _la_case("gla", 2, 64, 48, lens, 5, tau=tau, shift=shift)
    want, s = plain(0, 0, None)
    ctx = _ctx([0], lens, [1])
    for chunked in (0, 40):
        st = torch.zeros(2, 2 * 48 * 64, device=DEV)
        arr, meta = ops.linear_attention_plan(lens, chunked)
        y = ops.linear_attention(proj.to(DEV), sizes, ten, ctx.positions, ctx.q_start, ctx.state_slots, st, torch.bfloat16,
                                 (torch.from_numpy(arr).to(DEV), meta), chunked)
        assert bool(torch.isfinite(y.float()).all())
        assert _rel(y.float().cpu(), want) < 4e-3
        assert _rel(st[1].cpu().reshape(2, 48, 64).permute(0, 2, 1), s) < 5e-5


def test_fixed_decays_of_one_of_nothing_and_between_in_chunks():
    from atoma_infer_amd.kernels import ops
    lens, decay = [200, 65], [1.0, 0.0, 0.3, 0.999]
    for rot in (0, 8, 32):
        proj, sizes, ten, plain = _la_case("retention", 4, 32, 40, lens, 6, rot=rot, decay=decay)
        want = [plain(e, s, None) for e, s in ((0, 0), (1, 5000))]
        ctx = _ctx([0, 5000], lens, [1, 0])
        st = torch.zeros(2, 4 * 40 * 32, device=DEV)
        arr, meta = ops.linear_attention_plan(lens, 40)
        y = ops.linear_attention(proj.to(DEV), sizes, ten, ctx.positions, ctx.q_start, ctx.state_slots, st, torch.bfloat16,
                                 (torch.from_numpy(arr).to(DEV), meta), 40).float().cpu()
        assert _rel(y[:200], want[0][0]) < 4e-3
        assert _rel(y[200:], want[1][0]) < 5e-3          # (angles of thousands of radians in float32)
        assert _rel(st[1].cpu().reshape(4, 40, 32).permute(0, 2, 1), want[0][1]) < 5e-5


RECURRENT_CUTS = ([(0, 1), (1, 2)], [(0, 2)], [(1, 1), (0, 1)], [(0, 30), (1, 6)], [(0, 3)], [(0, 64), (1, 17)], [(0, 250)],
                  [(0, 16), (1, 100)], [(1, 3), (0, 100)])


def _recurrent_case(part, hs, dtype, state_width):
    """Two requests side by side in portions of one token, two, a few and hundreds, each carried by its state slot."""
    state = torch.full((4, state_width), float("nan"), dtype=torch.float32, device=DEV)
    state[1].fill_(7.0)                       # another request's slot must stay as it is
    state[0].zero_()
    state[3].zero_()
    cache = types.SimpleNamespace(state=state)
    got, at = [[], []], [0, 0]
    for cuts in RECURRENT_CUTS:
        ctx = _ctx([at[r] for r, _ in cuts], [c for _, c in cuts], [3 if r == 0 else 0 for r, _ in cuts])
        x = torch.cat([hs[r][at[r]: at[r] + c] for r, c in cuts]).to(DEV, dtype)
        y = _flat(part.forward(x, ctx, cache))
        o = 0
        for r, c in cuts:
            got[r].append(y[o: o + c])
            o += c
            at[r] += c
    assert at == [len(h) for h in hs] and bool((state[1] == 7.0).all()) and bool(state[2].isnan().all())
    return [torch.cat(g) for g in got]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [gla(3, 24, 40, 8.0, 6), gla(4, 64, 128, 16.0, 16), gla(1, 7, 3, 1.0, 3), gla(2, 48, 64, 20.0, 33),
                               retention(3, 16, 24), retention(2, 64, 64, 3000.0, 32, [0.97, 0.999]),
                               retention(4, 10, 5, rot_dims=0, decay=[1.0, 0.0, 0.3, 0.9]), retention(2, 128, 256, 5e4)])
def test_both_linear_attentions_alone_whole_and_in_portions(m, dtype):
    from atoma_infer_amd.parts import DecayedLinearAttention
    width, gated = 64, "tau" in m
    if gated:
        part = DecayedLinearAttention(width, m["heads"], m["dim"], m["vdim"], 1e-5, tau=m["tau"], rank=m["rank"],
                                      q_scale=m["dim"] ** -0.5, norm_weight=True)
    else:
        rot = m.get("rot", {"base": 1.5, "dims": 0})
        part = DecayedLinearAttention(width, m["heads"], m["dim"], m["vdim"], 1e-5, decay=m["decay"], rotary_base=rot["base"],
                                      rotary_dim=rot["dims"], k_scale=m["dim"] ** -0.5)
    w = _drawn(part, "l.", 5, boost=(("q", 4), ("k", 4), ("v", 4), ("g", 8), ("a1", 3)))
    _load(part, w, dtype)
    hs = _inputs((467, 129), width, m["dim"])
    n = as_numpy(w, "m.")
    want = [pd.gla(h.double().numpy(), n, "m.", m, 1e-5)[0] if gated else
            pd.retention(h.double().numpy(), np.arange(len(h)), n, "m.", m, 1e-5)[0] for h in hs]
    got = _recurrent_case(part, hs, dtype, m["heads"] * m["vdim"] * m["dim"])
    for r in range(2):
        # (rotation: float32 angles of hundreds of radians)
        assert _rel(got[r], want[r]) < (4e-5 if dtype is torch.float32 else PART_TOL[dtype]), r


@pytest.mark.parametrize("kind", ["gla", "retention"])
def test_a_far_token_stays_in_a_state_that_hardly_decays(kind):
    """One early token with a large value; hundreds of tokens later the read-out still holds it.  A state that is lost,
    cleared or carried by the wrong slot changes the late outputs entirely."""
    from atoma_infer_amd.parts import DecayedLinearAttention
    width = 64
    if kind == "gla":
        m = gla(2, 32, 16, 16.0, 4)
        part = DecayedLinearAttention(width, 2, 32, 16, 1e-5, tau=16.0, rank=4, q_scale=32 ** -0.5, norm_weight=True)
    else:
        m = retention(2, 32, 16, 1e4, 16, [0.9995, 0.5])
        part = DecayedLinearAttention(width, 2, 32, 16, 1e-5, decay=m["decay"], rotary_base=1e4, rotary_dim=16, k_scale=32 ** -0.5)
    w = _drawn(part, "m.", 9, boost=(("q", 4), ("k", 4), ("v", 4)))
    if kind == "gla":
        w["a2.b"] = torch.full_like(w["a2.b"], 6.0)        # alpha = sigmoid(6)^(1/16), 0.99985, where W_a1 x is small
        w["a1"] = w["a1"] * 0.125
    _load(part, w, torch.float32)
    n = as_numpy(w, "m.")
    plain = lambda h: pd.gla(h.double().numpy(), n, "m.", m, 1e-5)[0] if kind == "gla" else \
        pd.retention(h.double().numpy(), np.arange(len(h)), n, "m.", m, 1e-5)[0]
    h = _inputs([400], width, 1)[0] * 0.3
    h[5] = h[5] * 100
    want = plain(h)
    h2 = h.clone()
    h2[5] = h[5] / 100
    assert np.linalg.norm(plain(h2)[-20:] - want[-20:]) > 0.2 * np.linalg.norm(want[-20:])
    cache = types.SimpleNamespace(state=torch.zeros((2, 2 * 16 * 32), dtype=torch.float32, device=DEV))
    got, at = [], 0
    for c in [300, 63, 2] + [1] * 35:
        got.append(_flat(part.forward(h[at: at + c].to(DEV), _ctx([at], [c], [1]), cache)))
        at += c
    got = torch.cat(got)
    assert _rel(got, want) < 4e-5 and _rel(got[-20:], want[-20:]) < 4e-5


# ---- latent attention with a window alone ---------------------------------------------------------------------------

def _paged_case(part, plain, dtype, cuts_of_steps, page, seed, width=64, hs=None):
    """A mixer over a paged cache on hand-made steps over pages that are dealt out of order: per request the outputs
    of all its portions, and the plain function's on the whole request."""
    lens = [sum(c for r2, c in sum(cuts_of_steps, []) if r2 == r) for r in range(2)]
    g = torch.Generator().manual_seed(seed)
    hs = hs if hs is not None else [torch.randn(c, width, generator=g).to(torch.bfloat16).float() for c in lens]
    want = [plain(h.double().numpy()) for h in hs if len(h)]
    cs = part.cache_spec()
    n_pages = sum(-(-c // page) for c in lens) + 3
    order = torch.randperm(n_pages, generator=g).tolist()
    tables = [[order.pop() for _ in range(-(-c // page))] for c in lens]
    max_blocks = max(len(tb) for tb in tables)
    k = torch.zeros((n_pages, cs.kv_heads, page * cs.head_size), dtype=dtype, device=DEV)
    v = torch.zeros_like(k)
    got, at = [[], []], [0, 0]
    for cuts in cuts_of_steps:
        ctx = _ctx([at[r] for r, _ in cuts], [c for _, c in cuts], [0] * len(cuts))
        bt = torch.tensor([tables[r] + [0] * (max_blocks - len(tables[r])) for r, _ in cuts], dtype=torch.int32, device=DEV)
        slots = [tables[r][(at[r] + j) // page] * page + (at[r] + j) % page for r, c in cuts for j in range(c)]
        x = torch.cat([hs[r][at[r]: at[r] + c] for r, c in cuts]).to(DEV, dtype)
        cache = types.SimpleNamespace(k=k, v=v, page_size=page, writable=True, block_tables=bt,
                                      slot_mapping=torch.tensor(slots, dtype=torch.int32, device=DEV))
        y = _flat(part.forward(x, ctx, cache))
        o = 0
        for r, c in cuts:
            got[r].append(y[o: o + c])
            o += c
            at[r] += c
    return [torch.cat(x) for x in got if x], want


def _latent_part(m):
    from atoma_infer_amd.parts import RotaryLatentAttention
    rot = m.get("rot", {"base": 10000.0, "dims": 0})
    return RotaryLatentAttention(64, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"], m["scale"], 1e-5,
                                 rot["base"], rot["dims"], interleaved=False, gated=False,
                                 window=m["mask"]["size"] if "mask" in m else None)


CUTS = [[(0, 20), (1, 3)], [(0, 1), (1, 1)], [(0, 2)], [(1, 40), (0, 1)], [(0, 50)], [(0, 1)], [(1, 1)], [(0, 1), (1, 2)]]
BOOST = (("uq", 3), ("uk", 3), ("dq", 10), ("dkv", 10), ("o", 5))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m, page", [(latent(window=13), 16), (latent(32, 2, 64, 48, 32, 16, 0.15, 500.0, 16), 32),
                                     (latent(10, 3, 20, 12, 6, 6, 0.4, 30.0, None), 16), (latent(8, 1, 16, 8, 2, 8, 1.0, 2.0, 1), 48),
                                     (latent(24, 5, 100, 72, 12, 40, 0.1, 1e4, 33), 16), (latent(16, 2, 48, 24, 0, 16, 0.3, window=5), 16)])
def test_latent_attention_with_half_split_pairs_a_window_and_no_gate_alone(m, page, dtype):
    part = _latent_part(m)
    assert "g" not in part.weight_specs() and part.cache_spec().window == (m["mask"]["size"] if "mask" in m else None)
    w = _drawn(part, "a.", 11, boost=BOOST)
    _load(part, w, dtype)
    plain = lambda h: pd.latent_attention(h, np.arange(len(h)), as_numpy(w, "m."), "m.", m, 1e-5)
    got, want = _paged_case(part, plain, dtype, CUTS, page, m["dim"])
    for g, wt in zip(got, want):
        assert _rel(g, wt) < PART_TOL[dtype]


@pytest.mark.parametrize("far, window", [(3, 64), (16, 40), (63, 40), (100, 17), (5, 1), (7, 2), (0, 255), (40, None)])
def test_one_key_that_stands_out_is_seen_to_the_windows_edge_and_not_beyond(far, window):
    """The latent's first column carries a mark through W_dkv, and every head's key and query read it: the marked
    position's key stands out for every later query that sees it, and only for those, whether they come in a prompt, in
    a portion that begins anywhere, or alone."""
    m = latent(16, 2, 32, 16, 8, 16, 0.5, 100.0, window)
    part = _latent_part(m)
    w = _drawn(part, "f.", 23, boost=(("o", 5), ("uv", 2)))
    w["dkv"][0] = 0.0
    w["dkv"][0, 0] = 8.0                      # latent column 0 = the mark
    w["dq"][0] = 0.0
    w["dq"][0, 1] = 8.0                       # query latent column 0 = the constant
    for a in range(2):
        w["uk"][a * 16 + 15] = 0.0
        w["uk"][a * 16 + 15, 0] = 4.0
        w["uq"][a * 24 + 15] = 0.0
        w["uq"][a * 24 + 15, 0] = 4.0
    _load(part, w, torch.float32)
    total = 270
    hs = _inputs((total, 0), 64, 3)
    for h in hs:
        h[:, 0], h[:, 1] = 0.0, 1.0
    hs[0][far, 0] = 6.0
    plain = lambda h: pd.latent_attention(h, np.arange(len(h)), as_numpy(w, "m."), "m.", m, 1e-5)
    edge = far + (window or 10 ** 6)
    near = max(1, min(edge, total - 1) - 3)
    for cuts in ([[(0, total)]], [[(0, 7)], [(0, 121)], [(0, 2)], [(0, 70)], [(0, 70)]],
                 [[(0, near)]] + [[(0, 1)]] * min(8, total - near) + ([[(0, total - near - 8)]] if total - near > 8 else [])):
        got, want = _paged_case(part, plain, torch.float32, cuts, 16, 1, hs=hs)
        assert (got[0].double() - torch.from_numpy(want[0])).abs().max() < 1e-4 * np.abs(want[0]).max()
    hs0 = [h.clone() for h in hs]
    hs0[0][far, 0] = 0.0
    a, b = plain(hs[0].double().numpy()), plain(hs0[0].double().numpy())
    moved = np.abs(a - b).max(axis=1) > 1e-3 * np.abs(a).max()
    end = min(total, edge)
    assert moved[far + 1: end].all() and not moved[end:].any() and not moved[:far].any()


# ---- the whole model ------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_whole_prompts_portions_and_single_tokens_agree_with_the_plain_model(dirs, name, dtype):
    d = dirs[name]
    vocab = plain_config(d)["vocab"]
    toks = tokens(150, vocab, 7)
    want = oracle(d, toks)
    runner = make_runner(d, dtype, 256, 16, 2)
    schedules = {"whole": [[(0, 150)]],
                 "tokens": [[(0, 1)]] * 150,
                 "portions": [[(0, c)] for c in (5, 2, 1, 1, 9, 2, 30, 1, 33, 2, 16, 16, 3, 29)],
                 "portions of two": [[(0, 2)]] * 75,
                 "prompt then tokens": [[(0, 97)]] + [[(0, 1)]] * 53}
    for what, sched in schedules.items():
        got = run_schedule(runner, {0: toks}, sched)[0]
        assert_logits(got, want, dtype, d, toks, what)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_batches_of_unequal_requests_equal_each_alone_over_pages_and_slots_used_again(dirs, name, dtype):
    """Five requests through a pool of three slots and just enough pages: portions of some beside single tokens of
    others; a request that ends gives its pages and its slot to the next."""
    d = dirs[name]
    vocab = plain_config(d)["vocab"]
    reqs = {r: tokens(n, vocab, 20 + r) for r, n in enumerate((70, 33, 90, 2, 41))}
    want = {r: oracle(d, t) for r, t in reqs.items()}
    runner = make_runner(d, dtype, 256, 16, 3)
    sched = [[(0, 30), (1, 5)], [(0, 1), (1, 28), (2, 17)], [(0, 39), (2, 1)], [(2, 40), (3, 2)], [(2, 1), (4, 1)],
             [(2, 31), (4, 40)]]
    got = run_schedule(runner, reqs, sched)
    for r in reqs:
        assert_logits(got[r], want[r], dtype, d, reqs[r], r)


@pytest.mark.parametrize("seed", [2, 15, 28, 41, 59, 82])
def test_configurations_drawn_at_random_agree_with_the_plain_model(tmp_path, seed):
    """Layers of the three kinds in any order with sizes drawn at random: a whole prompt, a prompt and single tokens,
    portions, and a mixed batch over four slots."""
    import random
    cfg = random_config(random.Random(seed))
    d = write_model(str(tmp_path / "m"), cfg, seed, _lively)
    reqs = {r: tokens(n, cfg["vocab"], 100 * seed + r) for r, n in enumerate((230, 33, 150, 2, 77))}
    want = {r: oracle(d, t) for r, t in reqs.items()}
    for dtype in ("float32", "bfloat16"):
        runner = make_runner(d, dtype, 512, 16, 4)
        runs = {"whole": run_schedule(runner, {0: reqs[0]}, [[(0, 230)]]),
                "tokens": run_schedule(runner, {0: reqs[0]}, [[(0, 190)]] + [[(0, 1)]] * 40),
                "portions": run_schedule(runner, {0: reqs[0]}, [[(0, c)] for c in (5, 2, 60, 1, 33, 2, 100, 3, 24)]),
                "mixed": run_schedule(runner, reqs, [[(0, 100), (1, 5)], [(0, 1), (1, 28), (2, 17)], [(0, 100), (2, 1), (3, 1)],
                                                     [(0, 29), (2, 40), (3, 1)], [(2, 1), (4, 1)], [(2, 91), (4, 76)]])}
        for what, got in runs.items():
            for r, rows in got.items():
                assert_logits(rows, want[r], dtype, d, reqs[r], (what, r))


def test_long_decoding_over_many_windows_and_pages(dirs):
    d = dirs["A"]
    toks = tokens(420, plain_config(d)["vocab"], 9)
    want = oracle(d, toks)
    runner = make_runner(d, "float32", 448, 16, 1)
    got = run_schedule(runner, {0: toks}, [[(0, 20)]] + [[(0, 1)]] * 400)[0]
    assert_logits(got, want, "float32", d, toks)


def test_decode_steps_and_lone_prompts_replayed_as_graphs_equal_the_direct_ones(dirs):
    """Decode steps of one shape are recorded the second time they are seen and lone prompts the third time, and replayed
    afterwards, with the program's own direct work between the replays: every replay against the plain model."""
    d = dirs["B"]
    vocab = plain_config(d)["vocab"]
    reqs = {0: tokens(60, vocab, 1), 1: tokens(45, vocab, 2), 2: tokens(30, vocab, 3)}
    want = {r: oracle(d, t) for r, t in reqs.items()}
    runner = make_runner(d, "float32", 256, 16, 3)
    assert runner.use_graphs
    sched = [[(0, 20), (1, 5)]] + [[(0, 1), (1, 1)]] * 10 + [[(2, 30)]] + [[(0, 1), (1, 1)]] * 30
    got = run_schedule(runner, reqs, sched)
    for r in (0, 1, 2):
        assert_logits(got[r], want[r][: len(got[r])], "float32", d, reqs[r], r)
    from atoma_infer_amd.engine.step import StepEntry
    runner = make_runner(d, "bfloat16", 640, 16, 2)
    for i in range(5):
        toks = tokens(300, vocab, 40 + i)
        runner.add_request(7)
        logits = runner.step([StepEntry(7, toks, 0, [299])]).float().cpu().clone()
        assert float(row_errors(logits, oracle(d, toks)[-1:]).max()) < 2 * TOL["bfloat16"], i
        runner.free_request(7)
        run_schedule(runner, {1: reqs[1]}, [[(1, 40)]] + [[(1, 1)]] * 5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine_and_its_scheduler(dirs, dtype):
    """Requests of unequal lengths through ``LlmEngine.generate``: continuous batching with prompts in portions (a token
    budget below the longest prompt) beside decoding requests, greedy tokens against the plain model."""
    from atoma_infer_amd.config.engine import CacheConfig, SchedulerConfig
    from atoma_infer_amd.engine.engine import LlmEngine
    from atoma_infer_amd.sampling.params import GenerateParameters
    d = dirs["A"]
    cfg, w = plain_config(d), numpy_weights(d)
    prompts = [tokens(n, cfg["vocab"], 60 + n) for n in (3, 41, 17, 1, 29)]
    eng = LlmEngine(d, dtype, cache=CacheConfig(block_size=16, num_gpu_blocks_override=24),
                    scheduler=SchedulerConfig(max_num_batched_tokens=24, max_num_sequences=4, max_model_len=128,
                                              enable_chunked_prefill=True))
    outs = eng.generate(prompts, GenerateParameters(do_sample=False, max_new_tokens=12, ignore_eos_token=True))
    off = 0
    for p, o in zip(prompts, outs):
        got = o.inference_outputs[0].token_ids
        assert len(got) == 12
        rows = pd.forward(list(p) + got, w, cfg)[0][len(p) - 1: -1]
        for step, tok in enumerate(got):
            gap = float(rows[step].max() - rows[step][tok])
            off += gap > (1e-4 if dtype == "float32" else 0.08) * float(np.abs(rows[step]).max())
    # (bfloat16: a router's close call may go the other way)
    assert off <= (0 if dtype == "float32" else 3), off


def test_the_trace_program_and_the_command_line_run_the_design(dirs, tmp_path):
    import subprocess
    import sys
    d = dirs["D"]
    toks = tokens(30, plain_config(d)["vocab"], 8)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:9], "want": [0, 8]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[9:], "want": [20]},
                                     {"id": "y", "tokens": toks[:4], "want": [3]}], "end": ["x", "y"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = str(tmp_path / "out")
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d, "--dtype", "float32",
                           "--out", out, "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                          capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1"]
    want = oracle(d, toks)
    a = torch.from_numpy(np.fromfile(os.path.join(out, "0.f32"), dtype="<f4").reshape(2, -1))
    b = torch.from_numpy(np.fromfile(os.path.join(out, "1.f32"), dtype="<f4").reshape(2, -1))
    assert float(row_errors(a, want[[0, 8]]).max()) < TOL["float32"]
    assert float(row_errors(b, want[[29, 3]]).max()) < TOL["float32"]


def test_the_command_line_writes_random_weights_and_generates(tmp_path):
    """``random-weights`` from a config.json of the design, then ``generate``: greedy tokens are the plain model's, and
    sampling with a seed (temperature, top-k, top-p through the framework's sampler) gives the same tokens twice."""
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    env = dict(os.environ, PYTHONPATH=root)
    cfg_file, d = tmp_path / "config.json", str(tmp_path / "m")
    cfg_file.write_text(json.dumps(DUD_A))
    run = lambda *a: subprocess.run([sys.executable, "-m", "atoma_infer_amd", *a], capture_output=True, text=True, env=env,
                                    timeout=300, cwd=root)
    proc = run("random-weights", "--config", str(cfg_file), "--out", d, "--seed", "4", "--norm-jitter", "0.1")
    assert proc.returncode == 0, proc.stderr[-2000:]
    prompt = tokens(9, DUD_A["vocab"], 2)
    common = ["generate", "--model", d, "--block-size", "16", "--num-gpu-blocks-override", "16", "--max-model-len", "64",
              "--max-num-batched-tokens", "64", "--max-num-sequences", "4", "--max-new-tokens", "6", "--ignore-eos-token",
              "--prompt-ids", ",".join(str(t) for t in prompt)]
    proc = run(*common, "--dtype", "f32", "--greedy")
    assert proc.returncode == 0, proc.stderr[-2000:]
    got = json.loads(proc.stdout.strip().splitlines()[-1])["inference_outputs"][0]["token_ids"]
    w, cfg, seq = numpy_weights(d), plain_config(d), list(prompt)
    for _ in range(6):
        seq.append(int(pd.forward(seq, w, cfg)[0][-1].argmax()))
    assert got == seq[len(prompt):]
    drawn = []
    for _ in range(2):
        proc = run(*common, "--dtype", "bf16", "--temperature", "1.5", "--top-k", "20", "--top-p", "0.9", "--random-seed", "11")
        assert proc.returncode == 0, proc.stderr[-2000:]
        drawn.append(json.loads(proc.stdout.strip().splitlines()[-1])["inference_outputs"][0]["token_ids"])
    assert drawn[0] == drawn[1] and len(drawn[0]) == 6 and all(0 <= t < DUD_A["vocab"] for t in drawn[0])
