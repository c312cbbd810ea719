"""Gerorax on the GPU against the plain implementation: every mechanism alone, then the whole model through the
runner's step function (portions, batches, pages and slots used again) and through the engine's own entry point."""
import json
import os
import types

import numpy as np
import pytest
import torch

import plain_gerorax as pg
from gerorax_util import GER_A, GER_B, GER_C, GER_D, as_numpy, attention, moe, numpy_weights, random_config
from somesun_util import make_runner, plain_config, row_errors, run_schedule, tokens, write_model
from util import force_chunked_decode

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
# float32: the engine's sums run in another order than the plain model's float64 ones; bfloat16: activations are
# rounded to 8 bits about ten times a layer
TOL = {"float32": 3e-5, "bfloat16": 4e-2}
PART_TOL = {torch.float32: 2e-5, torch.bfloat16: 2.5e-2}
CONFIGS = {"A": GER_A, "B": GER_B, "C": GER_C, "D": GER_D}


def _lively(t):
    """Scores that tell keys apart, norms away from one, routers that decide clearly, gates that reach their bounds."""
    g = torch.Generator().manual_seed(5)
    for k in t:
        if k.endswith((".q.norm", ".k.norm")):
            t[k] = t[k] * (1.5 + 0.3 * torch.randn(t[k].shape, generator=g))
        elif k.endswith((".gate", ".up")):
            t[k] = t[k] * 8
        elif k.endswith(".router"):
            t[k] = t[k] + torch.randn(t[k].shape, generator=g)
        elif k.endswith((".ls1", ".ls2")):
            t[k] = t[k] + 0.3 * torch.randn(t[k].shape, generator=g)


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("gerorax")
    return {n: write_model(str(root / n), c, 51 + i, _lively) for i, (n, c) in enumerate(CONFIGS.items())}


def oracle(path, toks):
    return torch.from_numpy(pg.forward(list(toks), numpy_weights(path), plain_config(path))[0]).float()


def sensitivity(path, toks, dtype, want):
    """Row errors of the plain model whose norms put out rounded values (to bfloat16, or by a few units in the last
    place of float32) against itself: what rounding alone does to these weights and tokens."""
    rng, exact = np.random.default_rng(0), pg.norm
    if dtype == "float32":
        rough = lambda x, wt, eps: exact(x, wt, eps) * (1.0 + 3e-7 * rng.standard_normal(x.shape))
    else:
        rough = lambda x, wt, eps: torch.from_numpy(exact(x, wt, eps)).to(torch.bfloat16).double().numpy()
    pg.norm = rough
    try:
        return row_errors(oracle(path, toks), want)
    finally:
        pg.norm = exact


def assert_logits(got, want, dtype, path, toks, what=""):
    """float32: every row within the tolerance, or within a few times what rounding alone does.  bfloat16: rounding now
    and then sends a token of random weights to another expert, whose row then differs by more: half of the rows within
    half of the tolerance and nine in ten within it (or a few times what rounding does), which no fault of a cache or a
    mask passes."""
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


def _ctx(starts, counts, slots=None):
    """What a part reads of a step, for entries of ``counts`` tokens at ``starts``, built by hand."""
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
    seq = [e for e, c in enumerate(counts) for _ in range(c)]
    pos = [s + j for s, c in zip(starts, counts) for j in range(c)]
    return types.SimpleNamespace(n_tokens=int(sum(counts)), n_entries=len(counts), positions=i32(pos), token_seq=i32(seq),
                                 h_starts=np.asarray(starts, dtype=np.int32), h_counts=np.asarray(counts, dtype=np.int32),
                                 plans={}, scratch={}, decode_bucket=None)


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


# ---- embedding, norms and loop steps ------------------------------------------------------------------------------

@pytest.mark.parametrize("width", [64, 36, 7, 1])
def test_the_embedding_is_multiplied_and_joined_by_a_sinusoid_at_any_position(width):
    from atoma_infer_amd.parts import OutputHead, TokenEmbedding
    emb = TokenEmbedding(50, width, name="embed", scale=2.5, sinusoid_base=10000.0)
    w = _drawn(emb, "e.", 2)
    _load(emb, w, torch.bfloat16)
    pos = [0, 1, 31, 1000, 54321, (1 << 20) - 1]
    toks = torch.tensor([3, 49, 0, 3, 12, 60], dtype=torch.int32, device=DEV)
    got = emb.forward(toks, positions=torch.tensor(pos, dtype=torch.int32, device=DEV)).cpu()
    want = w["embed"][[3, 49, 0, 3, 12]].double().numpy() * 2.5 + pg.sinusoid(pos, width)[:5]
    assert np.abs(got[:5].double().numpy() - want).max() < 1e-6 and bool(got[5].isnan().all())
    out = torch.zeros(6, width, device=DEV)
    rows, begun = emb.forward(toks, norm=object(), out=out, positions=torch.tensor(pos, dtype=torch.int32, device=DEV))
    assert begun is None and rows is out and torch.equal(rows[:5].cpu(), got[:5])
    # the head reads the table alone
    head = OutputHead(width, 50, tied_to=emb)
    head.load(None, torch.device(DEV), torch.float32)
    h = _inputs([3], width, 1)[0]
    assert _rel(head.forward(h.to(DEV)).cpu(), h.double() @ w["embed"].double().T) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [64, 40, 33, 2048, 5000])
def test_a_norm_behind_a_sublayer_with_its_layer_scale_and_multiplier(width, dtype):
    from atoma_infer_amd.parts.base import make_part
    post = make_part("norm", "rmsnorm", width=width, eps=1e-4, name="b", gain="ls", factor=0.4)
    nxt = make_part("norm", "rmsnorm", width=width, eps=1e-4, name="n")
    wp, wn = _drawn(post, "p.", 3), _drawn(nxt, "n.", 4)
    assert set(wp) == {"b", "ls"}
    _load(post, wp, dtype)
    _load(nxt, wn, dtype)
    for t in (1, 9, 70):
        x, d = _inputs([t, t], width, t)
        resid = x.clone().to(DEV)
        out = post.add_normed(resid, d.to(DEV), nxt)
        a = as_numpy({**wp, **wn})
        want = x.double().numpy() + 0.4 * (a["ls"] * pg.norm(d.double().numpy(), a["b"], 1e-4))
        assert _rel(resid.cpu(), want) < 1e-6
        assert _rel(out.float().cpu(), pg.norm(want, a["n"], 1e-4)) < (2e-6 if dtype is torch.float32 else 4e-3)


@pytest.mark.parametrize("width", [64, 30, 37])
def test_a_loop_step_adds_the_embedding_before_every_pass_but_the_first(width):
    from atoma_infer_amd.parts import LoopStep
    from atoma_infer_amd.parts.base import make_part
    step = LoopStep(width, 3)
    nxt = make_part("norm", "rmsnorm", width=width, eps=1e-5, name="n")
    ws, wn = _drawn(step, "s.", 5), _drawn(nxt, "n.", 6)
    _load(step, ws, torch.float32)
    _load(nxt, wn, torch.float32)
    x, e, d = _inputs([11] * 3, width, width)
    for turn in range(3):
        for norm in (nxt, None):
            for delta in (None, d):
                resid = x.clone().to(DEV)
                y = step.forward(resid, None if delta is None else delta.to(DEV), None, None, embedded=e.to(DEV), turn=turn,
                                 next_norm=norm)
                want = x.double() + (e.double() if turn else 0) + ws["step"][turn].double() + (0 if delta is None else d.double())
                assert _rel(resid.cpu(), want) < 1e-6
                assert (y is None) == (norm is None)
                if norm is not None:
                    assert y.norm is nxt and _rel(y.data.cpu(), pg.norm(want.numpy(), wn["n"].double().numpy(), 1e-5)) < 2e-6
    for bad in (dict(turn=3, embedded=e), dict(turn=-1, embedded=e), dict(turn=1)):
        with pytest.raises(RuntimeError, match="loop step"):
            step.forward(x.clone().to(DEV), None, None, None, **bad)
    assert not LoopStep(width, 1).reads_embedding and LoopStep(width, 1, embedding_from=0).reads_embedding


# ---- routers and experts ------------------------------------------------------------------------------------------

@pytest.mark.parametrize("experts, top, groups", [
    (8, 3, (2, 1)), (6, 2, (3, 2)), (64, 6, (8, 3)), (64, 64, (4, 4)), (60, 5, (12, 2)), (70, 6, (7, 3)), (200, 50, (4, 1)),
    (1024, 8, (64, 5)), (1000, 3, (1000, 7)), (128, 4, (1, 1)), (1, 1, (1, 1)), (16, 2, (16, 2)), (12, 4, None), (100, 7, None)])
@pytest.mark.parametrize("score", ["softmax", "sigmoid"])
def test_experts_are_chosen_inside_the_groups_with_the_best_expert(experts, top, groups, score):
    from atoma_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(experts + top)
    t = 37
    z = torch.randn(t, experts, generator=g) * 3
    z[3, : experts // 2] = 1.25                      # ties: the lower index wins, of groups and of experts
    z[4] = 0.5
    ids, wts = ops.route_topk(z.to(DEV), top, score, groups=groups, scale=0.5)
    if score == "softmax":
        want_ids, want_w = pg.route(z.double().numpy(), top, {"count": groups[0], "keep": groups[1]} if groups else None)
    else:
        s = 1 / (1 + np.exp(-z.double().numpy()))
        want_ids = pg.route(z.double().numpy(), top, {"count": groups[0], "keep": groups[1]} if groups else None)[0]
        want_w = np.take_along_axis(s, want_ids, axis=1)
    # (float32 scores of different logits may be equal where the sigmoid is flat: the weights say whether it matters)
    same = np.asarray(ids.cpu()) == want_ids
    assert same.all() or score == "sigmoid" and same.mean() > 0.99
    assert np.abs(wts.cpu().double().numpy() - 0.5 * want_w).max() < 1e-6


@pytest.mark.parametrize("experts, groups", [(8, (2, 1)), (48, None), (128, (8, 2)), (300, None)])
def test_logits_that_are_no_numbers_still_choose_experts_of_the_layer(experts, groups):
    from atoma_infer_amd.kernels import ops
    z = torch.randn(9, experts, generator=torch.Generator().manual_seed(1))
    z[2] = float("nan")
    z[5, ::2] = float("nan")
    z[6] = float("inf")
    z[7] = -float("inf")
    for score in ("softmax", "sigmoid", "softmax_chosen"):
        if score == "softmax_chosen" and groups:
            continue
        ids = ops.route_topk(z.to(DEV), 4, score, groups=groups)[0].cpu()
        assert int(ids.min()) >= 0 and int(ids.max()) < experts


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width, m", [
    (64, moe(32, 6, 2, (3, 2), 1.5, (48, 0.7))), (128, moe(64, 12, 4, (2, 1), 0.5, (64, 0.5))), (40, moe(10, 4, 3, (2, 2), 0.8, None)),
    (96, moe(96, 70, 6, (7, 2), 1.0, (20, 2.0))), (64, moe(16, 1, 1, (1, 1), 0.3, (16, 9.0)))])
def test_clamped_experts_of_the_kept_groups_weighed_on_their_outputs_beside_a_shared_one(width, m, dtype):
    from atoma_infer_amd.parts.base import make_part
    act = lambda l: ("clamped_sigmoid", l, 1.702)
    r, e, s = m["router"], m["expert"], m.get("shared")
    part = make_part("feed_forward", "routed_experts", width=width, intermediate=e["ff"], experts=r["experts"], top=r["top"],
                     score="softmax", activation=act(e["limit"]), weigh="output",
                     groups=(r["groups"]["count"], r["groups"]["keep"]), shared=s["ff"] if s else 0,
                     shared_activation=act(s["limit"]) if s else None)
    w = _drawn(part, "x.", 7, boost=[("router", 3)] + [(f"{x}.{n}", 6) for x in ["shared"] + [f"e{i}" for i in range(r["experts"])]
                                                       for n in ("gate", "up")])
    _load(part, w, dtype)
    for t in (1, 9, 150):
        h = _inputs([t], width, e["ff"] + t)[0]
        got = _flat(part.forward(h.to(DEV, dtype), None))
        n, hn = as_numpy(w, "m."), h.double().numpy()
        want = torch.from_numpy(pg.moe(hn, n, "m.", m))
        # tokens whose choice, of groups or of experts, is no close call
        z = hn @ n["m.router"].T
        best = np.sort(z.reshape(t, r["groups"]["count"], -1).max(2), axis=1)[:, ::-1]
        kept = r["groups"]["keep"]
        clear = best[:, kept - 1] - best[:, kept] > 2e-3 if kept < r["groups"]["count"] else np.ones(t, dtype=bool)
        rough = z + np.random.default_rng(0).uniform(-1e-3, 1e-3, z.shape)
        clear &= (pg.route(rough, r["top"], r["groups"])[0] == pg.route(z, r["top"], r["groups"])[0]).all(1)
        clear = torch.from_numpy(clear)
        assert int(clear.sum()) > 0.8 * t
        assert _rel(got[clear], want[clear]) < PART_TOL[dtype], t


# ---- attention alone ----------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh, nkv, hd, vd, page", [(6, 2, 24, 40, 16), (4, 4, 64, 64, 16), (3, 1, 10, 5, 20), (8, 2, 128, 32, 48),
                                                   (2, 1, 7, 3, 16), (5, 5, 1, 1, 4), (4, 2, 256, 200, 32), (2, 2, 100, 256, 16)])
def test_heads_are_normed_and_the_tiles_filled(nh, nkv, hd, vd, page, dtype):
    from atoma_infer_amd.cache.layout import unpack_keys, unpack_values
    from atoma_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(hd)
    t, ho, vo = 29, -(-hd // 16) * 16, -(-vd // 16) * 16
    ld = -(-((nh + nkv) * hd + nkv * vd) // 64) * 64
    proj = torch.randn(t, ld, generator=g) * torch.rand(t, 1, generator=g) * 3
    wq, wk = torch.randn(hd, generator=g), torch.randn(hd, generator=g)
    pages = -(-t // page) + 2
    kc = torch.full((pages, nkv, page * ho), 7.0, dtype=dtype, device=DEV)
    vc = torch.full((pages, nkv, page * vo), 7.0, dtype=dtype, device=DEV)
    slots = torch.randperm(pages * page, generator=g)[:t].int()
    q = ops.head_norm(proj.to(DEV), wq.to(DEV), wk.to(DEV), 1e-3, kc, vc, slots.to(DEV), page, nh, nkv, hd, vd, ho, vo, dtype)
    x = proj.double().numpy()
    pad = lambda a, to: np.pad(a, ((0, 0), (0, 0), (0, to - a.shape[2])))
    wantq = pad(pg.norm(x[:, : nh * hd].reshape(t, nh, hd), wq.double().numpy(), 1e-3), ho).reshape(t, -1)
    wantk = pad(pg.norm(x[:, nh * hd: (nh + nkv) * hd].reshape(t, nkv, hd), wk.double().numpy(), 1e-3), ho)
    wantv = pad(x[:, (nh + nkv) * hd: (nh + nkv) * hd + nkv * vd].reshape(t, nkv, vd), vo)
    ks = unpack_keys(kc.cpu(), page, ho).permute(0, 2, 1, 3).reshape(pages * page, nkv, ho)
    vs = unpack_values(vc.cpu(), page, vo).permute(0, 3, 1, 2).reshape(pages * page, nkv, vo)
    tol = 1e-6 if dtype is torch.float32 else 4e-3
    assert _rel(q.float().cpu(), wantq) < tol
    idx = slots.long()
    assert _rel(ks[idx].float(), wantk) < tol and _rel(vs[idx].float(), wantv) < tol
    rest = torch.ones(pages * page, dtype=torch.bool)
    rest[idx] = False
    assert bool((ks[rest] == 7.0).all()) and bool((vs[rest] == 7.0).all())


def _cached(lens, nkv, hd, vd, page, dtype, seed):
    """Keys and values of requests in shuffled pages: (ks, vs, key tiles, value tiles, block tables)."""
    from atoma_infer_amd.cache.layout import pack_keys, pack_values
    g = torch.Generator().manual_seed(seed)
    ks = [torch.randn(n, nkv, hd, generator=g).to(dtype) for n in lens]
    vs = [torch.randn(n, nkv, vd, generator=g).to(dtype) for n in lens]
    blocks = [-(-n // page) for n in lens]
    perm = torch.randperm(sum(blocks) + 3, generator=g).tolist()
    kc = torch.randn(len(perm), nkv, page, hd, generator=g).to(dtype)          # unused slots hold noise
    vc = torch.randn(len(perm), nkv, vd, page, generator=g).to(dtype)
    bt = torch.zeros(len(lens), max(blocks), dtype=torch.int32)
    for e, n in enumerate(lens):
        for b in range(blocks[e]):
            bt[e, b] = pgn = perm.pop()
            lo, hi = b * page, min((b + 1) * page, n)
            kc[pgn, :, : hi - lo] = ks[e][lo:hi].permute(1, 0, 2)
            vc[pgn, :, :, : hi - lo] = vs[e][lo:hi].permute(1, 2, 0)
    return ks, vs, pack_keys(kc).to(DEV), pack_values(vc).to(DEV), bt


BIASED_CASES = [
    # (nh, nkv, hd, vd, page, window, keep, slopes, [(start, count), ...])
    (4, 2, 64, 64, 16, 50, 5, True, [(0, 40), (0, 1), (39, 1), (700, 1), (100, 20)]),
    (6, 2, 32, 48, 16, 13, 3, True, [(0, 70), (5, 9), (64, 2), (300, 33)]),
    (3, 1, 48, 32, 16, 0, 0, True, [(0, 130), (600, 1), (1030, 3), (511, 1)]),
    (8, 8, 16, 64, 16, 33, 40, True, [(0, 150), (41, 1), (72, 2), (73, 1), (500, 5)]),
    (4, 1, 64, 128, 16, 32, 32, True, [(0, 100), (63, 1), (64, 1), (95, 1), (1000, 40)]),
    (5, 1, 128, 64, 16, 600, 1, True, [(0, 700), (900, 150), (2047, 1), (1500, 3)]),
    (8, 2, 128, 128, 16, 100, 17, True, [(0, 300), (1500, 1), (95, 2)]),
    (4, 2, 64, 64, 16, 900, 33, False, [(0, 1300), (1200, 40), (3000, 1)]),
    (4, 2, 96, 96, 16, 0, 0, True, [(0, 260), (4000, 1), (4000, 3)]),
    (2, 1, 160, 32, 16, 70, 4, True, [(0, 90), (500, 1)]),
    (2, 2, 192, 192, 16, 70, 4, True, [(0, 90), (500, 1), (800, 2)]),
    (3, 1, 208, 64, 16, 90, 64, True, [(0, 200), (700, 1)]),
    (2, 1, 64, 208, 16, 90, 31, True, [(0, 200), (700, 1)]),
    (2, 1, 256, 256, 16, 40, 3, True, [(0, 80), (520, 2), (520, 1)]),
    (8, 2, 64, 64, 32, 600, 40, True, [(0, 1100), (900, 1), (640, 5)]),
    (8, 2, 64, 64, 64, 48, 4, True, [(0, 130), (600, 1), (1030, 3)]),
    (4, 2, 32, 48, 48, 100, 47, True, [(0, 300), (1500, 1), (95, 2)]),
    (4, 2, 128, 64, 32, -50, 0, True, [(0, 130), (600, 1), (149, 1), (150, 1)]),
    # so many keys that a wave works on two pieces of rows, and decoded tokens with long walks
    (4, 1, 64, 64, 16, 0, 0, True, [(17000, 70)]),
    (4, 1, 64, 64, 16, 9000, 40, True, [(17000, 70), (30000, 1)]),
    (8, 8, 64, 64, 16, 17000, 64, True, [(20000, 1), (16500, 1), (3, 1)]),
]


@pytest.mark.parametrize("nh,nkv,hd,vd,page,window,keep,biased,entries", BIASED_CASES)
@pytest.mark.parametrize("kind", ["generic_f32", "generic_bf16", "mfma", "mfma_chunks", "mfma_merge"])
def test_biased_attention_with_kept_keys_sinks_and_values_of_their_own_width(nh, nkv, hd, vd, page, window, keep, biased,
                                                                             entries, kind, monkeypatch):
    from atoma_infer_amd.kernels import attention_bf16, ops
    if kind == "mfma_chunks":
        force_chunked_decode(monkeypatch)
    elif kind == "mfma_merge":
        force_chunked_decode(monkeypatch, second_kernel=True)
    dtype = torch.float32 if kind == "generic_f32" else torch.bfloat16
    starts, counts = [s for s, _ in entries], [c for _, c in entries]
    ks, vs, kc, vc, bt = _cached([s + c for s, c in entries], nkv, hd, vd, page, dtype, hd + nh)
    # pages that a window has passed hold other things by now, and their entries say page 0
    if window > 0:
        for e, (s, _) in enumerate(entries):
            dead = [b for b in range(bt.shape[1]) if (b + 1) * page <= s - window + 1 and b * page >= keep]
            for b in dead:
                kc[int(bt[e, b])], vc[int(bt[e, b])] = 50.0, 50.0
                bt[e, b] = 0
    bt = bt.to(DEV)
    g = torch.Generator().manual_seed(1)
    t = sum(counts)
    q = (torch.randn(t, nh * hd, generator=g) * 1.5).to(dtype)
    slopes = torch.tensor(pg.slopes(nh), dtype=torch.float32, device=DEV) if biased else None
    sinks = torch.randn(nh, generator=g) * 3
    out = torch.full((t, nh * vd), float("nan"), dtype=dtype, device=DEV)
    ctx, cache = _ctx(starts, counts), types.SimpleNamespace(block_tables=bt, page_size=page)
    scale = hd ** -0.5
    if kind.startswith("mfma"):
        assert attention_bf16.try_attention(q.to(DEV), kc, vc, out, ctx, cache, scale, window, nh, nkv, hd, sinks.to(DEV), vd=vd,
                                            keep=keep, slopes=slopes)
    else:
        ops.paged_attention_generic(q.to(DEV), kc, vc, out, bt, ctx.token_seq, ctx.positions, scale, max(window, 0), page, nh, nkv,
                                    hd, slopes, max(-window, 0), sinks.to(DEV), keep, vd)
    row = 0
    for e, (s, c) in enumerate(entries):
        p, j = np.arange(s, s + c)[:, None], np.arange(s + c)[None, :]
        seen = j <= p
        if window > 0:
            seen = seen & ((p - j < window) | (j < keep))
        elif window < 0:
            seen = seen & (j >= p // -window * -window)
        qq = q[row: row + c].double().view(c, nh, hd).numpy()
        kk, vv = ks[e].double().numpy(), vs[e].double().numpy()
        for h in range(nh):
            sc = qq[:, h] @ kk[:, h // (nh // nkv)].T * scale - (pg.slopes(nh)[h] if biased else 0.0) * (p - j)
            sc = np.where(seen, sc, -np.inf)
            top = np.maximum(sc.max(1, keepdims=True), float(sinks[h]))
            ex = np.exp(sc - top)
            want = (ex / (ex.sum(1, keepdims=True) + np.exp(float(sinks[h]) - top))) @ vv[:, h // (nh // nkv)]
            got = out[row: row + c].double().cpu().numpy()[:, h * vd: (h + 1) * vd]
            err = np.abs(got - want).max() / max(np.abs(want).max(), 0.05)
            assert err < (2e-5 if dtype is torch.float32 else 2e-2), (e, h, err)
        row += c


@pytest.mark.parametrize("chunks", [None, "kernel", "second kernel"])
@pytest.mark.parametrize("nh, nkv, hd, vd, window, keep", [(8, 2, 64, 64, 300, 20), (4, 4, 32, 32, 1024, 4), (6, 1, 128, 64, 40, 33),
                                                           (3, 1, 16, 16, 700, 64)])
def test_decode_steps_of_a_bucket_walk_kept_keys_and_window(nh, nkv, hd, vd, window, keep, chunks, monkeypatch):
    """Steps as the runner plans them, every entry one token: whole ranges and chunks of the walk, contexts on both sides
    of where the gap opens, tables with more entries than a request holds."""
    from atoma_infer_amd.kernels import attention_bf16 as A
    if chunks:
        force_chunked_decode(monkeypatch, second_kernel=chunks != "kernel")
    starts = [0, 5, window - 1, window, window + 31, window + keep, window + keep + 32, window + keep + 63, 1500, 1531, 1532]
    counts, page = [1] * len(starts), 16
    ks, vs, kc, vc, bt = _cached([s + 1 for s in starts], nkv, hd, vd, page, torch.bfloat16, nh)
    bucket = -(-(max(starts) + 1) // 256) * 256
    arr, meta = A.build_tasks(np.asarray(starts, dtype=np.int32), np.asarray(counts, dtype=np.int32), nh // nkv, window, bucket,
                              kv_heads=nkv, max_waves=A.max_waves_for(hd, vd), head_size=hd, keep=keep)
    ctx = _ctx(starts, counts)
    ctx.plans = {A.plan_key(nh // nkv, window, nkv, hd, vd, keep): (torch.from_numpy(arr).to(DEV), meta)}
    wide = torch.zeros(len(starts), bucket // page, dtype=torch.int32)
    wide[:, : bt.shape[1]] = bt
    g = torch.Generator().manual_seed(2)
    q = (torch.randn(len(starts), nh * hd, generator=g) * 1.5).to(torch.bfloat16)
    slopes, sinks = torch.tensor(pg.slopes(nh), dtype=torch.float32, device=DEV), torch.randn(nh, generator=g)
    for _ in range(2):          # (the counters of merged chunks are left as they were)
        out = torch.full((len(starts), nh * vd), float("nan"), dtype=torch.bfloat16, device=DEV)
        assert A.try_attention(q.to(DEV), kc, vc, out, ctx, types.SimpleNamespace(block_tables=wide.to(DEV), page_size=page), 0.2,
                               window, nh, nkv, hd, sinks.to(DEV), vd=vd, keep=keep, slopes=slopes)
        for e, s in enumerate(starts):
            j = np.arange(s + 1)
            seen = (s - j < window) | (j < keep)
            for h in range(nh):
                sc = ks[e].double().numpy()[:, h // (nh // nkv)] @ q[e].double().numpy()[h * hd: (h + 1) * hd] * 0.2 \
                    - pg.slopes(nh)[h] * (s - j)
                sc = np.where(seen, sc, -np.inf)
                ex = np.exp(sc)
                want = ex @ vs[e].double().numpy()[:, h // (nh // nkv)] / (ex.sum() + np.exp(float(sinks[h])))
                got = out[e].double().cpu().numpy()[h * vd: (h + 1) * vd]
                assert np.abs(got - want).max() < 2e-2 * max(np.abs(want).max(), 0.05), (e, h)


def _paged_case(part, plain, dtype, cuts_of_steps, page, seed, width=64, hs=None):
    """A mixer over a paged cache on hand-made steps over pages that are dealt out of order: per request the outputs
    of all its portions, and the plain function's on the whole request.  Behind every step, pages that no later token
    sees are filled with something else and leave the tables, as pages do that another request uses by then."""
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
    v = torch.zeros((n_pages, cs.kv_heads, page * cs.value_elements), dtype=dtype, device=DEV)
    got, at = [[], []], [0, 0]
    for cuts in cuts_of_steps:
        ctx = _ctx([at[r] for r, _ in cuts], [c for _, c in cuts])
        bt = torch.tensor([[p or 0 for p in tables[r]] + [0] * (max_blocks - len(tables[r])) for r, _ in cuts],
                          dtype=torch.int32, device=DEV)
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
            if cs.window:
                for b in range(-(-cs.keep_first // page), max(0, at[r] - cs.window + 1) // page):
                    if b < len(tables[r]) and tables[r][b] is not None:
                        k[tables[r][b]], v[tables[r][b]] = 30.0, 30.0
                        tables[r][b] = None
    return [torch.cat(x) for x in got if x], want


def _part(m, width=64):
    from atoma_infer_amd.parts.base import make_part
    mask = m.get("mask")
    return make_part("mixer", "head_norm_attention", width=width, num_heads=m["heads"], num_kv_heads=m["kv_heads"],
                     head_size=m["dim"], value_size=m["vdim"], scale=m["scale"], norm_eps=1e-5,
                     position=make_part("position", "distance_bias"), window=mask["size"] if mask else None,
                     keep_first=mask["keep_first"] if mask else 0)


CUTS = [[(0, 20), (1, 3)], [(0, 1), (1, 1)], [(0, 2)], [(1, 40), (0, 1)], [(0, 50)], [(0, 1)], [(1, 1)], [(0, 1), (1, 2)]]
BOOST = (("q.norm", 2), ("k.norm", 2), ("v", 20), ("o", 5))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m, page", [
    (attention(24, 6, 2, 40, 0.2, 13, 3), 16), (attention(64, 8, 4, 64, 0.125, 50, 5), 32), (attention(10, 3, 3, 5, 0.4, 1, 2), 16),
    (attention(18, 2, 2, 33, 0.3, None), 48), (attention(16, 2, 1, 56, 0.25, 50, 33), 16), (attention(7, 5, 1, 3, 0.5, 9, 0), 20),
    (attention(2, 1, 1, 1, 1.0, 1, 1), 16), (attention(48, 12, 2, 80, 0.1, 33, 16), 16), (attention(1, 2, 1, 8, 3.0, 2, 1), 16)])
def test_attention_with_normed_heads_alone_whole_and_in_portions(m, page, dtype):
    part = _part(m)
    w = _drawn(part, "a.", 11, boost=BOOST)
    _load(part, w, dtype)
    plain = lambda h: pg.attention(h, np.arange(len(h)), as_numpy(w, "m."), "m.", m, 1e-5)
    got, want = _paged_case(part, plain, dtype, CUTS, page, m["dim"])
    for g, wt in zip(got, want):
        assert _rel(g, wt) < PART_TOL[dtype]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("far, window, keep", [
    (3, 64, 3), (3, 64, 4), (16, 40, 16), (16, 40, 17), (15, 40, 16), (63, 40, 5), (100, 17, 1), (5, 1, 0), (7, 2, 40), (0, 255, 0),
    (0, 17, 1), (40, None, 0), (31, 33, 32), (32, 33, 32), (95, 64, 96), (1, 1, 2)])
def test_one_key_that_stands_out_is_seen_to_the_windows_edge_or_for_good(far, window, keep, dtype):
    """One position's key matches what every query asks for: it stands out for every later query that sees it, and
    only for those, whether they come in a prompt, in a portion that begins anywhere, or alone.  Among the first
    ``keep`` positions it is seen for good."""
    m = attention(16, 2, 1, 16, 1.5, window, keep)
    part = _part(m)
    w = _drawn(part, "f.", 23, boost=(("o", 5), ("v", 20)))
    # column 0 of a head: a query's is large (the constant), a key's only at the marked position
    w["q"][0::16], w["k"][0] = 0.0, 0.0
    w["q"][0::16, 1] = 4.0
    w["k"][0, 0] = 4.0
    w["q.norm"][:] = 0.5
    w["k.norm"][:] = 0.5
    w["q.norm"][0] = w["k.norm"][0] = 6.0
    w["sink"][:] = -1.0
    _load(part, w, dtype)
    total = 270
    hs = _inputs((total, 0), 64, 3)
    for h in hs:
        h[:, 0], h[:, 1] = 0.0, 1.0
    hs[0][far, 0] = 6.0
    plain = lambda h: pg.attention(h, np.arange(len(h)), as_numpy(w, "m."), "m.", m, 1e-5)
    edge = far + (window or 10 ** 6)
    near = max(1, min(edge, total - 1) - 3)
    for cuts in ([[(0, total)]], [[(0, 7)], [(0, 121)], [(0, 2)], [(0, 70)], [(0, 70)]],
                 [[(0, near)]] + [[(0, 1)]] * min(8, total - near) + ([[(0, total - near - 8)]] if total - near > 8 else [])):
        got, want = _paged_case(part, plain, dtype, cuts, 16, 1, hs=hs)
        per_row = (got[0].double() - torch.from_numpy(want[0])).abs().amax(1) / np.abs(want[0]).max()
        assert float(per_row.max()) < (1e-4 if dtype is torch.float32 else 4e-2), int(per_row.argmax())
    hs0 = [h.clone() for h in hs]
    hs0[0][far, 0] = 0.0
    a, b = plain(hs[0].double().numpy()), plain(hs0[0].double().numpy())
    moved = np.abs(a - b).max(axis=1) > 0.1 * np.abs(a).max()
    end = total if far < keep else min(total, edge)
    near_end = min(end, far + 100)         # (the bias makes the mark fade at a distance)
    assert moved[far + 1: near_end].all() and not moved[end:].any() and not moved[:far].any()


def test_first_and_last_tokens_of_a_sequence_share_with_the_sink():
    """A sequence of one token is its value shared with the sink; a sink that outweighs all keys leaves nothing."""
    for dtype in (torch.float32, torch.bfloat16):
        m = attention(32, 4, 2, 32, 0.3, 5, 1)
        part = _part(m)
        w = _drawn(part, "s.", 3, boost=BOOST)
        w["sink"] = torch.tensor([30.0, -30.0, 0.0, 2.0])
        w["o"] = torch.nn.functional.pad(torch.eye(64), (0, 64))          # the first two heads' values
        _load(part, w, dtype)
        plain = lambda h: pg.attention(h, np.arange(len(h)), as_numpy(w, "m."), "m.", m, 1e-5)
        got, want = _paged_case(part, plain, dtype, [[(0, 1)], [(1, 30)], [(1, 1)], [(0, 1)]], 16, 4)
        for g, wt in zip(got, want):
            assert (g.double() - torch.from_numpy(wt)).abs().max() < (1e-5 if dtype is torch.float32 else 2e-2) * np.abs(wt).max()
            assert float(g[:, :32].abs().max()) < 1e-4 * float(g[:, 32:].abs().max())


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


@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_the_stream_behind_every_layer_run(dirs, name):
    from atoma_infer_amd.engine.step import StepEntry
    d = dirs[name]
    cfg = plain_config(d)
    toks = tokens(40, cfg["vocab"], 3)
    want = pg.forward(toks, numpy_weights(d), cfg)[1]
    runner = make_runner(d, "float32", 64, 16, 1)
    seen, steps = [], {i for i, c in enumerate(runner.model.spec.run_order) if c.layer == len(cfg["layers"])}
    runner.model.after_block = lambda pos, resid, pending: seen.append(resid.cpu().clone()) if pos not in steps else None
    runner.add_request(0)
    runner.step([StepEntry(0, toks, 0, [0])])
    assert len(seen) == len(want)
    for i, (g, w) in enumerate(zip(seen, want)):
        assert _rel(g, w) < 2e-5, i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_batches_of_unequal_requests_equal_each_alone_over_pages_and_slots_used_again(dirs, name, dtype):
    """Five requests through a pool of three slots and just enough pages: portions of some beside single tokens of
    others; a request that ends gives its pages and its slot to the next, and pages that a window has passed serve the
    others while the request still runs."""
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
    runner.manager.check()
    assert runner.manager.num_free_slots() == 3
    for gi in range(len(runner.pool.plan.groups)):
        assert runner.manager.num_free_pages(gi) == runner.manager.num_pages(gi)


@pytest.mark.parametrize("seed", [2, 15, 28, 41, 59, 82])
def test_configurations_drawn_at_random_agree_with_the_plain_model(tmp_path, seed):
    """Layers with sizes drawn at random: a whole prompt, a prompt and single tokens, portions, and a mixed batch over
    four slots."""
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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_over_many_windows_and_pages(dirs, dtype):
    d = dirs["A"]
    toks = tokens(420, plain_config(d)["vocab"], 9)
    want = oracle(d, toks)
    runner = make_runner(d, dtype, 448, 16, 1)
    got = run_schedule(runner, {0: toks}, [[(0, 20)]] + [[(0, 1)]] * 400)[0]
    assert_logits(got, want, dtype, d, toks)


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
        rows = pg.forward(list(p) + got, w, cfg)[0][len(p) - 1: -1]
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
    """``random-weights`` from a config.json of the design, then ``generate``: greedy tokens are the plain model's."""
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    env = dict(os.environ, PYTHONPATH=root)
    cfg_file, d = tmp_path / "config.json", str(tmp_path / "m")
    cfg_file.write_text(json.dumps(GER_A))
    run = lambda *a: subprocess.run([sys.executable, "-m", "atoma_infer_amd", *a], capture_output=True, text=True, env=env,
                                    timeout=300, cwd=root)
    proc = run("random-weights", "--config", str(cfg_file), "--out", d, "--seed", "4", "--norm-jitter", "0.1")
    assert proc.returncode == 0, proc.stderr[-2000:]
    prompt = tokens(9, GER_A["vocab"], 2)
    proc = run("generate", "--model", d, "--block-size", "16", "--num-gpu-blocks-override", "16", "--max-model-len", "64",
               "--max-num-batched-tokens", "64", "--max-num-sequences", "4", "--max-new-tokens", "6", "--ignore-eos-token",
               "--prompt-ids", ",".join(str(t) for t in prompt), "--dtype", "f32", "--greedy")
    assert proc.returncode == 0, proc.stderr[-2000:]
    got = json.loads(proc.stdout.strip().splitlines()[-1])["inference_outputs"][0]["token_ids"]
    w, cfg, seq = numpy_weights(d), plain_config(d), list(prompt)
    for _ in range(6):
        seq.append(int(pg.forward(seq, w, cfg)[0][-1].argmax()))
    assert got == seq[len(prompt):]
