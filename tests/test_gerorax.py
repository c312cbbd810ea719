"""What pins the plain Gerorax (closed forms worked by hand) and what the configuration, the builder and the cache manager
do, on the CPU."""
import copy
import math

import numpy as np
import pytest

import plain_gerorax as pg
from gerorax_util import GER_A, GER_B, GER_C, GER_D


# ---- the plain implementation ------------------------------------------------------------------------------------

def test_the_sinusoid_alternates_sine_and_cosine_of_slowing_angles():
    s = pg.sinusoid([0, 3], 6)
    assert np.allclose(s[0], [0, 1, 0, 1, 0, 1])
    f = [1.0, 10000.0 ** (-1 / 3), 10000.0 ** (-2 / 3)]
    assert np.allclose(s[1], [g(3 * x) for x in f for g in (math.sin, math.cos)])
    cfg = {"embedding": {"scale": 4.0}, "width": 2}
    assert np.allclose(pg.embed([1], [2], {"embed": np.array([[0.0, 0.0], [1.0, -2.0]])}, cfg),
                       [[4 + math.sin(2), -8 + math.cos(2)]])


def test_slopes_halve_at_eight_heads_and_fall_faster_with_fewer():
    assert np.allclose(pg.slopes(8), [2.0 ** -i for i in range(1, 9)])
    assert np.allclose(pg.slopes(1), [2.0 ** -8]) and np.allclose(pg.slopes(3), [2.0 ** (-8 / 3), 2.0 ** (-16 / 3), 2.0 ** -8])


def test_a_window_keeps_the_first_tokens():
    seen = pg.visible(range(8), {"size": 2, "keep_first": 3})
    assert [np.flatnonzero(r).tolist() for r in seen] == [
        [0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 2, 4, 5], [0, 1, 2, 5, 6], [0, 1, 2, 6, 7]]
    assert np.array_equal(pg.visible(range(5), {"size": 3}), pg.visible(range(5), {"size": 3, "keep_first": 0}))
    assert np.array_equal(pg.visible(range(5), None), np.tril(np.ones((5, 5), dtype=bool)))


def test_biased_scores_and_the_sink_in_closed_form():
    # two heads over one key head, slopes 2^-4 and 2^-8; scores zero but for the bias; values 1, 10, 100
    q, k, v = np.zeros((3, 2, 4)), np.zeros((3, 1, 4)), np.array([1.0, 10.0, 100.0]).reshape(3, 1, 1)
    sink = np.array([0.5, -2.0])
    o = pg.biased_softmax(q, k, v, np.arange(3), 1.0, None, sink)[2, :, 0]
    for h, s in enumerate((2.0 ** -4, 2.0 ** -8)):
        e = [math.exp(-2 * s), math.exp(-s), 1.0]
        assert math.isclose(o[h], (e[0] + 10 * e[1] + 100 * e[2]) / (sum(e) + math.exp(sink[h])))
    # the bias is not scaled, and the sink neither scaled nor biased
    q[2, 0, 0], k[0, 0, 0] = 2.0, 3.0
    o = pg.biased_softmax(q, k, v, np.arange(3), 0.25, None, sink)[2, 0, 0]
    e = [math.exp(6 * 0.25 - 2 / 16), math.exp(-1 / 16), 1.0]
    assert math.isclose(o, (e[0] + 10 * e[1] + 100 * e[2]) / (sum(e) + math.exp(0.5)))
    # a kept key keeps its true distance
    q[:], k[:] = 0.0, 0.0
    o = pg.biased_softmax(q, k, v, np.arange(3), 1.0, {"size": 1, "keep_first": 1})[2, 0, 0]
    assert math.isclose(o, (math.exp(-2 / 16) + 100) / (math.exp(-2 / 16) + 1))


def test_heads_are_normed_one_by_one_with_a_shared_weight():
    m = {"heads": 2, "kv_heads": 1, "dim": 2, "vdim": 1, "scale": 1.0}
    w = {"m.q": np.array([[3.0, 0], [0, 4.0], [0, 0], [0, 2.0]]), "m.k": np.eye(2), "m.v": np.array([[1.0, 0.0]]),
         "m.q.norm": np.array([1.0, 2.0]), "m.k.norm": np.array([1.0, 1.0]), "m.sink": np.array([0.0, 0.0]), "m.o": np.eye(2)}
    h = np.array([[1.0, 1.0], [2.0, 1.0]])
    out = pg.attention(h, np.arange(2), w, "m.", m, 0.0)
    unit = lambda x: x / math.sqrt((x ** 2).mean())
    k = [unit(h[0]), unit(h[1])]
    for hh, q in enumerate((unit(np.array([6.0, 4.0])) * [1, 2], unit(np.array([0.0, 2.0])) * [1, 2])):
        s = [q @ k[0] - 2.0 ** (-4 * (hh + 1)), q @ k[1]]
        e = np.exp(s)
        assert math.isclose(out[1, hh], (e[0] * 1 + e[1] * 2) / (e.sum() + 1.0))


def test_the_router_looks_for_experts_in_the_best_groups_only():
    z = np.array([[5.0, 0.0, 4.0, 3.9, 1.0, 4.5]])
    s = np.exp(z[0]) / np.exp(z[0]).sum()
    for groups, want in ((None, [0, 5, 2]), ({"count": 3, "keep": 2}, [0, 5, 4]), ({"count": 2, "keep": 1}, [0, 2, 1]),
                         ({"count": 3, "keep": 3}, [0, 5, 2])):
        ids, wts = pg.route(z, 3, groups)
        assert ids[0].tolist() == want and np.allclose(wts[0], s[want])          # not renormalised


def test_feed_forwards_in_closed_form():
    w = {"m.gate": np.array([[1.0, 0.0]]), "m.up": np.array([[0.0, 1.0]]), "m.down": np.array([[1.0]])}
    h = np.array([[5.0, 9.0], [-5.0, -9.0], [0.5, 0.25]])
    sg = lambda z: 1 / (1 + math.exp(-z))
    want = [2 * sg(1.702 * 2) * 3, -5 * sg(-1.702 * 5) * -1, 0.5 * sg(0.851) * 1.25]
    assert np.allclose(pg.expert(h, w, "m.", 2.0)[:, 0], want)
    g = 0.25 * (1 + math.tanh(math.sqrt(2 / math.pi) * (0.5 + 0.044715 / 8)))
    assert np.allclose(pg.dense(h, w, "m.")[2, 0], g * 0.25)


def test_the_order_of_layer_runs_and_what_joins_before_a_pass():
    assert pg.runs({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == [
        (0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert pg.runs({"layers": [0] * 2}) == [(0, None), (1, None)]
    # layers that add nothing leave the stream to the steps and the embedding
    cfg = {"layers": [{"mixer": {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 1, "scale": 1.0}, "mlp": None}],
           "loop": {"start": 0, "stop": 1, "times": 3}, "norm": {"eps": 1e-5}, "residual_mult": 1.0, "width": 2,
           "embedding": {"scale": 1.0}}
    w = {"embed": np.array([[1.0, 2.0]]), "loop.step": np.array([[1.0, 0], [0, 10.0], [100.0, 0]]), "final.norm": np.ones(2),
         "l0.norm1": np.ones(2), "l0.norm1b": np.ones(2), "l0.ls1": np.zeros(2), "l0.mix.q": np.eye(2), "l0.mix.k": np.eye(2),
         "l0.mix.v": np.ones((1, 2)), "l0.mix.o": np.ones((2, 1)), "l0.mix.q.norm": np.ones(2), "l0.mix.k.norm": np.ones(2),
         "l0.mix.sink": np.zeros(1)}
    x0 = np.array([1.0, 3.0])
    seen = pg.forward([0], w, cfg)[1][:, 0]
    assert np.allclose(seen, [x0 + [1, 0], 2 * x0 + [1, 10], 3 * x0 + [101, 10]])


def test_a_sublayer_s_output_is_normed_scaled_by_column_and_multiplied():
    cfg = {"layers": [{"mixer": {"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 1.0}, "mlp": {"kind": "dense", "ff": 1}}],
           "norm": {"eps": 0.0}, "residual_mult": 0.5, "width": 2, "embedding": {"scale": 1.0}}
    w = {"l0.norm1": np.ones(2), "l0.norm1b": np.array([2.0, 1.0]), "l0.ls1": np.array([1.0, 3.0]), "l0.norm2": np.ones(2),
         "l0.norm2b": np.ones(2), "l0.ls2": np.array([0.0, 4.0]), "l0.mix.q": np.ones((1, 2)), "l0.mix.k": np.ones((1, 2)),
         "l0.mix.v": np.ones((1, 2)), "l0.mix.o": np.array([[1.0], [7.0]]), "l0.mix.q.norm": np.ones(1),
         "l0.mix.k.norm": np.ones(1), "l0.mix.sink": np.full(1, -1e9), "l0.mlp.gate": np.ones((1, 2)),
         "l0.mlp.up": np.ones((1, 2)), "l0.mlp.down": np.array([[3.0], [3.0]])}
    x = pg.layer(np.array([[1.0, 1.0]]), [0], w, 0, cfg)
    assert np.allclose(x, [[1 + 0.5 * 2 * 1 / 5, 1 + 0.5 * (3 * 7 / 5 + 4)]])


# ---- configuration and builder -----------------------------------------------------------------------------------

def _spec(cfg):
    from atoma_infer_amd.config.registry import resolve_architecture
    arch = resolve_architecture(cfg)
    return arch.build(arch.config_cls.from_dict(copy.deepcopy(cfg)))


def _shapes(cfg):
    from atoma_infer_amd.weights.loader import expected_tensors
    return {n: ws.shape for n, ws in expected_tensors(_spec(cfg)).items()}


@pytest.mark.parametrize("cfg", [GER_A, GER_B, GER_C, GER_D])
def test_a_configuration_reads_back_equal_and_declares_its_tensors(cfg):
    from atoma_infer_amd.config.gerorax import GeroraxConfig
    c = GeroraxConfig.from_dict(copy.deepcopy(cfg))
    assert GeroraxConfig.from_dict(c.to_dict()) == c and c.to_dict() == cfg
    shapes, W = _shapes(cfg), cfg["width"]
    assert "head" not in shapes and shapes["embed"] == (cfg["vocab"], W) and shapes["final.norm"] == (W,)
    assert shapes.get("loop.step") == ((cfg["loop"]["times"], W) if "loop" in cfg else None)
    for i, l in enumerate(cfg["layers"]):
        m, f, pre = l["mixer"], l["mlp"], f"l{i}."
        for n in ("norm2", "norm2b", "ls2"):
            assert (pre + n in shapes) == (f is not None)
        assert {shapes[pre + n] for n in ("norm1", "norm1b", "ls1")} == {(W,)}
        assert shapes[pre + "mix.q"] == (m["heads"] * m["dim"], W) and shapes[pre + "mix.v"] == (m["kv_heads"] * m["vdim"], W)
        assert shapes[pre + "mix.o"] == (W, m["heads"] * m["vdim"]) and shapes[pre + "mix.sink"] == (m["heads"],)
        assert shapes[pre + "mix.q.norm"] == shapes[pre + "mix.k.norm"] == (m["dim"],)
        if f and f["kind"] == "moe":
            assert shapes[pre + "mlp.router"] == (f["router"]["experts"], W) and pre + "mlp.router.b" not in shapes
            assert (pre + "mlp.shared.gate" in shapes) == ("shared" in f)
            assert shapes[pre + f"mlp.e{f['router']['experts'] - 1}.up"] == (f["expert"]["ff"], W)


def test_every_pass_of_a_loop_has_a_cache_of_its_own_in_its_layers_group():
    from atoma_infer_amd.cache.pool import plan_cache
    spec = _spec(GER_A)
    assert [c.layer for c in spec.run_order] == [0, 4, 1, 2, 4, 1, 2, 4, 1, 2, 3]
    plan = plan_cache(spec)
    groups = {(g.spec.window, g.spec.keep_first, g.spec.head_size, g.spec.value_elements): g.calls for g in plan.groups}
    assert groups == {(13, 3, 32, 48): [0], (21, 18, 16, 16): [2, 5, 8], (None, 0, 48, 32): [3, 6, 9], (50, 33, 16, 64): [10]}
    assert not plan.states


def test_a_layer_without_a_feed_forward_may_carry_the_tensors_around_one():
    import re
    spec = _spec(GER_A)
    assert all(any(re.fullmatch(p, n) for p in spec.ignorable) for n in ("l2.norm2", "l2.norm2b", "l2.ls2"))
    assert not any(re.fullmatch(p, n) for p in spec.ignorable for n in ("l1.norm2", "l2.norm1", "l2.ls1"))


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0]["mixer"].update(heads=5), "not a multiple of kv_heads"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=300), "more than 256 columns"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "positive"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1), "not negative"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "is not possible"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "is not possible"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "is not possible"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=-1.0), "positive"),
    (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "kind must be one of"),
    (lambda c: c["layers"][0].update(type="convolution"), "is not supported"),
    (lambda c: c["loop"].update(stop=5), "does not lie within"),
    (lambda c: c["loop"].update(times=0), "positive"),
    (lambda c: c.pop("norm"), "missing key 'norm'"),
])
def test_a_configuration_the_engine_cannot_run_is_refused_with_the_reason(change, message):
    from atoma_infer_amd.config.base import ConfigError
    from atoma_infer_amd.config.gerorax import GeroraxConfig
    c = copy.deepcopy(GER_A)
    change(c)
    with pytest.raises(ConfigError, match=message):
        GeroraxConfig.from_dict(c)


def test_parts_refuse_what_they_cannot_mean():
    from atoma_infer_amd.parts.base import CacheSpec, make_part
    ex = dict(width=8, intermediate=4, experts=6, top=3)
    for bad in ((4, 2), (3, 0), (3, 4), (3, 1)):
        with pytest.raises(ValueError, match="groups"):
            make_part("feed_forward", "routed_experts", **ex, groups=bad)
    rot = make_part("position", "rotary", head_size=8, theta=100.0, max_positions=4)
    rot.cos = rot.sin = 0
    with pytest.raises(ValueError, match="rotation"):
        make_part("mixer", "head_norm_attention", width=8, num_heads=1, num_kv_heads=1, head_size=8, value_size=8, scale=1.0,
                  norm_eps=1e-5, position=rot)
    for bad in (dict(keep_first=3), dict(window=4, keep_first=-1)):
        with pytest.raises(ValueError, match="invalid cache spec"):
            CacheSpec(1, 16, **bad)
    # without a window every key is seen: nothing is kept beside it
    assert make_part("mixer", "attention", width=8, num_heads=1, num_kv_heads=1, head_size=8, keep_first=3).cache_spec() \
        == CacheSpec(1, 8)


# ---- the cache manager -------------------------------------------------------------------------------------------

def test_pages_of_the_first_tokens_stay_while_a_window_moves_on():
    from atoma_infer_amd.cache.manager import CacheError, CacheManager, GroupGeometry
    m = CacheManager([GroupGeometry(4, 20, window=6, keep_first=5), GroupGeometry(4, 20, window=6)], 2)
    m.add(1)
    m.reserve(1, 40)
    assert m.release_behind(1, 8) == 0                 # the next token sees 3 .. 8
    # the token at 40 sees 35 .. 40 and 0 .. 4: blocks 2 .. 7 go in the first group, 0 .. 7 in the second
    assert m.release_behind(1, 40) == 6 + 8
    t0, t1 = m.table(1, 0), m.table(1, 1)
    assert [b for b, p in enumerate(t0) if p >= 0] == [0, 1, 8, 9] and [b for b, p in enumerate(t1) if p >= 0] == [8, 9]
    m.check()
    m.reserve(1, 48)
    assert m.release_behind(1, 48) == 2 + 2 and m.table(1, 0)[:2] == t0[:2]
    assert m.release_behind(1, 48) == 0
    m.check()
    m.free(1)
    m.check()
    assert m.num_free_pages(0) == 20 and m.num_free_pages(1) == 20
    for bad in (GroupGeometry(4, 4, keep_first=2), GroupGeometry(4, 4, window=4, keep_first=-1),
                GroupGeometry(4, 4, chunk=4, keep_first=2)):
        with pytest.raises(CacheError, match="invalid cache geometry"):
            CacheManager([bad], 1)


def test_admission_counts_the_kept_pages_beside_the_window():
    from atoma_infer_amd.cache.manager import CacheManager, GroupGeometry
    # a request in full swing holds the window's three pages, the page the next token opens and two kept ones
    g = lambda n: CacheManager([GroupGeometry(4, n, window=10, keep_first=5)], 4)
    assert g(6).fits_at_all(10 ** 6) and not g(5).fits_at_all(10 ** 6) and g(5).fits_at_all(20)
    m = g(12)
    assert m.can_admit(1000, 8)
    m.add(1)
    m.reserve(1, 8)                                    # two pages, four more to come
    assert m.can_admit(1000, 8) and not m.can_admit(1000, 25)
    m.add(2)
    m.reserve(2, 8)
    assert not m.can_admit(4, 4)
    m.reserve(1, 24)
    m.release_behind(1, 24)                            # holds the pages 0, 1 and 3 .. 5
    assert [p >= 0 for p in m.table(1)] == [True, True, False, True, True, True]
    m.free(2)
    assert m.num_free_pages() == 7 and m.can_admit(1000, 24) and not m.can_admit(1000, 28)


def test_random_traffic_never_loses_a_kept_page_or_one_of_the_window():
    import random
    from atoma_infer_amd.cache.manager import CacheManager, GroupGeometry
    rng = random.Random(3)
    for page, window, keep in ((4, 6, 5), (16, 40, 1), (2, 1, 9), (8, 100, 8)):
        m = CacheManager([GroupGeometry(page, 400, window=window, keep_first=keep)], 3)
        at = {}
        for _ in range(400):
            r = rng.randint(0, 2)
            if r not in at:
                m.add(r)
                at[r] = 0
            n = rng.choice([1, 1, 2, 5, 30])
            m.reserve(r, at[r] + n)
            t = m.table(r)
            for pos in range(at[r], at[r] + n):        # every key that these tokens see has its page
                for key in list(range(max(0, pos - window + 1), pos + 1)) + list(range(min(keep, pos + 1))):
                    assert t[key // page] >= 0
            at[r] += n
            m.release_behind(r, at[r])
            held = sum(p >= 0 for p in m.table(r))
            assert held <= -(-window // page) + 1 + -(-keep // page)
            m.check()
            if rng.random() < 0.05:
                m.free(r)
                del at[r]
