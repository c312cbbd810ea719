"""What pins the plain Duduvik (closed forms worked by hand) and what the configuration and the builder do, on the CPU."""
import copy
import math

import numpy as np
import pytest

import plain_duduvik as pd
from duduvik_util import DUD_A, DUD_B, DUD_C, DUD_D


# ---- the plain implementation ------------------------------------------------------------------------------------

def test_half_split_pairs_turn_by_the_position_and_the_rest_passes():
    x = np.zeros((1, 1, 6))
    x[0, 0] = [1, 0, 0, 5, 0, 7]
    rot = {"base": 4.0, "dims": 4}
    f = [1.0, 0.5]
    got = pd.rotate_half(x, [3], rot)[0, 0]
    want = [math.cos(3 * f[0]), -5 * math.sin(3 * f[1]), math.sin(3 * f[0]), 5 * math.cos(3 * f[1]), 0, 7]
    assert np.allclose(got, want)
    assert np.array_equal(pd.rotate_half(x, [3], {"base": 4.0, "dims": 0}), x) and np.array_equal(pd.rotate_half(x, [3], None), x)
    # scores depend on the distance alone
    g = np.random.default_rng(0)
    q, k = g.standard_normal((1, 1, 6)), g.standard_normal((1, 1, 6))
    s = [(pd.rotate_half(q, [a], rot) * pd.rotate_half(k, [b], rot)).sum() for a, b in ((9, 4), (105, 100))]
    assert abs(s[0] - s[1]) < 1e-9


def test_the_decay_acts_on_rows_of_key_channels_before_the_token_joins():
    q = np.array([[[1.0, 1.0]], [[2.0, 3.0]]])
    k = np.array([[[1.0, 2.0]], [[5.0, 0.0]]])
    v = np.array([[[4.0]], [[1.0]]])
    al = np.array([[[0.9, 0.9]], [[0.5, 0.25]]])
    o, S = pd.decayed_sum(q, k, v, al)
    assert np.allclose(o[:, 0, 0], [12.0, 2 * (0.5 * 4 + 5) + 3 * (0.25 * 8)])
    assert np.allclose(S[0, :, 0], [7.0, 2.0])
    a, Sa = pd.decayed_sum(q[:1], k[:1], v[:1], al[:1])
    b, Sb = pd.decayed_sum(q[1:], k[1:], v[1:], al[1:], Sa)
    assert np.allclose(np.concatenate([a, b]), o) and np.allclose(Sb, S)


def test_gated_linear_attention_in_closed_form():
    m = {"heads": 1, "dim": 2, "vdim": 1, "tau": 2.0}
    eye = np.eye(2)
    w = {"m.q": eye, "m.k": eye, "m.v": np.array([[1.0, 0.0]]), "m.g": np.array([[0.0, 1.0]]), "m.norm": np.array([3.0]),
         "m.o": np.array([[2.0]]), "m.a1": np.array([[1.0, 0.0]]), "m.a2": np.array([[1.0], [0.0]]),
         "m.a2.b": np.array([0.0, math.log(3.0)])}
    h = np.array([[1.0, 2.0], [0.0, -1.0]])
    al = pd.gla_decay(h, w, "m.", m)
    assert np.allclose(al[1, 0], [math.sqrt(0.5), math.sqrt(0.75)])      # sigmoid(0)^(1/2), sigmoid(log 3)^(1/2)
    S = np.array([1.0, 2.0])
    o = [(S @ h[0]) / math.sqrt(2)]
    S = al[1, 0] * S + 0.0
    o.append((S @ h[1]) / math.sqrt(2))
    want = [2 * 3 * x / math.sqrt(x * x + 1e-6) * pd.silu(g) for x, g in zip(o, h[:, 1])]
    assert np.allclose(pd.gla(h, w, "m.", m, 1e-6)[0][:, 0], want)
    # logits far below zero give no NaN, and no decay above one
    big = np.full((1, 2), -800.0)
    w2 = dict(w)
    w2["m.a1"] = np.array([[1.0, 1.0]])
    assert np.all(pd.gla_decay(big, w2, "m.", m) >= 0.0) and np.all(pd.gla_decay(-big, w2, "m.", m) <= 1.0)


def test_retention_in_closed_form_and_scaled_after_rotation():
    m = {"heads": 2, "dim": 2, "vdim": 1, "decay": [0.5, 1.0], "rot": {"base": 10.0, "dims": 2}}
    one = np.ones((4, 1))
    w = {"m.q": one, "m.k": one, "m.v": np.ones((2, 1)), "m.g": np.full((2, 1), 2.0), "m.o": np.eye(2)}
    h = np.ones((3, 1))
    # q . k between positions d apart is 2 cos(d), over sqrt(2)
    sc = [2 * math.cos(d) / math.sqrt(2) for d in range(3)]
    o = [[sc[0], sc[0]], [sc[0] + 0.5 * sc[1], sc[0] + sc[1]], [sc[0] + 0.5 * sc[1] + 0.25 * sc[2], sc[0] + sc[1] + sc[2]]]
    want = np.array([[x / math.sqrt(x * x + 1e-3) for x in row] for row in o]) * pd.silu(2.0)
    got, S = pd.retention(h, np.arange(3), w, "m.", m, 1e-3)
    assert np.allclose(got, want) and S.shape == (2, 2, 1)
    tail, _ = pd.retention(h[2:], [2], w, "m.", m, 1e-3, pd.retention(h[:2], [0, 1], w, "m.", m, 1e-3)[1])
    assert np.allclose(tail, want[2:])


def test_a_window_sees_itself_and_the_tokens_just_before_it():
    T = 6
    z, v = np.zeros((T, 1, 2)), np.arange(T, dtype=float).reshape(T, 1, 1)
    o = pd.windowed_softmax(z, z, v, np.arange(T), 1.0, 3)[:, 0, 0]
    assert np.allclose(o, [0, 0.5, 1, 2, 3, 4])
    assert np.allclose(pd.windowed_softmax(z, z, v, np.arange(T), 1.0, 1)[:, 0, 0], np.arange(T))
    assert np.allclose(pd.windowed_softmax(z, z, v, np.arange(T), 1.0)[:, 0, 0], np.arange(T) / 2)


def test_the_router_chooses_by_biased_logits_and_weighs_by_the_chosen_ones():
    w = {"m.router": np.eye(3), "m.router.b": np.array([0.0, 2.0, -5.0])}
    ids, wts = pd.route(np.array([[1.0, 0.5, 3.0]]), w, "m.", 2)
    assert ids.tolist() == [[1, 0]]                                  # 1, 2.5, -2
    assert np.allclose(wts, [[1 / (1 + math.exp(-1.5)), 1 / (1 + math.exp(1.5))]])


def test_an_expert_bounds_its_gate_from_above_and_its_up_value_on_both_sides():
    w = {"m.gate": np.array([[1.0, 0.0]]), "m.up": np.array([[0.0, 1.0]]), "m.down": np.array([[1.0]])}
    h = np.array([[5.0, 9.0], [-5.0, -9.0], [0.5, 0.25]])
    sg = lambda z: 1 / (1 + math.exp(-z))
    want = [2 * sg(1.702 * 2) * 3, -5 * sg(-1.702 * 5) * -1, 0.5 * sg(0.851) * 1.25]
    assert np.allclose(pd.expert(h, w, "m.", 2.0)[:, 0], want)
    assert np.allclose(pd.dense(h, w, "m.")[:, 0], [45.0, 0.0, 0.125])


def test_the_head_is_the_table_without_its_factor():
    cfg = {"embedding": {"scale": 4.0}, "norm": {"eps": 1e-6}, "layers": []}
    w = {"embed": np.array([[1.0, 2.0], [3.0, -1.0]]), "final.norm": np.array([0.0, 1.0])}
    x = 4 * w["embed"][1]
    n = x / math.sqrt(np.mean(x * x) + 1e-6) * np.array([1.0, 2.0])
    assert np.allclose(pd.embed([1], w, cfg)[0], x)
    assert np.allclose(_head([1], w, cfg), n @ w["embed"].T)


def _head(toks, w, cfg):
    x = pd.embed(toks, w, cfg)
    return (pd.norm_one_plus(x, w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T)[0]


# ---- configuration and builder -----------------------------------------------------------------------------------

def _shapes(cfg):
    """Tensor names and shapes of a configuration, from the engine's own declaration of them."""
    from atoma_infer_amd.config.registry import resolve_architecture
    from atoma_infer_amd.weights.loader import expected_tensors
    arch = resolve_architecture(cfg)
    return {n: ws.shape for n, ws in expected_tensors(arch.build(arch.config_cls.from_dict(cfg))).items()}


@pytest.mark.parametrize("cfg", [DUD_A, DUD_B, DUD_C, DUD_D])
def test_a_configuration_reads_back_equal_and_declares_its_tensors(cfg):
    from atoma_infer_amd.config.duduvik import DuduvikConfig
    c = DuduvikConfig.from_dict(copy.deepcopy(cfg))
    assert DuduvikConfig.from_dict(c.to_dict()) == c and c.to_dict() == cfg
    shapes = _shapes(cfg)
    assert "head" not in shapes and shapes["embed"] == (cfg["vocab"], cfg["width"])
    for i, l in enumerate(cfg["layers"]):
        m, f, pre = l["mixer"], l["mlp"], f"l{i}."
        assert pre + "norm1b" in shapes and (pre + "norm2b" in shapes) == (f is not None)
        if l["type"] == "gla":
            assert shapes[pre + "mix.a1"] == (m["rank"], cfg["width"]) and shapes[pre + "mix.norm"] == (m["vdim"],)
            assert shapes[pre + "mix.a2.b"] == (m["heads"] * m["dim"],)
        if l["type"] == "retention":
            assert pre + "mix.norm" not in shapes and pre + "mix.a1" not in shapes
            assert shapes[pre + "mix.g"] == (m["heads"] * m["vdim"], cfg["width"])
        if l["type"] == "latent_attention":
            assert pre + "mix.g" not in shapes and shapes[pre + "mix.dkv"] == (m["kv_rank"] + m["rot_dim"], cfg["width"])
        if f and f["kind"] == "moe":
            assert shapes[pre + "mlp.router.b"] == (f["router"]["experts"],)
            assert (pre + "mlp.shared.gate" in shapes) == ("shared" in f)
            if "shared" in f:
                assert shapes[pre + "mlp.shared.down"] == (cfg["width"], f["shared"]["ff"])
            assert shapes[pre + f"mlp.e{f['router']['experts'] - 1}.up"] == (f["expert"]["ff"], cfg["width"])


def test_the_inner_size_of_the_decays_map_is_the_checkpoints():
    from atoma_infer_amd.parts.base import FREE
    c = copy.deepcopy(DUD_B)
    del c["layers"][1]["mixer"]["rank"]
    shapes = _shapes(c)
    assert shapes["l1.mix.a1"] == (FREE, c["width"]) and shapes["l1.mix.a2"] == (4 * 64, FREE)


def test_windows_get_groups_of_pages_and_recurrences_states():
    from atoma_infer_amd.cache.pool import plan_cache
    from atoma_infer_amd.config.registry import resolve_architecture
    arch = resolve_architecture(DUD_B)
    spec = arch.build(arch.config_cls.from_dict(copy.deepcopy(DUD_B)))
    plan = plan_cache(spec)
    assert sorted(g.spec.window for g in plan.groups) == [16, 50]
    assert plan.states == {1: ((4 * 64 * 128,), "float32"), 2: ((2 * 64 * 64,), "float32")}


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5]), "decays for"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 1.5, 0.1]), "between 0 and 1"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "cannot hold"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3), "even"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10), "cannot hold"),
    (lambda c: c["layers"][1]["mixer"].update(kv_rank=300), "more than the attention kernels"),
    (lambda c: c["layers"][2]["mixer"].update(tau=0.0), "positive"),
    (lambda c: c["layers"][2]["mixer"].update(dim=300), "beyond 256"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "is not possible"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=-1.0), "positive"),
    (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "kind must be one of"),
    (lambda c: c["layers"][0].update(type="convolution"), "is not supported"),
])
def test_a_configuration_the_engine_cannot_run_is_refused_with_the_reason(change, message):
    from atoma_infer_amd.config.base import ConfigError
    from atoma_infer_amd.config.duduvik import DuduvikConfig
    c = copy.deepcopy(DUD_A)
    change(c)
    with pytest.raises(ConfigError, match=message):
        DuduvikConfig.from_dict(c)


def test_the_chunk_plan_lists_every_token_of_a_long_entry_once():
    from atoma_infer_amd.kernels import ops
    arr, (nc, nl, short) = ops.linear_attention_plan([3, 130, 39, 64, 40], 40)
    rows = arr.reshape(-1, 4).tolist()
    assert (nc, nl, short) == (5, 3, 39) == (len(rows) - nl, 3, 39)
    assert rows[:nc] == [[1, 3, 64, 0], [1, 67, 64, 0], [1, 131, 2, 0], [3, 172, 64, 0], [4, 236, 40, 0]]
    assert rows[nc:] == [[1, 0, 3, 0], [3, 3, 1, 0], [4, 4, 1, 0]]
    assert ops.linear_attention_plan([1, 1], 40)[1] == (0, 0, 1)
    assert ops.linear_attention_plan([100], 0)[1] == (0, 0, 100)
    assert ops.linear_attention_plan([64, 40], 40)[1] == (2, 2, 0)


def test_gate_activations_that_do_not_exist_are_refused():
    from atoma_infer_amd.kernels import ops
    for bad in ("tanh", ("silu", 1.0), "clamped_sigmoid", ("clamped_sigmoid", 1.0), ("clamped_sigmoid", 0.0, 1.7)):
        with pytest.raises(ValueError, match="not supported"):
            ops.gate_activation(bad)
    assert ops.gate_activation("relu")[0] == 2 and ops.gate_activation(("clamped_sigmoid", 2, 1.5)) == (3, 2.0, 1.5)


def test_parts_refuse_what_they_cannot_mean():
    from atoma_infer_amd.parts.base import make_part
    la = dict(width=8, heads=2, dim=4, vdim=4, norm_eps=1e-5)
    for bad, message in (({}, "one of the two"), ({"decay": [0.5, 0.5], "tau": 2.0}, "one of the two"),
                         ({"decay": [0.5]}, "decays for"), ({"tau": 2.0, "rotary_dim": 2}, "no rotation"),
                         ({"decay": [0.5, 0.5], "rotary_dim": 6}, "fit the 4")):
        with pytest.raises(ValueError, match=message):
            make_part("mixer", "decayed_linear_attention", **la, **bad)
    ex = dict(width=8, intermediate=4, experts=3, top=2)
    for bad, message in (({"weigh": "twice"}, "'input' or its 'output'"), ({"score": "max"}, "scores are one of"),
                         ({"score": "softmax_chosen", "correction": True}, "does not have")):
        with pytest.raises(ValueError, match=message):
            make_part("feed_forward", "routed_experts", **ex, **bad)
