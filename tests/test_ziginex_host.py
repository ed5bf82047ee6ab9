"""Host-side tests of the Ziginex design that need no GPU: hand-derived values of the plain restatement (tests/ziginex_ref.py), one per
mechanism, and the native loader's refusals that come before any device call."""
import math

import numpy as np
import pytest

import __graft_entry__ as ge
import ziginex_ref as R


@pytest.fixture(scope="module")
def hy():
    from importlib import import_module
    ge.load_package()
    return import_module(ge.PKG_NAME + ".hybrid")


def test_ref_turn_pairs():
    x = np.array([[[1.0, 2.0, 3.0, 4.0, 9.0]]] * 2)
    rot = {"base": 100.0, "dims": 4}                              # frequencies 1 and 0.1
    f, mul = R.frequencies(rot)
    assert np.allclose(f, [1.0, 0.1]) and mul == 1.0
    inter, half = R.turn(x, [0, 3], rot, True)[1, 0], R.turn(x, [0, 3], rot, False)[1, 0]
    c, s, c1, s1 = math.cos(3.0), math.sin(3.0), math.cos(0.3), math.sin(0.3)
    assert np.allclose(inter, [c - 2 * s, 2 * c + s, 3 * c1 - 4 * s1, 4 * c1 + 3 * s1, 9.0])
    assert np.allclose(half, [c - 3 * s, 2 * c1 - 4 * s1, 3 * c + s, 4 * c1 + 2 * s1, 9.0])
    assert np.allclose(R.turn(x, [0, 3], rot, True)[0], x[0])


def test_ref_blended_frequencies():
    # n = 8, base e^4: where(t) = ln(original / (2 pi t)); original = 2 pi e^3: fast = 1 / e -> 4 -> hi clipped below, fast = e -> 2, slow = 1 -> 3
    rot = {"base": math.exp(4.0), "dims": 8, "scaling": {"factor": 4.0, "original": 2 * math.pi * math.exp(3.0), "fast": math.exp(1.5), "slow": math.exp(-0.5)}}
    f, mul = R.frequencies(rot)                                   # lo = floor(1.5) = 1, hi = ceil(3.5) = 4: ramps 0, 0, 1/3, 2/3
    base = [math.exp(-i) for i in range(4)]
    assert np.allclose(f, [base[0], base[1], base[2] * (2 / 3 + 1 / 12), base[3] * (1 / 3 + 2 / 12)])
    assert np.isclose(mul, 0.1 * math.log(4.0) + 1.0)
    same = dict(rot["scaling"], fast=1e9, slow=math.exp(9.0))     # lo = 0, hi = -6 clipped to max(hi - lo, 0.001): pair 0 stays, the others divide
    assert np.allclose(R.frequencies(dict(rot, scaling=same))[0], [base[0]] + [b / 4 for b in base[1:]])


def test_ref_sink_counts_once():
    s = np.array([[0.0, math.log(2.0), -np.inf]])
    assert np.allclose(R.sink_softmax(s, np.array([math.log(5.0)])), [[1 / 8, 2 / 8, 0.0]])
    assert np.allclose(R.sink_softmax(s + 700, np.array([-1000.0])), [[1 / 3, 2 / 3, 0.0]])


def test_ref_chunks_are_counted_from_the_first_position():
    seen = R.chunk_mask(7, 3)
    assert [list(np.nonzero(r)[0]) for r in seen] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    assert list(np.nonzero(R.chunk_mask(7, 0)[5])[0]) == [0, 1, 2, 3, 4, 5]
    assert list(np.nonzero(R.chunk_mask(7, 3, chunk_shift=1)[2])[0]) == [2]          # the runs' edges moved one token earlier


def test_ref_scores_are_tempered_capped_then_mixed():
    q = np.array([[[1.0], [3.0]]])                                # one token, two heads, one key head
    k = np.array([[[2.0]]])
    c = {"scale": 0.5, "softcap": 4.0}
    s = R.head_scores(q, k, c, np.array([1.0, 2.0]))
    assert np.allclose(s[:, 0, 0], [4 * math.tanh(1.0 / 4), 4 * math.tanh(6.0 / 4)])
    assert np.allclose(R.head_scores(q, k, {"scale": 0.5}, np.array([1.0, 2.0]))[:, 0, 0], [1.0, 6.0])
    # one token: its weight is e^m / (e^m + e^sink) with m the mixed score
    one = np.array([[1.0]])
    p = {"q": np.array([[1.0], [1.0]]), "k": one, "v": np.array([[5.0]]), "q.norm": np.array([2.0]), "k.norm": np.array([3.0]), "temp": np.array([1.0, 0.5]),
         "talk": np.array([[0.0, 1.0], [2.0, -1.0]]), "sink": np.array([0.3, -0.2]), "o": np.eye(2)}
    cfg = {"heads": 2, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 0.25, "softcap": 2.0}
    out = R.mixed_attention(np.array([[7.0]]), p, cfg, 0.0)       # q = 2, k = 3 whatever the input's size
    s = [2 * math.tanh(1.5 / 2), 2 * math.tanh(0.75 / 2)]
    m = [s[1], 2 * s[0] - s[1]]
    assert np.allclose(out, [[35 * math.exp(m[0]) / (math.exp(m[0]) + math.exp(0.3)), 35 * math.exp(m[1]) / (math.exp(m[1]) + math.exp(-0.2))]])


def test_ref_delta_rule_replaces_what_a_key_recalls():
    k = np.array([[[1.0, 0.0]], [[1.0, 0.0]], [[0.0, 1.0]]])
    v = np.array([[[5.0]], [[2.0]], [[7.0]]])
    ones = np.ones((3, 1))
    o = R.delta_memory(k, k, v, ones, ones)
    assert np.allclose(o[:, 0, 0], [5.0, 2.0, 7.0])               # beta = 1, no decay: the key's value is replaced, not added
    q = np.array([[[1.0, 1.0]]] * 3)
    o = R.delta_memory(q, k, v, np.array([[1.0], [0.5], [0.5]]), np.array([[1.0], [0.25], [1.0]]))
    second = 0.5 * 5 + 0.25 * (2 - 0.5 * 5)                       # the decay comes first, the read-out sees the current write
    assert np.allclose(o[:, 0, 0], [5.0, second, 0.5 * second + 7.0])


def test_ref_delta_gates_and_unit():
    g, b = R.delta_gates(np.array([[2.0]]), {"a": np.array([[1.0]]), "b": np.array([[-1.0]]), "A_log": np.array([0.5]), "dt_bias": np.array([-1.0])})
    assert np.isclose(g[0, 0], math.exp(-math.exp(0.5) * math.log(1 + math.exp(1.0)))) and np.isclose(b[0, 0], 1 / (1 + math.exp(2.0)))
    assert np.allclose(R.unit(np.array([3.0, 4.0])), np.array([3.0, 4.0]) / math.sqrt(25 + 1e-6))


def test_ref_short_convolution_ends_at_the_current_token():
    u = np.array([[1.0], [10.0], [100.0], [1000.0]])
    assert list(R.short_conv(u, np.array([[5.0, 3.0, 2.0]]))[:, 0]) == [2.0, 23.0, 235.0, 2350.0]


def test_ref_router_takes_groups_by_their_largest_and_keeps_plain_scores():
    z = np.log(np.array([0.05, 0.2, 0.1, 0.25, 0.15, 0.25]))
    p = {"router": z[:, None], "correction": np.array([-1.0, -0.6, -0.3, -0.9, -0.2, -2.0])}
    c = {"router": {"experts": 4, "identity": 2, "top": 2, "groups": {"count": 3, "keep": 1}}}
    choice, w = R.route(np.array([[1.0]]), p, c)                  # choice scores -0.95 -0.4 | -0.2 -0.65 | -0.05 -1.75: the last group, both identity
    assert list(choice[0]) == [4, 5] and np.allclose(w[0], [0.15, 0.25])
    c["router"]["groups"] = None
    choice, w = R.route(np.array([[1.0]]), p, c)
    assert list(choice[0]) == [4, 2] and np.allclose(w[0], [0.15, 0.1])


def test_ref_identity_choice_returns_the_input():
    p = {"router": np.zeros((2, 2)), "correction": np.array([0.0, 1.0]), "e0.gate": np.ones((1, 2)), "e0.up": np.ones((1, 2)), "e0.down": np.ones((2, 1))}
    c = {"router": {"experts": 1, "identity": 1, "top": 1}}
    assert np.allclose(R.moe_ff(np.array([[3.0, -8.0]]), p, c), [[1.5, -4.0]])


def test_ref_token_input_by_hand():
    y = R.token_input(np.array([[1.0, 2.0]]), np.array([[3.0]]), np.array([[1.0, 1.0]]), np.array([[1.0], [-2.0]]), np.array([10.0, 100.0]), 0.5)
    g = 3 * R.gelu_tanh(3.0)
    r = math.sqrt((g * g + 4 * g * g) / 2 + 0.5)
    assert np.allclose(y, [[10 * g / r, -200 * g / r]])
    assert np.isclose(R.gelu_tanh(1.0), 0.8411919906)


def test_ref_sublayers_read_the_residual_and_norms_stand_behind():
    cfg = {"vocab": 3, "width": 2, "norm": {"eps": 0.25}, "layers": [{"type": "latent_attention", "mlp": {"kind": "dense", "ff": 1},
           "mixer": {"heads": 1, "dim": 1, "vdim": 1, "kv_rank": 1, "q_rank": 1, "scale": 1.0}}]}
    w = R.to_f64(R.random_weights(cfg, 3))
    taps = []
    R.forward(cfg, w, [2], taps)
    x = w["embed"][[2]]
    y = R.latent_attention(x, R.sub(w, "l0.mix."), cfg["layers"][0]["mixer"], 0.25)
    x = x + y / np.sqrt((y ** 2).mean() + 0.25) * w["l0.norm1"]
    f = R.silu(x @ w["l0.mlp.gate"].T) * (x @ w["l0.mlp.up"].T) @ w["l0.mlp.down"].T
    x = x + f / np.sqrt((f ** 2).mean() + 0.25) * w["l0.norm2"]
    assert np.allclose(taps[0], x)


def test_ref_prefix_property():
    """Causal: the first tokens' logits do not depend on what follows."""
    cfg = {"vocab": 31, "width": 16, "norm": {"eps": 1e-5}, "token_side": {"dim": 3}, "layers": [
        {"type": "parallel", "mlp": None, "mixer": {"left": {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 3, "scale": 0.5, "softcap": 5.0, "mask": {"size": 4},
                                                             "rot": {"base": 10.0, "dims": 2}},
                                                    "right": {"heads": 2, "kv_heads": 1, "dim": 3, "vdim": 4, "conv": 3}}}]}
    w = R.to_f64(R.random_weights(cfg, 1))
    t = np.random.default_rng(0).integers(0, 31, 12)
    assert np.allclose(R.forward(cfg, w, t)[:7], R.forward(cfg, w, t[:7]))


def test_shapes_of_the_random_folder_agree(hy):
    """The two independent lists of tensor names and shapes (the framework's random folders, the restatement's) are the same."""
    import bench
    for z in bench.ZIGINEX_SIZES.values():
        cfg = bench.ziginex_config(z)
        assert hy.ziginex_tensor_shapes(cfg) == R.tensor_shapes(cfg)


@pytest.mark.parametrize("change", [
    lambda c: c.pop("width"), lambda c: c.pop("norm"), lambda c: c.update(layers=[]), lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][0]["mixer"].pop("right"),
    lambda c: c["layers"][0]["mixer"]["left"].pop("scale"), lambda c: c["layers"][0]["mixer"]["left"].update(heads=3), lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0),
    lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=3), lambda c: c["layers"][0]["mixer"]["right"].pop("conv"), lambda c: c["layers"][0]["mixer"]["right"].update(heads=3),
    lambda c: c["layers"][0]["mlp"].update(kind="wide"), lambda c: c["layers"][0]["mlp"]["router"].update(top=4), lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4),
    lambda c: c["layers"][0]["mixer"]["left"].update(heads=130, kv_heads=2), lambda c: c["layers"][1]["mixer"].update(q_rank=0), lambda c: c["layers"][1]["mixer"]["rot"].update(dims=2)])
def test_loader_refuses_bad_configurations(hy, tmp_path, change):
    cfg = {"architecture": "Ziginex", "vocab": 9, "width": 8, "norm": {"eps": 1e-5}, "layers": [
        {"type": "parallel", "mixer": {"left": {"heads": 2, "kv_heads": 2, "dim": 4, "vdim": 4, "scale": 0.5, "mask": {"size": 4}, "rot": {"base": 10.0, "dims": 2}},
                                       "right": {"heads": 2, "kv_heads": 2, "dim": 3, "vdim": 4, "conv": 3}},
         "mlp": {"kind": "moe", "expert": {"ff": 4}, "router": {"experts": 4, "identity": 2, "top": 2, "groups": {"count": 2, "keep": 1}}}},
        {"type": "latent_attention", "mlp": None, "mixer": {"heads": 2, "dim": 4, "rot_dim": 4, "vdim": 4, "kv_rank": 5, "q_rank": 3, "scale": 1.0, "rot": {"base": 10.0, "dims": 4}}}]}
    change(cfg)
    hy.save_model_dir(str(tmp_path / "bad"), cfg, {"final.norm": np.ones(8, np.float32)})
    with pytest.raises(hy.hip.Gl3Error) as e:
        hy.HybridPlan.from_dir(str(tmp_path / "bad"))
    assert e.value.code in (hy.hip.E_ARG, hy.hip.E_UNSUPPORTED), e.value
