"""Host-side tests of the Tutedra design that need no GPU: hand-derived values of the plain restatement (tests/tutedra_ref.py), one per
mechanism, and the native loader's refusals that come before any device call."""
import math

import numpy as np
import pytest

import __graft_entry__ as ge
import tutedra_ref as R


@pytest.fixture(scope="module")
def hy():
    from importlib import import_module
    ge.load_package()
    return import_module(ge.PKG_NAME + ".hybrid")


def test_ref_pair_rows_by_hand():
    b = {"buckets": 10, "mul_prev": 3, "mul_cur": 4}
    assert R.bigram_rows([2, 5, 9], b) == [10, (2 * 3 + 5 * 4) % 10, (5 * 3 + 9 * 4) % 10] == [10, 6, 1]
    w = {"embed": np.arange(10.0)[:, None], "bigram": 100.0 * np.arange(11.0)[:, None]}
    assert list(R.embedding([2, 5, 9], w, {"embedding": {"bigram": b}})[:, 0]) == [1002.0, 605.0, 109.0]
    assert list(R.embedding([2, 5], w, {})[:, 0]) == [2.0, 5.0]


def test_ref_token_shift_reads_the_unshifted_row():
    h = np.array([[1.0, 2.0], [3.0, 6.0], [5.0, 0.0]])
    mu = np.array([1.0, 0.25])
    assert np.allclose(R.token_shift(h, mu), [[0.0, 1.5], [1.0, 5.0], [3.0, 1.5]])


def test_ref_channel_gates_are_a_product_of_the_gates_since():
    rng = np.random.default_rng(0)
    T, H, D, V = 5, 2, 3, 4
    q, v, f = rng.standard_normal((T, H, D)), rng.standard_normal((T, H, V)), rng.uniform(0.0, 1.0, (T, H, D))
    want = np.zeros((T, H, V))
    for t in range(T):
        for s in range(t + 1):
            keep = np.prod(f[s + 1:t + 1], axis=0) * (1.0 - f[s])
            want[t] += (q[t] * keep).sum(axis=1)[:, None] * v[s]
    assert np.allclose(R.channel_gated_memory(q, f, v), want)


def test_ref_hgrn2_by_hand():
    # one head, one channel, one value, one input: with W_f = 0 and f.b = 0 the gate is l + (1 - l) / 2 = 0.75
    p = {"q": np.array([[1.0]]), "f": np.array([[0.0]]), "f.b": np.array([0.0]), "lower": np.array([0.5]), "v": np.array([[2.0]]), "norm": np.array([3.0]), "o": np.array([[1.0]])}
    h = np.array([[1.0], [-1.0]])
    s0 = 0.25 * 2.0
    s1 = 0.75 * s0 + 0.25 * -2.0
    o = np.array([s0 / (1 + math.exp(-1.0)), s1 * -1.0 / (1 + math.exp(1.0))])
    assert np.allclose(R.hgrn2(h, p, {"heads": 1, "dim": 1, "vdim": 1}, 0.5)[:, 0], 3.0 * o / np.sqrt(o ** 2 + 0.5))


def test_ref_exponential_gates_start_from_a_maximum_of_zero():
    one = np.ones((2, 1, 1))
    i, f = np.array([[-3.0], [2.0]]), np.array([[-1.0], [-0.5]])
    o = R.exp_gated_memory(one, one, 5.0 * one, i, f)
    # token 0: m = max(-1, -3) = -1, S = e^(-3 + 1) 5, n = e^-2, bound e^1
    assert np.isclose(o[0, 0, 0], 5 * math.exp(-2) / (math.exp(1.0) + 1e-6))
    # token 1: m = max(-1.5, 2) = 2: S = e^(-3.5) S + 5, n = e^(-3.5) n + 1 > e^-2
    n = math.exp(-3.5) * math.exp(-2) + 1
    assert np.isclose(o[1, 0, 0], 5 * n / (n + 1e-6))
    zi, zf = R.log_gates(np.array([[2.0]]), {"i": np.array([[1.0]]), "i.b": np.array([1.0]), "f": np.array([[-1.0]]), "f.b": np.array([0.5])}, 4.0)
    assert np.isclose(zi[0, 0], 4 * math.tanh(0.75)) and np.isclose(zf[0, 0], -math.log(1 + math.exp(-4 * math.tanh(-1.5 / 4))))


def test_ref_short_convolution_ends_at_the_current_token():
    u = np.array([[1.0], [10.0], [100.0], [1000.0]])
    assert list(R.short_conv(u, np.array([[5.0, 3.0, 2.0]]))[:, 0]) == [2.0, 23.0, 235.0, 2350.0]
    assert list(R.short_conv(u, np.array([[7.0]]))[:, 0]) == [7.0, 70.0, 700.0, 7000.0]


def test_ref_frequencies_by_wavelength():
    # base 16, 8 entries: f = 1, 1/2, 1/4, 1/8; original / wavelength = original f / (2 pi) = 8, 4, 2, 1 for original = 16 pi
    rot = {"dims": 8, "base": 16.0, "scaling": {"factor": 10.0, "high": 5.0, "low": 1.5, "original": 16 * math.pi}}
    f = lambda x, s: (1 - s) * x / 10 + s * x
    assert np.allclose(R.frequencies(rot), [1.0, f(0.5, 2.5 / 3.5), f(0.25, 0.5 / 3.5), 0.0125])
    assert np.allclose(R.frequencies({"dims": 8, "base": 16.0}), [1.0, 0.5, 0.25, 0.125])


def test_ref_values_are_the_keys_before_norm_and_turn():
    # one head of two entries, both turned; W_q = 0: all scores are equal and the output is the mean of the convolved keys so far
    c = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0, "conv": 2, "rot": {"dims": 2, "base": 10.0}}
    p = {"q": np.zeros((2, 2)), "k": np.eye(2), "q.conv": np.ones((2, 2)), "k.conv": np.array([[1.0, 1.0], [0.0, 2.0]]), "q.norm": np.ones(2), "k.norm": np.full(2, 9.0), "o": np.eye(2)}
    h = np.array([[1.0, 1.0], [2.0, 3.0], [4.0, 5.0]])
    v = np.array([[1.0, 2.0], [3.0, 6.0], [6.0, 10.0]])
    assert np.allclose(R.attention(h, p, c, 1e-6), np.cumsum(v, axis=0) / np.array([[1], [2], [3]]))


def test_ref_attention_norms_turns_and_scales():
    # two query heads on one key head; position 1's scores by hand
    c = {"heads": 2, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 0.5, "rot": {"dims": 2, "base": 10.0}}
    p = {"q": np.array([[1.0, 0], [0, 1], [0, 1], [1, 0]]), "k": np.eye(2), "q.norm": np.array([2.0, 1.0]), "k.norm": np.array([1.0, 3.0]), "o": np.eye(4)}
    h = np.array([[1.0, 0.0], [3.0, 4.0]])
    rms = math.sqrt(12.5)
    spin = lambda u, v: (u * math.cos(1) - v * math.sin(1), v * math.cos(1) + u * math.sin(1))
    k0, k1 = np.array([math.sqrt(2), 0.0]), np.array(spin(3 / rms, 3 * 4 / rms))
    out = R.attention(h, p, c, 0.0)
    for hd, (a, b) in enumerate(((3.0, 4.0), (4.0, 3.0))):
        q = np.array(spin(2 * a / rms, b / rms))
        s = np.exp(0.5 * np.array([q @ k0, q @ k1]))
        assert np.allclose(out[1, 2 * hd:2 * hd + 2], (s[0] * h[0] + s[1] * h[1]) / s.sum())


def test_ref_polynomial_activation_by_hand():
    z = np.array([[1.0, -2.0]])
    n = [math.sqrt(2.5 + 0.1), math.sqrt(8.5 + 0.1), math.sqrt(32.5 + 0.1)]
    want = [2 / n[0] + 3 / n[1] + 5 / n[2] + 7, -4 / n[0] + 12 / n[1] - 40 / n[2] + 7]
    assert np.allclose(R.poly_norm(z, [2.0, 3.0, 5.0, 7.0], 0.1)[0], want)


def test_ref_router_by_hand():
    c = {"router": {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}}}
    s = np.array([0.9, 0.1, 0.5, 0.55, 0.2, 0.3])
    p = {"router": np.log(s / (1 - s))[:, None], "correction": np.zeros(6)}
    choice, w = R.route(np.ones((1, 1)), p, c)
    assert list(choice[0]) == [3, 2] and np.allclose(w[0], [0.55, 0.5])             # 0.5 + 0.55 beats 0.9 + 0.1; the weights are the plain scores
    p["correction"] = np.array([-1.0, -1.0, -1.0, -1.0, -0.1, -0.1])
    choice, w = R.route(np.ones((1, 1)), p, c)
    assert list(choice[0]) == [5, 4] and np.allclose(w[0], [0.3, 0.2])
    p["correction"] = np.array([-2.0] * 6)                                         # every choice score negative: closed experts stay closed
    assert list(R.route(np.ones((1, 1)), p, c)[0][0]) == [3, 2]
    tie = R.route(np.zeros((1, 1)), dict(p, correction=np.zeros(6)), c)[0][0]
    assert list(tie) == [0, 1]                                                     # ties: the lowest group, the lowest expert


def test_ref_layer_scales_and_norms_around_zero():
    """An attention layer whose output projection is zero leaves the feed-forward alone to move x."""
    cfg = {"vocab": 3, "width": 2, "norm": {"eps": 1e-6},
           "layers": [{"type": "attention", "mixer": {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0}, "mlp": {"kind": "moe", "expert": {"ff": 1},
                       "router": {"experts": 1, "top": 1}, "shared": {"ff": 1}}}]}
    w = {"embed": np.array([[1.0, 0.5], [0.0, 1.0], [2.0, 2.0]]), "l0.norm1": np.zeros(2), "l0.shift": np.ones(2), "l0.mix.q": np.eye(2), "l0.mix.k": np.eye(2),
         "l0.mix.q.norm": np.ones(2), "l0.mix.k.norm": np.ones(2), "l0.mix.o": np.zeros((2, 2)), "l0.ls1": np.ones(2), "l0.ls2": np.array([0.5, 10.0]),
         "l0.norm2": np.array([1.0, -0.5]), "l0.mlp.e0.up": np.array([[1.0, 0.0]]), "l0.mlp.e0.down": np.array([[1.0], [1.0]]), "l0.mlp.router": np.array([[0.0, 0.0]]),
         "l0.mlp.correction": np.array([5.0]), "l0.mlp.shared.up": np.array([[0.0, -1.0]]), "l0.mlp.shared.down": np.array([[1.0], [1.0]]), "l0.mlp.shared.sg": np.array([[0.0, 0.0]]),
         "final.norm": np.array([0.0, 1.0])}
    hn = np.array([2.0, 2.0]) / math.sqrt(4 + 1e-6) * np.array([2.0, 0.5])
    x = np.array([2.0, 2.0]) + np.array([0.5, 10.0]) * 0.5 * hn[0] ** 2             # the expert at score 1/2; the shared expert's relu passes nothing
    z = w["embed"] @ (x / math.sqrt((x ** 2).mean() + 1e-6) * np.array([1.0, 2.0]))
    assert np.allclose(R.forward(cfg, w, [2])[0], z)


def test_native_loader_refuses_before_touching_a_device(hy, tmp_path):
    L = hy.hip.lib()
    base = '{"architecture": "Tutedra", "vocab": 8, "width": 8, "norm": {"eps": 1e-6}%s, "layers": [%s]}'
    at = '{"type": "attention", "mixer": {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": %d, "scale": 1.0%s}%s}'
    hg = '{"type": "hgrn2", "mixer": {"heads": 2, "dim": 4, "vdim": 4}%s}'
    mo = ', "mlp": {"kind": "moe", "expert": {"ff": 4}, "router": {"experts": 4, "top": %d, "groups": {"count": %d, "keep": %d}}}'
    for i, text in enumerate(['{"architecture": "Tutedra", "vocab": 8}', base % ("", '{"type": "lightning", "mixer": {"heads": 1, "dim": 1, "vdim": 1}}'), base % ("", '{"type": "hgrn2"}'),
                              base % (', "embedding": {"bigram": {"buckets": 5}}', hg % ""), base % (', "embedding": {"bigram": {"buckets": 0, "mul_prev": 1, "mul_cur": 1}}', hg % ""),
                              base % ("", at % (5, "", "")),                                              # values are keys: another size
                              base % ("", at % (4, ', "rot": {"dims": 4}', "")),                          # no base
                              base % ("", at % (4, ', "rot": {"dims": 4, "base": 10.0, "scaling": {"factor": 2.0}}', "")),
                              base % ("", at % (4, ', "rot": {"dims": 6, "base": 10.0}', "")),
                              base % ("", '{"type": "mlstm", "mixer": {"heads": 1, "dim": 4, "vdim": 4}}'),  # no gate_cap
                              base % ("", hg % ', "mlp": {"kind": "glu", "ff": 4}'), base % ("", hg % ', "mlp": {"kind": "moe", "expert": {"ff": 4}}'),
                              base % ("", hg % (mo % (2, 3, 1))), base % ("", hg % (mo % (3, 2, 1))), base % ("", hg % (mo % (2, 2, 3)))]):
        d = tmp_path / ("c%d" % i)
        d.mkdir()
        (d / "config.json").write_text(text)
        (d / "model.safetensors").write_bytes((2).to_bytes(8, "little") + b"{}")
        assert L.gl3_is_model_dir(str(d).encode()) == 1
        with pytest.raises(hy.hip.Gl3Error) as e:
            hy.HybridPlan.from_dir(str(d))
        assert e.value.code in (hy.hip.E_ARG, hy.hip.E_UNSUPPORTED) and len(str(e.value)) > 20, text
