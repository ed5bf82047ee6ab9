"""The Tutedra design (layer-list family: token-pair embedding, token shift, layer scales; HGRN2, mLSTM and attention layers with short
convolutions; polynomial feed-forward; relu^2 experts chosen among groups) on the GPU against the plain float64 restatement in
tests/tutedra_ref.py.

Every test makes its own small configuration and random bfloat16-representable weights, writes them as a model folder and loads that
through the product's loader.  float32 plans are held to 2e-4 (root mean square of the logit difference over the root mean square of
the logits), bfloat16 plans to 6e-2.  Where random weights would hide a fault, the first attention layer is turned into a look-up (W_q
repeats W_k, the rotated entries of q are zero), so that a token attends to the earlier occurrences of the same token wherever they
are; hiding one key, or moving the causal edge by one, then moves the logits by far more than the bound, and the tests check that on
the restatement itself.
"""
import copy
import json
import os
import subprocess

import numpy as np
import pytest

import __graft_entry__ as ge
import tutedra_ref as R

pytestmark = pytest.mark.gpu
F32_TOL, BF16_TOL = 2e-4, 6e-2


@pytest.fixture(scope="module")
def hy():
    from importlib import import_module
    ge.load_package()
    return import_module(ge.PKG_NAME + ".hybrid")


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, shared=40, groups=(3, 2)):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r, "shared": {"ff": shared} if shared else None}


def hgrn(heads=3, dim=16, vdim=24, mlp="dense"):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": dense() if mlp == "dense" else mlp}


def mls(heads=3, dim=12, vdim=20, cap=9.0, mlp="dense"):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": dense() if mlp == "dense" else mlp}


WAVES = {"factor": 5.0, "high": 4.0, "low": 1.5, "original": 96}


def att(heads=4, kv_heads=2, dim=20, rot=12, conv=4, base=600.0, scaling=WAVES, scale=0.25, mlp="dense"):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if conv:
        m["conv"] = conv
    if rot:
        m["rot"] = {"base": base, "dims": rot}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    return {"type": "attention", "mixer": m, "mlp": dense() if mlp == "dense" else mlp}


def config(layers, width=88, vocab=131, eps=1e-5, bigram=(211, 31, 7)):
    c = {"architecture": "Tutedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if bigram:
        c["embedding"] = {"bigram": {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}}
    return c


class Model:
    def __init__(self, hy, tmp_path, cfg, seed, tweak=None):
        self.cfg, self.w = cfg, R.random_weights(cfg, seed)
        if tweak:
            tweak(cfg, self.w)
            self.w = {k: R.bf16_round(v) for k, v in self.w.items()}
        self.dir = str(tmp_path / ("m%d" % seed))
        hy.save_model_dir(self.dir, cfg, self.w)
        self.w64 = R.to_f64(self.w)
        self.hy = hy

    def plan(self, dtype="float32", **kw):
        return self.hy.HybridPlan.from_dir(self.dir, dtype=dtype, **kw)

    def ref(self, tokens, **kw):
        return R.forward(self.cfg, self.w64, tokens, **kw)

    def tokens(self, n, seed=0, vocab=None):
        toks = np.random.default_rng(1000 + seed).integers(0, vocab or self.cfg["vocab"], n).astype(np.int32)
        return toks, self.ref(toks)


def err_rows(got, want):
    d = got - want
    d = d - d.mean(axis=-1, keepdims=True)
    w = want - want.mean(axis=-1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=-1)) / np.sqrt((w ** 2).mean())


def err(got, want):
    return float(err_rows(got, want).max())


def bf16_ok(m, toks, got, ref=None):
    """A bfloat16 plan is held to the restatement with its products' inputs rounded alike: then both choose the same experts, but for a token
    whose choice scores tie to the last bits (that one, and through state and cache those after it, leave by more than rounding; up to five
    routers in a row here): three rows in four.  Against the unrounded restatement the median row is held to the bound."""
    refb = m.ref(toks, round_inputs=True)
    ref = m.ref(toks) if ref is None else ref
    return np.quantile(err_rows(got, refb[:len(got)]), 0.75) < BF16_TOL / 3 and np.median(err_rows(got, ref[:len(got)])) < BF16_TOL


def whole(plan, toks, want=None):
    want = list(range(len(toks))) if want is None else want
    s = plan.acquire()
    out = plan.step(s, toks, 0, want)
    plan.release(s)
    return out


def stepwise(plan, toks, sizes):
    """The sequence in steps of the given sizes (the last size repeats), all logits."""
    s = plan.acquire()
    rows, p, i = [], 0, 0
    while p < len(toks):
        c = min(sizes[min(i, len(sizes) - 1)], len(toks) - p)
        rows.append(plan.step(s, toks[p:p + c], p, list(range(c))))
        p += c
        i += 1
    plan.release(s)
    return np.concatenate(rows)


# ---- each mechanism alone: one or two layers, the mechanism's sizes and constants varied ---------------------------------------------
SINGLE = [
    ("hgrn2_plain", [hgrn()], {}),
    ("hgrn2_no_feed_forward", [hgrn(mlp=None)], {}),
    ("hgrn2_one_wide_head", [hgrn(heads=1, dim=72, vdim=130)], {}),
    ("hgrn2_many_small_heads", [hgrn(heads=11, dim=4, vdim=6)], {}),
    ("hgrn2_one_channel", [hgrn(heads=2, dim=1, vdim=3)], {}),
    ("hgrn2_one_value", [hgrn(heads=2, dim=5, vdim=1)], {}),
    ("hgrn2_long_keys", [hgrn(heads=1, dim=300, vdim=20, mlp=None)], {}),
    ("mlstm_plain", [mls()], {}),
    ("mlstm_small_cap_one_head", [mls(heads=1, dim=40, vdim=70, cap=1.5, mlp=None)], {}),
    ("mlstm_many_heads", [mls(heads=9, dim=5, vdim=7, cap=20.0)], {}),
    ("attention_plain", [att()], {}),
    ("attention_no_feed_forward", [att(mlp=None)], {}),
    ("attention_one_head", [att(heads=1, kv_heads=1, dim=48, rot=48)], {}),
    ("attention_one_key_head_for_many", [att(heads=12, kv_heads=1, dim=10, rot=2)], {}),
    ("attention_a_key_head_each", [att(heads=5, kv_heads=5, dim=16)], {}),
    ("attention_no_rotation", [att(rot=0)], {}),
    ("attention_plain_frequencies", [att(scaling=None, base=10000.0)], {}),
    ("attention_all_waves_kept", [att(scaling={"factor": 8.0, "high": 4.0, "low": 1.0, "original": 100000})], {}),
    ("attention_all_waves_divided", [att(scaling={"factor": 8.0, "high": 4.0, "low": 1.0, "original": 3})], {}),
    ("attention_waves_without_a_blend", [att(scaling={"factor": 8.0, "high": 2.0, "low": 2.0, "original": 96})], {}),
    ("attention_no_convolution", [att(conv=0)], {}),
    ("attention_one_tap", [att(conv=1)], {}),
    ("attention_two_taps", [att(conv=2)], {}),
    ("attention_many_taps", [att(conv=11)], {}),
    ("attention_large_heads", [att(heads=2, kv_heads=1, dim=192, rot=64, scale=0.08)], {}),
    ("dense_odd_width", [hgrn(mlp=dense(33))], {}),
    ("dense_wide", [hgrn(mlp=dense(1500))], {}),
    ("dense_one", [hgrn(mlp=dense(1))], {}),
    ("dense_wider_than_the_kept_part", [hgrn(heads=1, dim=8, vdim=8, mlp=dense(16500))], {"width": 24, "vocab": 40, "n": 20}),
    ("experts_plain", [hgrn(mlp=moe())], {}),
    ("experts_without_shared", [mls(mlp=moe(shared=0))], {}),
    ("experts_without_groups", [hgrn(mlp=moe(groups=None))], {}),
    ("experts_one_group", [hgrn(mlp=moe(groups=(1, 1)))], {}),
    ("experts_groups_of_one", [hgrn(mlp=moe(experts=7, top=3, groups=(7, 4)))], {}),
    ("experts_all_of_the_kept_groups", [att(mlp=moe(experts=12, top=6, groups=(4, 2)))], {}),
    ("experts_all_groups_kept", [att(mlp=moe(experts=8, top=3, groups=(4, 4)))], {}),
    ("experts_many", [att(mlp=moe(experts=140, top=9, ff=8, shared=8, groups=(70, 5)))], {}),
    ("experts_one", [hgrn(mlp=moe(experts=1, top=1, groups=(1, 1)))], {}),
    ("no_pair_embedding", [hgrn(), att()], {"bigram": None}),
    ("one_pair_bucket", [hgrn()], {"bigram": (1, 3, 5)}),
    ("pair_products_past_32_bits", [hgrn()], {"bigram": (997, 1900000001, 1700000009)}),
    ("widths_not_multiples_of_four", [hgrn(heads=3, dim=10, vdim=9, mlp=dense(17)), att(heads=6, kv_heads=3, dim=9, rot=6, conv=3, mlp=moe(ff=9, shared=13)),
                                      mls(heads=3, dim=7, vdim=5, mlp=None)], {"width": 75, "vocab": 53}),
    ("wide_model", [hgrn(heads=2, dim=32, vdim=32, mlp=dense(2048)), att(heads=4, kv_heads=2, dim=32, rot=16, mlp=moe(ff=64, shared=2048)), mls(heads=2, dim=32, vdim=32, mlp=None)],
     {"width": 1024, "vocab": 64, "n": 40}),
    ("width_past_the_registers", [hgrn(heads=1, dim=8, vdim=8, mlp=None), att(heads=1, kv_heads=1, dim=8, rot=4, mlp=dense(16))], {"width": 8300, "vocab": 40, "n": 40}),
]


@pytest.mark.parametrize("name,layers,kw", SINGLE, ids=[s[0] for s in SINGLE])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_single_mechanism(hy, tmp_path, name, layers, kw, dtype):
    kw = dict(kw)
    n = kw.pop("n", 75)
    m = Model(hy, tmp_path, config(copy.deepcopy(layers), **kw), seed=len(name))
    toks, ref = m.tokens(n)
    plan = m.plan(dtype, ctx=max(128, n))
    got = whole(plan, toks)
    dec = stepwise(plan, toks[:12], [1])
    plan.close()
    if dtype == "float32":
        assert err(got, ref) < F32_TOL
        assert err(dec, ref[:12]) < F32_TOL
    elif any((l["mlp"] or {}).get("kind") == "moe" for l in layers):
        assert bf16_ok(m, toks, got, ref) and bf16_ok(m, toks, dec, ref)
    else:
        assert err(got, ref) < BF16_TOL
        assert err(dec, ref[:12]) < BF16_TOL


MIXED = [hgrn(heads=2, dim=24, vdim=16, mlp=None), att(mlp=moe(experts=8, top=3, groups=(4, 2))),
         mls(heads=4, dim=12, vdim=28, mlp=dense(72)), att(heads=3, kv_heads=1, dim=32, rot=32, conv=2, base=50.0, scaling=None, scale=0.2, mlp=dense(24)),
         hgrn(heads=5, dim=8, vdim=12, mlp=moe(experts=9, top=2, ff=16, shared=0, groups=(3, 1))), mls(heads=1, dim=20, vdim=36, cap=3.0, mlp=None)]


def test_layer_taps(hy, tmp_path):
    """The residual that leaves every layer against the restatement, layer by layer."""
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED), width=96), seed=41)
    toks, ref = m.tokens(90)
    plan = m.plan("float32", ctx=96, layer_taps=True)
    taps = []
    m.ref(toks, taps=taps)
    got = whole(plan, toks)
    for l, t in enumerate(taps):
        rows = plan.layer_rows(l, len(toks))
        assert np.abs(rows - t).max() < 1e-4 * max(1.0, np.abs(t).max()), l
    plan.close()
    assert err(got, ref) < F32_TOL


def random_config(seed):
    """Layer order, every size and every constant drawn at random (sizes that are no multiples of anything included)."""
    rng = np.random.default_rng(seed)
    pick = lambda *xs: xs[int(rng.integers(len(xs)))]

    def mlp():
        kind = pick("none", "dense", "moe", "moe")
        if kind == "none":
            return None
        if kind == "dense":
            return dense(int(rng.integers(4, 150)))
        G, per = int(rng.integers(1, 6)), int(rng.integers(1, 6))
        keep = int(rng.integers(1, G + 1))
        return moe(experts=G * per, top=int(rng.integers(1, keep * per + 1)), ff=int(rng.integers(4, 40)), shared=pick(0, int(rng.integers(4, 60))), groups=(G, keep))

    layers = []
    for i in range(int(rng.integers(2, 7))):
        kind = pick("hgrn2", "mlstm", "attention")
        H = int(rng.integers(1, 7))
        if kind == "hgrn2":
            layers.append(hgrn(heads=H, dim=int(rng.integers(2, 60)), vdim=int(rng.integers(2, 70)), mlp=mlp()))
        elif kind == "mlstm":
            layers.append(mls(heads=H, dim=int(rng.integers(2, 50)), vdim=int(rng.integers(2, 60)), cap=float(rng.uniform(2.0, 25.0)), mlp=mlp()))
        else:
            G, D = int(rng.integers(1, 4)), int(rng.integers(4, 60))
            sc = pick(None, {"factor": float(rng.uniform(1.5, 16.0)), "high": float(rng.uniform(2.0, 8.0)), "low": float(rng.uniform(0.5, 2.0)), "original": int(rng.integers(16, 2000))})
            layers.append(att(heads=G * int(rng.integers(1, 5)), kv_heads=G, dim=D, rot=2 * int(rng.integers(1, D // 2 + 1)), conv=int(rng.integers(1, 7)),
                              base=float(rng.uniform(5.0, 1e6)), scaling=sc, scale=float(rng.uniform(0.05, 0.4)), mlp=mlp()))
    return config(layers, width=int(rng.integers(20, 140)), vocab=int(rng.integers(30, 300)), eps=float(10.0 ** -rng.uniform(4, 7)),
                  bigram=(int(rng.integers(50, 2000)), int(rng.integers(1, 500)), int(rng.integers(1, 500))))


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(hy, tmp_path, seed):
    m = Model(hy, tmp_path, random_config(seed), seed=100 + seed)
    n = 140
    toks, ref = m.tokens(n, seed=seed)
    for dtype in ("float32", "bfloat16"):
        plan = m.plan(dtype, ctx=n + 4, max_batch=48)
        for got in (whole(plan, toks), stepwise(plan, toks, [50, 2, 1, 31, 7, 1])):
            assert err(got, ref) < F32_TOL if dtype == "float32" else bf16_ok(m, toks, got, ref)
        plan.close()


# ---- prompts cut into portions, decoding token by token ---------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prefill_equals_token_by_token_and_portions(hy, tmp_path, dtype):
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED)), seed=7)
    n = 150
    toks, ref = m.tokens(n)
    ok = (lambda got: err(got, ref) < F32_TOL) if dtype == "float32" else (lambda got: bf16_ok(m, toks, got, ref))
    plan = m.plan(dtype, ctx=160, max_batch=64)              # the whole prompt runs as portions of 64 inside one step, too
    assert ok(whole(plan, toks))
    assert ok(stepwise(plan, toks, [1]))
    for sizes in ([2, 3, 2, 64, 5, 1, 1, 37, 2, 33], [70, 2, 2, 2, 74], [1, 149], [9, 2], [8, 9, 8], [2]):
        assert ok(stepwise(plan, toks, sizes)), sizes
    plan.close()


def test_logits_do_not_depend_on_the_cut(hy, tmp_path):
    """float32: the same position through different cuts agrees to rounding."""
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED)), seed=8)
    toks, _ = m.tokens(90)
    plan = m.plan("float32", ctx=128)
    a = whole(plan, toks)
    b = stepwise(plan, toks, [41, 2, 47])
    c = stepwise(plan, toks, [1])
    plan.close()
    assert err(b, a) < 2e-5 and err(c, a) < 2e-5


@pytest.mark.parametrize("taps", [2, 3, 5, 9])
def test_convolution_tail_across_portions(hy, tmp_path, taps):
    """A convolution reaches taps - 1 tokens back over any number of short steps, single tokens and portions shorter than its reach mixed; with
    all the weight on its oldest tap each key is the projection of the token taps - 1 earlier, and the restatement with the weight one tap
    later differs by far more than the bound."""
    def tweak(cfg, w):
        for n in ("l0.mix.q.conv", "l0.mix.k.conv"):
            w[n] = np.zeros_like(w[n])
            w[n][:, 0] = 1.0

    m = Model(hy, tmp_path, config([att(conv=taps, mlp=None)], bigram=None), seed=60 + taps, tweak=tweak)
    toks, ref = m.tokens(50)
    other = dict(m.w64)
    for n in ("l0.mix.q.conv", "l0.mix.k.conv"):
        other[n] = np.roll(m.w64[n], 1, axis=1)
    assert err(R.forward(m.cfg, other, toks), ref) > 20 * F32_TOL
    plan = m.plan("float32", ctx=64, n_seqs=2)
    for sizes in ([50], [1], [2], [1, 2, 1, 1, 3, 2, 1, 4, 1, 20, 1, 1, 2], [20, 1, 1, 28], [20, 2, 28]):
        assert err(stepwise(plan, toks, sizes), ref) < F32_TOL, sizes
    plan.close()


def test_previous_token_across_portions(hy, tmp_path):
    """What the previous token leaves behind — its row of the pair table and its share of the shifted input — made large: every cut sees the
    token before the cut, and a sequence's first token sees none, also in a slot that held another sequence."""
    def tweak(cfg, w):
        w["bigram"] = w["bigram"] * 4.0
        w["l0.shift"] = np.ones_like(w["l0.shift"])          # the mixer reads the previous token's row alone
        w["l1.shift"] = np.full_like(w["l1.shift"], 0.75)

    m = Model(hy, tmp_path, config([hgrn(mlp=dense(24)), mls(mlp=None)]), seed=65, tweak=tweak)
    (ta, ra), (tb, rb) = m.tokens(40, 1), m.tokens(40, 2)
    swapped = ta.copy()
    swapped[19] = (ta[19] + 1) % 131
    assert err(m.ref(swapped)[20:21], ra[20:21]) > 20 * F32_TOL
    plan = m.plan("float32", ctx=48, max_batch=16)
    for toks, ref in ((ta, ra), (tb, rb)):
        for sizes in ([40], [1], [20, 1, 19], [2], [3, 17, 2, 1, 1, 16]):
            assert err(stepwise(plan, toks, sizes), ref) < F32_TOL, sizes
    plan.close()


# ---- slots -------------------------------------------------------------------------------------------------------------------------------
def test_interleaved_requests_and_slot_reuse(hy, tmp_path):
    """Unequal requests whose steps alternate give what each gives alone; a slot that a long request left (cache rows, states, running maxima,
    convolution tails, the previous token and its row) is clean for the next."""
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED)), seed=9)
    (ta, ra), (tb, rb), (tc, rc) = m.tokens(60, 1), m.tokens(45, 2), m.tokens(30, 3)
    plan = m.plan("float32", ctx=64, n_seqs=2)
    a, b = plan.acquire(), plan.acquire()
    assert a != b
    with pytest.raises(hy.hip.Gl3Error):
        plan.acquire()                                   # both slots are taken
    ga, gb = [], []
    ga.append(plan.step(a, ta[:20], 0, list(range(20))))
    gb.append(plan.step(b, tb[:7], 0, list(range(7))))
    ga.append(plan.step(a, ta[20:21], 20, [0]))
    gb.append(plan.step(b, tb[7:40], 7, list(range(33))))
    ga.append(plan.step(a, ta[21:], 21, list(range(39))))
    for i in range(40, 45):
        gb.append(plan.step(b, tb[i:i + 1], i, [0]))
    assert err(np.concatenate(ga), ra) < F32_TOL and err(np.concatenate(gb), rb) < F32_TOL
    plan.release(a)
    c = plan.acquire()
    assert c == a
    gc = [plan.step(c, tc[:1], 0, [0]), plan.step(c, tc[1:3], 1, [0, 1]), plan.step(c, tc[3:], 3, list(range(27)))]
    assert err(np.concatenate(gc), rc) < F32_TOL
    with pytest.raises(hy.hip.Gl3Error):
        plan.step(c, tc[:2], 7, [])                      # neither a continuation nor a restart
    assert err(plan.step(b, tc, 0, list(range(30))), rc) < F32_TOL          # a restart at position 0 on a live slot starts clean as well
    plan.close()


def test_decode_batch_over_slots(hy, tmp_path):
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED[:3])), seed=10)
    (ta, ra), (tb, rb) = m.tokens(12, 4), m.tokens(9, 5)
    plan = m.plan("float32", ctx=32, n_seqs=2)
    a, b = plan.acquire(), plan.acquire()
    plan.step(a, ta[:11], 0, [])
    plan.step(b, tb[:8], 0, [])
    logits, ids = plan.forward_decode_batch([ta[11], tb[8]], [a, b], [11, 8])
    plan.close()
    assert err(logits, np.stack([ra[11], rb[8]])) < F32_TOL and list(ids) == list(np.argmax(logits, axis=1))


# ---- far keys, the causal edge, key tiles: a token looks for its own earlier occurrences -------------------------------------------------
def lookup_attention(cfg, w, copy_score=9.0):
    """Layer 0 becomes a look-up: every query head repeats its key head's projection, the convolutions pass the current token alone, nothing is
    shifted in, and the q norm's weights are zero on the rotated entries and level on the others: the score of a key depends on the two
    tokens only, and a token finds every earlier copy of itself about `copy_score` above the other keys."""
    mx = cfg["layers"][0]["mixer"]
    H, G, D, n = mx["heads"], mx["kv_heads"], mx["dim"], mx["rot"]["dims"]
    assert cfg["layers"][0]["type"] == "attention" and not cfg.get("embedding")
    w["l0.shift"] = np.zeros_like(w["l0.shift"])
    k = w["l0.mix.k"].reshape(G, D, -1)
    w["l0.mix.q"] = np.repeat(k, H // G, axis=0).reshape(H * D, -1)
    for name in ("l0.mix.q.conv", "l0.mix.k.conv"):
        w[name] = np.zeros_like(w[name])
        w[name][:, -1] = 1.0
    w["l0.mix.k.norm"] = np.ones_like(w["l0.mix.k.norm"])
    w["l0.mix.q.norm"] = np.where(np.arange(D) < n, 0.0, copy_score / (mx["scale"] * (D - n)))
    w["l0.ls1"] = np.full_like(w["l0.ls1"], 4.0)


def lookup_model(hy, tmp_path, seed, extra=()):
    layers = [att(heads=4, kv_heads=2, dim=40, rot=8, conv=3, scale=0.5, mlp=None)] + list(extra)
    return Model(hy, tmp_path, config(layers, width=64, vocab=97, bigram=None), seed=seed, tweak=lookup_attention)


@pytest.mark.parametrize("n,decode_from", [(150, 120), (200, 190), (330, 300), (129, 60), (530, 505)])
def test_causal_edge_and_key_tiles(hy, tmp_path, n, decode_from):
    """A small vocabulary and a look-up layer: every query has earlier copies of its token at all distances, in every key tile (tiles are
    64 keys wide; decode steps split the keys over workgroups by tile), in the prompt and while decoding.  The restatement with the
    causal edge moved by one (a query that also sees the next key) differs by more than 10 times the bound: a kernel that is off by
    one at the edge cannot pass."""
    m = lookup_model(hy, tmp_path, n, extra=[att(heads=2, kv_heads=1, dim=12, rot=8, mlp=dense(16))])
    toks, ref = m.tokens(n, vocab=23)
    assert err(m.ref(toks, causal_shift=1), ref) > 10 * F32_TOL
    plan = m.plan("float32", ctx=n + 8, max_batch=96)
    assert err(whole(plan, toks), ref) < F32_TOL
    s = plan.acquire()
    got = [plan.step(s, toks[:decode_from], 0, list(range(decode_from)))]
    got += [plan.step(s, toks[i:i + 1], i, [0]) for i in range(decode_from, n)]
    plan.release(s)
    assert err(np.concatenate(got), ref) < F32_TOL
    assert err(stepwise(plan, toks, [61, 2, 3, 64, 2, 67]), ref) < F32_TOL
    plan.close()


@pytest.mark.parametrize("far", [0, 3, 63, 64, 127, 128, 191])
def test_one_far_key_among_hundreds(hy, tmp_path, far):
    """One token stands at position `far` and again at the very end, nowhere else: the last query's look-up finds that one key among
    hundreds (at a tile's first or last row, in the first tile or a later one).  Hiding the key in the restatement moves the last logits
    by far more than the bound; the plan follows with the prompt whole, in portions, and with the last tokens decoded (the keys are
    then split over workgroups)."""
    m = lookup_model(hy, tmp_path, 300 + far, extra=[hgrn(heads=2, dim=8, vdim=8, mlp=None)])
    n = 450
    toks = np.random.default_rng(far).integers(1, 97, n).astype(np.int32)
    toks[far] = toks[n - 1] = 0
    ref = m.ref(toks)
    assert err(m.ref(toks, drop_keys=[far])[-1:], ref[-1:]) > 20 * F32_TOL
    for dtype, tol in (("float32", F32_TOL), ("bfloat16", BF16_TOL)):
        plan = m.plan(dtype, ctx=n, max_batch=200)
        assert err(whole(plan, toks, [n - 1]), ref[-1:]) < tol
        s = plan.acquire()
        plan.step(s, toks[:n - 5], 0, [])
        got = np.concatenate([plan.step(s, toks[i:i + 1], i, [0]) for i in range(n - 5, n)])
        plan.release(s)
        assert err(got, ref[n - 5:]) < tol
        assert err(stepwise(plan, toks, [190, 2, 130, 127, 1])[-1:], ref[-1:]) < tol
        plan.close()


@pytest.mark.parametrize("kind", ["hgrn2", "mlstm"])
def test_far_tokens_reach_the_memories(hy, tmp_path, kind):
    """The first tokens of a long prompt decide the last logits only through one recurrence's states, whose gates are nearly shut for
    forgetting: changing two early tokens moves the restatement's last logits by far more than the bound, and the plan follows, whole and
    decoded."""
    layers = [hgrn(heads=2, dim=16, vdim=16, mlp=None) if kind == "hgrn2" else mls(heads=2, dim=16, vdim=16, mlp=None)]

    def tweak(cfg, w):
        if kind == "hgrn2":
            w["l0.mix.lower"] = np.full_like(w["l0.mix.lower"], 0.998)
        else:
            w["l0.mix.f.b"] = np.full_like(w["l0.mix.f.b"], 8.0)
            w["l0.mix.f"] = w["l0.mix.f"] * 0.1
            w["l0.mix.i"] = w["l0.mix.i"] * 0.1
        w["l0.ls1"] = np.full_like(w["l0.ls1"], 3.0)

    m = Model(hy, tmp_path, config(layers, width=48, vocab=61), seed=77, tweak=tweak)
    n = 700
    toks, ref = m.tokens(n)
    other = toks.copy()
    other[3], other[4] = (toks[3] + 1) % 61, (toks[4] + 7) % 61
    assert err(m.ref(other)[-1:], ref[-1:]) > 20 * F32_TOL
    plan = m.plan("float32", ctx=n, max_batch=256)
    assert err(whole(plan, toks, [n - 1]), ref[-1:]) < F32_TOL
    s = plan.acquire()
    plan.step(s, toks[:n - 40], 0, [])
    got = np.concatenate([plan.step(s, toks[i:i + 1], i, [0]) for i in range(n - 40, n)])
    plan.release(s)
    plan.close()
    assert err(got, ref[n - 40:]) < F32_TOL


def test_gates_near_one_and_zero(hy, tmp_path):
    """Channels that never forget (lower bound 1), channels whose gate follows its input over its whole range, and saturated gates side by side."""
    def tweak(cfg, w):
        low = w["l0.mix.lower"].reshape(3, 16)
        low[0], low[1, ::2] = 1.0, 0.0
        b = w["l0.mix.f.b"].reshape(3, 16)
        b[1], b[2] = 0.0, np.where(np.arange(16) % 2, 30.0, -30.0)

    m = Model(hy, tmp_path, config([hgrn()]), seed=78, tweak=tweak)
    toks, ref = m.tokens(120)
    plan = m.plan("float32", ctx=128)
    assert err(whole(plan, toks), ref) < F32_TOL
    assert err(stepwise(plan, toks, [30, 2, 1]), ref) < F32_TOL
    plan.close()


def test_running_maximum_from_zero(hy, tmp_path):
    """Input gates far below zero: the running maximum starts at zero and falls with the forget gate, so the normaliser's lower bound e^(-m)
    decides the first outputs; then a token with a large input gate takes the maximum over."""
    def tweak(cfg, w):
        w["l0.mix.i.b"] = np.array([-6.0, 0.0, 7.0], np.float32)
        w["l0.mix.f.b"] = np.array([0.0, -5.0, 5.0], np.float32)

    m = Model(hy, tmp_path, config([mls()]), seed=79, tweak=tweak)
    toks, ref = m.tokens(80)
    plan = m.plan("float32", ctx=96)
    for sizes in ([80], [1], [2, 1, 5, 30]):
        assert err(stepwise(plan, toks, sizes), ref) < F32_TOL, sizes
    plan.close()


def test_first_tokens(hy, tmp_path):
    """Positions 0 .. 4 and a one-token sequence (through the decode kernels)."""
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED)), seed=21)
    toks, ref = m.tokens(5)
    plan = m.plan("float32", ctx=8)
    assert err(whole(plan, toks), ref) < F32_TOL
    assert err(whole(plan, toks[:1]), ref[:1]) < F32_TOL
    assert err(stepwise(plan, toks, [1]), ref) < F32_TOL
    assert err(stepwise(plan, toks, [2]), ref) < F32_TOL
    plan.close()


def test_long_decoding(hy, tmp_path):
    layers = [att(heads=2, kv_heads=1, dim=16, rot=8, mlp=dense(16)), hgrn(heads=2, dim=16, vdim=16, mlp=None), mls(heads=2, dim=8, vdim=8, mlp=dense(40))]
    m = Model(hy, tmp_path, config(layers, width=48, vocab=61), seed=33)
    n = 420
    toks, ref = m.tokens(n)
    for dtype, tol in (("float32", F32_TOL), ("bfloat16", BF16_TOL)):
        plan = m.plan(dtype, ctx=n)
        s = plan.acquire()
        plan.step(s, toks[:3], 0, [])
        got = np.concatenate([plan.step(s, toks[i:i + 1], i, [0]) for i in range(3, n)])
        plan.release(s)
        plan.close()
        assert err(got, ref[3:]) < tol, dtype


def test_rotation_is_by_position_not_by_place_in_the_step(hy, tmp_path):
    """With a small base and no scaling the turns are large, and a portion that starts late must turn by its true positions."""
    m = Model(hy, tmp_path, config([att(dim=24, rot=24, base=3.0, scaling=None, scale=1.0)]), seed=61)
    toks, ref = m.tokens(70)
    plan = m.plan("float32", ctx=80)
    assert err(stepwise(plan, toks, [33, 2, 1, 20, 14]), ref) < F32_TOL
    plan.close()


def test_groups_close_experts_with_negative_choice_scores(hy, tmp_path):
    """Corrections that put every choice score below zero, and the largest single score into a group whose two best are not the best pair:
    the closed groups' experts stay closed (a closed expert counts as minus infinity, not as zero)."""
    layers = [hgrn(mlp=moe(experts=8, top=3, ff=16, shared=0, groups=(4, 2)))]

    def tweak(cfg, w):
        w["l0.mlp.correction"] = np.array([-2.0, -19.0, -4.0, -4.0, -5.0, -5.0, -8.0, -8.0], np.float32)

    m = Model(hy, tmp_path, config(layers), seed=88, tweak=tweak)
    toks, ref = m.tokens(40)
    h = np.random.default_rng(0).standard_normal((9, 88))
    choice, wts = R.route(h, R.sub(m.w64, "l0.mlp."), m.cfg["layers"][0]["mlp"])
    assert all(set(c) <= {2, 3, 4, 5} for c in choice)                   # expert 0 has the largest choice score, but its group ranks third
    plan = m.plan("float32", ctx=64)
    assert err(whole(plan, toks), ref) < F32_TOL
    assert err(stepwise(plan, toks, [1]), ref) < F32_TOL
    plan.close()


# ---- the framework's own entry points ----------------------------------------------------------------------------------------------------
def check_greedy(m, prompt, ids):
    """Every generated id is the reference's arg max given the ids before it (ties within 1e-4 of the maximum are allowed)."""
    full = list(prompt) + list(ids)
    ref = m.ref(np.array(full[:-1], np.int32))
    for i, t in enumerate(ids):
        row = ref[len(prompt) - 1 + i]
        assert row[t] >= row.max() - 1e-4 * max(1.0, abs(row.max())), i


def test_greedy_generation_python_entry(hy, tmp_path):
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED)), seed=51)
    prompt, _ = m.tokens(37)
    plan = m.plan("float32", ctx=64, max_batch=16)
    ids = plan.generate(prompt, 20)
    check_greedy(m, prompt, ids)
    plan.prefill(prompt[:-1], 0)
    lg = plan.forward_decode(int(prompt[-1]), len(prompt) - 1)
    assert int(np.argmax(lg)) == ids[0]
    plan.prefill(prompt[:-1], 0)
    t = plan.forward_decode_sample(int(prompt[-1]), len(prompt) - 1, 0.7, 0.9, 0.3)
    assert 0 <= t < m.cfg["vocab"]
    plan.close()


def test_greedy_generation_command_line(hy, tmp_path):
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED)), seed=52)
    prompt, _ = m.tokens(21)
    exe = os.path.join(ge.ROOT, "tools", "gl3_run")
    out = subprocess.run([exe, "-m", m.dir, "--ids", ",".join(map(str, prompt)), "-n", "40", "-b", "8", "--f32"], capture_output=True, text=True, timeout=120)
    assert out.returncode == 0, out.stderr
    ids = [int(x) for x in out.stdout.split("generated:")[1].split()]
    assert len(ids) == 40 - len(prompt) + 1
    check_greedy(m, prompt, ids)


def test_trace_replay_tool(hy, tmp_path):
    m = Model(hy, tmp_path, config(copy.deepcopy(MIXED[:4])), seed=53)
    toks, ref = m.tokens(50)
    outdir = tmp_path / "out"
    outdir.mkdir()
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:30].tolist(), "want": [3, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[30:32].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[32:].tolist(), "want": [17]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": toks[:5].tolist(), "want": [4]}], "end": ["y"]}]
    for dtype, tol in (("float32", F32_TOL), ("bfloat16", BF16_TOL)):
        p = subprocess.run([os.path.join(ge.ROOT, "bin", "trace_run"), "--model", m.dir, "--dtype", dtype, "--out", str(outdir), "--max-tokens", "64"],
                           input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
        assert p.returncode == 0, p.stderr
        assert [l for l in p.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
        assert not (outdir / "1.f32").exists()
        got = np.concatenate([np.fromfile(outdir / ("%d.f32" % i), np.float32).reshape(-1, m.cfg["vocab"]) for i in (0, 2, 3)])
        want = ref[[3, 29, 49, 4]] if dtype == "float32" else m.ref(toks, round_inputs=True)[[3, 29, 49, 4]]
        assert np.median(err_rows(got, want)) < tol if dtype == "bfloat16" else err(got, want) < tol


def test_loader_refuses_what_it_cannot_run(hy, tmp_path):
    m = Model(hy, tmp_path, config([att(mlp=moe()), hgrn(), mls(mlp=None)]), seed=54)
    for name in ("bigram", "l0.shift", "l0.ls1", "l0.ls2", "l0.mix.q.norm", "l0.mix.k.norm", "l0.mix.q.conv", "l0.mix.k.conv", "l0.mlp.correction", "l0.mlp.e3.up", "l0.mlp.shared.sg",
                 "l0.mlp.shared.up", "l1.mix.f", "l1.mix.f.b", "l1.mix.lower", "l1.mix.norm", "l1.mlp.act", "l1.mlp.up", "l2.mix.i.b", "l2.mix.g", "l2.mix.norm", "final.norm"):
        w = dict(m.w)
        del w[name]
        hy.save_model_dir(str(tmp_path / "bad"), m.cfg, w)
        with pytest.raises(hy.hip.Gl3Error):
            hy.HybridPlan.from_dir(str(tmp_path / "bad"))
    for name in ("bigram", "l0.mlp.correction", "l0.mix.k.conv", "l1.mix.lower", "l1.mlp.act", "l1.mix.norm"):
        w = dict(m.w)
        w[name] = np.concatenate([w[name], w[name]])
        hy.save_model_dir(str(tmp_path / "bad"), m.cfg, w)
        with pytest.raises(hy.hip.Gl3Error):
            hy.HybridPlan.from_dir(str(tmp_path / "bad"))


# ---- a mechanism is a parameter of the family, not of one design ------------------------------------------------------------------------
def test_channel_gates_beside_attention_of_another_kind(hy):
    """The descriptor combines the new mechanisms with older ones: one that cannot be combined is refused before any device memory is taken."""
    hip = hy.hip

    def create(layer, **model):
        d = hip.ModelDesc()
        d.struct_size, d.arch, d.dim, d.vocab, d.ctx, d.max_batch, d.weight_type, d.n_layers, d.rms_eps = hip.C.sizeof(hip.ModelDesc), 6, 16, 8, 8, 4, 30, 1, 1e-5
        l = hip.LayerDesc()
        for k, v in dict(dict(mixer=0, heads=2, kv_heads=1, dim=8, vdim=8, scale=1.0), **layer).items():
            setattr(l, k, v)
        for k, v in model.items():
            setattr(d, k, v)
        d.layer_descs = hip.C.pointer(l)
        p = hip.C.c_void_p()
        r = hip.lib().gl3_create(hip.C.byref(d), hip.C.byref(p))
        if p:
            hip.lib().gl3_destroy(p)
        return r

    assert create({}) == 0
    assert create({"qk_conv": 3}) == 0 and create({"v_from_k": 1, "qk_unit_norm": 3, "window": 4}) == 0
    assert create({"mixer": 3, "mem_gates": 2, "mem_gate_act": 1}) == 0
    assert create({"ff": 8, "ff_act": 3}, post_norms=1, layer_scale=1, token_shift=1, bigram_buckets=5) == 0
    for layer, model in (({"v_from_k": 1, "vdim": 4}, {}), ({"v_from_k": 1, "v_unit_norm": 1}, {}), ({"qk_conv": 3, "qk_bias": 1}, {}), ({"qk_conv": 65}, {}),
                         ({"mixer": 3, "qk_conv": 2}, {}), ({"mixer": 3, "mem_gates": 3}, {}), ({"mixer": 3, "mem_gates": 2, "rot_dims": 2, "rot_base": 10.0}, {}),
                         ({"ff": 8, "ff_act": 3, "experts": 2, "top": 1}, {}), ({"ff": 8, "ff_act": 2, "experts": 2, "top": 1}, {}),
                         ({"ff": 8, "experts": 4, "top": 3, "route_groups": 2, "route_keep": 1}, {}), ({"ff": 8, "experts": 5, "top": 1, "route_groups": 2, "route_keep": 1}, {}),
                         ({"rot_dims": 2, "rot_base": 10.0, "rot_wave_factor": 2.0}, {}), ({}, {"parallel_block": 1, "token_shift": 1}), ({}, {"streams": 1, "layer_scale": 1})):
        assert create(layer, **model) != 0, (layer, model)
