"""The Ziginex design (layer-list family: norms behind the sublayers only; attention with tempered, capped and mixed head scores inside chunks
beside a gated delta rule; latent attention with a learned sink; experts and identity choices; per-layer token input) on the GPU against
the plain float64 restatement in tests/ziginex_ref.py.

Every test makes its own small configuration and random bfloat16-representable weights, writes them as a model folder and loads that
through the product's loader.  float32 plans are held to 2e-4 (root mean square of the logit difference over the root mean square of
the logits), bfloat16 plans to 6e-2.  Where random weights would hide a fault, the first layer's attention is turned into a look-up: the
second half of a token's embedding is the first half of the next token id's, keys read the first half and queries the second, so that a
token attends to the earlier occurrences of its successor wherever they are inside its chunk; hiding one key, or moving the causal
edge or the chunks' edges by one, then moves the logits by far more than the bound, and the tests check that on the restatement itself.
"""
import copy
import ctypes as C
import json
import math
import os
import subprocess

import numpy as np
import pytest

import __graft_entry__ as ge
import ziginex_ref as R

pytestmark = pytest.mark.gpu
F32_TOL, BF16_TOL = 2e-4, 6e-2


@pytest.fixture(scope="module")
def hy():
    from importlib import import_module
    ge.load_package()
    return import_module(ge.PKG_NAME + ".hybrid")


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, identity=1, top=2, ff=24, groups=(3, 2)):
    r = {"experts": experts, "top": top}
    if identity:
        r["identity"] = identity
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def par(heads=4, kv_heads=2, dim=20, vdim=16, rot=12, base=600.0, scale=0.4, cap=6.0, chunk=24, d_heads=4, d_kv_heads=2, d_dim=12, d_vdim=20, conv=4, mlp="dense"):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if cap:
        left["softcap"] = cap
    if chunk:
        left["mask"] = {"size": chunk}
    if rot:
        left["rot"] = {"base": base, "dims": rot}
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": d_heads, "kv_heads": d_kv_heads, "dim": d_dim, "vdim": d_vdim, "conv": conv}},
            "mlp": dense() if mlp == "dense" else mlp}


BLEND = {"factor": 4.0, "original": 200, "fast": 12.0, "slow": 1.5}


def lat(heads=3, dim=12, rot=8, vdim=20, kv_rank=28, q_rank=18, base=900.0, scaling=BLEND, scale=0.3, mlp="dense"):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}
    if rot:
        m["rot_dim"] = rot
        m["rot"] = {"base": base, "dims": rot}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    return {"type": "latent_attention", "mixer": m, "mlp": dense() if mlp == "dense" else mlp}


def config(layers, width=88, vocab=131, eps=1e-5, side=10):
    c = {"architecture": "Ziginex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if side:
        c["token_side"] = {"dim": side}
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
    whose choice scores tie to the last bits (that one, and through state and cache those after it, leave by more than rounding): three
    rows in four.  Against the unrounded restatement the median row is held to the bound."""
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
    ("parallel_plain", [par()], {}),
    ("parallel_no_feed_forward", [par(mlp=None)], {}),
    ("no_token_input", [par(), lat()], {"side": 0}),
    ("token_input_one_entry", [par(mlp=None)], {"side": 1}),
    ("token_input_wide", [par(), lat(mlp=None)], {"side": 150}),
    ("scores_one_head", [par(heads=1, kv_heads=1, dim=32, vdim=32)], {}),
    ("scores_one_key_head_for_many", [par(heads=12, kv_heads=1, dim=16, vdim=16, rot=4)], {}),
    ("scores_a_key_head_each", [par(heads=5, kv_heads=5, dim=16, vdim=8)], {}),
    ("scores_past_sixteen_heads", [par(heads=21, kv_heads=7, dim=16, vdim=12, rot=8)], {}),
    ("scores_past_sixty_four_heads", [par(heads=70, kv_heads=5, dim=8, vdim=4, rot=8, mlp=None)], {}),
    ("scores_most_heads", [par(heads=128, kv_heads=32, dim=16, vdim=4, rot=8, mlp=None)], {"n": 40}),
    ("scores_heads_of_48_and_96", [par(heads=4, kv_heads=2, dim=48, vdim=96, rot=24)], {}),
    ("scores_large_heads", [par(heads=2, kv_heads=1, dim=192, vdim=160, rot=64, scale=0.08)], {}),
    ("scores_many_value_columns", [par(heads=12, kv_heads=12, dim=16, vdim=320, mlp=None)], {}),
    ("scores_odd_sizes", [par(heads=6, kv_heads=3, dim=18, vdim=13, rot=10)], {}),
    ("scores_no_rotation", [par(rot=0)], {}),
    ("scores_all_turned", [par(dim=24, rot=24, base=5.0)], {}),
    ("scores_no_cap", [par(cap=None)], {}),
    ("scores_tight_cap", [par(cap=0.7, scale=2.0)], {}),
    ("no_chunks", [par(chunk=None)], {}),
    ("chunks_of_one", [par(chunk=1)], {}),
    ("chunks_of_two", [par(chunk=2)], {}),
    ("chunks_of_a_key_tile", [par(dim=16, chunk=64)], {"n": 150}),
    ("chunks_past_the_end", [par(chunk=500)], {}),
    ("delta_one_tap", [par(conv=1)], {}),
    ("delta_two_taps", [par(conv=2)], {}),
    ("delta_many_taps", [par(conv=11)], {}),
    ("delta_one_head", [par(d_heads=1, d_kv_heads=1, d_dim=40, d_vdim=70, mlp=None)], {}),
    ("delta_a_key_head_each", [par(d_heads=5, d_kv_heads=5, d_dim=16, d_vdim=16)], {}),
    ("delta_one_key_head_for_many", [par(d_heads=9, d_kv_heads=1, d_dim=8, d_vdim=6)], {}),
    ("delta_one_key_entry", [par(d_dim=1, d_vdim=3)], {}),
    ("delta_one_value", [par(d_dim=5, d_vdim=1)], {}),
    ("delta_keys_of_64", [par(d_dim=64, d_vdim=32)], {}),
    ("delta_keys_of_128", [par(d_dim=128, d_vdim=128, mlp=None)], {}),
    ("delta_keys_of_200", [par(d_heads=2, d_kv_heads=1, d_dim=200, d_vdim=24, mlp=None)], {}),
    ("delta_keys_of_300", [par(d_heads=1, d_kv_heads=1, d_dim=300, d_vdim=20, mlp=None)], {}),
    ("delta_keys_of_601", [par(d_heads=2, d_kv_heads=2, d_dim=601, d_vdim=9, mlp=None)], {}),
    ("latent_plain", [lat()], {}),
    ("latent_no_feed_forward", [lat(mlp=None)], {}),
    ("latent_one_head", [lat(heads=1, dim=40, vdim=24, kv_rank=64, q_rank=32)], {}),
    ("latent_many_heads", [lat(heads=13, dim=5, rot=4, vdim=3, kv_rank=9, q_rank=7)], {}),
    ("latent_plain_frequencies", [lat(scaling=None, base=10000.0)], {}),
    ("latent_all_waves_divided", [lat(scaling={"factor": 8.0, "original": 2, "fast": 32.0, "slow": 1.0})], {}),
    ("latent_all_waves_kept", [lat(scaling={"factor": 8.0, "original": 10000000, "fast": 32.0, "slow": 1.0})], {}),
    ("latent_wide_rotation", [lat(dim=4, rot=48)], {}),
    ("latent_long_rows", [lat(heads=2, dim=24, kv_rank=560, q_rank=40, mlp=None)], {}),
    ("dense_odd_width", [par(mlp=dense(33))], {}),
    ("dense_wide", [lat(mlp=dense(1500))], {}),
    ("experts_plain", [par(mlp=moe())], {}),
    ("experts_without_identity", [par(mlp=moe(experts=6, identity=0))], {}),
    ("experts_without_groups", [par(mlp=moe(groups=None))], {}),
    ("experts_more_identity_than_experts", [lat(mlp=moe(experts=3, identity=9, top=5, groups=(4, 3)))], {}),
    ("experts_all_choices_taken", [lat(mlp=moe(experts=3, identity=2, top=5, groups=None))], {}),
    ("experts_one_group", [lat(mlp=moe(groups=(1, 1)))], {}),
    ("experts_groups_of_one", [lat(mlp=moe(experts=6, identity=1, top=3, groups=(7, 4)))], {}),
    ("experts_all_of_the_kept_groups", [par(mlp=moe(experts=9, identity=3, top=6, groups=(4, 2)))], {}),
    ("experts_past_sixty_four", [par(mlp=moe(experts=90, identity=10, top=9, ff=8, groups=(10, 4)))], {}),
    ("experts_past_256", [lat(mlp=moe(experts=270, identity=10, top=12, ff=4, groups=(28, 9)))], {"n": 40}),
    ("experts_one", [par(mlp=moe(experts=1, identity=0, top=1, groups=None))], {}),
    ("widths_not_multiples_of_four", [par(heads=3, kv_heads=3, dim=10, vdim=9, rot=6, d_heads=3, d_kv_heads=1, d_dim=7, d_vdim=5, conv=3, mlp=moe(ff=9)),
                                      lat(heads=3, dim=7, rot=6, vdim=5, kv_rank=11, q_rank=9, mlp=dense(17))], {"width": 75, "vocab": 53, "side": 7}),
    ("wide_model", [par(dim=32, vdim=32, d_dim=32, d_vdim=32, mlp=dense(2048)), lat(dim=32, rot=16, vdim=32, kv_rank=64, q_rank=64, mlp=moe(ff=64))],
     {"width": 1024, "vocab": 64, "n": 40, "side": 32}),
    ("width_past_the_registers", [par(heads=2, kv_heads=1, dim=16, vdim=8, d_heads=1, d_kv_heads=1, d_dim=8, d_vdim=8, mlp=moe(experts=2, identity=2, top=3, ff=8, groups=None))],
     {"width": 8300, "vocab": 40, "n": 40, "side": 4}),
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
    few = stepwise(plan, toks[:30], [7])
    plan.close()
    if dtype == "float32":
        assert err(got, ref) < F32_TOL
        assert err(dec, ref[:12]) < F32_TOL
        assert err(few, ref[:30]) < F32_TOL
    elif any((l["mlp"] or {}).get("kind") == "moe" for l in layers):
        assert bf16_ok(m, toks, got, ref) and bf16_ok(m, toks, dec, ref) and bf16_ok(m, toks, few, ref)
    else:
        assert err(got, ref) < BF16_TOL
        assert err(dec, ref[:12]) < BF16_TOL
        assert err(few, ref[:30]) < BF16_TOL


MIXED = [par(chunk=17, mlp=None), lat(mlp=moe(experts=6, identity=2, top=3, groups=(4, 2))), par(heads=6, kv_heads=3, dim=32, vdim=48, rot=16, chunk=40, d_heads=2, d_kv_heads=2, d_dim=24,
         d_vdim=12, conv=3, mlp=moe(experts=4, identity=2, top=2, ff=16, groups=None)), lat(heads=5, dim=16, rot=4, vdim=8, kv_rank=20, q_rank=33, scaling=None, base=50.0, mlp=None),
         par(heads=3, kv_heads=1, dim=9, vdim=7, rot=8, chunk=None, cap=None, d_heads=6, d_kv_heads=3, d_dim=6, d_vdim=10, conv=2, mlp=dense(40))]


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
    num = lambda a, b: int(rng.integers(a, b))

    def mlp():
        kind = pick("none", "dense", "moe", "moe")
        if kind == "none":
            return None
        if kind == "dense":
            return dense(num(4, 150))
        G, per = num(1, 6), num(1, 6)
        keep, ident = num(1, G + 1), num(0, G * per)
        return moe(experts=G * per - ident, identity=ident, top=num(1, keep * per + 1), ff=num(4, 40), groups=(G, keep))

    layers = []
    for i in range(num(2, 6)):
        if pick(True, True, False):
            G, D, K = num(1, 4), pick(16, 32, num(4, 60)), num(1, 4)
            layers.append(par(heads=G * num(1, 6), kv_heads=G, dim=D, vdim=pick(8, 32, num(2, 70)), rot=2 * num(1, D // 2 + 1), base=float(rng.uniform(5.0, 1e6)),
                              scale=float(rng.uniform(0.05, 0.6)), cap=pick(None, float(rng.uniform(1.0, 50.0))), chunk=pick(None, num(1, 120), num(30, 70)), d_heads=K * num(1, 5),
                              d_kv_heads=K, d_dim=num(2, 80), d_vdim=num(2, 60), conv=num(1, 7), mlp=mlp()))
        else:
            P = 2 * num(1, 14)
            sc = pick(None, {"factor": float(rng.uniform(1.5, 16.0)), "original": num(32, 4000), "fast": float(rng.uniform(8.0, 40.0)), "slow": float(rng.uniform(0.5, 4.0))})
            layers.append(lat(heads=num(1, 7), dim=num(2, 50), rot=P, vdim=num(2, 50), kv_rank=num(4, 90), q_rank=num(4, 80), base=float(rng.uniform(20.0, 1e6)), scaling=sc,
                              scale=float(rng.uniform(0.05, 0.4)), mlp=mlp()))
    return config(layers, width=num(20, 140), vocab=num(30, 300), eps=float(10.0 ** -rng.uniform(4, 7)), side=pick(0, num(1, 40)))


@pytest.mark.parametrize("seed", range(16))
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
    for sizes in ([2, 3, 2, 64, 5, 1, 1, 37, 2, 33], [70, 2, 2, 2, 74], [1, 149], [9, 2], [16, 17, 18], [8, 9, 8], [2]):
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
    """A convolution reaches taps - 1 tokens back over any number of short steps, single tokens and portions shorter than its reach mixed: with
    all the weight on its oldest tap q, k and v are those of the token taps - 1 earlier, and the restatement with the weight one tap later
    differs by far more than the bound."""
    names = ["l0.mix.right.%s.conv" % n for n in "qkv"]

    def tweak(cfg, w):
        for n in names:
            w[n] = np.zeros_like(w[n])
            w[n][:, 0] = 1.0

    m = Model(hy, tmp_path, config([par(conv=taps, mlp=None)], side=0), seed=60 + taps, tweak=tweak)
    toks, ref = m.tokens(50)
    other = dict(m.w64)
    for n in names:
        other[n] = np.roll(m.w64[n], 1, axis=1)
    assert err(R.forward(m.cfg, other, toks), ref) > 20 * F32_TOL
    plan = m.plan("float32", ctx=64, n_seqs=2)
    for sizes in ([50], [1], [2], [1, 2, 1, 1, 3, 2, 1, 4, 1, 20, 1, 1, 2], [20, 1, 1, 28], [20, 2, 28]):
        assert err(stepwise(plan, toks, sizes), ref) < F32_TOL, sizes
    plan.close()


# ---- slots -------------------------------------------------------------------------------------------------------------------------------
def test_interleaved_requests_and_slot_reuse(hy, tmp_path):
    """Unequal requests whose steps alternate give what each gives alone; a slot that a long request left (cache rows, latent rows, states,
    convolution tails) is clean for the next."""
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


# ---- far keys, the causal edge, chunk edges, key tiles: a token looks for its own earlier occurrences -------------------------------------
def successor_embedding(w):
    """Token t's row = [a_t | a_(t + 1)]; returns half the width."""
    half = w["embed"].shape[1] // 2
    w["embed"][:, half:] = np.roll(w["embed"][:, :half], -1, axis=0)
    return half


def lookup_attention(cfg, w, score=9.0):
    """Layer 0's attention becomes a look-up and its other mixer goes silent: every query head repeats its key head's projection on the successor's
    half and the q norm's weights are zero on the rotated entries and level on the others, so the score of a key depends on the two tokens
    only and a token finds every occurrence of its successor it may see about `score` above the other keys (no cap in these models; the heads
    still mix)."""
    mx = cfg["layers"][0]["mixer"]["left"]
    H, G, D, n = mx["heads"], mx["kv_heads"], mx["dim"], mx["rot"]["dims"]
    assert "softcap" not in mx
    p, half = "l0.mix.left.", successor_embedding(w)
    k = w[p + "k"]
    k[:, half:] = 0.0
    w[p + "q"] = np.repeat(np.roll(k, half, axis=1).reshape(G, D, -1), H // G, axis=0).reshape(H * D, -1)
    w[p + "k.norm"] = np.ones_like(w[p + "k.norm"])
    w[p + "q.norm"] = np.where(np.arange(D) < n, 0.0, score / (mx["scale"] * (D - n)))
    w[p + "temp"] = np.ones(H)
    w[p + "talk"] = np.eye(H) * 0.8 + 0.2 * np.roll(np.eye(H), 1, axis=1)
    w[p + "sink"] = np.full(H, -2.0)
    w["l0.mix.right.out"] = np.zeros_like(w["l0.mix.right.out"])
    w["l0.norm1"] = np.full_like(w["l0.norm1"], 2.0)


def lookup_model(hy, tmp_path, seed, chunk, extra=(), dim=48):
    layers = [par(heads=4, kv_heads=2, dim=dim, vdim=40, rot=8, scale=0.5, cap=None, chunk=chunk, mlp=None)] + list(extra)
    return Model(hy, tmp_path, config(layers, width=64, vocab=97, side=0), seed=seed, tweak=lookup_attention)


@pytest.mark.parametrize("n,decode_from,chunk", [(150, 120, 64), (200, 190, 63), (330, 250, 65), (129, 60, 7), (300, 250, 128), (530, 505, None), (180, 90, 16), (260, 200, 100)])
def test_causal_edge_chunk_edges_and_key_tiles(hy, tmp_path, n, decode_from, chunk):
    """A small vocabulary and a look-up layer: every query has earlier occurrences of its successor at all distances, before and behind its chunk's first
    position, in every key tile (64 or 16 keys wide; decode steps split the keys over workgroups by tile), in the prompt and while decoding.
    The restatement with the causal edge, or the chunks' edges either way, moved by one differs by more than 10 times the bound."""
    m = lookup_model(hy, tmp_path, n, chunk, extra=[lat(heads=2, dim=12, mlp=dense(16))])
    toks, ref = m.tokens(n, vocab=23)
    assert err(m.ref(toks, causal_shift=1), ref) > 10 * F32_TOL
    if chunk:
        assert err(m.ref(toks, chunk_shift=1), ref) > 10 * F32_TOL and err(m.ref(toks, chunk_shift=chunk - 1), ref) > 10 * F32_TOL
    plan = m.plan("float32", ctx=n + 8, max_batch=96)
    assert err(whole(plan, toks), ref) < F32_TOL
    s = plan.acquire()
    got = [plan.step(s, toks[:decode_from], 0, list(range(decode_from)))]
    got += [plan.step(s, toks[i:i + 1], i, [0]) for i in range(decode_from, n)]
    plan.release(s)
    assert err(np.concatenate(got), ref) < F32_TOL
    assert err(stepwise(plan, toks, [61, 2, 3, 64, 2, 67, 5, 12]), ref) < F32_TOL
    plan.close()


@pytest.mark.parametrize("back", [1, 2, 15, 16, 63, 64, 127])
@pytest.mark.parametrize("inside", [True, False])
def test_one_key_at_a_chunks_edge(hy, tmp_path, back, inside):
    """A token stands at its chunk's first position (inside) or one before it (outside), nowhere else, and the token that looks for it `back` tokens later.  Inside,
    hiding that key moves the last logits by far more than the bound; outside, hiding it changes nothing, while chunks moved by one token
    would show it.  The plan follows with the prompt whole, in portions, and with the last tokens decoded."""
    chunk, first = 192, 192
    m = lookup_model(hy, tmp_path, 400 + 2 * back + inside, chunk)
    at = first if inside else first - 1
    n = at + back + 1
    toks = np.random.default_rng(back).integers(2, 97, n).astype(np.int32)
    toks[at], toks[n - 1] = 1, 0
    ref = m.ref(toks)
    hidden = err(m.ref(toks, drop_keys=[at])[-1:], ref[-1:])
    assert hidden > 20 * F32_TOL if inside else hidden < 1e-9
    if not inside:
        assert err(m.ref(toks, chunk_shift=1)[-1:], ref[-1:]) > 20 * F32_TOL
    for dtype, tol in (("float32", F32_TOL), ("bfloat16", BF16_TOL)):
        plan = m.plan(dtype, ctx=n, max_batch=200)
        assert err(whole(plan, toks), ref) < tol
        s = plan.acquire()
        plan.step(s, toks[:n - 3], 0, [])
        got = np.concatenate([plan.step(s, toks[i:i + 1], i, [0]) for i in range(n - 3, n)])
        plan.release(s)
        assert err(got, ref[n - 3:]) < tol
        assert err(stepwise(plan, toks, [190, 2, 2, 90]), ref) < tol
        plan.close()


@pytest.mark.parametrize("far", [0, 3, 63, 64, 127, 128, 191])
def test_one_far_key_among_hundreds(hy, tmp_path, far):
    """A token stands at position `far`, nowhere else, and the one that looks for it at the very end of one long chunk: the last query's look-up finds that one key
    among hundreds.  Hiding the key in the restatement moves the last logits by far more than the bound; the plan follows with the prompt
    whole, in portions, and with the last tokens decoded (the keys are then split over workgroups)."""
    m = lookup_model(hy, tmp_path, 300 + far, 512, dim=48 if far % 2 else 45)
    n = 450
    toks = np.random.default_rng(far).integers(2, 97, n).astype(np.int32)
    toks[far], toks[n - 1] = 1, 0
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


def latent_lookup(cfg, w, score=10.0):
    """Layer 0's latent attention becomes a look-up: the query latent is the key latent of the successor, and both expansions pass the latent on."""
    m = cfg["layers"][0]["mixer"]
    H, D, P, Rk = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    assert m["q_rank"] == Rk and D == Rk
    half = successor_embedding(w)
    w["l0.mix.dkv"][:Rk, half:] = 0.0
    w["l0.mix.dq"] = np.roll(w["l0.mix.dkv"][:Rk], half, axis=1)
    w["l0.mix.dq.norm"] = np.ones(Rk)
    w["l0.mix.dkv.norm"] = np.ones(Rk)
    uq = np.zeros((H, D + P, Rk))
    uq[:, :D] = np.eye(D) * score / (Rk * m["scale"])
    w["l0.mix.uq"] = uq.reshape(H * (D + P), Rk)
    w["l0.mix.uk"] = np.tile(np.eye(D), (H, 1))
    w["l0.mix.sink"] = np.full(H, -2.0)
    w["l0.norm1"] = np.full_like(w["l0.norm1"], 2.0)


@pytest.mark.parametrize("far", [0, 5, 63, 64, 200])
def test_one_far_key_reaches_the_latent_attention(hy, tmp_path, far):
    m = Model(hy, tmp_path, config([lat(heads=2, dim=32, rot=8, vdim=24, kv_rank=32, q_rank=32, scale=0.25, mlp=None)], width=64, vocab=97, side=0), seed=500 + far, tweak=latent_lookup)
    n = 420
    toks = np.random.default_rng(far).integers(2, 97, n).astype(np.int32)
    toks[far], toks[n - 1] = 1, 0
    toks[30], toks[31] = 50, 51          # a successor one token ahead, for the causal edge
    ref = m.ref(toks)
    assert err(m.ref(toks, drop_keys=[far])[-1:], ref[-1:]) > 20 * F32_TOL and err(m.ref(toks, causal_shift=1), ref) > 10 * F32_TOL
    plan = m.plan("float32", ctx=n, max_batch=150)
    assert err(whole(plan, toks), ref) < F32_TOL
    s = plan.acquire()
    plan.step(s, toks[:n - 4], 0, [])
    got = np.concatenate([plan.step(s, toks[i:i + 1], i, [0]) for i in range(n - 4, n)])
    plan.release(s)
    plan.close()
    assert err(got, ref[n - 4:]) < F32_TOL


@pytest.mark.parametrize("kind", ["parallel", "latent"])
def test_sinks_weigh(hy, tmp_path, kind):
    """Large sinks of different size per head, on the first tokens (few keys beside them) and later: leaving them out, or swapping two heads',
    moves the restatement by far more than the bound.  (Each output passes a norm: only the heads' shares against each other show.)"""
    name = "l0.mix.left.sink" if kind == "parallel" else "l0.mix.sink"

    def tweak(cfg, w):
        w[name] = np.linspace(-3.0, 6.0, w[name].size)

    m = Model(hy, tmp_path, config([par(mlp=None) if kind == "parallel" else lat(mlp=None)], side=0), seed=70, tweak=tweak)
    toks, ref = m.tokens(60)
    for other in (np.full_like(m.w64[name], -100.0), np.roll(m.w64[name], 1)):
        assert err_rows(R.forward(m.cfg, dict(m.w64, **{name: other}), toks), ref).min() > 5 * F32_TOL
    plan = m.plan("float32", ctx=64)
    for sizes in ([60], [1], [2, 30, 3]):
        assert err(stepwise(plan, toks, sizes), ref) < F32_TOL, sizes
    plan.close()


def test_heads_mix_tempers_and_cap_matter(hy, tmp_path):
    """Each of the score's steps, left out of the restatement, or the mixing matrix turned over, moves the logits by far more than the bound."""
    m = Model(hy, tmp_path, config([par(cap=2.0, scale=0.5, mlp=None)], side=0), seed=72)
    toks, ref = m.tokens(60)
    p = "l0.mix.left."
    for name, v in (("talk", np.eye(4)), ("talk", m.w64[p + "talk"].T), ("temp", np.ones(4)), ("temp", np.roll(m.w64[p + "temp"], 1))):
        assert err(R.forward(m.cfg, dict(m.w64, **{p + name: v}), toks), ref) > 10 * F32_TOL, name
    free = copy.deepcopy(m.cfg)
    del free["layers"][0]["mixer"]["left"]["softcap"]
    assert err(R.forward(free, m.w64, toks), ref) > 10 * F32_TOL
    plan = m.plan("float32", ctx=64)
    assert err(whole(plan, toks), ref) < F32_TOL and err(stepwise(plan, toks, [1]), ref) < F32_TOL
    plan.close()


def test_far_tokens_reach_the_memory(hy, tmp_path):
    """The first tokens of a long prompt decide the last logits only through the delta rule's states, whose decay is nearly one and whose keys
    are long (so that later writes overwrite little): changing two early tokens moves the restatement's last logits by far more than the
    bound, and the plan follows, whole and decoded."""
    def tweak(cfg, w):
        w["l0.mix.right.A_log"] = np.full_like(w["l0.mix.right.A_log"], -9.0)
        w["l0.mix.right.b"] = w["l0.mix.right.b"] * 0.05
        w["l0.mix.left.out"] = np.zeros_like(w["l0.mix.left.out"])
        w["l0.norm1"] = np.full_like(w["l0.norm1"], 3.0)

    m = Model(hy, tmp_path, config([par(chunk=8, d_heads=2, d_kv_heads=1, d_dim=120, d_vdim=16, mlp=None)], width=48, vocab=61, side=0), seed=77, tweak=tweak)
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


def test_delta_gates_at_their_limits(hy, tmp_path):
    """Heads that forget everything, nothing, write everything, nothing, side by side."""
    def tweak(cfg, w):
        w["l0.mix.right.A_log"] = np.array([4.0, -12.0, 0.0, 0.0])
        w["l0.mix.right.dt_bias"] = np.array([6.0, -20.0, 25.0, -3.0])
        w["l0.mix.right.b"][2:] *= 30.0

    m = Model(hy, tmp_path, config([par(d_heads=4, d_kv_heads=2)]), seed=78, tweak=tweak)
    toks, ref = m.tokens(120)
    plan = m.plan("float32", ctx=128)
    assert err(whole(plan, toks), ref) < F32_TOL
    assert err(stepwise(plan, toks, [30, 2, 1]), ref) < F32_TOL
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
    layers = [par(heads=2, kv_heads=1, dim=16, vdim=16, rot=8, chunk=90, d_heads=2, d_kv_heads=1, d_dim=16, d_vdim=8, mlp=dense(16)), lat(heads=2, mlp=None)]
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


def test_rotation_is_by_position_not_by_place_in_the_step_or_chunk(hy, tmp_path):
    """With a small base the turns are large, and a portion or a chunk that starts late must turn by its true positions (in the latent attention
    and, seen through the mixed heads' scores of one chunk, in the other)."""
    m = Model(hy, tmp_path, config([par(dim=24, rot=24, base=3.0, scale=1.0, chunk=31), lat(rot=16, base=3.0, scaling=None)]), seed=61)
    toks, ref = m.tokens(70)
    plan = m.plan("float32", ctx=80)
    assert err(stepwise(plan, toks, [33, 2, 1, 20, 14]), ref) < F32_TOL
    plan.close()


def test_groups_close_choices_with_negative_scores(hy, tmp_path):
    """Corrections that put every choice score below zero: a closed group's choices stay closed (they count as minus infinity, not as zero), a
    group ranks by its largest choice score, not by its two largest, and identity choices among the open ones return the residual itself."""
    def tweak(cfg, w):
        w["l0.mlp.correction"] = np.array([-8.0, -8.0, -3.0, -19.0, -4.0, -4.0, -2.0, -30.0])

    m = Model(hy, tmp_path, config([par(mlp=moe(experts=6, identity=2, top=3, ff=16, groups=(4, 2)))]), seed=88, tweak=tweak)
    toks, ref = m.tokens(40)
    h = np.random.default_rng(0).standard_normal((9, 88))
    choice, _ = R.route(h, R.sub(m.w64, "l0.mlp."), m.cfg["layers"][0]["mlp"])
    assert all(list(c) == [6, 2, 3] for c in choice)                     # two largest summed would open the pair at -4
    plan = m.plan("float32", ctx=64)
    assert err(whole(plan, toks), ref) < F32_TOL
    assert err(stepwise(plan, toks, [1]), ref) < F32_TOL
    plan.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_tokens_without_any_expert(hy, tmp_path, dtype):
    """Every choice an identity choice, for all tokens and for none, in the same model: the feed-forward is then the normed residual."""
    def tweak(cfg, w):
        w["l0.mlp.correction"] = np.array([-9.0] * 4 + [5.0] * 4)
        w["l1.mlp.correction"] = np.array([5.0] * 4 + [-9.0] * 4)

    layers = [par(mlp=moe(experts=4, identity=4, top=3, groups=None)), lat(mlp=moe(experts=4, identity=4, top=3, groups=None))]
    m = Model(hy, tmp_path, config(layers), seed=89, tweak=tweak)
    toks, ref = m.tokens(40)
    plan = m.plan(dtype, ctx=64)
    for got in (whole(plan, toks), stepwise(plan, toks, [1])):
        assert err(got, ref) < F32_TOL if dtype == "float32" else bf16_ok(m, toks, got, ref)
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
    m = Model(hy, tmp_path, config([par(mlp=moe()), lat()]), seed=54)
    for name in ("embed", "side.embed", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.left.q.norm", "l0.mix.left.talk", "l0.mix.left.temp", "l0.mix.left.sink", "l0.mix.left.out",
                 "l0.mix.left.o", "l0.mix.right.q.conv", "l0.mix.right.v.conv", "l0.mix.right.a", "l0.mix.right.b", "l0.mix.right.A_log", "l0.mix.right.dt_bias", "l0.mix.right.norm",
                 "l0.mix.right.g", "l0.mix.right.o", "l0.mix.right.out", "l0.mlp.correction", "l0.mlp.router", "l0.mlp.e3.up", "l0.side.gate", "l0.side.norm", "l1.mix.dq.norm", "l1.mix.uq",
                 "l1.mix.sink", "l1.mix.g", "l1.mlp.up"):
        w = dict(m.w)
        del w[name]
        hy.save_model_dir(str(tmp_path / "bad"), m.cfg, w)
        with pytest.raises(hy.hip.Gl3Error):
            hy.HybridPlan.from_dir(str(tmp_path / "bad"))
    for name in ("l0.mlp.correction", "l0.mlp.router", "l0.mix.left.talk", "l0.mix.left.temp", "l0.mix.right.k.conv", "l0.mix.right.out", "l0.mix.right.v", "l0.mix.right.o", "l1.mix.sink"):
        w = dict(m.w)
        w[name] = np.concatenate([w[name], w[name]])
        hy.save_model_dir(str(tmp_path / "bad"), m.cfg, w)
        with pytest.raises(hy.hip.Gl3Error):
            hy.HybridPlan.from_dir(str(tmp_path / "bad"))


# ---- a mechanism is a parameter of the family, not of one design ------------------------------------------------------------------------
def describe(hip, layer, beside=None, **model):
    """(model descriptor, what must stay alive) of a one-layer model on the plain residual."""
    d = hip.ModelDesc()
    d.struct_size, d.arch, d.dim, d.vocab, d.ctx, d.max_batch, d.weight_type, d.n_layers, d.rms_eps = C.sizeof(hip.ModelDesc), 6, 16, 8, 64, 40, 30, 1, 1e-5
    ls = []
    for spec in (layer, beside):
        if spec is None:
            continue
        l = hip.LayerDesc()
        for k, v in dict(dict(mixer=0, heads=2, kv_heads=1, dim=8, vdim=8, scale=1.0), **spec).items():
            setattr(l, k, v)
        ls.append(l)
    if beside is not None:
        ls[0].beside = C.cast(C.pointer(ls[1]), C.c_void_p)
    for k, v in model.items():
        setattr(d, k, v)
    d.layer_descs = C.pointer(ls[0])
    return d, ls


def test_descriptor_takes_or_refuses_combinations(hy):
    """The descriptor combines the new mechanisms with older ones: one that cannot be combined is refused before any device memory is taken."""
    hip = hy.hip

    def create(layer, beside=None, **model):
        d, keep = describe(hip, layer, beside, **model)
        p = C.c_void_p()
        r = hip.lib().gl3_create(C.byref(d), C.byref(p))
        if p:
            hip.lib().gl3_destroy(p)
        return r

    delta = {"mixer": 3, "mem_gates": 3, "mem_conv": 3, "mem_qk_unit": 1}
    assert create({"chunk": 4}) == 0 and create({"score_softcap": 5.0, "softmax_sink": 1}) == 0 and create({"head_mix": 1, "out_gate": 2}) == 0 and create({"head_temp": 1, "v_rot": 1, "rot_base": 9.0}) == 0
    assert create(delta) == 0 and create(dict(delta, mem_gate_act=2)) == 0 and create({"mixer": 1, "kv_rank": 5, "softmax_sink": 2}) == 0
    assert create({}, delta) == 0 and create({"out_norm": 1}, dict(delta, out_norm=1), post_norms=1, side_dim=3) == 0
    assert create({"ff": 8}, post_norms=1, no_pre_norms=1, layer_scale=1) == 0 and create({"ff": 8, "experts": 3, "identity": 2, "top": 4, "route_on_output": 1}) == 0
    for layer, beside, model in (({"chunk": 4, "window": 3}, None, {}), ({"head_mix": 1, "slope_log2": 8.0}, None, {}), ({"head_mix": 1, "heads": 130}, None, {}), ({"chunk": -1}, None, {}),
                                 ({"mixer": 3, "mem_gates": 4}, None, {}), ({"mixer": 3, "mem_gates": 2, "mem_conv": 3}, None, {}), (dict(delta, mem_conv=0), None, {}), (dict(delta, mem_conv=65), None, {}),
                                 (dict(delta, heads=3, kv_heads=2), None, {}), (dict(delta, rot_dims=2, rot_base=9.0), None, {}), (dict(delta, dim=1025), None, {}),
                                 (dict(delta, chunk=3), None, {}), ({"out_norm": 1}, None, {}), ({"out_norm": 1}, delta, {}), ({}, dict(delta, out_norm=1), {}),
                                 ({"out_norm": 1}, dict(delta, out_norm=1), {"parallel_block": 1}), ({}, None, {"no_pre_norms": 1}), ({}, None, {"no_pre_norms": 1, "post_norms": 1, "token_shift": 1}),
                                 ({"ff": 8, "experts": 3, "identity": 2, "top": 4}, None, {}), ({"ff": 8, "identity": 2}, None, {}),
                                 ({"ff": 8, "experts": 3, "identity": 2, "top": 6, "route_on_output": 1}, None, {})):
        assert create(layer, beside, **model) != 0, (layer, beside, model)


@pytest.mark.parametrize("switches", [{"chunk": 5}, {"score_softcap": 0.8}, {"head_temp": 1}, {"head_mix": 1}, {"chunk": 7, "head_mix": 1, "out_gate": 1}])
def test_score_switches_alone(hy, switches):
    """A design of another kind — a norm in front of the mixer, no norm behind it, no feed-forward — that uses one of the score's switches without
    the others, built through the descriptor."""
    hip = hy.hip
    W, V, H, D, n = 16, 8, 2, 8, 40
    d, keep = describe(hip, dict(switches, scale=0.6), flags=hip.FLAG_F32_COMPUTE)
    ctx = C.c_void_p()
    hip.check(hip.lib().gl3_create(C.byref(d), C.byref(ctx)))
    rng = np.random.default_rng(5)
    w = {0: rng.standard_normal((V, W)), 1: np.ones(W), 3: 1 + 0.1 * rng.standard_normal(W), 4: rng.standard_normal((H * D, W)) / 4, 5: rng.standard_normal((D, W)) / 4,
         6: rng.standard_normal((D, W)) / 4, 7: rng.standard_normal((W, H * D)) / 4}
    if switches.get("head_temp"):
        w[65] = np.array([0.5, 2.0])
    if switches.get("head_mix"):
        w[66] = np.array([[0.3, 0.9], [-0.5, 1.1]])
    if switches.get("out_gate"):
        w[24] = rng.standard_normal((H * D, W)) / 4
    w = {k: np.ascontiguousarray(v, np.float32) for k, v in w.items()}
    for k, v in w.items():
        hip.check(hip.lib().gl3_upload_tensor(ctx, k, 0, v.ctypes.data_as(C.c_void_p), v.nbytes, hip.TYPE_F32), ctx)
    hip.check(hip.lib().gl3_finalize(ctx), ctx)
    plan = hy.HybridPlan(ctx)
    toks = rng.integers(0, V, n).astype(np.int32)
    x = np.asarray(w[0], np.float64)[toks]
    h = R.rms_norm(x, 1e-5, w[3])
    q, k, v = (h @ w[4].T.astype(np.float64)).reshape(n, H, D), (h @ w[5].T).reshape(n, 1, D), (h @ w[6].T).reshape(n, 1, D)
    s = R.head_scores(q, k, {"scale": 0.6, "softcap": switches.get("score_softcap")}, w.get(65, np.ones(H)))
    if 66 in w:
        s = np.einsum("hg,gij->hij", w[66], s)
    s = np.where(R.chunk_mask(n, switches.get("chunk", 0)), s, -np.inf)
    a = np.exp(s - s.max(axis=-1, keepdims=True))
    o = np.einsum("hij,jv->ihv", a / a.sum(axis=-1, keepdims=True), v[:, 0]).reshape(n, H * D)
    if 24 in w:
        o = o * R.sigmoid(h @ w[24].T)
    ref = R.rms_norm(x + o @ w[7].T, 1e-5) @ w[0].T
    for sizes in ([n], [1], [30, 3, 7]):
        assert err(stepwise(plan, toks, sizes), ref) < F32_TOL, sizes
    plan.close()
