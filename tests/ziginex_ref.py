"""Plain, slow restatement of the Ziginex design in float64 numpy: one function per mechanism, whole sequences at once, no cache
carried between calls.  It shares no code with the product path (csrc/gl3_hybrid*.h, csrc/gl3_hy*_kernels.h) and is the yardstick of
tests/test_ziginex*.py.

Notation: T tokens at positions 0 .. T - 1, W model width, h the [T, W] input of a sublayer, weights as [out, in] matrices applied as
h @ M.T.  A mixer's weights are a dict keyed by the tensor's name behind "<layer>.mix." ("left.q", "right.k.conv", "dkv.norm", ...), a
feed-forward's by the name behind "<layer>.mlp." ("up", "e3.down", "router", "correction").

The design: x_0 = embed[token]; every layer is
    x <- x + N(mixer(x), norm1);   x <- x + N(ff(x), norm2);   x <- x + N(W_proj (gelu_tanh(W_gate x) * e), side.norm)
(the second step only where the layer has a feed-forward; e = the layer's part of the token's row of a second table),
N(y, w) = y / rms(y) * w; logits = embed N(x, final.norm).  Mixers: "parallel" (attention whose heads' scores are capped and mixed with
each other, inside chunks of the sequence, beside a gated delta rule; the two outputs are normed and averaged) and "latent_attention"
(keys and values expanded from a cached latent, one rotated key part for all heads, a sink and an output gate).
"""
from __future__ import annotations

import math

import numpy as np


def bf16_round(a):
    """float32 values that bfloat16 holds exactly (round to nearest even)."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32).reshape(np.shape(a))


ROUND_INPUTS = False          # set by forward(round_inputs=True)


def inp(x):
    """The input of a matrix product: as it is, or (ROUND_INPUTS) rounded to bfloat16 as a bfloat16 plan rounds it."""
    return np.asarray(bf16_round(x), np.float64) if ROUND_INPUTS else x


def rms_norm(x, eps, w=None):
    """x / sqrt(mean(x^2) + eps) over the last axis, times w if given."""
    y = x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)
    return y if w is None else y * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- positions ----------------------------------------------------------------------------------------------------------------------
def frequencies(rot):
    """base^(-2 i / dims) per pair and the multiplier of cos and sin.  With rot.scaling the frequency of pair i leans towards f / factor
    along a ramp between the pair indices at which a wave makes `fast` and `slow` turns over `original` positions."""
    n, sc, base = rot["dims"], rot.get("scaling"), float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if not sc:
        return np.array(f), 1.0
    where = lambda turns: n * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(where(sc["fast"])), 0), min(math.ceil(where(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return np.array(out), 0.1 * math.log(sc["factor"]) + 1.0


def turn(x, pos, rot, interleaved):
    """Rotary turn of the first rot.dims entries of the last axis; pairs (2 i, 2 i + 1), or (i, i + dims / 2).  x: [T, heads, D]."""
    n = rot["dims"]
    f, mul = frequencies(rot)
    a = np.asarray(pos, np.float64)[:, None, None] * f
    c, s = mul * np.cos(a), mul * np.sin(a)
    first, second = (slice(0, n, 2), slice(1, n, 2)) if interleaved else (slice(0, n // 2), slice(n // 2, n))
    out = x.copy()
    u, v = x[..., first], x[..., second]
    out[..., first], out[..., second] = u * c - v * s, v * c + u * s
    return out


# ---- softmax ------------------------------------------------------------------------------------------------------------------------
def sink_softmax(s, sink):
    """exp(s) / (exp(sink) + sum exp(s)) over the last axis; -inf = not seen.  sink: a number per row of the last axis (broadcast)."""
    m = np.maximum(s.max(axis=-1, keepdims=True), sink[..., None])
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink[..., None] - m))


def chunk_mask(T, size, causal_shift=0, chunk_shift=0):
    """seen[i, j]: j <= i and both in the same run of `size` positions (counted from position 0; size 0: no runs).  The shifts are knobs
    for the tests' sensitivity checks: the causal edge, and the runs' first positions, moved by that many tokens (a token always sees itself)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = j <= i + causal_shift
    if size:
        seen &= (i + chunk_shift) // size == (j + chunk_shift) // size
    return seen | (i == j)


# ---- attention whose heads' scores mix ------------------------------------------------------------------------------------------------
def head_scores(q, k, c, temp):
    """cap tanh(scale temp_h q_h . k_g / cap) for every head, query and key: [H, T, T].  q: [T, H, D], k: [T, G, D]."""
    H, G = q.shape[1], k.shape[1]
    s = np.stack([q[:, h] @ k[:, h // (H // G)].T * c["scale"] * temp[h] for h in range(H)])
    return c["softcap"] * np.tanh(s / c["softcap"]) if c.get("softcap") else s


def mixed_attention(h, p, c, eps, causal_shift=0, chunk_shift=0, drop_keys=()):
    """drop_keys: positions hidden from later queries (a knob, as the shifts)."""
    T = h.shape[0]
    H, G, D, V = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    h = inp(h)
    q, k, v = (h @ p["q"].T).reshape(T, H, D), (h @ p["k"].T).reshape(T, G, D), (h @ p["v"].T).reshape(T, G, V)
    q, k = rms_norm(q, eps, p["q.norm"]), rms_norm(k, eps, p["k.norm"])
    if c.get("rot"):
        q, k = turn(q, np.arange(T), c["rot"], True), turn(k, np.arange(T), c["rot"], True)
    s = np.einsum("hg,gij->hij", p["talk"], head_scores(q, k, c, p["temp"]))
    seen = chunk_mask(T, (c.get("mask") or {}).get("size", 0), causal_shift, chunk_shift)
    for j in drop_keys:
        seen[j + 1:, j] = False
    w = sink_softmax(np.where(seen, s, -np.inf), np.broadcast_to(p["sink"][:, None], (H, T)))
    o = np.stack([w[hd] @ v[:, hd // (H // G)] for hd in range(H)], axis=1)
    return inp(o.reshape(T, H * V)) @ p["o"].T


# ---- gated delta rule -----------------------------------------------------------------------------------------------------------------
def short_conv(u, w):
    """y_t[c] = sum_j w[c, j] u_(t - taps + 1 + j)[c], zeros before the sequence.  u: [T, C], w: [C, taps]."""
    T, taps = u.shape[0], w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, u.shape[1])), u])
    return sum(pad[j:j + T] * w[:, j] for j in range(taps))


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_memory(q, k, v, g, beta):
    """Per head S <- g S; S <- S + k (beta (v - S^T k))^T; o = S^T q from S = 0.  q, k: [T, H, D], v: [T, H, V], g, beta: [T, H]."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]))
    o = np.zeros(v.shape)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o


def delta_gates(h, p):
    """decay g = exp(-exp(A_log) softplus(W_a h + dt_bias)) and write strength beta = sigmoid(W_b h), [T, heads] each."""
    return np.exp(-np.exp(p["A_log"]) * np.logaddexp(0.0, h @ p["a"].T + p["dt_bias"])), sigmoid(h @ p["b"].T)


def gated_delta(h, p, c, eps):
    T = h.shape[0]
    H, G, D, V = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    h = inp(h)
    q, k, v = (silu(short_conv(h @ p[n].T, p[n + ".conv"])) for n in "qkv")
    of = np.arange(H) // (H // G)                                  # the key head of every head
    q, k = unit(q.reshape(T, G, D))[:, of] / math.sqrt(D), unit(k.reshape(T, G, D))[:, of]
    o = delta_memory(q, k, v.reshape(T, H, V), *delta_gates(h, p))
    o = rms_norm(o, eps, p["norm"]).reshape(T, H * V) * silu(h @ p["g"].T)
    return inp(o) @ p["o"].T


def parallel(h, p, c, eps, **knobs):
    left, right = sub(p, "left."), sub(p, "right.")
    return 0.5 * (rms_norm(mixed_attention(h, left, c["left"], eps, **knobs), eps, left["out"]) + rms_norm(gated_delta(h, right, c["right"], eps), eps, right["out"]))


# ---- latent attention -------------------------------------------------------------------------------------------------------------------
def latent_attention(h, p, c, eps, causal_shift=0, drop_keys=(), **_):
    T = h.shape[0]
    H, D, P, V, R = c["heads"], c["dim"], c.get("rot_dim", 0), c["vdim"], c["kv_rank"]
    h = inp(h)
    q = (inp(rms_norm(h @ p["dq"].T, eps, p["dq.norm"])) @ p["uq"].T).reshape(T, H, D + P)
    down = h @ p["dkv"].T
    lat, kr = rms_norm(down[:, :R], eps, p["dkv.norm"]), down[:, None, R:]
    if P:
        kr = turn(kr, np.arange(T), c["rot"], False)
        q = np.concatenate([q[..., :D], turn(q[..., D:], np.arange(T), c["rot"], False)], axis=-1)
    k = np.concatenate([(lat @ p["uk"].T).reshape(T, H, D), np.broadcast_to(kr, (T, H, P))], axis=-1)
    v = (lat @ p["uv"].T).reshape(T, H, V)
    seen = chunk_mask(T, 0, causal_shift)
    for j in drop_keys:
        seen[j + 1:, j] = False
    s = np.einsum("ihd,jhd->hij", q, k) * c["scale"]
    w = sink_softmax(np.where(seen, s, -np.inf), np.broadcast_to(p["sink"][:, None], (H, T)))
    o = np.einsum("hij,jhv->ihv", w, v).reshape(T, H * V) * sigmoid(h @ p["g"].T)
    return inp(o) @ p["o"].T


# ---- feed-forward -----------------------------------------------------------------------------------------------------------------
def gated_ff(h, gate, up, down):
    h = inp(h)
    return inp(silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(h, p, c):
    """Chosen outputs [T, top] of the router and their weights.  Scores: softmax over all of its outputs (experts, then identity experts);
    choice scores = scores + correction.  The outputs form groups.count runs of neighbours; a group's score is its largest choice
    score; only the best groups.keep groups are open to the choice of the `top` largest choice scores (the lowest index wins a tie).  The
    weights are the plain scores, not renormalised."""
    r = c["router"]
    z = inp(h) @ p["router"].T
    z = np.exp(z - z.max(axis=-1, keepdims=True))
    s = z / z.sum(axis=-1, keepdims=True)
    cs = s + p["correction"]
    n, grp = cs.shape[-1], r.get("groups")
    if grp:
        score = cs.reshape(-1, grp["count"], n // grp["count"]).max(axis=-1)
        kept = np.argsort(-score, axis=-1, kind="stable")[:, :grp["keep"]]
        closed = np.ones(score.shape, bool)
        np.put_along_axis(closed, kept, False, axis=-1)
        cs = np.where(np.repeat(closed, n // grp["count"], axis=-1), -np.inf, cs)
    choice = np.argsort(-cs, axis=-1, kind="stable")[:, :r["top"]]
    return choice, np.take_along_axis(s, choice, axis=-1)


def moe_ff(h, p, c):
    choice, w = route(h, p, c)
    E = c["router"]["experts"]
    out = np.zeros(h.shape)
    for t in range(h.shape[0]):
        for e, we in zip(choice[t], w[t]):
            out[t] += we * (h[t] if e >= E else gated_ff(h[t:t + 1], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])[0])
    return out


# ---- per-layer token input ----------------------------------------------------------------------------------------------------------
def token_input(x, e, gate, proj, norm, eps):
    return rms_norm(inp(gelu_tanh(inp(x) @ gate.T) * e) @ proj.T, eps, norm)


# ---- the model --------------------------------------------------------------------------------------------------------------------
def sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, taps=None, round_inputs=False, **knobs):
    """Logits [T, vocab] of one sequence; taps (a list) receives the residual stream [T, W] after every layer.  weights: name -> float64
    array.  round_inputs: every matrix product's input is rounded to bfloat16 first (see inp).  knobs go to every attention."""
    global ROUND_INPUTS
    ROUND_INPUTS = round_inputs
    try:
        return _forward(cfg, weights, tokens, taps, knobs)
    finally:
        ROUND_INPUTS = False


def _forward(cfg, weights, tokens, taps, knobs):
    eps = cfg["norm"]["eps"]
    n = (cfg.get("token_side") or {}).get("dim", 0)
    tokens = np.asarray(tokens)
    x = weights["embed"][tokens]
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        mixer = {"parallel": parallel, "latent_attention": latent_attention}[layer["type"]]
        x = x + rms_norm(mixer(x, sub(weights, pre + "mix."), layer["mixer"], eps, **knobs), eps, weights[pre + "norm1"])
        mlp = layer.get("mlp")
        if mlp:
            f = sub(weights, pre + "mlp.")
            y = gated_ff(x, f["gate"], f["up"], f["down"]) if mlp["kind"] == "dense" else moe_ff(x, f, mlp)
            x = x + rms_norm(y, eps, weights[pre + "norm2"])
        if n:
            e = weights["side.embed"][tokens][:, i * n:(i + 1) * n]
            x = x + token_input(x, e, weights[pre + "side.gate"], weights[pre + "side.proj"], weights[pre + "side.norm"], eps)
        if taps is not None:
            taps.append(x.copy())
    return inp(rms_norm(x, eps, weights["final.norm"])) @ weights["embed"].T


# ---- random models for the tests ----------------------------------------------------------------------------------------------------
def tensor_shapes(cfg):
    """{tensor name: shape} of a configuration, in file order."""
    W, V = cfg["width"], cfg["vocab"]
    n = (cfg.get("token_side") or {}).get("dim", 0)
    out = {"embed": (V, W)}
    if n:
        out["side.embed"] = (V, n * len(cfg["layers"]))
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = "l%d." % i, layer["mixer"], layer.get("mlp")
        out[p + "norm1"] = (W,)
        if layer["type"] == "parallel":
            a, d = m["left"], m["right"]
            H = a["heads"]
            mix = {"left.q": (H * a["dim"], W), "left.k": (a["kv_heads"] * a["dim"], W), "left.v": (a["kv_heads"] * a["vdim"], W), "left.q.norm": (a["dim"],),
                   "left.k.norm": (a["dim"],), "left.talk": (H, H), "left.temp": (H,), "left.sink": (H,), "left.o": (W, H * a["vdim"])}
            H = d["heads"]
            for name, rows in (("q", d["kv_heads"] * d["dim"]), ("k", d["kv_heads"] * d["dim"]), ("v", H * d["vdim"])):
                mix["right." + name], mix["right." + name + ".conv"] = (rows, W), (rows, d["conv"])
            mix.update({"right.b": (H, W), "right.A_log": (H,), "right.norm": (d["vdim"],), "right.a": (H, W), "right.dt_bias": (H,), "right.g": (H * d["vdim"], W),
                        "right.o": (W, H * d["vdim"]), "left.out": (W,), "right.out": (W,)})
        else:
            H, P, R, od = m["heads"], m.get("rot_dim", 0), m["kv_rank"], m["heads"] * m["vdim"]
            mix = {"dq": (m["q_rank"], W), "dq.norm": (m["q_rank"],), "uq": (H * (m["dim"] + P), m["q_rank"]), "dkv": (R + P, W), "dkv.norm": (R,),
                   "uk": (H * m["dim"], R), "uv": (od, R), "sink": (H,), "g": (od, W), "o": (W, od)}
        out.update({p + "mix." + k: v for k, v in mix.items()})
        if ff:
            out[p + "norm2"] = (W,)
            if ff["kind"] == "dense":
                out.update({p + "mlp.gate": (ff["ff"], W), p + "mlp.up": (ff["ff"], W), p + "mlp.down": (W, ff["ff"])})
            else:
                f, r = ff["expert"]["ff"], ff["router"]
                for e in range(r["experts"]):
                    out.update({p + "mlp.e%d.gate" % e: (f, W), p + "mlp.e%d.up" % e: (f, W), p + "mlp.e%d.down" % e: (W, f)})
                out.update({p + "mlp.router": (r["experts"] + r.get("identity", 0), W), p + "mlp.correction": (r["experts"] + r.get("identity", 0),)})
        if n:
            out.update({p + "side.gate": (n, W), p + "side.proj": (W, n), p + "side.norm": (W,)})
    out["final.norm"] = (W,)
    return out


def random_weights(cfg, seed):
    """bfloat16-representable float32 weights: matrices ~ N(0, 1 / fan_in), gate and router projections larger (so that gates move and
    scores spread), norm weights around one (the sublayers' output norms around 0.6), the heads' mixing around the identity."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shp in tensor_shapes(cfg).items():
        leaf = name.split(".", 1)[1] if name[0] == "l" and name[1].isdigit() else name
        last = leaf.rsplit(".", 1)[-1]
        if leaf in ("norm1", "norm2", "side.norm"):
            a = 0.6 + 0.2 * rng.standard_normal(shp)
        elif last in ("norm", "out"):
            a = 1.0 + 0.2 * rng.standard_normal(shp)
        elif last == "talk":
            a = np.eye(shp[0]) + 0.4 * rng.standard_normal(shp) / math.sqrt(shp[0])
        elif last == "temp":
            a = rng.uniform(0.6, 1.8, shp)
        elif last == "sink":
            a = rng.standard_normal(shp)
        elif last == "A_log":
            a = rng.uniform(-2.5, 0.5, shp)
        elif last == "dt_bias":
            a = rng.uniform(-3.0, 0.5, shp)
        elif last == "conv":
            a = rng.standard_normal(shp) / math.sqrt(shp[1])
        elif last == "correction":
            a = 0.1 * rng.standard_normal(shp)
        elif leaf in ("embed", "side.embed"):
            a = rng.standard_normal(shp)
        elif last in ("g", "a", "b", "router"):
            a = 2.0 * rng.standard_normal(shp) / math.sqrt(shp[-1])
        else:
            a = rng.standard_normal(shp) / math.sqrt(shp[-1])
        out[name] = bf16_round(a)
    return out


def to_f64(w):
    return {k: np.asarray(v, np.float64) for k, v in w.items()}
