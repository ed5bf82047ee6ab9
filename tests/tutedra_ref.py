"""Plain, slow restatement of the Tutedra design in float64 numpy: one function per mechanism, whole sequences at once, no cache
carried between calls.  It shares no code with the product path (csrc/gl3_hybrid*.h, csrc/gl3_hy*_kernels.h) and is the yardstick of
tests/test_tutedra*.py.

Notation: T tokens at positions 0 .. T - 1, W model width, h the [T, W] input of a sublayer, weights as [out, in] matrices applied as
h @ M.T.  A mixer's weights are a dict keyed by the tensor's name behind "<layer>.mix." ("q", "k.conv", "f.b", ...), a feed-forward's by
the name behind "<layer>.mlp." ("up", "act", "e3.up", "shared.sg", "router", "correction").

The design: x_0 = embed[token] + bigram[row of the token pair]; every layer is
    h = norm(x, norm1);  h <- h + (previous token's h - h) * shift;  x <- x + mixer(h) * ls1;   x <- x + ff(norm(x, norm2)) * ls2
(the last step only where the layer has a feed-forward), norm(x, w) = x / rms(x) * (1 + w); logits = embed norm(x, final.norm).
Mixers: "hgrn2" (linear attention whose forget gate, one per channel, also writes), "mlstm" (matrix memory with exponential gates) and
"attention" (short convolutions on q and k, values = convolved keys, weighted q / k norms per head, partial rotary turn).
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


# ---- embedding --------------------------------------------------------------------------------------------------------------------
def bigram_rows(tokens, b):
    """Row of the pair table per token: (previous mul_prev + token mul_cur) mod buckets; the sequence's first token takes the row behind
    the last bucket."""
    rows = [b["buckets"]]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * b["mul_prev"] + int(cur) * b["mul_cur"]) % b["buckets"])
    return rows


def embedding(tokens, weights, cfg):
    x = weights["embed"][np.asarray(tokens)]
    b = (cfg.get("embedding") or {}).get("bigram")
    return x + weights["bigram"][bigram_rows(list(tokens), b)] if b else x


# ---- what stands between a norm and a mixer -----------------------------------------------------------------------------------------
def token_shift(h, shift):
    """h_t + (h_(t-1) - h_t) * shift, with zeros before the first token (h_(t-1) as it was before its own shift)."""
    prev = np.concatenate([np.zeros_like(h[:1]), h[:-1]])
    return h + (prev - h) * shift


# ---- hgrn2 ----------------------------------------------------------------------------------------------------------------------------
def channel_gated_memory(q, f, v):
    """Per head S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T, o_t = S_t^T q_t from S = 0.  q, f: [T, H, D], v: [T, H, V]."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]))
    o = np.zeros(v.shape)
    for t in range(T):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o


def hgrn2(h, p, c, eps):
    T = h.shape[0]
    H, D, V = c["heads"], c["dim"], c["vdim"]
    h = inp(h)
    q = silu(h @ p["q"].T)
    f = p["lower"] + (1.0 - p["lower"]) * sigmoid(h @ p["f"].T + p["f.b"])
    o = channel_gated_memory(q.reshape(T, H, D), f.reshape(T, H, D), (h @ p["v"].T).reshape(T, H, V))
    return inp(rms_norm(o, eps, p["norm"]).reshape(T, H * V)) @ p["o"].T


# ---- mlstm ----------------------------------------------------------------------------------------------------------------------------
def exp_gated_memory(q, k, v, i, f):
    """Per head, with log gates i and f ([T, H]): m_t = max(f + m_(t-1), i) from m = 0; S and n decay by exp(f + m_(t-1) - m_t) and gain
    exp(i - m_t) times k v^T and k; o = S^T q / (max(|n . q|, exp(-m)) + 1e-6)."""
    T, H, D = q.shape
    S, n, m = np.zeros((H, D, v.shape[2])), np.zeros((H, D)), np.zeros(H)
    o = np.zeros(v.shape)
    for t in range(T):
        m_new = np.maximum(f[t] + m, i[t])
        a, b = np.exp(f[t] + m - m_new), np.exp(i[t] - m_new)
        S = a[:, None, None] * S + b[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = a[:, None] * n + b[:, None] * k[t]
        m = m_new
        den = np.maximum(np.abs(np.einsum("hd,hd->h", n, q[t])), np.exp(-m)) + 1e-6
        o[t] = np.einsum("hdv,hd->hv", S, q[t]) / den[:, None]
    return o


def log_gates(h, p, cap):
    zi, zf = h @ p["i"].T + p["i.b"], h @ p["f"].T + p["f.b"]
    return cap * np.tanh(zi / cap), -np.logaddexp(0.0, -cap * np.tanh(zf / cap))


def mlstm(h, p, c, eps):
    T = h.shape[0]
    H, D, V = c["heads"], c["dim"], c["vdim"]
    h = inp(h)
    q = (h @ p["q"].T).reshape(T, H, D) / math.sqrt(D)
    i, f = log_gates(h, p, c["gate_cap"])
    o = exp_gated_memory(q, (h @ p["k"].T).reshape(T, H, D), (h @ p["v"].T).reshape(T, H, V), i, f)
    o = rms_norm(o, eps).reshape(T, H * V) * p["norm"] * sigmoid(h @ p["g"].T)
    return inp(o) @ p["o"].T


# ---- attention ----------------------------------------------------------------------------------------------------------------------
def short_conv(u, w):
    """y_t[c] = sum_j w[c, j] u_(t - taps + 1 + j)[c], zeros before the sequence.  u: [T, C], w: [C, taps]."""
    T, taps = u.shape[0], w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, u.shape[1])), u])
    return sum(pad[j:j + T] * w[:, j] for j in range(taps))


def frequencies(rot):
    """base^(-2 i / dims) per pair; with rot.scaling, by wavelength l = 2 pi / f: kept where l < original / high, divided by factor where
    l > original / low, and a blend in between whose weight of the kept frequency is (original / l - low) / (high - low)."""
    n, sc = rot["dims"], rot.get("scaling")
    out = []
    for i in range(n // 2):
        f = float(rot["base"]) ** (-2.0 * i / n)
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return np.array(out)


def turn(x, pos, rot):
    """Rotary turn of the first rot.dims entries of the last axis, entry i paired with entry i + dims / 2.  x: [T, heads, D]."""
    n = rot["dims"]
    a = np.asarray(pos, np.float64)[:, None, None] * frequencies(rot)
    out = x.copy()
    u, v = x[..., :n // 2], x[..., n // 2:n]
    out[..., :n // 2], out[..., n // 2:n] = u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)
    return out


def attention(h, p, c, eps, causal_shift=0, drop_keys=()):
    """causal_shift and drop_keys are knobs for the tests' sensitivity checks: query i sees j <= i + shift (always itself), and the
    listed keys are hidden from later queries."""
    T = h.shape[0]
    H, G, D = c["heads"], c["kv_heads"], c["dim"]
    h = inp(h)
    q, k = h @ p["q"].T, h @ p["k"].T
    if c.get("conv"):
        q, k = short_conv(q, p["q.conv"]), short_conv(k, p["k.conv"])
    q, k = q.reshape(T, H, D), k.reshape(T, G, D)
    v = k                                                      # the values: keys before norm and turn
    q, k = rms_norm(q, eps, p["q.norm"]), rms_norm(k, eps, p["k.norm"])
    if c.get("rot"):
        q, k = turn(q, np.arange(T), c["rot"]), turn(k, np.arange(T), c["rot"])
    seen = np.tril(np.ones((T, T), bool), causal_shift) | np.eye(T, dtype=bool)
    for j in drop_keys:
        seen[j + 1:, j] = False
    out = np.zeros((T, H, D))
    for hd in range(H):
        g = hd // (H // G)
        s = np.where(seen, (q[:, hd] @ k[:, g].T) * c["scale"], -np.inf)
        w = np.exp(s - s.max(axis=-1, keepdims=True))
        out[:, hd] = (w / w.sum(axis=-1, keepdims=True)) @ v[:, g]
    return inp(out.reshape(T, H * D)) @ p["o"].T


# ---- feed-forward -----------------------------------------------------------------------------------------------------------------
def poly_norm(z, act, eps):
    """a N(z) + b N(z^2) + c N(z^3) + e, N dividing a token's vector by its root mean square."""
    a, b, c, e = act
    return a * rms_norm(z, eps) + b * rms_norm(z ** 2, eps) + c * rms_norm(z ** 3, eps) + e


def dense_ff(h, p, eps):
    return inp(poly_norm(inp(h) @ p["up"].T, p["act"], eps)) @ p["down"].T


def expert(h, up, down):
    return inp(np.square(np.maximum(inp(h) @ up.T, 0.0))) @ down.T


def route(h, p, c):
    """Chosen experts [T, top] and their weights.  Scores sigmoid(W_router h); choice scores = scores + correction.  The experts form
    groups.count runs of neighbours; a group's score is the sum of its two largest choice scores; only the best groups.keep groups are
    open to the choice of the `top` largest choice scores (the lowest index wins a tie).  The weights are the plain scores."""
    s = sigmoid(inp(h) @ p["router"].T)
    cs = s + p["correction"]
    E, top = c["router"]["experts"], c["router"]["top"]
    grp = c["router"].get("groups")
    if grp:
        by = cs.reshape(-1, grp["count"], E // grp["count"])
        score = np.sort(by, axis=-1)[..., -2:].sum(axis=-1)
        kept = np.argsort(-score, axis=-1, kind="stable")[:, :grp["keep"]]
        closed = np.ones(score.shape, bool)
        np.put_along_axis(closed, kept, False, axis=-1)
        cs = np.where(np.repeat(closed, E // grp["count"], axis=-1), -np.inf, cs)
    choice = np.argsort(-cs, axis=-1, kind="stable")[:, :top]
    return choice, np.take_along_axis(s, choice, axis=-1)


def moe_ff(h, p, c):
    choice, w = route(h, p, c)
    out = np.zeros((h.shape[0], p["e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, we in zip(choice[t], w[t]):
            out[t] += we * expert(h[t:t + 1], p[f"e{e}.up"], p[f"e{e}.down"])[0]
    if c.get("shared"):
        out = out + sigmoid(inp(h) @ p["shared.sg"].T) * expert(h, p["shared.up"], p["shared.down"])
    return out


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
    x = embedding(tokens, weights, cfg)
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        m, c = sub(weights, pre + "mix."), layer["mixer"]
        h = token_shift(rms_norm(x, eps, 1.0 + weights[pre + "norm1"]), weights[pre + "shift"])
        if layer["type"] == "hgrn2":
            y = hgrn2(h, m, c, eps)
        elif layer["type"] == "mlstm":
            y = mlstm(h, m, c, eps)
        elif layer["type"] == "attention":
            y = attention(h, m, c, eps, **knobs)
        else:
            raise ValueError(layer["type"])
        x = x + y * weights[pre + "ls1"]
        mlp = layer.get("mlp")
        if mlp:
            f = sub(weights, pre + "mlp.")
            h = rms_norm(x, eps, 1.0 + weights[pre + "norm2"])
            y = dense_ff(h, f, eps) if mlp["kind"] == "dense" else moe_ff(h, f, mlp)
            x = x + y * weights[pre + "ls2"]
        if taps is not None:
            taps.append(x.copy())
    return inp(rms_norm(x, eps, 1.0 + weights["final.norm"])) @ weights["embed"].T


# ---- random models for the tests ----------------------------------------------------------------------------------------------------
def tensor_shapes(cfg):
    """{tensor name: shape} of a configuration, in file order."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W)}
    b = (cfg.get("embedding") or {}).get("bigram")
    if b:
        out["bigram"] = (b["buckets"] + 1, W)
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = "l%d." % i, layer["mixer"], layer.get("mlp")
        q = p + "mix."
        nq, od = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        out[p + "norm1"] = (W,)
        if layer["type"] == "hgrn2":
            out.update({q + "q": (nq, W), q + "f": (nq, W), q + "f.b": (nq,), q + "lower": (nq,), q + "v": (od, W), q + "norm": (m["vdim"],), q + "o": (W, od)})
        elif layer["type"] == "mlstm":
            out.update({q + "q": (nq, W), q + "k": (nq, W), q + "v": (od, W), q + "g": (od, W), q + "o": (W, od), q + "norm": (od,),
                        q + "i": (m["heads"], W), q + "i.b": (m["heads"],), q + "f": (m["heads"], W), q + "f.b": (m["heads"],)})
        else:
            nk = m["kv_heads"] * m["dim"]
            out.update({q + "q": (nq, W), q + "k": (nk, W), q + "q.norm": (m["dim"],), q + "k.norm": (m["dim"],)})
            if m.get("conv"):
                out.update({q + "q.conv": (nq, m["conv"]), q + "k.conv": (nk, m["conv"])})
            out[q + "o"] = (W, od)
        if ff:
            out[p + "norm2"] = (W,)
            if ff["kind"] == "dense":
                out.update({p + "mlp.up": (ff["ff"], W), p + "mlp.down": (W, ff["ff"]), p + "mlp.act": (4,)})
            else:
                f = ff["expert"]["ff"]
                for e in range(ff["router"]["experts"]):
                    out.update({p + "mlp.e%d.up" % e: (f, W), p + "mlp.e%d.down" % e: (W, f)})
                out.update({p + "mlp.router": (ff["router"]["experts"], W), p + "mlp.correction": (ff["router"]["experts"],)})
                if ff.get("shared"):
                    f = ff["shared"]["ff"]
                    out.update({p + "mlp.shared.up": (f, W), p + "mlp.shared.down": (W, f), p + "mlp.shared.sg": (1, W)})
            out[p + "ls2"] = (W,)
        out.update({p + "ls1": (W,), p + "shift": (W,)})
    out["final.norm"] = (W,)
    return out


def random_weights(cfg, seed):
    """bfloat16-representable float32 weights: matrices ~ N(0, 1 / fan_in), gate and router projections larger (so that gates move and
    the experts' scores spread), stored norm weights around zero, layer scales around one, shifts in [0, 1], lower bounds in [0, 0.95]."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shp in tensor_shapes(cfg).items():
        leaf = name.split(".", 1)[1] if name[0] == "l" and name[1].isdigit() else name
        if leaf in ("norm1", "norm2", "final.norm"):
            a = 0.2 * rng.standard_normal(shp)
        elif leaf in ("ls1", "ls2"):
            a = 0.7 + 0.2 * rng.standard_normal(shp)
        elif leaf == "shift":
            a = rng.uniform(0.0, 1.0, shp)
        elif leaf == "mix.lower":
            a = rng.uniform(0.0, 0.95, shp)
        elif leaf in ("mix.norm", "mix.q.norm", "mix.k.norm"):
            a = 1.0 + 0.2 * rng.standard_normal(shp)
        elif leaf == "mlp.act":
            a = np.array([0.6, 0.4, 0.3, 0.1]) + 0.1 * rng.standard_normal(4)
        elif leaf == "mlp.correction":
            a = 0.3 * rng.standard_normal(shp)
        elif leaf == "mix.f.b":
            a = 2.0 + rng.standard_normal(shp)
        elif leaf == "mix.i.b":
            a = rng.standard_normal(shp)
        elif leaf.endswith(".conv"):
            a = rng.standard_normal(shp) / math.sqrt(shp[1])
        elif leaf == "embed":
            a = rng.standard_normal(shp)
        elif leaf == "bigram":
            a = 0.5 * rng.standard_normal(shp)
        elif leaf in ("mix.g", "mix.i", "mlp.router", "mlp.shared.sg") or (leaf == "mix.f"):
            a = 2.0 * rng.standard_normal(shp) / math.sqrt(shp[-1])
        else:
            a = rng.standard_normal(shp) / math.sqrt(shp[-1])
        out[name] = bf16_round(a)
    return out


def to_f64(w):
    return {k: np.asarray(v, np.float64) for k, v in w.items()}
