"""Plain CPU restatement of the Lefalix decoder (numpy, float64): one function per mechanism, token loops for the recurrences, no cache,
no kernels, nothing shared with the package.  Test infrastructure only.

A model is (cfg, w): `cfg` the dictionary of config.json, `w` a dictionary name -> ndarray.  Notation: x [T, width] residual stream,
h [T, width] input of a sublayer, T tokens of one sequence from position 0.
"""
import math

import numpy as np

UNIT_EPS = 1e-6  # inside the root of the unit norm of the delta rule's queries and keys


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def sigmoid(x):
    with np.errstate(over="ignore"):
        return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(x, np.zeros_like(x))


_erf = np.vectorize(math.erf, otypes=[np.float64])


def gelu_erf(x):
    return 0.5 * x * (1.0 + _erf(x / math.sqrt(2.0)))


def causal_conv(u, taps):
    """per channel, the last tap on the current token, zeros before the start; u [T, C], taps [C, n]"""
    n = taps.shape[1]
    pad = np.concatenate([np.zeros((n - 1, u.shape[1]), u.dtype), u])
    return sum(pad[j:j + len(u)] * taps[:, j] for j in range(n))


# ---- rotation -----------------------------------------------------------------------------------------------------------------------
def rotation(rot):
    """(frequencies [dims / 2], factor of cosine and sine): geometric, with YaRN scaling where the configuration has it"""
    n, base = rot["dims"], rot["base"]
    f = base ** (-2.0 * np.arange(n // 2) / n)
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def pair(turns):
        return n * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(pair(s["fast"])), 0), min(math.ceil(pair(s["slow"])), n - 1)
    ramp = np.clip((np.arange(n // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate_pairs(x, rot):
    """neighbouring dimensions of the first rot.dims turn by position * frequency; x [T, heads, dim]"""
    freq, mult = rotation(rot)
    a = np.arange(len(x))[:, None, None] * freq
    u, v = x[..., 0:rot["dims"]:2], x[..., 1:rot["dims"]:2]
    y = x.copy()
    y[..., 0:rot["dims"]:2] = (u * np.cos(a) - v * np.sin(a)) * mult
    y[..., 1:rot["dims"]:2] = (v * np.cos(a) + u * np.sin(a)) * mult
    return y


# ---- windowed attention ---------------------------------------------------------------------------------------------------------------
def window(T, size):
    """[T, T]: row i sees the columns j with 0 <= i - j < size"""
    back = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (back >= 0) & (back < size)


def sink_softmax(scores, visible, sink):
    """softmax over the visible keys of every row with one more term exp(sink) in the denominator"""
    s = np.where(visible, scores, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - top))


def attention(h, m, w, p, eps):
    T, H, G, D = len(h), m["heads"], m["kv_heads"], m["dim"]
    q, k, v = (causal_conv(h @ w[p + n].T + w[p + n + ".b"], w[p + n + ".conv"]) for n in "qkv")
    q, k = (rms(rotate_pairs(a.reshape(T, -1, D), m["rot"]), eps) for a in (q, k))
    v = v.reshape(T, G, m["vdim"])
    visible = window(T, m["mask"]["size"])
    o = np.empty((T, H, m["vdim"]), h.dtype)
    for n in range(H):
        g = n // (H // G)
        o[:, n] = sink_softmax(q[:, n] @ k[:, g].T * m["scale"], visible, w[p + "sink"][n]) @ v[:, g]
    return o.reshape(T, -1) @ w[p + "o"].T + w[p + "o.b"]


# ---- gated delta rule -------------------------------------------------------------------------------------------------------------------
def delta_rule(q, k, v, g, beta):
    """S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q;  q, k, g [T, H, D], v [T, H, E], beta [T, H] -> o [T, H, E]"""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2]), q.dtype)
    o = np.empty(v.shape, q.dtype)
    for t in range(len(q)):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.matmul(k[t][:, None, :], S)[:, 0])
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.matmul(q[t][:, None, :], S)[:, 0]
    return o


def delta_inputs(h, m, w, p):
    """queries, keys [T, H, D] (a group's heads share theirs), values [T, H, E], write strengths [T, H]"""
    T, H, G, D = len(h), m["heads"], m["kv_heads"], m["dim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q, k = (np.repeat(unit(a.reshape(T, G, D)), H // G, axis=1) for a in (q, k))
    return q * D ** -0.5, k, v.reshape(T, H, m["vdim"]), sigmoid(h @ w[p + "b"].T)


def channel_decays(h, m, w, p):
    """a decay per head and key channel [T, H, D]"""
    z = ((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(len(h), m["heads"], m["dim"])
    return np.exp(-np.exp(w[p + "A_log"])[:, None] * softplus(z))


def head_decays(h, m, w, p):
    """one decay per head, on all of its key channels [T, H, D]"""
    g = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    return np.repeat(g[:, :, None], m["dim"], axis=2)


def channel_delta(h, m, w, p, eps):
    q, k, v, beta = delta_inputs(h, m, w, p)
    o = delta_rule(q, k, v, channel_decays(h, m, w, p), beta)
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(o.shape)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(len(h), -1) @ w[p + "o"].T


def head_delta(h, m, w, p, eps):
    q, k, v, beta = delta_inputs(h, m, w, p)
    o = delta_rule(q, k, v, head_decays(h, m, w, p), beta)
    gate = silu(h @ w[p + "g"].T).reshape(o.shape)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(len(h), -1) @ w[p + "o"].T


def parallel(h, m, w, p, eps):
    left, right = attention(h, m["left"], w, p + "left.", eps), head_delta(h, m["right"], w, p + "right.", eps)
    return 0.5 * (rms(left, eps) * w[p + "left.out"] + rms(right, eps) * w[p + "right.out"])


# ---- feed-forwards ------------------------------------------------------------------------------------------------------------------------
def dense(h, w, p):
    return gelu_erf(h @ w[p + "up"].T) @ w[p + "down"].T


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, r, w, p):
    """(chosen experts, their scores) of every token: softmax scores, the best groups by their largest score, the best experts in those"""
    z = h @ w[p + "router"].T
    s = np.exp(z - z.max(axis=-1, keepdims=True))
    s /= s.sum(axis=-1, keepdims=True)
    g = r.get("groups") or {"count": 1, "keep": 1}
    best = s.reshape(len(h), g["count"], -1).max(axis=-1)
    kept = np.argsort(-best, axis=-1, kind="stable")[:, :g["keep"]]
    open_group = np.zeros(best.shape, bool)
    np.put_along_axis(open_group, kept, True, axis=-1)
    can = np.where(np.repeat(open_group, r["experts"] // g["count"], axis=1), s, -1.0)
    idx = np.argsort(-can, axis=-1, kind="stable")[:, :r["top"]]
    return idx, np.take_along_axis(s, idx, axis=-1)


def experts(h, mlp, w, p):
    idx, wt = route(h, mlp["router"], w, p)
    y = np.zeros_like(h)
    for t in range(len(h)):
        for e, s in zip(idx[t], wt[t]):
            y[t] += s * expert(h[t:t + 1], w, f"{p}e{e}.")[0]
    return y


def feed_forward(h, mlp, w, p):
    return dense(h, w, p) if mlp["kind"] == "dense" else experts(h, mlp, w, p)


# ---- model ----------------------------------------------------------------------------------------------------------------------------------
def order(cfg):
    """[(layer, starts a pass but the first)] of every layer run"""
    n, loop = len(cfg["layers"]), cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    span = range(loop["start"], loop["stop"])
    runs = [(i, False) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t > 0 and i == loop["start"]) for i in span]
    return runs + [(i, False) for i in range(loop["stop"], n)]


MIXERS = {"parallel": parallel, "channel_delta": channel_delta}


def run(cfg, w, tokens):
    """-> (logits [T, vocab], residual stream after every layer run)"""
    eps = cfg["norm"]["eps"]
    first = w["embed"][np.asarray(tokens)]
    x, taps = first, []
    for i, again in order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + first
        y = MIXERS[layer["type"]](rms(x, eps) * w[p + "norm1"], layer["mixer"], w, p + "mix.", eps)
        x = x + rms(y, eps) * w[p + "norm1b"]
        if layer.get("mlp"):
            y = feed_forward(rms(x, eps) * w[p + "norm2"], layer["mlp"], w, p + "mlp.")
            x = x + rms(y, eps) * w[p + "norm2b"]
        taps.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T, taps


def greedy(cfg, w, prompt, n):
    """(ids, logits rows) of n greedy tokens (the last of equal maxima), the whole sequence run again for each"""
    toks, ids, rows = list(prompt), [], []
    for _ in range(n):
        r = run(cfg, w, toks)[0][-1]
        rows.append(r)
        ids.append(int(np.flatnonzero(r == r.max())[-1]))
        toks.append(ids[-1])
    return ids, rows


# ---- weights ----------------------------------------------------------------------------------------------------------------------------------
def _delta_shapes(m, W):
    G, H, D, E = m["kv_heads"], m["heads"], m["dim"], m["vdim"]
    out = {}
    for n, rows in (("q", G * D), ("k", G * D), ("v", H * E)):
        out[n], out[n + ".conv"] = (rows, W), (rows, m["conv"])
    out.update({"b": (H, W), "A_log": (H,), "norm": (E,), "o": (W, H * E)})
    return out


def tensor_shapes(cfg, rank=12):
    """`rank` rows of the first step of the two-step decay projection, three more of the gate's"""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        m, f, p = layer["mixer"], layer.get("mlp"), f"l{i}.mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            out[f"l{i}.{n}"] = (W,)
        if layer["type"] == "channel_delta":
            H, D, E = m["heads"], m["dim"], m["vdim"]
            out.update({p + k: s for k, s in _delta_shapes(m, W).items()})
            out.update({p + "a1": (rank, W), p + "a2": (H * D, rank), p + "dt_bias": (H * D,), p + "g1": (rank + 3, W), p + "g2": (H * E, rank + 3)})
        else:
            a, d = m["left"], m["right"]
            for n, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                out.update({f"{p}left.{n}": (rows, W), f"{p}left.{n}.b": (rows,), f"{p}left.{n}.conv": (rows, a["conv"])})
            out.update({p + "left.sink": (a["heads"],), p + "left.o": (W, a["heads"] * a["vdim"]), p + "left.o.b": (W,), p + "left.out": (W,), p + "right.out": (W,)})
            out.update({f"{p}right.{k}": s for k, s in _delta_shapes(d, W).items()})
            out.update({p + "right.a": (d["heads"], W), p + "right.dt_bias": (d["heads"],), p + "right.g": (d["heads"] * d["vdim"], W)})
        p = f"l{i}.mlp."
        if f and f["kind"] == "dense":
            out.update({p + "up": (f["ff"], W), p + "down": (W, f["ff"])})
        elif f:
            n = f["expert"]["ff"]
            for e in range(f["router"]["experts"]):
                out.update({f"{p}e{e}.gate": (n, W), f"{p}e{e}.up": (n, W), f"{p}e{e}.down": (W, n)})
            out[p + "router"] = (f["router"]["experts"], W)
    return out


def bf16(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32).reshape(np.shape(a))


def random_weights(cfg, seed=0, rank=12):
    """bf16-valued float64 weights: products of unit variance, norms near 1, decays from slow to fast, sinks that matter"""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_shapes(cfg, rank).items():
        if name.endswith(("norm", "norm1", "norm1b", "norm2", "norm2b", ".out")):
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif name.endswith("A_log"):
            a = rng.uniform(-5.0, 1.5, shape)
        elif name.endswith("dt_bias"):
            a = rng.uniform(-3.0, 1.0, shape)
        elif name.endswith("sink"):
            a = rng.uniform(-1.0, 2.5, shape)
        elif name.endswith(".b") and len(shape) == 1:
            a = 0.3 * rng.standard_normal(shape)
        elif name == "embed":
            a = rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) * shape[-1] ** -0.5
        w[name] = bf16(a).astype(np.float64)
    return w
