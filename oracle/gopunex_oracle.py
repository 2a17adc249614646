"""Plain CPU restatement of the Gopunex decoder (numpy, float64 unless told otherwise): one function per mechanism, token loops for
the recurrences, no cache, no kernels, nothing shared with the package.  Test infrastructure only.

A model is (cfg, w): `cfg` the dictionary of config.json, `w` a dictionary name -> ndarray.  Notation: x [T, width] residual
stream = input of every sublayer, T tokens of one sequence from position 0.
"""
import math

import numpy as np

UNIT_EPS = 1e-6  # inside the root of the unit norm of the delta rule's queries and keys


def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps) * weight, over the last axis"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def sigmoid(x):
    with np.errstate(over="ignore"):  # exp(inf) = inf gives 0, as it should
        return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(x, np.zeros_like(x))


def causal_conv(x, taps):
    """per channel: y_t = sum_i taps[:, i] x_{t - n + 1 + i}, zeros before the start; x [T, C], taps [C, n]"""
    n = taps.shape[1]
    y = np.zeros_like(x)
    for i in range(n):
        back = n - 1 - i
        if back < x.shape[0]:
            y[back:] += x[:x.shape[0] - back] * taps[:, i]
    return y


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def decay_linear_attention(q, k, v, decay):
    """S <- decay_h S + k v^T, o = S^T q;  q, k [T, H, D], v [T, H, E], decay [H] -> o [T, H, E]"""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]), q.dtype)
    o = np.empty(v.shape, q.dtype)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hde,hd->he", S, q[t])
    return o


def delta_rule(q, k, v, g, beta):
    """S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q;  q, k, g [T, H, D], v [T, H, E], beta [T, H] -> o [T, H, E]"""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]), q.dtype)
    o = np.empty(v.shape, q.dtype)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hde,hd->he", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hde,hd->he", S, q[t])
    return o


def bucket(distance, rows, far):
    """row of the bias table for a distance: exact below rows // 2, then logarithmic, the last row from about `far` on"""
    half = rows // 2
    if distance < half:
        return distance
    return min(rows - 1, half + int(math.floor(math.log(distance / half) / math.log(far / half) * (rows - half) + 1e-9)))


def distance_bias(T, table, far):
    """[H, T, T]: entry (h, i, j), j <= i"""
    row = np.array([bucket(n, table.shape[0], far) for n in range(T)])
    n = np.maximum(np.arange(T)[:, None] - np.arange(T)[None, :], 0)
    return np.moveaxis(table[row[n]], 2, 0)


def softmax_one(scores, visible):
    """exp(s_j) / (1 + sum_j exp(s_j)) over the visible keys of every row"""
    s = np.where(visible, scores, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), 0.0)
    e = np.exp(s - m)
    return e / (np.exp(-m) + e.sum(axis=-1, keepdims=True))


def lightning(x, m, w, p, eps):
    T, H = x.shape[0], m["heads"]
    q, k, v = (silu(x @ w[p + n].T).reshape(T, H, -1) for n in "qkv")
    o = decay_linear_attention(q, k, v, np.asarray(m["decay"], x.dtype)).reshape(T, -1)
    return (rms_norm(o, w[p + "norm"], eps) * sigmoid(x @ w[p + "g"].T)) @ w[p + "o"].T


def delta_decays(x, m, w, p):
    """log of g [T, H, D]"""
    z = (x @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    return -np.exp(w[p + "A_log"])[:, None] * softplus(z).reshape(x.shape[0], m["heads"], m["dim"])


def channel_delta(x, m, w, p, eps):
    T, H, G = x.shape[0], m["heads"], m["kv_heads"]
    q, k, v = (silu(causal_conv(x @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q, k = (np.repeat(unit(a.reshape(T, G, m["dim"])), H // G, axis=1) for a in (q, k))
    beta = sigmoid(x @ w[p + "b"].T)
    o = delta_rule(q * x.dtype.type(m["dim"]) ** -0.5, k, v.reshape(T, H, m["vdim"]), np.exp(delta_decays(x, m, w, p)), beta)
    gate = sigmoid((x @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(o.shape)
    return (rms_norm(o, w[p + "norm"], eps) * gate).reshape(T, -1) @ w[p + "o"].T


def attention(x, m, w, p, eps, v_first=None):
    """-> (output [T, width], the layer's own unmixed values)"""
    T, H, G = x.shape[0], m["heads"], m["kv_heads"]
    q, k, v = (x @ w[p + n].T + w[p + n + ".b"] for n in "qkv")
    q = rms_norm(q, w[p + "q.norm"], eps).reshape(T, H, m["dim"])
    k = rms_norm(k, w[p + "k.norm"], eps).reshape(T, G, m["dim"])
    own = v
    if v_first is not None:
        v = (1 - w[p + "vmix"]) * v + w[p + "vmix"] * v_first
    v = v.reshape(T, G, m["vdim"])
    bias = distance_bias(T, w[p + "rel"], m["bias_max"])
    visible = np.tril(np.ones((T, T), bool))
    out = np.empty((T, H, m["vdim"]), x.dtype)
    for h in range(H):
        g = h // (H // G)
        out[:, h] = softmax_one(q[:, h] @ k[:, g].T * x.dtype.type(m["scale"]) + bias[h], visible) @ v[:, g]
    return out.reshape(T, -1) @ w[p + "o"].T, own


def feed_forward(x, w, p):
    return np.maximum(x @ w[p + "up"].T, 0) ** 2 @ w[p + "down"].T


def forward(cfg, w, tokens, want=None, dtype=np.float64, layer_outputs=None):
    """logits [len(want) or T, vocab] of one sequence; layer_outputs (a list) collects the residual stream after every layer"""
    w = {k: np.asarray(v, dtype) for k, v in w.items()}
    eps, mult = dtype(cfg["norm"]["eps"]), dtype(cfg["residual_mult"])
    x = w["embed"][np.asarray(tokens)] * dtype(cfg["embedding"]["scale"])
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        if layer["type"] == "attention":
            mixes = bool(m.get("v_mix"))
            y, own = attention(x, m, w, p + "mix.", eps, v_first if mixes else None)
            if mixes and v_first is None:
                v_first = own
        else:
            y = {"lightning": lightning, "channel_delta": channel_delta}[layer["type"]](x, m, w, p + "mix.", eps)
        x = x + mult * rms_norm(y, 1 + w[p + "norm1"], eps)
        if layer.get("mlp"):
            x = x + mult * rms_norm(feed_forward(x, w, p + "mlp."), 1 + w[p + "norm2"], eps)
        if layer_outputs is not None:
            layer_outputs.append(x.copy())
    if want is not None:
        x = x[np.asarray(want, int)]
    return rms_norm(x, 1 + w["final.norm"], eps) @ w["head"].T


def greedy(cfg, w, prompt, n_new, dtype=np.float64):
    """n_new greedy tokens (last maximum wins) and the logits they came from, by full recomputation"""
    toks, rows = list(prompt), []
    for _ in range(n_new):
        lg = forward(cfg, w, toks, want=[len(toks) - 1], dtype=dtype)[0]
        rows.append(lg)
        toks.append(int(np.flatnonzero(lg == lg.max())[-1]))
    return toks[len(prompt):], np.array(rows)


def random_weights(cfg, seed=0, gain=1.0, rank=12, bias_rows=16):
    """bf16-valued random weights (float32 arrays): matrices ~ gain / sqrt(fan-in), plain norms near 1, others near 0; `rank` rows of
    the two-step projections, `bias_rows` rows of the distance tables"""
    rng = np.random.default_rng(seed)

    def bf16(a):
        u = np.ascontiguousarray(a, np.float32).view(np.uint32)
        return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32).reshape(np.shape(a))

    def mat(rows, cols):
        return bf16(rng.standard_normal((rows, cols)) * (gain / np.sqrt(cols)))

    def vec(n, mean=1.0):
        return bf16(mean + 0.2 * rng.standard_normal(n))

    W = cfg["width"]
    w = {"embed": bf16(rng.standard_normal((cfg["vocab"], W))), "head": mat(cfg["vocab"], W), "final.norm": vec(W, 0.0)}
    for l, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{l}.mix."
        H, D, E = m["heads"], m["dim"], m["vdim"]
        G = m.get("kv_heads", H)
        w[f"l{l}.norm1"] = vec(W, 0.0)
        w[p + "o"] = mat(W, H * E)
        if layer["type"] == "attention":
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * E)):
                w[p + n] = mat(rows, W)
                w[p + n + ".b"] = vec(rows, 0.0)
            w[p + "q.norm"], w[p + "k.norm"] = vec(H * D), vec(G * D)
            w[p + "rel"] = bf16(rng.standard_normal((bias_rows, H)))
            if m.get("v_mix"):
                w[p + "vmix"] = bf16(np.array(0.2 + 0.5 * rng.random()))
        elif layer["type"] == "lightning":
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * E), ("g", H * E)):
                w[p + n] = mat(rows, W)
            w[p + "norm"] = vec(H * E)
        else:
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * E)):
                w[p + n] = mat(rows, W)
                w[p + n + ".conv"] = bf16(rng.standard_normal((rows, m["conv"])) / np.sqrt(m["conv"]))
            w[p + "b"] = mat(H, W)
            w[p + "A_log"] = bf16(rng.uniform(-3.0, 0.5, H))
            w[p + "dt_bias"] = vec(H * D, -1.0)
            w[p + "norm"] = vec(E)
            w[p + "a1"], w[p + "a2"] = mat(rank, W), mat(H * D, rank)
            w[p + "g1"], w[p + "g2"] = mat(rank + 3, W), mat(H * E, rank + 3)
        if layer.get("mlp"):
            w[f"l{l}.norm2"] = vec(W, 0.0)
            w[f"l{l}.mlp.up"], w[f"l{l}.mlp.down"] = mat(layer["mlp"]["ff"], W), mat(W, layer["mlp"]["ff"])
    return w
