"""Plain CPU restatement of the Tafopel decoder (numpy, float64 unless told otherwise): one function per mechanism, whole sequences,
no cache, no kernels, nothing shared with the package.  Test infrastructure only.

A model is (cfg, w): `cfg` the dictionary of config.json, `w` a dictionary name -> ndarray.  Notation: x [T, width] residual stream,
h [T, width] the layer's normed input, c [T, rank] latents, r [T, rot] the rotated shared key part.
"""
import math

import numpy as np


def rms_norm(x, weight, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def layer_norm(x, weight, eps):
    """centred, divided by the standard deviation, weighted; no bias"""
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * weight


def sigmoid(x):
    return np.where(x >= 0, 1.0 / (1.0 + np.exp(-np.abs(x))), np.exp(-np.abs(x)) / (1.0 + np.exp(-np.abs(x))))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.maximum(x, 0) + np.log1p(np.exp(-np.abs(x)))


def gelu_tanh(x):
    return 0.5 * x * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def relu2(x):
    return np.maximum(x, 0) ** 2


# ---- rotation -------------------------------------------------------------------------------------------------------------------
def rotation(rot):
    """(frequency of every pair, factor of cos and sin)"""
    n, base = rot["dims"], float(rot["base"])
    freq = np.array([base ** (-2.0 * i / n) for i in range(n // 2)])
    sc = rot.get("scaling")
    if not sc:
        return freq, 1.0
    turns_at = lambda t: n * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo, hi = max(math.floor(turns_at(sc["fast"])), 0), min(math.ceil(turns_at(sc["slow"])), n - 1)
    for i in range(n // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        freq[i] = freq[i] / sc["factor"] * ramp + freq[i] * (1.0 - ramp)
    return freq, 0.1 * math.log(sc["factor"]) + 1.0


def rotary_pairs(x, positions, rot):
    """neighbouring dimensions (2i, 2i + 1) of the last axis turned by p * f_i; x [T, n]"""
    freq, mult = rotation(rot)
    ang = np.asarray(positions, np.float64)[:, None] * freq[None, :]
    cos, sin = (np.cos(ang) * mult).astype(x.dtype), (np.sin(ang) * mult).astype(x.dtype)
    out = np.empty_like(x)
    u, v = x[..., 0::2], x[..., 1::2]
    out[..., 0::2], out[..., 1::2] = u * cos - v * sin, v * cos + u * sin
    return out


# ---- latent attention -------------------------------------------------------------------------------------------------------------
def sink_softmax(scores, visible, sink):
    """softmax over the visible keys of every row with one more term exp(sink) in the denominator"""
    s = np.where(visible, scores, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - top))


def latents(h, mix, w, p, eps):
    """what a cache would hold: normed latents [T, rank] and the rotated key part [T, rot]"""
    d = h @ w[p + "dkv"].T
    rank = mix["kv_rank"]
    return rms_norm(d[:, :rank], w[p + "dkv.norm"], eps), rotary_pairs(d[:, rank:], np.arange(len(h)), mix["rot"])


def latent_attention(h, mix, w, p, eps, kv):
    """mixer output of a whole sequence; kv: (c, r) of this layer or of the one it borrows from"""
    T, H, dim, rot, vdim = len(h), mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    c, r = kv
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).reshape(T, H, dim + rot)
    visible = np.arange(T)[None, :] <= np.arange(T)[:, None]
    out = np.empty((T, H * vdim), h.dtype)
    for n in range(H):
        k = c @ w[p + "uk"][n * dim:(n + 1) * dim].T
        v = c @ w[p + "uv"][n * vdim:(n + 1) * vdim].T
        s = (q[:, n, :dim] @ k.T + rotary_pairs(q[:, n, dim:], np.arange(T), mix["rot"]) @ r.T) * mix["scale"]
        out[:, n * vdim:(n + 1) * vdim] = sink_softmax(s, visible, w[p + "sink"][n]) @ v
    return out @ w[p + "o"].T


# ---- selective scan -----------------------------------------------------------------------------------------------------------------
def causal_conv(x, kernel, bias):
    """per channel, last tap on the current token, zeros before the start; kernel [channels, taps]"""
    taps = kernel.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, x.shape[1]), x.dtype), x])
    return sum(pad[i:i + len(x)] * kernel[:, i] for i in range(taps)) + bias


def selective_scan(x, dt, A, B, C, D):
    """S <- exp(dt A) S + dt x B, y = S C + D x, token by token; x, dt [T, inner], A [inner, state], B, C [T, state]"""
    S, y = np.zeros(A.shape, x.dtype), np.empty_like(x)
    for t in range(len(x)):
        S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba(h, mix, w, p):
    n, state, rank = mix["inner"], mix["state"], mix["dt_rank"]
    xz = h @ w[p + "in"].T
    x, z = silu(causal_conv(xz[:, :n], w[p + "conv"], w[p + "conv.b"])), xz[:, n:]
    d = x @ w[p + "x"].T
    dt = softplus(d[:, :rank] @ w[p + "dt"].T + w[p + "dt.b"])
    y = selective_scan(x, dt, -np.exp(w[p + "A_log"]), d[:, rank:rank + state], d[:, rank + state:], w[p + "D"])
    return (y * silu(z)) @ w[p + "o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------------------------------------
def gated(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def plain(h, w, p):
    return relu2(h @ w[p + "up"].T) @ w[p + "down"].T


def route(h, w, p, top):
    """(chosen experts, their scores) of every token"""
    s = sigmoid(h @ w[p + "router"].T)
    idx = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return idx, np.take_along_axis(s, idx, axis=-1)


def experts(h, mlp, w, p):
    """the score multiplies the chosen expert's input; the shared expert's output is gated by one sigmoid per token"""
    idx, wt = route(h, w, p, mlp["router"]["top"])
    y = np.zeros_like(h)
    for t in range(len(h)):
        for e, g in zip(idx[t], wt[t]):
            y[t] += plain((g * h[t])[None], w, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        y = y + plain(h, w, p + "shared.") * sigmoid(h @ w[p + "shared.sg"].T)
    return y


def feed_forward(h, mlp, w, p):
    return gated(h, w, p) if mlp["kind"] == "dense" else experts(h, mlp, w, p)


# ---- model ------------------------------------------------------------------------------------------------------------------------------
def run(cfg, w, tokens):
    """-> (logits [T, vocab], residual stream after every layer)"""
    eps = cfg["norm"]["eps"]
    x, taps, kv = w["embed"][np.asarray(tokens)], [], {}
    for i, layer in enumerate(cfg["layers"]):
        p, mix = f"l{i}.", layer["mixer"]
        h = layer_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "mamba1":
            y = mamba(h, mix, w, p + "mix.")
        else:
            src = mix.get("kv_from")
            kv[i] = latents(h, mix, w, p + "mix.", eps) if src is None else kv[src]
            y = latent_attention(h, mix, w, p + "mix.", eps, kv[i])
        if layer.get("mlp"):
            y = y + feed_forward(h, layer["mlp"], w, p + "mlp.")
        x = x + y
        taps.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T, taps


def tensor_shapes(cfg):
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        m, p, f = layer["mixer"], f"l{i}.mix.", layer.get("mlp")
        out[f"l{i}.norm1"] = (W,)
        if layer["type"] == "mamba1":
            n, s, r = m["inner"], m["state"], m["dt_rank"]
            out.update({p + "in": (2 * n, W), p + "conv": (n, m["conv"]), p + "conv.b": (n,), p + "x": (r + 2 * s, n), p + "dt": (n, r), p + "dt.b": (n,),
                        p + "A_log": (n, s), p + "D": (n,), p + "o": (W, n)})
        else:
            H, d, ro, v, k, qr = (m[x] for x in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            out.update({p + "dq": (qr, W), p + "dq.norm": (qr,), p + "uq": (H * (d + ro), qr), p + "uk": (H * d, k), p + "uv": (H * v, k), p + "sink": (H,),
                        p + "o": (W, H * v)})
            if m.get("kv_from") is None:
                out.update({p + "dkv": (k + ro, W), p + "dkv.norm": (k,)})
        p = f"l{i}.mlp."
        if f and f["kind"] == "dense":
            out.update({p + "gate": (f["ff"], W), p + "up": (f["ff"], W), p + "down": (W, f["ff"])})
        elif f:
            for e in range(f["router"]["experts"]):
                out.update({f"{p}e{e}.up": (f["expert"]["ff"], W), f"{p}e{e}.down": (W, f["expert"]["ff"])})
            out[p + "router"] = (f["router"]["experts"], W)
            if f.get("shared"):
                out.update({p + "shared.up": (f["shared"]["ff"], W), p + "shared.down": (W, f["shared"]["ff"]), p + "shared.sg": (1, W)})
    return out


def random_weights(cfg, seed=0):
    """bf16-valued float64 weights: unit-variance products, norms near 1, decays from slow to fast"""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        if name.endswith("norm") or name.endswith("norm1"):
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif name.endswith("A_log"):
            a = rng.uniform(-2.0, 2.5, shape)
        elif name.endswith("dt.b"):
            a = rng.uniform(-4.0, 0.5, shape)
        elif name.endswith((".D", "conv.b")):
            a = rng.uniform(-0.5, 1.0, shape)
        elif name.endswith("sink"):
            a = rng.uniform(-1.0, 2.0, shape)
        elif name == "embed":
            a = rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) * shape[-1] ** -0.5
        w[name] = bf16(a).astype(np.float64)
    return w


def bf16(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32).reshape(np.shape(a))


def greedy(cfg, w, prompt, n):
    """(ids, logits rows) of n greedy tokens, the whole sequence run again for each"""
    toks, ids, rows = list(prompt), [], []
    for _ in range(n):
        r = run(cfg, w, toks)[0][-1]
        rows.append(r)
        ids.append(int(len(r) - 1 - np.argmax(r[::-1])))  # the last of equal maxima
        toks.append(ids[-1])
    return ids, rows
