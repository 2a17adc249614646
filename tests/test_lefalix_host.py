"""Lefalix without a GPU: configuration, registry, and the CPU restatement against itself (each function alone; what mistakes the GPU tests
would show)."""
import json
import math

import numpy as np
import pytest

import nano_vllm_candle_amd as pkg
from nano_vllm_candle_amd import _lib, registry
from nano_vllm_candle_amd.causal_lm import tensor_shapes
from oracle import lefalix_oracle as L
from tests.berevik_util import row_err
from tests.lefalix_util import CONFIGS, MIXED, TOL, YARN, beacon_config, beacon_weights, config, delta, moe, par, weights, win
from tests.util import write_checkpoint


def shapes(w):
    return {k: np.shape(v) for k, v in w.items()}


def test_config_reads_every_field(tmp_path):
    w = L.random_weights(MIXED)
    write_checkpoint(tmp_path, MIXED, {k: v.astype(np.float32) for k, v in w.items()})
    c = pkg.LefalixConfig.from_dir(str(tmp_path))
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.loop) == (333, 72, 1e-5, (1, 4, 3))
    (m,), f = c.layers[0]
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.conv, m.decay_rank, m.gate_rank) == (4, 2, 24, 20, 2, 12, 15)
    assert (f.experts, f.top, f.ff, f.groups, f.kept) == (6, 2, 24, 3, 2)
    (a, m), f = c.layers[1]
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.conv, a.rot_dim, a.rot_base) == (6, 2, 20, 18, 0.5, 21, 3, 12, 300.0)
    assert (a.yarn.factor, a.yarn.original, a.yarn.fast, a.yarn.slow) == (5.0, 48.0, 6.0, 0.7)
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.conv, m.decay_rank, m.gate_rank) == (4, 2, 24, 20, 4, 0, 0) and f.ff == 56
    assert c.layers[2][0][0].yarn is None and c.layers[2][1] is None and c.layers[5][1].kept == 1
    assert c.tensor_shapes() == shapes(w) == tensor_shapes(str(tmp_path))
    assert registry.model_class(str(tmp_path)) is pkg.LefalixForCausalLM
    cc, ls = c.to_c(True)
    assert cc.f32 == 1 and cc.pre_norm == 1 and cc.norm_offset == 0.0 and (cc.loop_start, cc.loop_stop, cc.loop_times) == (1, 4, 3)
    assert [l.branches for l in ls] == [1, 2, 2, 1, 2, 1] and [l.mixer for l in ls] == [2, 0, 0, 2, 0, 2] and [l.side.mixer for l in ls][1] == 2
    l = ls[1]
    assert (l.sink, l.qk_norm, l.out_bias, l.window, l.rot_dim, l.yarn_factor, l.act) == (_lib.SINK_HEAD, _lib.QK_NORM_HEAD, 1, 21, 12, 5.0, _lib.ACT_GELU)
    assert ls[2].yarn_factor == 0.0 and ls[4].experts == 9 and (ls[5].groups, ls[5].groups_kept) == (2, 1) and ls[0].decay_rank == 12 and l.side.decay_rank == 0


def test_config_without_loop_or_groups():
    d = config([delta(moe())])
    del d["layers"][0]["mlp"]["router"]["groups"]
    for loop in (None, {"start": 1, "stop": 1, "times": 4}):
        d["loop"] = loop
        c = pkg.LefalixConfig.from_dict(d, shapes(L.random_weights(d)))
        assert c.loop == (0, 0, 1) and (c.layers[0][1].groups, c.layers[0][1].kept) == (1, 1)
    del d["loop"]
    assert pkg.LefalixConfig.from_dict(d, shapes(L.random_weights(d))).loop == (0, 0, 1)


@pytest.mark.parametrize("edit, text", [
    (lambda d: d.pop("norm"), "missing field"),
    (lambda d: d["layers"][0].update(type="other"), "mixer type"),
    (lambda d: d["layers"][1]["mlp"].update(kind="other"), "feed-forward kind"),
    (lambda d: d["layers"][1]["mixer"].pop("right"), "missing field"),
    (lambda d: d["layers"][1]["mixer"]["left"]["rot"]["scaling"].pop("slow"), "missing field"),
    (lambda d: d["layers"][1]["mixer"]["left"].pop("mask"), "missing field"),
])
def test_config_refuses_what_it_does_not_know(edit, text):
    d = json.loads(json.dumps(MIXED))
    edit(d)
    with pytest.raises(RuntimeError, match=text):
        pkg.LefalixConfig.from_dict(d, shapes(L.random_weights(MIXED)))


def test_random_tensors_cover_every_shape():
    c = pkg.LefalixConfig.from_dict(MIXED, shapes(L.random_weights(MIXED)))
    rng = np.random.default_rng(0)
    for name, shape in c.tensor_shapes().items():
        assert np.shape(c.random_tensor(name, shape, rng)) == shape, name


def test_oracle_pieces():
    rng = np.random.default_rng(0)
    x = rng.standard_normal((6, 5))
    assert np.allclose(L.rms(np.full((1, 4), 2.0), 12.0), 0.5) and np.allclose((L.unit(x) ** 2).sum(1), 1, atol=1e-5)
    k = rng.standard_normal((5, 3))
    y = L.causal_conv(x, k)
    assert np.allclose(y[0], x[0] * k[:, 2]) and np.allclose(y[4], x[4] * k[:, 2] + x[3] * k[:, 1] + x[2] * k[:, 0])
    assert np.allclose(L.gelu_erf(np.array([-10.0, 0.0, 10.0])), [0.0, 0.0, 10.0]) and np.isclose(L.gelu_erf(np.array(1.0)), 0.8413447461)
    assert np.isclose(L.softplus(np.array(800.0)), 800.0) and np.isclose(L.sigmoid(np.array(-800.0)), 0.0)
    assert L.window(5, 2).tolist() == [[j in (i - 1, i) for j in range(5)] for i in range(5)]
    s, seen = np.array([[0.0, np.log(3.0), 5.0]]), np.array([[True, True, False]])
    assert np.allclose(L.sink_softmax(s, seen, 0.0), [[0.2, 0.6, 0.0]]) and np.allclose(L.sink_softmax(s - 1000, seen, -1000.0), [[0.2, 0.6, 0.0]])
    assert np.allclose(L.sink_softmax(s, seen, -1000.0), [[0.25, 0.75, 0.0]])


def test_oracle_rotation():
    f, mult = L.rotation({"dims": 8, "base": 100.0})
    assert mult == 1.0 and np.allclose(f, [1.0, 100 ** -0.25, 0.1, 100 ** -0.75])
    rot = {"dims": 16, "base": 300.0, "scaling": YARN}
    g, mult = L.rotation(rot)
    ratio = g / L.rotation({"dims": 16, "base": 300.0})[0]
    assert np.isclose(mult, 0.1 * math.log(5.0) + 1) and ratio[0] == 1.0 and np.isclose(ratio[-1], 0.2) and ((ratio > 0.21) & (ratio < 0.99)).any()
    x = np.random.default_rng(1).standard_normal((10, 2, 20))
    y = L.rotate_pairs(x, rot)
    assert np.allclose(y[..., 16:], x[..., 16:]) and np.allclose(y[0, :, :16], x[0, :, :16] * mult)
    assert np.allclose(y[9, 1, 2] + 1j * y[9, 1, 3], (x[9, 1, 2] + 1j * x[9, 1, 3]) * np.exp(9j * g[1]) * mult)
    assert np.isfinite(L.rotation({"dims": 4, "base": 10.0, "scaling": {"factor": 2.0, "original": 10000, "fast": 1.0, "slow": 1.0}})[0]).all()


def test_oracle_delta_rule_against_the_matrix_form():
    # S_t = (I - beta k k^T) diag(g) S_{t-1} + beta k v^T
    rng = np.random.default_rng(2)
    T, H, D, E = 7, 2, 4, 3
    q, k, v = rng.standard_normal((T, H, D)), L.unit(rng.standard_normal((T, H, D))), rng.standard_normal((T, H, E))
    g, beta = rng.uniform(0.2, 1, (T, H, D)), rng.uniform(0, 1, (T, H))
    o = L.delta_rule(q, k, v, g, beta)
    for h in range(H):
        S = np.zeros((D, E))
        for t in range(T):
            S = (np.eye(D) - beta[t, h] * np.outer(k[t, h], k[t, h])) @ (g[t, h][:, None] * S) + beta[t, h] * np.outer(k[t, h], v[t, h])
            assert np.allclose(o[t, h], q[t, h] @ S)


def test_oracle_decays_per_head_are_those_per_channel_made_equal():
    cfg = config([par()])
    w = L.random_weights(cfg, 4)
    m, h = cfg["layers"][0]["mixer"]["right"], np.random.default_rng(0).standard_normal((9, 72))
    g = L.head_decays(h, m, w, "l0.mix.right.")
    assert g.shape == (9, 4, 24) and (g == g[:, :, :1]).all() and 0 < g.min() < g.max() < 1


def test_oracle_routing():
    w = {"router": np.eye(8)}
    z = np.log([[9.0, 1.0, 8.0, 7.0, 1.0, 1.0, 10.0, 6.5], [1.0, 2.0, 3.0, 4.0, 5.0, 6.0, 7.0, 8.0]])
    r = {"experts": 8, "top": 3, "groups": {"count": 4, "keep": 2}}
    idx, s = L.route(z, r, w, "")
    assert idx.tolist() == [[6, 0, 7], [7, 6, 5]]  # groups (0, 1) and (6, 7): expert 2 is closed though its score is larger than 7's
    p = np.exp(z) / np.exp(z).sum(1, keepdims=True)
    assert np.allclose(s, np.take_along_axis(p, idx, 1))
    assert L.route(z, dict(r, groups={"count": 4, "keep": 4}), w, "")[0].tolist() == L.route(z, {"experts": 8, "top": 3}, w, "")[0].tolist() == [[6, 0, 2], [7, 6, 5]]


def test_oracle_order_of_layers():
    assert L.order(MIXED) == [(0, False), (1, False), (2, False), (3, False), (1, True), (2, False), (3, False), (1, True), (2, False), (3, False), (4, False), (5, False)]
    assert L.order(config([delta(), delta()])) == [(0, False), (1, False)]
    assert L.order(config([delta(), delta()], loop=(0, 1, 2))) == [(0, False), (0, True), (1, False)]


@pytest.mark.parametrize("name", ["mixed", "even", "wide"])
def test_clear_choices_are_clear(name):
    cfg = CONFIGS[name]
    w = weights(cfg, 1)
    toks = np.random.default_rng(0).integers(0, cfg["vocab"], 30)
    eps, x, first = cfg["norm"]["eps"], w["embed"][toks], w["embed"][toks]
    for i, again in L.order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        x = x + first if again else x
        x = x + L.rms(L.MIXERS[layer["type"]](L.rms(x, eps) * w[p + "norm1"], layer["mixer"], w, p + "mix.", eps), eps) * w[p + "norm1b"]
        f = layer.get("mlp")
        if not f:
            continue
        h = L.rms(x, eps) * w[p + "norm2"]
        if f["kind"] == "moe":
            z = np.sort(h @ w[p + "mlp.router"].T, axis=1)[:, -f["router"]["top"] - 1:]
            assert f["router"]["experts"] == 1 or np.diff(z, axis=1).min() > 0.02, i
            assert len({tuple(r) for r in L.route(h, f["router"], w, p + "mlp.")[0].tolist()}) > 1
        x = x + L.rms(L.feed_forward(h, f, w, p + "mlp."), eps) * w[p + "norm2b"]


def each(kind, edit):
    """edit every mixer of a kind (left, right, channel_delta)"""
    def go(c, w):
        for i, l in enumerate(c["layers"]):
            if kind == "channel_delta" and l["type"] == kind:
                edit(l["mixer"], w, f"l{i}.mix.")
            elif kind != "channel_delta" and l["type"] == "parallel":
                edit(l["mixer"][kind], w, f"l{i}.mix.{kind}.")
    return go


def mistakes():
    yield "no sink", each("left", lambda m, w, p: w.update({p + "sink": w[p + "sink"] - 50}))
    yield "window one token wide", each("left", lambda m, w, p: m["mask"].update(size=m["mask"]["size"] + 1))
    yield "window one token narrow", each("left", lambda m, w, p: m["mask"].update(size=max(1, m["mask"]["size"] - 1)))
    yield "no YaRN", each("left", lambda m, w, p: m["rot"].pop("scaling", None))
    yield "no rotation", each("left", lambda m, w, p: m["rot"].update(base=1e30, scaling=None))
    yield "no projection bias", each("left", lambda m, w, p: w.update({p + n + ".b": w[p + n + ".b"] * 0 for n in "qkv"}))
    yield "no output bias", each("left", lambda m, w, p: w.update({p + "o.b": w[p + "o.b"] * 0}))
    yield "convolution backwards", each("left", lambda m, w, p: w.update({p + n + ".conv": w[p + n + ".conv"][:, ::-1] for n in "qkv"}))
    yield "no decay", each("right", lambda m, w, p: w.update({p + "A_log": w[p + "A_log"] - 50}))
    yield "no decay per channel", each("channel_delta", lambda m, w, p: w.update({p + "A_log": w[p + "A_log"] - 50}))
    yield "no step", each("right", lambda m, w, p: w.update({p + "dt_bias": w[p + "dt_bias"] * 0}))
    yield "no branch norm", each("right", lambda m, w, p: w.update({p + "out": w[p + "out"] * 0 + 1}))
    yield "one pass fewer", lambda c, w: c["loop"].update(times=2)
    yield "one expert fewer", lambda c, w: c["layers"][4]["mlp"]["router"].update(top=3)
    yield "groups open", lambda c, w: c["layers"][5]["mlp"]["router"]["groups"].update(keep=2)
    yield "one group fewer", lambda c, w: c["layers"][0]["mlp"]["router"]["groups"].update(keep=1)


@pytest.mark.parametrize("what", [m[0] for m in mistakes()])
def test_mistakes_would_show(what):
    """the comparison the GPU tests make tells every one of these apart, by far"""
    cfg, w = json.loads(json.dumps(MIXED)), weights(MIXED)
    toks = np.random.default_rng(5).integers(0, 333, 60)
    ref, _ = L.run(MIXED, w, toks)
    dict(mistakes())[what](cfg, w)
    got, _ = L.run(cfg, w, toks)
    assert row_err(got, ref) > 4 * TOL["bfloat16"], row_err(got, ref)


def test_embedding_output_enters_every_later_pass():
    w = weights(MIXED)
    toks = np.random.default_rng(5).integers(0, 333, 20)
    ref, taps = L.run(MIXED, w, toks)
    single = {**MIXED, "layers": MIXED["layers"][:1] + MIXED["layers"][1:4] * 3 + MIXED["layers"][4:], "loop": None}
    renamed = {}
    for i, (j, _) in enumerate(L.order(MIXED)):
        renamed.update({f"l{i}." + k.split(".", 1)[1]: v for k, v in w.items() if k.startswith(f"l{j}.")})
    renamed.update({k: w[k] for k in ("embed", "head", "final.norm")})
    got, taps1 = L.run(single, renamed, toks)
    assert all(np.allclose(a, b) for a, b in zip(taps[:4], taps1[:4])) and row_err(got, ref) > 4 * TOL["bfloat16"]


def test_beacon_holds_every_head():
    cfg = beacon_config(1000)
    w = beacon_weights(cfg, 63)
    toks = np.random.default_rng(0).integers(0, 60, 300)
    toks[37] = 63
    m, p = cfg["layers"][0]["mixer"]["left"], "l0.mix.left."
    h = L.rms(w["embed"][toks], 1e-5) * w["l0.norm1"]
    q, k = (L.causal_conv(h @ w[p + n].T + w[p + n + ".b"], w[p + n + ".conv"]).reshape(300, -1, m["dim"]) for n in "qk")
    q, k = (L.rms(L.rotate_pairs(a, m["rot"]), 1e-5) for a in (q, k))
    for n in range(m["heads"]):
        prob = L.sink_softmax(q[:, n] @ k[:, n // 2].T * m["scale"], L.window(300, 1000), w[p + "sink"][n])
        assert prob[38:, 37].min() > 0.5, (n, prob[38:, 37].min())
    # ... and its absence shows in the logits: just inside against just outside a window
    for window in (40, 41):
        c = beacon_config(window)
        a = L.run(c, w, toks[:78])[0][77]
        other = toks[:78].copy()
        other[37] = 5
        b = L.run(c, w, other)[0][77]
        assert (row_err(a[None], b[None]) > 10 * TOL["bfloat16"]) == (window == 41)
