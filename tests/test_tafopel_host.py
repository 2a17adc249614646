"""Tafopel without a GPU: configuration, registry, and the CPU restatement against itself (each function alone; what mistakes the GPU
tests would show)."""
import json

import numpy as np
import pytest

import nano_vllm_candle_amd as pkg
from nano_vllm_candle_amd import _lib, registry
from nano_vllm_candle_amd.causal_lm import tensor_shapes
from oracle import tafopel_oracle as T
from tests.berevik_util import row_err
from tests.tafopel_util import BEACON, CONFIGS, MIXED, TOL, YARN, attn, beacon_weights, clear_choices, config, mamba, moe, weights
from tests.util import write_checkpoint


def test_config_reads_every_field(tmp_path):
    w = T.random_weights(MIXED)
    write_checkpoint(tmp_path, MIXED, w)
    c = pkg.TafopelConfig.from_dir(str(tmp_path))
    assert (c.vocab_size, c.hidden_size, c.norm_eps) == (333, 72, 1e-5)
    m, f = c.layers[0]
    assert (m.inner, m.state, m.conv, m.dt_rank, f.ff) == (40, 6, 3, 5, 56)
    m, f = c.layers[1]
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.q_rank, m.rot_base, m.scale, m.kv_from) == (3, 20, 12, 18, 40, 36, 300.0, 32 ** -0.5, None)
    assert (m.yarn.factor, m.yarn.original, m.yarn.fast, m.yarn.slow) == (5.0, 48.0, 6.0, 0.7) and (f.experts, f.top, f.ff, f.shared_ff) == (6, 2, 24, 40)
    assert c.layers[2][0].kv_from == 1 and c.layers[2][1] is None and c.layers[3][1].shared_ff == 0 and c.layers[4][0].yarn is None
    assert c.tensor_shapes() == {k: np.shape(v) for k, v in w.items()} == tensor_shapes(str(tmp_path))
    assert registry.model_class(str(tmp_path)) is pkg.TafopelForCausalLM
    cc, ls = c.to_c(True)
    assert cc.f32 == 1 and cc.norm == _lib.NORM_LAYER and cc.one_norm == 1
    assert [l.mixer for l in ls] == [1, 0, 0, 1, 0, 0, 0, 1] and [l.kv_from for l in ls] == [-1, -1, 1, -1, -1, 1, 4, -1]
    assert ls[1].rot_pairs == 1 and ls[1].sink == 1 and ls[1].yarn_factor == 5.0 and ls[4].yarn_factor == 0.0 and ls[5].top == 4 and ls[5].expert_weight_in == 1
    assert ls[7].state == 19 and ls[0].glu == _lib.GLU_GELU and ls[3].shared_ff == 0


@pytest.mark.parametrize("edit, text", [
    (lambda d: d.pop("norm"), "missing field"),
    (lambda d: d["layers"][0].update(type="other"), "mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="other"), "feed-forward kind"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=10), "rot.dims"),
    (lambda d: d["layers"][2]["mixer"].update(kv_from=0), "no latent cache"),
    (lambda d: d["layers"][2]["mixer"].update(kv_from=2), "no latent cache"),
    (lambda d: d["layers"][5]["mixer"].update(kv_from=2), "no latent cache"),
    (lambda d: d["layers"][2]["mixer"].update(kv_rank=41), "differ"),
    (lambda d: d["layers"][2]["mixer"]["rot"]["scaling"].update(factor=2.0), "differ"),
    (lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].pop("slow"), "missing field"),
])
def test_config_refuses_what_it_does_not_know(edit, text):
    d = json.loads(json.dumps(MIXED))
    edit(d)
    with pytest.raises(RuntimeError, match=text):
        pkg.TafopelConfig.from_dict(d)


def test_random_tensors_cover_every_shape():
    c = pkg.TafopelConfig.from_dict(MIXED)
    rng = np.random.default_rng(0)
    for name, shape in c.tensor_shapes().items():
        assert np.shape(c.random_tensor(name, shape, rng)) == shape, name


def test_oracle_functions():
    rng = np.random.default_rng(0)
    x = rng.standard_normal((6, 5))
    n = T.layer_norm(x + 100.0, np.ones(5), 0.0)
    assert np.allclose(n.mean(1), 0) and np.allclose((n * n).mean(1), 1) and np.allclose(n, T.layer_norm(x, np.ones(5), 0.0))
    assert np.allclose(T.layer_norm(np.full((1, 4), 3.0), np.ones(4), 1e-3), 0.0)
    assert np.allclose(T.rms_norm(np.full((1, 4), 2.0), np.ones(4), 12.0), 0.5)
    k, b = rng.standard_normal((5, 3)), rng.standard_normal(5)
    y = T.causal_conv(x, k, b)
    assert np.allclose(y[0], x[0] * k[:, 2] + b) and np.allclose(y[4], x[4] * k[:, 2] + x[3] * k[:, 1] + x[2] * k[:, 0] + b)
    assert np.allclose(T.gelu_tanh(np.array([-10.0, 0.0, 10.0])), [0.0, 0.0, 10.0]) and np.isclose(T.gelu_tanh(1.0), 0.8411919906)
    assert np.isclose(T.softplus(np.array(800.0)), 800.0) and np.isclose(T.softplus(np.array(-800.0)), 0.0) and np.isclose(T.sigmoid(np.array(-800.0)), 0.0)
    assert np.allclose(T.relu2(np.array([-3.0, 2.0])), [0.0, 4.0])


def test_oracle_sink():
    s = np.array([[0.0, np.log(3.0), 5.0]])
    seen = np.array([[True, True, False]])
    assert np.allclose(T.sink_softmax(s, seen, 0.0), [[0.2, 0.6, 0.0]])
    assert np.allclose(T.sink_softmax(s, seen, -1000.0), [[0.25, 0.75, 0.0]]) and np.allclose(T.sink_softmax(s, seen, 1000.0), 0.0)
    assert np.allclose(T.sink_softmax(s - 1000, seen, -1000.0), [[0.2, 0.6, 0.0]])


def test_oracle_rotation():
    f, mult = T.rotation({"dims": 8, "base": 100.0})
    assert mult == 1.0 and np.allclose(f, [1.0, 100 ** -0.25, 0.1, 100 ** -0.75])
    g, mult = T.rotation({"dims": 16, "base": 300.0, "scaling": YARN})
    f, _ = T.rotation({"dims": 16, "base": 300.0})
    ratio = g / f
    assert np.isclose(mult, 0.1 * np.log(5.0) + 1) and ratio[0] == 1.0 and np.isclose(ratio[-1], 0.2) and (np.diff(ratio) <= 1e-12).all() and ((ratio > 0.21) & (ratio < 0.99)).any()
    x = np.random.default_rng(1).standard_normal((4, 16))
    y = T.rotary_pairs(x, [0, 1, 2, 9], {"dims": 16, "base": 300.0})
    assert np.allclose(y[0], x[0]) and np.allclose(np.linalg.norm(y, axis=1), np.linalg.norm(x, axis=1))
    assert np.allclose(y[3, 0] + 1j * y[3, 1], (x[3, 0] + 1j * x[3, 1]) * np.exp(9j))
    # one step for fast and slow pairs: the ramp has no width, and no division by zero
    g, _ = T.rotation({"dims": 4, "base": 10.0, "scaling": {"factor": 2.0, "original": 10000, "fast": 1.0, "slow": 1.0}})
    assert np.isfinite(g).all()


def test_oracle_scan_against_the_closed_form():
    rng = np.random.default_rng(2)
    n, s, t = 3, 4, 7
    x, dt = rng.standard_normal((t, n)), rng.uniform(0.1, 1, (t, n))
    A, B, C, D = -rng.uniform(0.2, 2, (n, s)), rng.standard_normal((t, s)), rng.standard_normal((t, s)), rng.standard_normal(n)
    y = T.selective_scan(x, dt, A, B, C, D)
    for i in range(t):
        want = D * x[i]
        for j in range(i + 1):
            decay = np.exp(A * dt[j + 1:i + 1].sum(0)[:, None])
            want = want + ((decay * B[j]) @ C[i]) * dt[j] * x[j]
        assert np.allclose(y[i], want)


def test_oracle_experts():
    cfg = config([mamba(mlp=moe(4, 2, 6, 5))], width=8, vocab=9)
    w = T.random_weights(cfg, 3)
    h = np.random.default_rng(0).standard_normal((5, 8))
    idx, s = T.route(h, w, "l0.mlp.", 2)
    z = h @ w["l0.mlp.router"].T
    for t in range(5):
        assert set(idx[t]) == set(np.argsort(z[t])[-2:]) and np.allclose(s[t], 1 / (1 + np.exp(-z[t][idx[t]])))
    y = T.experts(h, cfg["layers"][0]["mlp"], w, "l0.mlp.")
    one = sum(g * g * T.plain(h[:1], w, f"l0.mlp.e{e}.") for e, g in zip(idx[0], s[0]))  # squared ReLU: an input factor comes out squared
    shared = T.plain(h[:1], w, "l0.mlp.shared.") * T.sigmoid(h[:1] @ w["l0.mlp.shared.sg"].T)
    assert np.allclose(y[0], one + shared)


def test_clear_choices_are_clear():
    for cfg in (MIXED, CONFIGS["even"]):
        w = weights(cfg, 1)
        toks = np.random.default_rng(0).integers(0, cfg["vocab"], 40)
        _, taps = T.run(cfg, w, toks)
        xs = [w["embed"][toks]] + taps
        for i, l in enumerate(cfg["layers"]):
            if not l.get("mlp") or l["mlp"]["kind"] != "moe":
                continue
            z = np.sort(T.layer_norm(xs[i], w[f"l{i}.norm1"], 1e-5) @ w[f"l{i}.mlp.router"].T, axis=1)
            assert np.diff(z, axis=1).min() > 0.02 * np.abs(z).max(), i
            assert len({tuple(r) for r in T.route(T.layer_norm(xs[i], w[f"l{i}.norm1"], 1e-5), w, f"l{i}.mlp.", l["mlp"]["router"]["top"])[0].tolist()}) > 1


def mistakes():
    yield "no sink", lambda c, w: [w.update({k: v - 50 for k, v in w.items() if k.endswith("sink")})]
    yield "no YaRN", lambda c, w: [l["mixer"]["rot"].pop("scaling", None) for l in c["layers"] if l["type"] == "latent_attention"]
    yield "cache of another layer", lambda c, w: c["layers"][5]["mixer"].pop("kv_from") and w.update({"l5.mix.dkv": w["l1.mix.dkv"], "l5.mix.dkv.norm": w["l1.mix.dkv.norm"]})
    yield "no convolution bias", lambda c, w: w.update({k: v * 0 for k, v in w.items() if k.endswith("conv.b")})
    yield "no skip", lambda c, w: w.update({k: v * 0 for k, v in w.items() if k.endswith(".D")})
    yield "one expert fewer", lambda c, w: c["layers"][5]["mlp"]["router"].update(top=3)
    yield "no shared expert", lambda c, w: c["layers"][5]["mlp"].pop("shared")
    yield "shared gate at one half", lambda c, w: w.update({"l1.mlp.shared.sg": w["l1.mlp.shared.sg"] * 0})


@pytest.mark.parametrize("what", [m[0] for m in mistakes()])
def test_mistakes_would_show(what):
    """the comparison the GPU tests make tells every one of these apart, by far"""
    cfg, w = json.loads(json.dumps(MIXED)), weights(MIXED)
    toks = np.random.default_rng(5).integers(0, 333, 60)
    ref, _ = T.run(MIXED, w, toks)
    dict(mistakes())[what](cfg, w)
    got, _ = T.run(cfg, w, toks)
    assert row_err(got, ref) > 4 * TOL["bfloat16"], row_err(got, ref)


def test_beacon_holds_every_head():
    w = beacon_weights(BEACON, 63)
    toks = np.random.default_rng(0).integers(0, 60, 400)
    toks[37] = 63
    h = T.layer_norm(w["embed"][toks], w["l0.norm1"], 1e-5)
    m = BEACON["layers"][0]["mixer"]
    c, r = T.latents(h, m, w, "l0.mix.", 1e-5)
    q = (T.rms_norm(h @ w["l0.mix.dq"].T, w["l0.mix.dq.norm"], 1e-5) @ w["l0.mix.uq"].T).reshape(400, 4, 48)
    for n in range(4):
        s = (q[:, n, :32] @ (c @ w["l0.mix.uk"][n * 32:(n + 1) * 32].T).T + T.rotary_pairs(q[:, n, 32:], np.arange(400), m["rot"]) @ r.T) * m["scale"]
        p = T.sink_softmax(s, np.tril(np.ones((400, 400), bool)), w["l0.mix.sink"][n])
        assert p[38:, 37].min() > 0.5, (n, p[38:, 37].min())


def test_clear_choices_leave_plain_models_alone():
    cfg = config([attn()])
    w = T.random_weights(cfg)
    assert clear_choices(cfg, dict(w)) == w
