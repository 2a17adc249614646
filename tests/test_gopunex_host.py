"""Gopunex without a GPU: configuration, registry, and the CPU restatement against itself (each function alone; what the planted mistakes
of the GPU tests must show)."""
import json

import numpy as np
import pytest

import nano_vllm_candle_amd as pkg
from nano_vllm_candle_amd import registry
from nano_vllm_candle_amd.causal_lm import tensor_shapes
from oracle import gopunex_oracle as G
from tests.berevik_util import row_err
from tests.gopunex_util import BEACON, MIXED, attn, beacon_weights, config, delta, light, sharp_weights
from tests.util import write_checkpoint


def test_config_reads_every_field(tmp_path):
    w = G.random_weights(MIXED)
    write_checkpoint(tmp_path, MIXED, w)
    c = pkg.GopunexConfig.from_dir(str(tmp_path))
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.embed_scale, c.residual_mult) == (333, 72, 1e-5, 2.0, 0.4)
    m, ff = c.layers[1]
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.bias_rows, m.bias_max, m.v_mix, m.sink, ff) == (6, 2, 40, 24, 40 ** -0.5, 16, 100.0, True, True, 88)
    m, ff = c.layers[4]
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.conv, m.decay_rank, m.gate_rank, ff) == (3, 3, 70, 33, 2, 12, 15, 0)
    m, ff = c.layers[6]
    assert (m.heads, m.dim, m.vdim, m.decay, ff) == (2, 65, 40, (1.0, 0.97), 0)
    assert c.tensor_shapes() == {k: np.shape(v) for k, v in w.items()} == tensor_shapes(str(tmp_path))
    assert registry.model_class(str(tmp_path)) is pkg.GopunexForCausalLM
    cc, ls = c.to_c(True)
    assert cc.f32 == 1 and cc.norm_offset == 1.0 and [l.mixer for l in ls] == [1, 0, 2, 0, 2, 0, 1]
    assert [ls[6].decay[i] for i in range(2)] == [1.0, 0.97] and ls[3].v_mix == 0 and ls[5].v_mix == 1 and ls[1].sink == 1


@pytest.mark.parametrize("edit, text", [
    (lambda d: d.pop("residual_mult"), "missing field"),
    (lambda d: d["layers"][0].update(type="other"), "mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="other"), "feed-forward kind"),
    (lambda d: d["layers"][0]["mixer"].update(decay=[0.5]), "decays"),
    (lambda d: d["layers"][2]["mixer"].pop("conv"), "missing field"),
])
def test_config_refuses_what_it_does_not_know(edit, text):
    d = json.loads(json.dumps(MIXED))
    edit(d)
    with pytest.raises(RuntimeError, match=text):
        pkg.GopunexConfig.from_dict(d, {k: np.shape(v) for k, v in G.random_weights(MIXED).items()})
    with pytest.raises(RuntimeError, match="missing field or tensor"):
        pkg.GopunexConfig.from_dict(MIXED, {})


def test_oracle_mechanisms():
    rng = np.random.default_rng(0)
    x = rng.standard_normal((6, 5))
    taps = rng.standard_normal((5, 3))
    y = G.causal_conv(x, taps)
    assert np.allclose(y[0], x[0] * taps[:, 2]) and np.allclose(y[4], x[4] * taps[:, 2] + x[3] * taps[:, 1] + x[2] * taps[:, 0])
    assert np.allclose(np.linalg.norm(G.unit(x * 100), axis=-1), 1.0)
    assert np.isclose(G.softplus(np.array(800.0)), 800.0) and np.isclose(G.softplus(np.array(-800.0)), 0.0) and np.isclose(G.sigmoid(np.array(-800.0)), 0.0)
    # the softmax with a sink: weights sum to less than one, to l / (1 + l)
    s = np.array([[0.0, np.log(3.0), 5.0]])
    assert np.allclose(G.softmax_one(s, np.array([[True, True, False]])), [[0.2, 0.6, 0.0]])
    assert np.allclose(G.softmax_one(s - 1000, np.ones((1, 3), bool)), 0.0)


def test_oracle_buckets():
    b = [G.bucket(n, 16, 100) for n in range(200)]
    assert b[:8] == list(range(8)) and b[8] == 8 and max(b) == 15 and b[100:] == [15] * 100 and (np.diff(b) >= 0).all()
    assert G.bucket(79, 32, 1024) < G.bucket(1023, 32, 1024) <= 31
    # exact powers sit on their edge: 16 * 2^k of a table that doubles every 4 rows
    assert [G.bucket(n, 32, 256) for n in (31, 32, 63, 64, 127, 128)] == [19, 20, 23, 24, 27, 28]
    d = G.distance_bias(5, np.arange(8.0).reshape(4, 2), 100)
    assert d.shape == (2, 5, 5) and d[1, 4, 3] == 3.0 and d[0, 1, 0] == 2.0 and d[0, 2, 2] == 0.0


def test_oracle_recurrences_against_closed_forms():
    rng = np.random.default_rng(1)
    T, H, D, E = 7, 2, 4, 3
    q, k = rng.standard_normal((2, T, H, D))
    v = rng.standard_normal((T, H, E))
    lam = np.array([0.7, 1.0])
    o = G.decay_linear_attention(q, k, v, lam)
    for t in range(T):
        for h in range(H):
            assert np.allclose(o[t, h], sum(lam[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1)))
    # the delta rule with beta 1, no decay and orthonormal keys stores every value exactly; an equal key replaces its value
    eye = np.tile(np.eye(4)[:, None, :], (1, H, 1))
    k2 = np.concatenate([eye, eye[1:2]])
    v2 = rng.standard_normal((5, H, E))
    o = G.delta_rule(np.tile(eye[1:2], (5, 1, 1)), k2, v2, np.ones_like(k2), np.ones((5, H)))
    assert np.allclose(o[0], 0) and np.allclose(o[1], v2[1]) and np.allclose(o[3], v2[1]) and np.allclose(o[4], v2[4])
    # without writes only the decays act, each on its key channel
    g = np.full_like(k2, 0.5)
    o = G.delta_rule(np.tile(eye[1:2], (5, 1, 1)), k2, v2, g, np.array([1.0, 1, 0, 0, 0])[:, None] * np.ones(H))
    assert np.allclose(o[4], 0.125 * v2[1])


def test_oracle_prefix_property():
    w = sharp_weights(MIXED)
    toks = list(range(40))
    assert np.allclose(G.forward(MIXED, w, toks, [17]), G.forward(MIXED, w, toks[:18], [-1]), atol=1e-9)


def test_values_are_mixed_from_the_first_mixing_layer_only():
    cfg = config([attn(v_mix=False), attn(), light(), attn()])
    w = sharp_weights(cfg, 2)
    toks = list(range(12))
    ref = G.forward(cfg, w, toks)
    moved = dict(w)
    moved["l1.mix.vmix"] = w["l1.mix.vmix"] + 1  # the first layer's own lambda is unused
    assert np.array_equal(G.forward(cfg, moved, toks), ref)
    moved = dict(w)
    moved["l3.mix.vmix"] = w["l3.mix.vmix"] + 1
    assert row_err(G.forward(cfg, moved, toks), ref) > 0.02


def test_planted_mistakes_show(monkeypatch):
    # a far key left out
    w = beacon_weights(BEACON, 63)
    toks = [t % 60 for t in range(300)]
    toks[5] = 63
    ref = G.forward(BEACON, w, toks, [4, 299])
    toks[5] = 7
    gone = G.forward(BEACON, w, toks, [4, 299])
    assert np.array_equal(gone[0], ref[0]) and row_err(gone[1:], ref[1:]) > 0.1
    # a distance one off, another logarithmic range, no sink, the state lost at position 20, a convolution tap left out
    cfg = config([attn(heads=4, far=60, v_mix=False, ff=0)])
    w, toks = sharp_weights(cfg, 3), list(range(120))
    ref = G.forward(cfg, w, toks)
    assert row_err(G.forward(config([attn(heads=4, far=66, v_mix=False, ff=0)]), w, toks), ref) > 0.02
    real = G.bucket
    monkeypatch.setattr(G, "bucket", lambda n, rows, far: real(n + 1, rows, far))
    assert row_err(G.forward(cfg, w, toks), ref) > 0.05
    monkeypatch.setattr(G, "bucket", real)
    soft = G.softmax_one
    monkeypatch.setattr(G, "softmax_one", lambda s, v: soft(s, v) / soft(s, v).sum(-1, keepdims=True))
    assert row_err(G.forward(cfg, w, toks)[:4], ref[:4]) > 0.05
    monkeypatch.setattr(G, "softmax_one", soft)
    for layers in ([delta(ff=0)], [light(ff=0, decay=[1.0, 0.999, 0.99])]):
        cfg = config(layers)
        w = sharp_weights(cfg, 4)
        assert row_err(G.forward(cfg, w, toks[20:40]), G.forward(cfg, w, toks[:40])[20:]) > 0.05
    cfg = config([delta(ff=0)])
    w = sharp_weights(cfg, 4)
    ref = G.forward(cfg, w, toks)
    w["l0.mix.k.conv"] = w["l0.mix.k.conv"] * np.array([0, 1, 1, 1], np.float32)
    assert row_err(G.forward(cfg, w, toks), ref) > 0.05
