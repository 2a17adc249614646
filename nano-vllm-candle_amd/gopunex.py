"""Gopunex: a decoder whose layers mix tokens by attention with a learned distance bias, by a recurrence with constant decays
("lightning") or by a gated delta rule with a decay per key channel ("channel_delta"), each sublayer normed on its output.
Configuration reader and model class over the C ABI's hybrid decoder."""
import ctypes as C
import json
import os
from dataclasses import dataclass, field

import numpy as np

from . import _lib
from .causal_lm import LayeredCausalLM, random_matrix, tensor_shapes

NORM_OFFSET = 1.0  # layer and output norm weights are stored minus this


@dataclass
class BiasAttentionConfig:
    """grouped-query attention; `bias_rows` rows of the distance table, logarithmic up to distance `bias_max`; the softmax has a sink"""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_rows: int
    bias_max: float
    v_mix: bool = False
    sink: bool = True


@dataclass
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple


@dataclass
class ChannelDeltaConfig:
    """`conv` taps of the short convolutions; ranks of the two-step projections of decays and output gate"""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int
    gate_rank: int


@dataclass
class GopunexConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)  # [(mixer configuration, feed-forward width or 0)]
    norm_eps: float = 1e-6
    embed_scale: float = 1.0
    residual_mult: float = 1.0
    eos_token_id: int = None  # the design names no end-of-sequence token

    @classmethod
    def from_dict(cls, d, shapes):
        """the keys of config.json; `shapes` (tensor name -> shape) supplies the sizes config.json leaves to the checkpoint"""
        try:
            layers = []
            for i, e in enumerate(d["layers"]):
                m, p = e["mixer"], f"l{i}.mix."
                if e["type"] == "attention":
                    mix = BiasAttentionConfig(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]), shapes[p + "rel"][0], float(m["bias_max"]),
                                              bool(m.get("v_mix")))
                elif e["type"] == "lightning":
                    mix = LightningConfig(m["heads"], m["dim"], m["vdim"], tuple(float(x) for x in m["decay"]))
                    if len(mix.decay) != mix.heads:
                        raise RuntimeError(f"layer {i}: {len(mix.decay)} decays for {mix.heads} heads")
                elif e["type"] == "channel_delta":
                    mix = ChannelDeltaConfig(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], shapes[p + "a1"][0], shapes[p + "g1"][0])
                else:
                    raise RuntimeError(f"layer {i}: mixer type {e['type']!r} unknown (attention, lightning, channel_delta)")
                mlp = e.get("mlp")
                if mlp is not None and mlp["kind"] != "dense":
                    raise RuntimeError(f"layer {i}: feed-forward kind {mlp['kind']!r} unknown (dense)")
                layers.append((mix, mlp["ff"] if mlp is not None else 0))
            return cls(d["vocab"], d["width"], layers, float(d["norm"]["eps"]), float(d["embedding"]["scale"]), float(d["residual_mult"]))
        except KeyError as e:
            raise RuntimeError(f"Gopunex config: missing field or tensor {e}") from e

    @classmethod
    def from_dir(cls, model_dir):
        with open(os.path.join(model_dir, "config.json")) as f:
            return cls.from_dict(json.load(f), tensor_shapes(model_dir))

    def tensor_shapes(self):
        """checkpoint tensor names -> shapes"""
        w = self.hidden_size
        out = {"embed": (self.vocab_size, w), "head": (self.vocab_size, w), "final.norm": (w,)}
        for i, (m, ff) in enumerate(self.layers):
            p = f"l{i}.mix."
            out[f"l{i}.norm1"] = (w,)
            if isinstance(m, BiasAttentionConfig):
                for n, rows in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
                    out[p + n], out[p + n + ".b"] = (rows, w), (rows,)
                out[p + "q.norm"], out[p + "k.norm"] = (m.heads * m.dim,), (m.kv_heads * m.dim,)
                out[p + "rel"] = (m.bias_rows, m.heads)
                if m.v_mix:
                    out[p + "vmix"] = ()
            elif isinstance(m, LightningConfig):
                for n, rows in (("q", m.heads * m.dim), ("k", m.heads * m.dim), ("v", m.heads * m.vdim), ("g", m.heads * m.vdim)):
                    out[p + n] = (rows, w)
                out[p + "norm"] = (m.heads * m.vdim,)
            else:
                for n, rows in (("q", m.kv_heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.heads * m.vdim)):
                    out[p + n], out[p + n + ".conv"] = (rows, w), (rows, m.conv)
                out[p + "b"], out[p + "A_log"], out[p + "dt_bias"], out[p + "norm"] = (m.heads, w), (m.heads,), (m.heads * m.dim,), (m.vdim,)
                out[p + "a1"], out[p + "a2"] = (m.decay_rank, w), (m.heads * m.dim, m.decay_rank)
                out[p + "g1"], out[p + "g2"] = (m.gate_rank, w), (m.heads * m.vdim, m.gate_rank)
            out[p + "o"] = (w, m.heads * m.vdim)
            if ff:
                out[f"l{i}.norm2"], out[f"l{i}.mlp.up"], out[f"l{i}.mlp.down"] = (w,), (ff, w), (w, ff)
        return out

    def random_tensor(self, name, shape, rng):
        if len(shape) == 2:
            return random_matrix(shape, rng)
        ones = name.endswith(("q.norm", "k.norm", "mix.norm"))
        fill = 0.5 if name.endswith("vmix") else -1.0 if name.endswith(("A_log", "dt_bias")) else float(ones)
        return np.full(shape, fill, np.float32)

    def to_c(self, f32):
        c = _lib.HybridConfigC(self.vocab_size, self.hidden_size, len(self.layers), self.norm_eps, self.embed_scale, self.residual_mult, NORM_OFFSET, int(f32))
        ls = (_lib.HybridLayerC * max(len(self.layers), 1))()
        for l, (m, ff) in zip(ls, self.layers):
            l.heads, l.kv_heads, l.dim, l.vdim, l.ff = m.heads, getattr(m, "kv_heads", m.heads), m.dim, m.vdim, ff
            if isinstance(m, BiasAttentionConfig):
                l.mixer, l.scale, l.bias_rows, l.bias_max, l.sink, l.v_mix = _lib.MIXER_ATTENTION, m.scale, m.bias_rows, m.bias_max, m.sink, m.v_mix
            elif isinstance(m, LightningConfig):
                l.mixer, l.decay = _lib.MIXER_LINEAR, (C.c_double * m.heads)(*m.decay)
            else:
                l.mixer, l.conv_taps, l.decay_rank, l.gate_rank = _lib.MIXER_DELTA, m.conv, m.decay_rank, m.gate_rank
        return c, ls


class GopunexForCausalLM(LayeredCausalLM):
    """Both dtypes of LayeredCausalLM.  What the design computes in 32-bit (norms, scores, softmax, residual, gates and state of the
    recurrences) is so in both."""

    CONFIG = GopunexConfig

    def _create(self, cfg, f32, out):
        cc, layers = cfg.to_c(f32)
        return _lib.lib().nvllm_model_create_hybrid(self.ctx.h, C.byref(cc), layers, out)
