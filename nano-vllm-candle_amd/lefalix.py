"""Lefalix: a decoder whose sublayers are normed on both sides.  A layer mixes tokens by windowed attention (short convolutions, rotated
pairs with YaRN scaling, norms per head, a learned sink) beside a gated delta rule with one decay per head ("parallel"), or by a gated
delta rule with a decay per key channel ("channel_delta"); its feed-forward is an exact-GELU one, routed to gated experts, or absent.  A
range of layers may be passed through several times.  Configuration reader and model class over the C ABI's hybrid decoder."""
import ctypes as C
import json
import os
from dataclasses import dataclass, field

import numpy as np

from . import _lib
from .causal_lm import LayeredCausalLM, Yarn, random_matrix, tensor_shapes


@dataclass
class WindowAttentionConfig:
    """`window` visible positions; `conv` taps; the first `rot_dim` dimensions of a head turn"""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int
    conv: int
    rot_dim: int
    rot_base: float
    yarn: Yarn = None

    @classmethod
    def from_dict(cls, m):
        rot = m["rot"]
        return cls(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]), m["mask"]["size"], m["conv"], rot["dims"], float(rot["base"]),
                   Yarn.from_dict(rot.get("scaling")))

    def tensor_shapes(self, p, w):
        out = {}
        for n, rows in (("q", self.heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.kv_heads * self.vdim)):
            out[p + n], out[p + n + ".b"], out[p + n + ".conv"] = (rows, w), (rows,), (rows, self.conv)
        out[p + "sink"], out[p + "o"], out[p + "o.b"] = (self.heads,), (w, self.heads * self.vdim), (w,)
        return out

    def to_c(self, l):
        l.mixer, l.qk_norm, l.sink, l.out_bias = _lib.MIXER_ATTENTION, _lib.QK_NORM_HEAD, _lib.SINK_HEAD, 1
        l.heads, l.kv_heads, l.dim, l.vdim, l.scale, l.window, l.conv_taps = self.heads, self.kv_heads, self.dim, self.vdim, self.scale, self.window, self.conv
        l.rot_dim, l.rot_base = self.rot_dim, self.rot_base
        if self.yarn:
            l.yarn_factor, l.yarn_original, l.yarn_fast, l.yarn_slow = self.yarn.factor, self.yarn.original, self.yarn.fast, self.yarn.slow


@dataclass
class DeltaConfig:
    """gated delta rule with `conv` taps; ranks of the two-step projections of decays and output gate (0: one decay per head, a gate of one
    projection)"""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int = 0
    gate_rank: int = 0

    @classmethod
    def from_dict(cls, m, decay_rank=0, gate_rank=0):
        return cls(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], decay_rank, gate_rank)

    def tensor_shapes(self, p, w):
        out = {}
        for n, rows in (("q", self.kv_heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.heads * self.vdim)):
            out[p + n], out[p + n + ".conv"] = (rows, w), (rows, self.conv)
        out[p + "b"], out[p + "A_log"], out[p + "norm"], out[p + "o"] = (self.heads, w), (self.heads,), (self.vdim,), (w, self.heads * self.vdim)
        if self.decay_rank:
            out[p + "a1"], out[p + "a2"], out[p + "dt_bias"] = (self.decay_rank, w), (self.heads * self.dim, self.decay_rank), (self.heads * self.dim,)
            out[p + "g1"], out[p + "g2"] = (self.gate_rank, w), (self.heads * self.vdim, self.gate_rank)
        else:
            out[p + "a"], out[p + "dt_bias"], out[p + "g"] = (self.heads, w), (self.heads,), (self.heads * self.vdim, w)
        return out

    def to_c(self, l):
        l.mixer, l.heads, l.kv_heads, l.dim, l.vdim = _lib.MIXER_DELTA, self.heads, self.kv_heads, self.dim, self.vdim
        l.conv_taps, l.decay_rank, l.gate_rank = self.conv, self.decay_rank, self.gate_rank


@dataclass
class DenseConfig:
    ff: int


@dataclass
class RoutedConfig:
    """`top` of `experts` gated feed-forwards of width `ff`, out of the best `kept` of `groups` groups of neighbours"""
    experts: int
    top: int
    ff: int
    groups: int = 1
    kept: int = 1


@dataclass
class LefalixConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)  # [((mixer configuration,) or (left, right), feed-forward configuration or None)]
    loop: tuple = (0, 0, 1)                     # first layer, layer behind the last, passes
    norm_eps: float = 1e-6
    eos_token_id: int = None  # the design names no end-of-sequence token

    @classmethod
    def from_dict(cls, d, shapes):
        """the keys of config.json; `shapes` (tensor name -> shape) supplies the sizes config.json leaves to the checkpoint"""
        try:
            layers = []
            for i, e in enumerate(d["layers"]):
                m, p = e["mixer"], f"l{i}.mix."
                if e["type"] == "parallel":
                    mix = (WindowAttentionConfig.from_dict(m["left"]), DeltaConfig.from_dict(m["right"]))
                elif e["type"] == "channel_delta":
                    mix = (DeltaConfig.from_dict(m, shapes[p + "a1"][0], shapes[p + "g1"][0]),)
                else:
                    raise RuntimeError(f"layer {i}: mixer type {e['type']!r} unknown (parallel, channel_delta)")
                f = e.get("mlp")
                if f is None:
                    mlp = None
                elif f["kind"] == "dense":
                    mlp = DenseConfig(f["ff"])
                elif f["kind"] == "moe":
                    r, g = f["router"], f["router"].get("groups")
                    mlp = RoutedConfig(r["experts"], r["top"], f["expert"]["ff"], *((g["count"], g["keep"]) if g else ()))
                else:
                    raise RuntimeError(f"layer {i}: feed-forward kind {f['kind']!r} unknown (dense, moe)")
                layers.append((mix, mlp))
            loop = d.get("loop")
            loop = (loop["start"], loop["stop"], loop["times"]) if loop and loop["stop"] > loop["start"] else (0, 0, 1)
            return cls(d["vocab"], d["width"], layers, loop, float(d["norm"]["eps"]))
        except KeyError as e:
            raise RuntimeError(f"Lefalix config: missing field or tensor {e}") from e

    @classmethod
    def from_dir(cls, model_dir):
        with open(os.path.join(model_dir, "config.json")) as f:
            return cls.from_dict(json.load(f), tensor_shapes(model_dir))

    def tensor_shapes(self):
        """checkpoint tensor names -> shapes"""
        w = self.hidden_size
        out = {"embed": (self.vocab_size, w), "head": (self.vocab_size, w), "final.norm": (w,)}
        for i, (mix, mlp) in enumerate(self.layers):
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
                out[f"l{i}.{n}"] = (w,)
            for m, side in zip(mix, ("left.", "right.") if len(mix) == 2 else ("",)):
                out.update(m.tensor_shapes(f"l{i}.mix.{side}", w))
                if side:
                    out[f"l{i}.mix.{side}out"] = (w,)
            p = f"l{i}.mlp."
            if isinstance(mlp, DenseConfig):
                out[p + "up"], out[p + "down"] = (mlp.ff, w), (w, mlp.ff)
            elif mlp is not None:
                for e in range(mlp.experts):
                    out[f"{p}e{e}.gate"], out[f"{p}e{e}.up"], out[f"{p}e{e}.down"] = (mlp.ff, w), (mlp.ff, w), (w, mlp.ff)
                out[p + "router"] = (mlp.experts, w)
        return out

    def random_tensor(self, name, shape, rng):
        if len(shape) == 2:
            return random_matrix(shape, rng)
        fill = -1.0 if name.endswith(("A_log", "dt_bias")) else 0.0 if name.endswith((".b", "sink")) else 1.0
        return np.full(shape, fill, np.float32)

    def to_c(self, f32):
        c = _lib.HybridConfigC(self.vocab_size, self.hidden_size, len(self.layers), self.norm_eps, 1.0, 1.0, 0.0, int(f32), 1, *self.loop)
        ls = (_lib.HybridLayerC * max(len(self.layers), 1))()
        for l, (mix, mlp) in zip(ls, self.layers):
            l.branches = len(mix)
            for m, side in zip(mix, (l.mix, l.side)):
                m.to_c(side)
            if isinstance(mlp, DenseConfig):
                l.ff, l.act = mlp.ff, _lib.ACT_GELU
            elif mlp is not None:
                l.experts, l.top, l.expert_ff, l.groups, l.groups_kept = mlp.experts, mlp.top, mlp.ff, mlp.groups, mlp.kept
        return c, ls


class LefalixForCausalLM(LayeredCausalLM):
    """Both dtypes of LayeredCausalLM.  What the design computes in 32-bit (norms, rotation, scores, softmax, routers, residual, gates and
    state of the recurrences) is so in both."""

    CONFIG = LefalixConfig

    def _create(self, cfg, f32, out):
        cc, layers = cfg.to_c(f32)
        return _lib.lib().nvllm_model_create_hybrid(self.ctx.h, C.byref(cc), layers, out)
