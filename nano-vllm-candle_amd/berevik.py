"""Berevik: a decoder of parallel layers (windowed latent attention beside a clamped gated feed-forward, a norm for each), with
an optional looped range of layers, scaled embeddings and a soft-capped head.  Configuration reader and model class over the
C ABI's latent-attention decoder."""
import ctypes as C
import json
import os
from dataclasses import dataclass, field

import numpy as np

from . import _lib
from .causal_lm import LayeredCausalLM, random_matrix

GLU_ALPHA = 1.702  # gate slope of the feed-forward's sigmoid
GLU_SHIFT = 1.0    # added to the clamped up branch


@dataclass
class LatentAttentionConfig:
    """one layer's mixer: per head `dim` unrotated + `rot_dim` rotated query/key dimensions, value size `vdim`; latent size
    `kv_rank`; position i sees the last `window` positions, itself included (0: all)"""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    window: int
    rot_base: float
    scale: float


@dataclass
class GatedMlpConfig:
    ff: int
    limit: float
    alpha: float = GLU_ALPHA
    shift: float = GLU_SHIFT


@dataclass
class BerevikConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)  # [(LatentAttentionConfig, GatedMlpConfig or None)]
    norm_eps: float = 1e-6
    embed_scale: float = 1.0
    logit_softcap: float = 0.0
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    eos_token_id: int = None  # the design names no end-of-sequence token

    @property
    def num_runs(self):
        """layer runs of one forward pass (a looped layer counts every time)"""
        n = len(self.layers)
        return n + (self.loop_stop - self.loop_start) * (self.loop_times - 1)

    @classmethod
    def from_dict(cls, d):
        """the keys of config.json"""
        try:
            layers = []
            for i, e in enumerate(d["layers"]):
                if e["type"] != "latent_attention":
                    raise RuntimeError(f"layer {i}: mixer type {e['type']!r} unknown (latent_attention)")
                m, rot, mask = e["mixer"], e["mixer"]["rot"], e["mixer"].get("mask")
                if rot["dims"] != m["rot_dim"]:
                    raise RuntimeError(f"layer {i}: rot.dims {rot['dims']} differs from rot_dim {m['rot_dim']}")
                mix = LatentAttentionConfig(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], mask["size"] if mask else 0,
                                            float(rot["base"]), float(m["scale"]))
                mlp = e.get("mlp")
                if mlp is not None:
                    if mlp["kind"] != "dense":
                        raise RuntimeError(f"layer {i}: feed-forward kind {mlp['kind']!r} unknown (dense)")
                    mlp = GatedMlpConfig(mlp["ff"], float(mlp["limit"]))
                layers.append((mix, mlp))
            loop = d.get("loop") or {"start": 0, "stop": 0, "times": 1}
            return cls(d["vocab"], d["width"], layers, float(d["norm"]["eps"]), float(d["embedding"]["scale"]),
                       float(d.get("logit_softcap") or 0.0), loop["start"], loop["stop"], loop["times"])
        except KeyError as e:
            raise RuntimeError(f"Berevik config: missing field {e}") from e

    @classmethod
    def from_dir(cls, model_dir):
        with open(os.path.join(model_dir, "config.json")) as f:
            return cls.from_dict(json.load(f))

    def tensor_shapes(self):
        """checkpoint tensor names -> shapes"""
        w = self.hidden_size
        out = {"embed": (self.vocab_size, w), "head": (self.vocab_size, w), "final.norm": (w,)}
        for i, (m, mlp) in enumerate(self.layers):
            p = f"l{i}."
            out[p + "norm1"] = (w,)
            out[p + "mix.q"] = (m.heads * (m.dim + m.rot_dim), w)
            out[p + "mix.dkv"] = (m.kv_rank + m.rot_dim, w)
            out[p + "mix.dkv.norm"] = (m.kv_rank,)
            out[p + "mix.uk"] = (m.heads * m.dim, m.kv_rank)
            out[p + "mix.uv"] = (m.heads * m.vdim, m.kv_rank)
            out[p + "mix.o"] = (w, m.heads * m.vdim)
            if mlp is not None:
                out[p + "norm2"] = (w,)
                out[p + "mlp.gate"] = (mlp.ff, w)
                out[p + "mlp.up"] = (mlp.ff, w)
                out[p + "mlp.down"] = (w, mlp.ff)
        return out

    def random_tensor(self, name, shape, rng):
        return np.ones(shape, np.float32) if len(shape) == 1 else random_matrix(shape, rng)

    def to_c(self, f32):
        c = _lib.LatentConfigC(self.vocab_size, self.hidden_size, len(self.layers), self.loop_start, self.loop_stop, self.loop_times,
                               self.norm_eps, self.embed_scale, self.logit_softcap, _lib.NORM_RMS, 0, int(f32))
        ls = (_lib.LatentLayerC * max(len(self.layers), 1))()
        for l, (m, mlp) in zip(ls, self.layers):
            l.heads, l.dim, l.rot_dim, l.vdim, l.kv_rank, l.window = m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.window
            l.rot_base, l.scale, l.kv_from = m.rot_base, m.scale, -1
            if mlp is not None:
                l.ff, l.glu_limit, l.glu_alpha, l.glu_shift = mlp.ff, mlp.limit, mlp.alpha, mlp.shift
        return c, ls


class BerevikForCausalLM(LayeredCausalLM):
    """Both dtypes of LayeredCausalLM.  What the design computes in 32-bit (norms, rotation, scores, softmax, residual) is so in both."""

    CONFIG = BerevikConfig

    def _create(self, cfg, f32, out):
        cc, layers = cfg.to_c(f32)
        return _lib.lib().nvllm_model_create_latent(self.ctx.h, C.byref(cc), layers, out)
