"""Tafopel: a decoder of parallel layers on one layer norm each.  A layer mixes tokens by latent attention (query latents, rotated pairs
with YaRN scaling, a softmax sink, caches that later layers may share) or by a selective scan, beside a gated or a routed feed-forward or
none.  Configuration reader and model class over the C ABI's latent-attention decoder."""
import ctypes as C
import json
import os
from dataclasses import dataclass, field

import numpy as np

from . import _lib
from .causal_lm import LayeredCausalLM, Yarn, random_matrix


@dataclass
class LatentMixerConfig:
    """per head `dim` unrotated + `rot_dim` rotated query/key dimensions, value size `vdim`; latents of keys and values (`kv_rank`) and
    of queries (`q_rank`); `kv_from`: the layer whose cache this one reads (None: its own)"""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    rot_base: float
    scale: float
    yarn: Yarn = None
    kv_from: int = None


@dataclass
class ScanMixerConfig:
    """`inner` channels of `state` states, a convolution of `conv` taps, step sizes of rank `dt_rank`"""
    inner: int
    state: int
    conv: int
    dt_rank: int


@dataclass
class GeluMlpConfig:
    ff: int


@dataclass
class ExpertsConfig:
    """`top` of `experts` squared-ReLU feed-forwards of width `ff`; a shared one of width `shared_ff` (0: none)"""
    experts: int
    top: int
    ff: int
    shared_ff: int = 0


@dataclass
class TafopelConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)  # [(mixer configuration, feed-forward configuration or None)]
    norm_eps: float = 1e-6
    eos_token_id: int = None  # the design names no end-of-sequence token

    @classmethod
    def from_dict(cls, d):
        """the keys of config.json"""
        try:
            layers = []
            for i, e in enumerate(d["layers"]):
                m = e["mixer"]
                if e["type"] == "latent_attention":
                    rot = m["rot"]
                    if rot["dims"] != m["rot_dim"]:
                        raise RuntimeError(f"layer {i}: rot.dims {rot['dims']} differs from rot_dim {m['rot_dim']}")
                    yarn = Yarn.from_dict(rot.get("scaling"))
                    mix = LatentMixerConfig(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"], float(rot["base"]), float(m["scale"]), yarn,
                                            m.get("kv_from"))
                elif e["type"] == "mamba1":
                    mix = ScanMixerConfig(m["inner"], m["state"], m["conv"], m["dt_rank"])
                else:
                    raise RuntimeError(f"layer {i}: mixer type {e['type']!r} unknown (latent_attention, mamba1)")
                f = e.get("mlp")
                if f is None:
                    mlp = None
                elif f["kind"] == "dense":
                    mlp = GeluMlpConfig(f["ff"])
                elif f["kind"] == "moe":
                    mlp = ExpertsConfig(f["router"]["experts"], f["router"]["top"], f["expert"]["ff"], f["shared"]["ff"] if f.get("shared") else 0)
                else:
                    raise RuntimeError(f"layer {i}: feed-forward kind {f['kind']!r} unknown (dense, moe)")
                layers.append((mix, mlp))
            for i, (m, _) in enumerate(layers):
                j = getattr(m, "kv_from", None)
                if j is None:
                    continue
                k = layers[j][0] if 0 <= j < i else None
                if not isinstance(k, LatentMixerConfig) or k.kv_from is not None:
                    raise RuntimeError(f"layer {i}: layer {j} has no latent cache of its own before it")
                if (m.kv_rank, m.rot_dim, m.rot_base, m.yarn) != (k.kv_rank, k.rot_dim, k.rot_base, k.yarn):
                    raise RuntimeError(f"layer {i} reads the cache of layer {j}, whose sizes or rotation differ")
            return cls(d["vocab"], d["width"], layers, float(d["norm"]["eps"]))
        except KeyError as e:
            raise RuntimeError(f"Tafopel config: missing field {e}") from e

    @classmethod
    def from_dir(cls, model_dir):
        with open(os.path.join(model_dir, "config.json")) as f:
            return cls.from_dict(json.load(f))

    def tensor_shapes(self):
        """checkpoint tensor names -> shapes"""
        w = self.hidden_size
        out = {"embed": (self.vocab_size, w), "head": (self.vocab_size, w), "final.norm": (w,)}
        for i, (m, mlp) in enumerate(self.layers):
            out[f"l{i}.norm1"] = (w,)
            p = f"l{i}.mix."
            if isinstance(m, ScanMixerConfig):
                out[p + "in"], out[p + "conv"], out[p + "conv.b"] = (2 * m.inner, w), (m.inner, m.conv), (m.inner,)
                out[p + "x"], out[p + "dt"], out[p + "dt.b"] = (m.dt_rank + 2 * m.state, m.inner), (m.inner, m.dt_rank), (m.inner,)
                out[p + "A_log"], out[p + "D"], out[p + "o"] = (m.inner, m.state), (m.inner,), (w, m.inner)
            else:
                out[p + "dq"], out[p + "dq.norm"], out[p + "uq"] = (m.q_rank, w), (m.q_rank,), (m.heads * (m.dim + m.rot_dim), m.q_rank)
                if m.kv_from is None:
                    out[p + "dkv"], out[p + "dkv.norm"] = (m.kv_rank + m.rot_dim, w), (m.kv_rank,)
                out[p + "uk"], out[p + "uv"], out[p + "sink"] = (m.heads * m.dim, m.kv_rank), (m.heads * m.vdim, m.kv_rank), (m.heads,)
                out[p + "o"] = (w, m.heads * m.vdim)
            p = f"l{i}.mlp."
            if isinstance(mlp, GeluMlpConfig):
                out[p + "gate"], out[p + "up"], out[p + "down"] = (mlp.ff, w), (mlp.ff, w), (w, mlp.ff)
            elif mlp is not None:
                for e in range(mlp.experts):
                    out[f"{p}e{e}.up"], out[f"{p}e{e}.down"] = (mlp.ff, w), (w, mlp.ff)
                out[p + "router"] = (mlp.experts, w)
                if mlp.shared_ff:
                    out[p + "shared.up"], out[p + "shared.down"], out[p + "shared.sg"] = (mlp.shared_ff, w), (w, mlp.shared_ff), (1, w)
        return out

    def random_tensor(self, name, shape, rng):
        if name.endswith("A_log"):
            return np.log(np.broadcast_to(np.arange(1, shape[1] + 1, dtype=np.float32), shape))
        if len(shape) == 2:
            return random_matrix(shape, rng)
        fill = -4.0 if name.endswith("dt.b") else 0.0 if name.endswith(("conv.b", "sink")) else 1.0
        return np.full(shape, fill, np.float32)

    def to_c(self, f32):
        c = _lib.LatentConfigC(self.vocab_size, self.hidden_size, len(self.layers), 0, 0, 1, self.norm_eps, 1.0, 0.0, _lib.NORM_LAYER, 1, int(f32))
        ls = (_lib.LatentLayerC * max(len(self.layers), 1))()
        for l, (m, mlp) in zip(ls, self.layers):
            l.kv_from = -1
            if isinstance(m, ScanMixerConfig):
                l.mixer, l.inner, l.state, l.conv_taps, l.dt_rank = _lib.SELECTIVE_SCAN, m.inner, m.state, m.conv, m.dt_rank
            else:
                l.mixer, l.sink, l.rot_pairs = _lib.LATENT_ATTENTION, 1, 1
                l.heads, l.dim, l.rot_dim, l.vdim, l.kv_rank, l.q_rank = m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.q_rank
                l.rot_base, l.scale = m.rot_base, m.scale
                if m.kv_from is not None:
                    l.kv_from = m.kv_from
                if m.yarn:
                    l.yarn_factor, l.yarn_original, l.yarn_fast, l.yarn_slow = m.yarn.factor, m.yarn.original, m.yarn.fast, m.yarn.slow
            if isinstance(mlp, GeluMlpConfig):
                l.ff, l.glu = mlp.ff, _lib.GLU_GELU
            elif mlp is not None:
                l.experts, l.top, l.expert_ff, l.shared_ff, l.expert_weight_in = mlp.experts, mlp.top, mlp.ff, mlp.shared_ff, 1
        return c, ls


class TafopelForCausalLM(LayeredCausalLM):
    """Both dtypes of LayeredCausalLM.  What the design computes in 32-bit (norms, rotation, scores, softmax, routers, residual, step sizes
    and state of the scan) is so in both."""

    CONFIG = TafopelConfig

    def _create(self, cfg, f32, out):
        cc, layers = cfg.to_c(f32)
        return _lib.lib().nvllm_model_create_latent(self.ctx.h, C.byref(cc), layers, out)
