"""`bench.py --gopunex`: prefill and decode throughput of the Gopunex design at layer sizes of real models (random weights), beside Qwen3
layers of equal size (same width, heads, feed-forward parameters, depth, vocabulary, prompts and batch).  Prints one JSON line per size
and mixer (every layer the same mixer, and all three in turn), with HIP-event times per kernel class and the fraction of its roofline
that the mixer's own kernel reaches."""
import json

import numpy as np

from bench_berevik import HBM_GBS, MFMA_TFLOPS, measure, rooflines

F32_TFLOPS = 157.3  # f32 matrix rate: the recurrences are computed in 32-bit

# width, heads (all of 128), kv heads of the attention layers and of the Qwen3 twin, feed-forward width of the twin (two thirds of a
# two-matrix feed-forward of equal parameters), layers
SIZES = {
    "1k": dict(width=1024, heads=16, kv=8, ff=3072, layers=12),
    "2k": dict(width=2048, heads=16, kv=8, ff=6144, layers=6),
    "4k": dict(width=4096, heads=32, kv=8, ff=12288, layers=3),
}
MIXERS = ("attention", "channel_delta", "lightning", "mixed")
CLASSES = ("attn", "recur", "gemm", "norm", "qk", "silu", "lm_head")


def mixer(kind, z):
    from nano_vllm_candle_amd.gopunex import BiasAttentionConfig, ChannelDeltaConfig, LightningConfig

    h = z["heads"]
    if kind == "attention":
        return BiasAttentionConfig(h, z["kv"], 128, 128, 128 ** -0.5, 32, 512.0, True)
    if kind == "lightning":
        return LightningConfig(h, 128, 128, tuple(float(np.exp(-8.0 * (i + 1) / h / 16)) for i in range(h)))
    return ChannelDeltaConfig(h, h, 128, 128, 4, 128, 128)


def gopunex_config(pkg, z, kind, vocab):
    kinds = MIXERS[:3] if kind == "mixed" else (kind,)
    layers = [(mixer(kinds[i % len(kinds)], z), z["ff"] * 3 // 2) for i in range(z["layers"])]
    return pkg.GopunexConfig(vocab, z["width"], layers, 1e-6, 1.0, 0.5)


def recurrence_rooflines(r, z, kind, batch, prompt):
    """decode: the state read and written once over HBM; prefill: the token recurrence's own operations over the f32 matrix rate"""
    elems = z["heads"] * 128 * 128
    r["decode_recur_hbm_frac"] = round(z["layers"] * batch * elems * 8 / (r["decode_class_ms"]["recur"][0] * 1e-3) / 1e9 / HBM_GBS, 4)
    flops = (7 if kind == "channel_delta" else 5) * elems
    r["prefill_recur_f32_frac"] = round(z["layers"] * batch * prompt * flops / (r["prefill_class_ms"]["recur"][0] * 1e-3) / 1e12 / F32_TFLOPS, 4)


def main(sizes=None, batch=64, prompt=1024, steps=32, vocab=32768, mixers=MIXERS, with_qwen=True):
    import nano_vllm_candle_amd as pkg

    for name in sizes or SIZES:
        z = SIZES[name]
        for kind in mixers:
            m = pkg.GopunexForCausalLM.from_random(gopunex_config(pkg, z, kind, vocab))
            r = measure(m, batch, prompt, steps, np.random.default_rng(0), vocab, CLASSES)
            r["weight_bytes"], r["kv_bytes_per_token"] = m.weight_bytes, m.kv_bytes_per_token
            if kind == "attention":
                rooflines(r, z["layers"], batch, prompt, 1 << 30, m.kv_bytes_per_token // z["layers"], z["heads"] * 2 * 256, prompt + steps + 10)
            elif kind != "mixed":
                recurrence_rooflines(r, z, kind, batch, prompt)
            m.close()
            print(json.dumps({"size": name, **z, "mixer": kind, "batch": batch, "prompt": prompt, "vocab": vocab, "gopunex": r}), flush=True)
        if with_qwen:
            m = pkg.Qwen3ForCausalLM.from_synthetic(pkg.Qwen3Config(vocab, z["width"], 128, z["layers"], z["heads"], z["kv"], z["ff"], 40960), seed=0)
            r = measure(m, batch, prompt, steps, np.random.default_rng(0), vocab, CLASSES)
            r["weight_bytes"], r["kv_bytes_per_token"] = m.weight_bytes, m.kv_bytes_per_token
            rooflines(r, z["layers"], batch, prompt, 1 << 30, m.kv_bytes_per_token // z["layers"], z["heads"] * 2 * 256, prompt + steps + 10)
            m.close()
            print(json.dumps({"size": name, **z, "batch": batch, "prompt": prompt, "vocab": vocab, "qwen3": r}), flush=True)
