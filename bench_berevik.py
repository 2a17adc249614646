"""`bench.py --berevik`: prefill and decode throughput of the Berevik design at layer sizes of real models (random weights), beside
Qwen3 layers of equal size (same width, heads, feed-forward width, depth, vocabulary, prompts and batch).  Prints one JSON line per
size, with HIP-event times per kernel class and, for the attention kernels, the fraction of their roofline."""
import json
import time

import numpy as np

HBM_GBS, MFMA_TFLOPS = 8000.0, 2500.0

# width, heads, kv heads of the Qwen3 twin, unrotated / rotated / value size per head, latent size, feed-forward width, layers
SIZES = {
    "1k": dict(width=1024, heads=16, kv=8, dim=64, rot=64, vdim=128, rank=256, ff=3072, layers=14),
    "2k": dict(width=2048, heads=16, kv=8, dim=128, rot=64, vdim=128, rank=512, ff=6144, layers=8),
    "4k": dict(width=4096, heads=32, kv=8, dim=128, rot=64, vdim=128, rank=512, ff=12288, layers=4),
}
CLASSES = ("attn", "gemm", "norm", "qk", "silu", "lm_head")


def berevik_config(pkg, z, vocab, window):
    from nano_vllm_candle_amd.berevik import GatedMlpConfig, LatentAttentionConfig

    mix = LatentAttentionConfig(z["heads"], z["dim"], z["rot"], z["vdim"], z["rank"], window, 1e4, (z["dim"] + z["rot"]) ** -0.5)
    return pkg.BerevikConfig(vocab, z["width"], [(mix, GatedMlpConfig(z["ff"], 7.0))] * z["layers"], 1e-6, 1.0, 30.0)


def measure(model, batch, prompt, steps, rng, vocab, classes=CLASSES):
    model.kv_alloc(batch * -(-(prompt + 4 * steps + 64) // 256), batch, max_batched_tokens=8192)
    toks = [rng.integers(0, vocab, prompt, dtype=np.uint32) for _ in range(batch)]
    ids = list(range(batch))
    model.step(ids, toks, True)  # warm-up
    out = {}
    best = float("inf")
    for _ in range(3):
        t0 = time.perf_counter()
        model.step(ids, toks, True)
        model.ctx.synchronize()
        best = min(best, time.perf_counter() - t0)
    out["prefill_ms"], out["prefill_tokens_per_s"] = best * 1e3, batch * prompt / best
    out["prefill_class_ms"] = {}
    for c in classes:
        model.profile_kernel(c)
        model.step(ids, toks, True)
        ms, n = model.profile_read()
        if n:
            out["prefill_class_ms"][c] = [round(ms, 3), int(n)]
    model.profile_kernel(None)
    for _ in range(8):
        model.decode_next(False)
    model.ctx.synchronize()
    t0 = time.perf_counter()
    model.decode_enqueue()
    for _ in range(steps - 1):
        model.decode_enqueue()
        model.decode_collect()
    model.decode_collect()
    dt = (time.perf_counter() - t0) / steps
    out["decode_ms_per_step"], out["decode_tokens_per_s"] = dt * 1e3, batch / dt
    out["decode_class_ms"] = {}
    for c in classes:
        model.profile_kernel(c)
        for _ in range(4):
            model.decode_next(False)
        ms, n = model.profile_read()
        if n:
            out["decode_class_ms"][c] = [round(ms / 4, 4), int(n // 4)]
    model.profile_kernel(None)
    return out


def rooflines(r, layers, batch, prompt, window, token_bytes, qk_plus_v_flops, ctx):
    """attention class against its bound: decode = cache bytes over HBM, prefill = visible pairs over the dense f16 peak"""
    seen = min(ctx, window)
    dec = r["decode_class_ms"]["attn"][0] * 1e-3
    r["decode_attn_hbm_frac"] = round(layers * batch * seen * token_bytes / dec / 1e9 / HBM_GBS, 4)
    pairs = sum(min(i + 1, window) for i in range(prompt)) * batch
    pre = r["prefill_class_ms"]["attn"][0] * 1e-3
    r["prefill_attn_mfma_frac"] = round(layers * pairs * qk_plus_v_flops / pre / 1e12 / MFMA_TFLOPS, 4)


def main(sizes=None, batch=64, prompt=1024, steps=32, vocab=32768, window=1 << 20, with_qwen=True):
    import nano_vllm_candle_amd as pkg

    for name in sizes or SIZES:
        z = SIZES[name]
        out = {"size": name, **z, "batch": batch, "prompt": prompt, "vocab": vocab, "window": window}
        m = pkg.BerevikForCausalLM.from_random(berevik_config(pkg, z, vocab, window))
        out["berevik"] = r = measure(m, batch, prompt, steps, np.random.default_rng(0), vocab)
        out["berevik"]["weight_bytes"], out["berevik"]["kv_bytes_per_token"] = m.weight_bytes, m.kv_bytes_per_token
        rooflines(r, z["layers"], batch, prompt, window, m.kv_bytes_per_token // z["layers"],
                  z["heads"] * 2 * (z["dim"] + z["rot"] + z["vdim"]), prompt + steps + 10)
        m.close()
        print("size", name, "berevik done", flush=True)
        if with_qwen:
            cfg = pkg.Qwen3Config(vocab, z["width"], 128, z["layers"], z["heads"], z["kv"], z["ff"], 40960)
            m = pkg.Qwen3ForCausalLM.from_synthetic(cfg, seed=0)
            out["qwen3"] = r = measure(m, batch, prompt, steps, np.random.default_rng(0), vocab)
            out["qwen3"]["weight_bytes"], out["qwen3"]["kv_bytes_per_token"] = m.weight_bytes, m.kv_bytes_per_token
            rooflines(r, z["layers"], batch, prompt, 1 << 30, m.kv_bytes_per_token // z["layers"], z["heads"] * 2 * 256, prompt + steps + 10)
            m.close()
        print(json.dumps(out), flush=True)
