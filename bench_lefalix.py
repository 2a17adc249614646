"""`bench.py --lefalix`: prefill and decode throughput of the Lefalix design at layer sizes of real models (random weights), beside the
framework's closest design at equal size (same width, depth, vocabulary, prompts and batch): Gopunex for attention and for the delta rule,
Tafopel for routed experts.  Prints one JSON line per size and kind of layer, with HIP-event times per kernel class and the fraction of
its roofline that the mixers' own kernels reach."""
import json

import numpy as np

from bench_berevik import measure, rooflines
from bench_gopunex import CLASSES, gopunex_config, recurrence_rooflines
from bench_tafopel import tafopel_config

# width, heads (all of 128, attention and delta rule alike), key/value heads of both, rotated dimensions, width of the Qwen3-like gated
# feed-forward of equal parameters (the two-matrix one is half as wide again), experts of which two are chosen, layers; the rest: Tafopel's
SIZES = {
    "1k": dict(width=1024, heads=16, kv=8, rot=64, ff=3072, experts=16, top=2, expert_ff=768, layers=10),
    "2k": dict(width=2048, heads=16, kv=8, rot=64, ff=6144, experts=16, top=2, expert_ff=1536, layers=5),
    "4k": dict(width=4096, heads=32, kv=8, rot=64, ff=12288, experts=8, top=2, expert_ff=3072, layers=3),
}
KINDS = ("parallel", "window", "channel_delta", "experts", "mixed")
WINDOW = 256  # of the kind `window`
LATENT = {"1k": dict(dim=64, vdim=128, rank=256, q_rank=512), "2k": dict(dim=128, vdim=128, rank=512, q_rank=1024), "4k": dict(dim=128, vdim=128, rank=512, q_rank=1536)}


def lefalix_config(pkg, z, kind, vocab):
    """parallel, window: two mixers (attention over everything, over WINDOW tokens) and a dense feed-forward; channel_delta: that mixer and a
    dense feed-forward; experts: two mixers and routed ones; mixed: all of them in turn, half of the layers run twice"""
    from nano_vllm_candle_amd.causal_lm import Yarn
    from nano_vllm_candle_amd.lefalix import DeltaConfig, DenseConfig, RoutedConfig, WindowAttentionConfig

    h, g = z["heads"], z["kv"]
    dense, moe = DenseConfig(z["ff"] * 3 // 2), RoutedConfig(z["experts"], z["top"], z["expert_ff"], 4, 2)

    def par(window):
        return WindowAttentionConfig(h, g, 128, 128, 128 ** -0.5, window, 4, z["rot"], 1e6, Yarn(8.0, 4096.0, 32.0, 1.0)), DeltaConfig(h, g, 128, 128, 4)

    rule = (DeltaConfig(h, h, 128, 128, 4, 128, 128),)
    n = z["layers"]
    if kind == "mixed":
        kinds = ((par(WINDOW), dense), (rule, moe), (par(WINDOW), moe), (rule, dense))
        layers = [kinds[i % 4] for i in range((n * 2 + 2) // 3)]
        return pkg.LefalixConfig(vocab, z["width"], layers, (0, n - len(layers), 2))
    mix = {"parallel": par(1 << 20), "window": par(WINDOW), "channel_delta": rule, "experts": par(1 << 20)}[kind]
    return pkg.LefalixConfig(vocab, z["width"], [(mix, moe if kind == "experts" else dense)] * n)


def main(sizes=None, batch=64, prompt=1024, steps=32, vocab=32768, kinds=KINDS, with_twins=True):
    import nano_vllm_candle_amd as pkg

    def run(name, z, label, m, extra):
        r = measure(m, batch, prompt, steps, np.random.default_rng(0), vocab, CLASSES)
        r["weight_bytes"], r["kv_bytes_per_token"] = m.weight_bytes, m.kv_bytes_per_token
        for e in extra:
            e(r)
        m.close()
        print(json.dumps({"size": name, **z, "model": label, "batch": batch, "prompt": prompt, "vocab": vocab, "result": r}), flush=True)

    for name in sizes or SIZES:
        z = SIZES[name]

        def attention(window):
            return lambda r: rooflines(r, z["layers"], batch, prompt, window, 2 * z["kv"] * 256, z["heads"] * 2 * 256, prompt + steps + 10)

        def rule(r):
            recurrence_rooflines(r, z, "channel_delta", batch, prompt)

        both = [attention(1 << 30), rule]
        extras = {"parallel": both, "window": [attention(WINDOW), rule], "channel_delta": [rule], "experts": both, "mixed": []}
        for kind in kinds:
            run(name, z, "lefalix " + kind, pkg.LefalixForCausalLM.from_random(lefalix_config(pkg, z, kind, vocab)), extras[kind])
        if with_twins:
            run(name, z, "gopunex attention", pkg.GopunexForCausalLM.from_random(gopunex_config(pkg, z, "attention", vocab)), [attention(1 << 30)])
            run(name, z, "gopunex channel_delta", pkg.GopunexForCausalLM.from_random(gopunex_config(pkg, z, "channel_delta", vocab)), [rule])
            run(name, z, "tafopel experts", pkg.TafopelForCausalLM.from_random(tafopel_config(pkg, {**z, **LATENT[name], "inner": 2 * z["width"], "state": 16, "dt_rank": z["width"] // 16}, "experts", vocab)), [])
