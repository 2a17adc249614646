"""`bench.py --tafopel`: prefill and decode throughput of the Tafopel design at layer sizes of real models (random weights), beside the
framework's closest designs at equal size (same width, depth, vocabulary, prompts and batch): Berevik for latent attention with a gated
feed-forward, Gopunex's delta rule for the scan.  Prints one JSON line per size and kind of layer, with HIP-event times per kernel class
and the fraction of its roofline that the mixer's own kernel reaches."""
import json

import numpy as np

from bench_berevik import HBM_GBS, berevik_config, measure, rooflines
from bench_gopunex import CLASSES, gopunex_config, recurrence_rooflines

# width, heads, unrotated / rotated / value size per head, latent sizes, channels / states / step rank of the scan, dense width, experts of
# one half or a quarter of it (two are chosen), layers; kv: key/value heads the twins' configurations want
SIZES = {
    "1k": dict(width=1024, heads=16, kv=8, dim=64, rot=64, vdim=128, rank=256, q_rank=512, inner=2048, state=16, dt_rank=64, ff=3072, experts=16, top=2, expert_ff=768, layers=10),
    "2k": dict(width=2048, heads=16, kv=8, dim=128, rot=64, vdim=128, rank=512, q_rank=1024, inner=4096, state=16, dt_rank=128, ff=6144, experts=16, top=2, expert_ff=1536, layers=5),
    "4k": dict(width=4096, heads=32, kv=8, dim=128, rot=64, vdim=128, rank=512, q_rank=1536, inner=8192, state=16, dt_rank=256, ff=12288, experts=8, top=2, expert_ff=3072, layers=3),
}
KINDS = ("attention", "scan", "experts", "mixed")


def tafopel_config(pkg, z, kind, vocab):
    """attention, scan: every layer that mixer with a gated feed-forward; experts: attention with routed ones, every other layer on the
    cache of the layer before; mixed: scans and attention in turn, mostly routed"""
    from nano_vllm_candle_amd.tafopel import ExpertsConfig, GeluMlpConfig, LatentMixerConfig, ScanMixerConfig, Yarn

    def attn(src=None):
        return LatentMixerConfig(z["heads"], z["dim"], z["rot"], z["vdim"], z["rank"], z["q_rank"], 1e6, (z["dim"] + z["rot"]) ** -0.5, Yarn(8.0, 4096.0, 32.0, 1.0), src)

    scan = ScanMixerConfig(z["inner"], z["state"], 4, z["dt_rank"])
    dense, moe = GeluMlpConfig(z["ff"]), ExpertsConfig(z["experts"], z["top"], z["expert_ff"], z["expert_ff"])
    layers = []
    for i in range(z["layers"]):
        if kind == "attention":
            layers.append((attn(), dense))
        elif kind == "scan":
            layers.append((scan, dense))
        elif kind == "experts":
            layers.append((attn(i - 1 if i % 2 else None), moe))
        else:
            layers.append([(scan, dense), (scan, moe), (attn(), moe), (attn(i - 1), moe), (scan, moe)][i % 5])
    return pkg.TafopelConfig(vocab, z["width"], layers, 1e-6)


def scan_rooflines(r, z, batch, prompt):
    """state read and written once (decode); input, gate and step sizes read, output planes written once (prefill)"""
    r["decode_recur_hbm_frac"] = round(z["layers"] * batch * z["inner"] * z["state"] * 8 / (r["decode_class_ms"]["recur"][0] * 1e-3) / 1e9 / HBM_GBS, 4)
    r["prefill_recur_hbm_frac"] = round(z["layers"] * batch * prompt * z["inner"] * 16 / (r["prefill_class_ms"]["recur"][0] * 1e-3) / 1e9 / HBM_GBS, 4)


def main(sizes=None, batch=64, prompt=1024, steps=32, vocab=32768, kinds=KINDS, with_twins=True):
    import nano_vllm_candle_amd as pkg

    def run(name, z, label, m, extra):
        r = measure(m, batch, prompt, steps, np.random.default_rng(0), vocab, CLASSES)
        r["weight_bytes"], r["kv_bytes_per_token"] = m.weight_bytes, m.kv_bytes_per_token
        extra(r)
        m.close()
        print(json.dumps({"size": name, **z, "model": label, "batch": batch, "prompt": prompt, "vocab": vocab, "result": r}), flush=True)

    for name in sizes or SIZES:
        z = SIZES[name]
        attention = lambda r: rooflines(r, z["layers"], batch, prompt, 1 << 30, 2 * (z["rank"] + z["rot"]), z["heads"] * 2 * (z["dim"] + z["rot"] + z["vdim"]), prompt + steps + 10)  # noqa: E731
        for kind in kinds:
            extra = {"attention": attention, "experts": attention, "scan": lambda r: scan_rooflines(r, z, batch, prompt)}.get(kind, lambda r: None)
            run(name, z, "tafopel " + kind, pkg.TafopelForCausalLM.from_random(tafopel_config(pkg, z, kind, vocab)), extra)
        if with_twins:
            run(name, z, "berevik", pkg.BerevikForCausalLM.from_random(berevik_config(pkg, z, vocab, 1 << 20)), attention)
            run(name, z, "gopunex channel_delta", pkg.GopunexForCausalLM.from_random(gopunex_config(pkg, z, "channel_delta", vocab)),
                lambda r: recurrence_rooflines(r, z, "channel_delta", batch, prompt))
