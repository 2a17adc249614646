"""Small Gopunex configurations and weights for the tests."""
import numpy as np

from oracle import gopunex_oracle as G


def attn(heads=6, kv=2, dim=40, vdim=24, scale=None, far=100, v_mix=True, ff=88):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "bias_max": far, "v_mix": v_mix,
                                           "scale": dim ** -0.5 if scale is None else scale},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def light(heads=3, dim=20, vdim=28, decay=None, ff=72):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay or [0.5 ** (2.0 ** -i / 2) for i in range(heads)]},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads=4, kv=2, dim=24, vdim=20, conv=4, ff=96):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, width=72, vocab=333, eps=1e-5, embed=2.0, mult=0.4):
    return {"architecture": "Gopunex", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": embed},
            "residual_mult": mult}


# every mixer with ragged sizes, layers without feed-forward (the last one too), values mixed across other layers, a layer that does not mix
MIXED = config([light(), attn(), delta(), attn(heads=3, kv=3, dim=17, vdim=16, far=30, v_mix=False, ff=0), delta(heads=3, kv=3, dim=70, vdim=33, conv=2, ff=0),
                attn(heads=4, kv=2, dim=33, vdim=24, far=500), light(heads=2, dim=65, vdim=40, decay=[1.0, 0.97], ff=0)])
# sizes on the tile boundaries, one key / value head for many queries
EVEN = config([delta(heads=8, kv=4, dim=64, vdim=64, ff=256), attn(heads=32, kv=1, dim=64, vdim=32, ff=128), light(heads=4, dim=64, vdim=32, ff=128),
               attn(heads=4, kv=1, dim=128, vdim=32, ff=128)], width=256, vocab=512)
# the smallest sizes; a convolution of one tap; feed-forward nowhere
ONE = config([delta(heads=1, kv=1, dim=1, vdim=1, conv=1, ff=0), attn(heads=1, kv=1, dim=1, vdim=1, ff=0), light(heads=1, dim=1, vdim=1, decay=[0.9], ff=0),
              delta(heads=2, kv=1, dim=3, vdim=2, conv=7, ff=0)], width=16, vocab=16)
# sizes beyond the matrix-core instances of the attention kernels; keys of the recurrences above 128
WIDE = config([attn(heads=2, kv=1, dim=300, vdim=40, ff=0), attn(heads=2, kv=2, dim=40, vdim=280, ff=0, v_mix=False), delta(heads=2, kv=1, dim=200, vdim=130),
               light(heads=1, dim=330, vdim=70, decay=[0.8])], width=100)
# every instance size of the matrix-core attention kernels
SIZES = config([attn(heads=4, kv=2, dim=d, vdim=v, ff=0, v_mix=False) for d, v in
                ((8, 30), (32, 64), (50, 100), (64, 200), (96, 32), (90, 60), (128, 128), (120, 256), (256, 20), (200, 64), (130, 128), (250, 250),
                 (20, 128), (30, 256), (60, 20), (64, 128), (80, 128), (96, 256), (110, 32), (128, 50))], width=64, vocab=200)
# no attention at all
STATE = config([delta(), light(ff=0), delta(heads=2, kv=2, conv=3)])

# key sizes whose padding is no power of two, and above what runs in pieces
KEYS = config([delta(heads=2, kv=2, dim=190, vdim=40, conv=3, ff=0), light(heads=2, dim=140, vdim=96, ff=0), delta(heads=1, kv=1, dim=400, vdim=50),
               light(heads=1, dim=512, vdim=17, decay=[0.95])], width=100, vocab=64)

CONFIGS = {"mixed": MIXED, "even": EVEN, "one": ONE, "wide": WIDE, "sizes": SIZES, "state": STATE, "keys": KEYS}
TOL = {"bfloat16": 4e-3, "float32": 3e-5}


def bf16(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32).reshape(np.shape(a))


def sharp_weights(cfg, seed=0, gain=2.0, bias=2.0):
    """random weights with wide spreads: peaked attention, distance biases that differ much from row to row, decays from almost one to
    almost nothing"""
    w = {k: v.copy() for k, v in G.random_weights(cfg, seed).items()}
    rng = np.random.default_rng(seed + 1000)
    for k in w:
        if k.endswith("q.norm"):
            w[k] = bf16(w[k] * gain)
        if k.endswith(".rel"):
            w[k] = bf16(w[k] * bias)
        if k.endswith("A_log"):
            w[k] = bf16(rng.uniform(-6.0, 3.0, w[k].shape))
    return w


def beacon_weights(cfg, token, seed=0):
    """`token` is a key that every head of attention layer 0 rests on wherever it is: residual channel 0 marks it, key dimension 0 of every
    group reads the mark, query dimension 0 is large for every token (a bias), and the score scale does the rest"""
    w = {k: v.copy() for k, v in G.random_weights(cfg, seed).items()}
    m, p = cfg["layers"][0]["mixer"], "l0.mix."
    w["embed"][:, 0] = 0.0
    w["embed"][token, 0] = 4.0
    for g in range(m["kv_heads"]):
        w[p + "k"][g * m["dim"], :] = 0.0
        w[p + "k"][g * m["dim"], 0] = 8.0
        w[p + "k.b"][g * m["dim"]] = 0.0
    for h in range(m["heads"]):
        w[p + "q"][h * m["dim"], :] = 0.0
        w[p + "q.b"][h * m["dim"]] = 12.0
    w[p + "q.norm"][:] = 1.0
    w[p + "k.norm"][:] = 1.0
    return {k: bf16(v) for k, v in w.items()}


BEACON = config([attn(heads=4, kv=2, dim=32, vdim=24, scale=0.6, far=60, v_mix=False, ff=0)], vocab=64)
