"""Small Lefalix configurations and weights for the tests."""
import numpy as np

from oracle import lefalix_oracle as L
from oracle.lefalix_oracle import bf16

TOL = {"bfloat16": 4e-3, "float32": 4e-5}
YARN = {"factor": 5.0, "original": 48, "fast": 6.0, "slow": 0.7}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, groups=(3, 2)):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": groups[0], "keep": groups[1]}}, "expert": {"ff": ff}}


def win(heads=6, kv=2, dim=20, vdim=18, conv=3, window=21, rot=12, scale=0.5, base=300.0, yarn=YARN):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv, "mask": {"size": window}, "scale": scale, "rot": {"base": base, "dims": rot}}
    if yarn:
        m["rot"]["scaling"] = dict(yarn)
    return m


def rule(heads=4, kv=2, dim=24, vdim=20, conv=4):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def par(left=None, right=None, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or win(), "right": right or rule()}, "mlp": mlp}


def delta(mlp=None, **sizes):
    return {"type": "channel_delta", "mixer": rule(**sizes), "mlp": mlp}


def config(layers, width=72, vocab=333, eps=1e-5, loop=None):
    return {"architecture": "Lefalix", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}, "loop": loop and dict(zip(("start", "stop", "times"), loop))}


# ragged sizes, every mixer beside every feed-forward and none, layers in the loop and around it
MIXED = config([delta(moe(), conv=2), par(mlp=dense()), par(win(heads=3, kv=3, dim=33, vdim=10, conv=1, window=7, rot=4, yarn=None), rule(heads=3, kv=3, dim=70, vdim=33, conv=2)),
                delta(dense(33), heads=5, kv=5, dim=17, vdim=9), par(win(heads=4, kv=1, dim=9, vdim=40, conv=5, window=130, rot=8, scale=1.1), rule(heads=2, kv=1, dim=5, vdim=7, conv=6), moe(9, 4, 17, (3, 3))),
                delta(moe(8, 3, 40, (2, 1)))], loop=(1, 4, 3))
# sizes on the tile boundaries, one key / value head for many queries; the first layers run twice
EVEN = config([par(win(heads=32, kv=1, dim=64, vdim=32, window=300, rot=64), rule(heads=8, kv=4, dim=64, vdim=64), dense(256)), delta(moe(8, 4, 128, (4, 2)), heads=8, kv=8, dim=64, vdim=32),
               par(win(heads=4, kv=4, dim=32, vdim=64, window=64, rot=32, base=5000.0), rule(heads=2, kv=2, dim=128, vdim=128), moe(16, 2, 64, (2, 1)))], width=256, vocab=512, loop=(0, 2, 2))
# the smallest sizes; windows of one and two tokens; the loop covers everything
ONE = config([par(win(heads=1, kv=1, dim=2, vdim=1, conv=1, window=1, rot=2, yarn=None), rule(heads=1, kv=1, dim=2, vdim=2, conv=1), moe(1, 1, 1, (1, 1))),
              delta(dense(1), heads=2, kv=1, dim=3, vdim=2, conv=7), par(win(heads=2, kv=1, dim=3, vdim=2, conv=2, window=2, rot=2), rule(heads=2, kv=2, dim=4, vdim=3, conv=2))],
             width=16, vocab=16, loop=(0, 3, 2))
# heads beyond the matrix-core attention and the piecewise recurrence; more than 64 experts, in groups of one too
WIDE = config([par(win(heads=2, kv=1, dim=300, vdim=40, window=50, rot=200, scale=0.1), rule(heads=2, kv=1, dim=190, vdim=130), moe(70, 5, 16, (70, 9))),
               par(win(heads=2, kv=2, dim=40, vdim=280, window=33, rot=40), rule(heads=1, kv=1, dim=400, vdim=50, conv=3), moe(130, 3, 8, (2, 1)))], width=100)
# every instance size of the matrix-core attention kernels, key sizes of every padding
SIZES = config([par(win(heads=4, kv=2, dim=d, vdim=v, window=40 + 13 * i, rot=d // 4 * 2, scale=1.5 * d ** -0.5), rule(heads=2, kv=1, dim=20 + 12 * i, vdim=16 + 5 * i, conv=1 + i % 5))
                for i, (d, v) in enumerate(((8, 30), (32, 64), (50, 100), (64, 200), (96, 32), (90, 60), (128, 128), (120, 250), (256, 20), (200, 64)))], width=64, vocab=200)
# no attention: nothing is cached
STATE = config([delta(dense()), delta(heads=2, kv=2, conv=3)], loop=(0, 1, 2))
CONFIGS = {"mixed": MIXED, "even": EVEN, "one": ONE, "wide": WIDE, "sizes": SIZES, "state": STATE}


def clear_choices(cfg, w, seed=0):
    """router scores far apart for every token: the residual's first channels hold a spaced permutation that no sublayer changes and that
    the routers read"""
    routed = [l["mlp"]["router"]["experts"] for l in cfg["layers"] if l.get("mlp") and l["mlp"]["kind"] == "moe"]
    n = min(max(routed, default=0), cfg["width"] // 2)
    if n < 2:
        return w
    rng = np.random.default_rng(seed + 77)
    w["embed"][:, :n] = np.stack([rng.permutation(n) for _ in range(cfg["vocab"])]) * (3.0 / n) - 1.5
    for i, l in enumerate(cfg["layers"]):
        w[f"l{i}.norm1b"][:n] = 0.0
        if not l.get("mlp"):
            continue
        w[f"l{i}.norm2"][:n], w[f"l{i}.norm2b"][:n] = 1.0, 0.0
        if l["mlp"]["kind"] == "moe":
            e = l["mlp"]["router"]["experts"]
            w[f"l{i}.mlp.router"][:] = 0.0
            # expert j reads channel pi(j) (more experts than channels: the others far below); every layer another choice
            for j in range(e):
                w[f"l{i}.mlp.router"][j, j % n] = 2.0 if j < n else -0.01
            w[f"l{i}.mlp.router"][:] = w[f"l{i}.mlp.router"][rng.permutation(e)]
    return w


def weights(cfg, seed=0):
    """random weights with clear choices of experts"""
    return {k: bf16(v).astype(np.float64) for k, v in clear_choices(cfg, L.random_weights(cfg, seed), seed).items()}


def beacon_config(window, heads=4, kv=2, dim=32, vdim=24, conv=3):
    return config([par(win(heads=heads, kv=kv, dim=dim, vdim=vdim, conv=conv, window=window, rot=16, scale=0.45), rule(heads=1, kv=1, dim=8, vdim=8, conv=1))], vocab=64)


def beacon_weights(cfg, token, seed=0):
    """`token` is a key that every head of attention layer 0 rests on wherever it is seen: residual channel 0 marks it, the last key dimension
    (not rotated) of every group reads the mark, the last query dimension is large for every token (a bias)"""
    w = L.random_weights(cfg, seed)
    m, p = cfg["layers"][0]["mixer"]["left"], "l0.mix.left."
    D = m["dim"]
    w["embed"][:, 0], w["embed"][token, 0] = 0.0, 6.0
    w["l0.norm1"][0] = 1.0
    for g in range(m["kv_heads"]):
        r = g * D + D - 1
        w[p + "k"][r], w[p + "k"][r, 0], w[p + "k.b"][r] = 0.0, 16.0, 0.0
    for h in range(m["heads"]):
        r = h * D + D - 1
        w[p + "q"][r], w[p + "q.b"][r] = 0.0, 24.0
    for n in "qk":
        w[p + n + ".conv"][:, :-1] *= 0.1
        w[p + n + ".conv"][:, -1] = 1.0
        w[p + n + ".conv"][D - 1::D, :-1] = 0.0
    w["l0.mix.right.out"][:] *= 0.2
    return {k: bf16(v).astype(np.float64) for k, v in w.items()}
