"""Small Tafopel configurations and weights for the tests."""
import numpy as np

from oracle import tafopel_oracle as T
from oracle.tafopel_oracle import bf16

TOL = {"bfloat16": 4e-3, "float32": 4e-5}
YARN = {"factor": 5.0, "original": 48, "fast": 6.0, "slow": 0.7}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, shared=40):
    m = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def attn(heads=3, dim=20, rot=12, vdim=18, rank=40, q_rank=36, scale=None, base=300.0, yarn=YARN, src=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": scale or (dim + rot) ** -0.5,
         "rot": {"base": base, "dims": rot}}
    if yarn:
        m["rot"]["scaling"] = dict(yarn)
    if src is not None:
        m["kv_from"] = src
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def mamba(inner=40, state=6, conv=3, rank=5, mlp=None):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "conv": conv, "dt_rank": rank}, "mlp": mlp}


def config(layers, width=72, vocab=333, eps=1e-5):
    return {"architecture": "Tafopel", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}}


# ragged sizes; every mixer beside every feed-forward and none; caches shared with other head counts and over other layers
MIXED = config([mamba(mlp=dense()), attn(mlp=moe()), attn(heads=5, dim=33, vdim=10, q_rank=50, src=1, scale=0.3), mamba(inner=27, conv=1, state=1, rank=1, mlp=moe(3, 1, 17, 0)),
                attn(heads=2, dim=7, rot=40, vdim=70, rank=33, q_rank=9, yarn=None, mlp=dense(33)), attn(heads=1, src=1, mlp=moe(9, 4, 8, 12)),
                attn(heads=3, dim=9, rot=40, vdim=20, rank=33, q_rank=20, yarn=None, src=4), mamba(inner=70, conv=6, state=19, rank=40, mlp=moe(4, 4, 30, 30))])
# sizes on the tile boundaries
EVEN = config([attn(heads=4, dim=64, rot=32, vdim=64, rank=128, q_rank=128, base=5000.0, mlp=moe(8, 2, 128, 128)), mamba(inner=256, state=16, conv=4, rank=32, mlp=dense(256)),
               attn(heads=8, dim=32, rot=32, vdim=32, rank=128, q_rank=128, base=5000.0, src=0, mlp=dense(128)), mamba(inner=128, state=64, conv=2, rank=16)], width=256, vocab=512)
# the smallest sizes
ONE = config([attn(heads=1, dim=1, rot=2, vdim=1, rank=1, q_rank=1, mlp=moe(1, 1, 1, 1)), mamba(inner=1, state=1, conv=1, rank=1, mlp=dense(1)), attn(heads=2, dim=1, rot=2, vdim=1, rank=1, q_rank=2, src=0),
              mamba(inner=3, state=2, conv=2, rank=2, mlp=moe(2, 1, 1, 0))], width=16, vocab=16)
# no attention, every group of lanes the scan has, beyond one wave too; no latent, no expert
STATE = config([mamba(inner=20, state=s, conv=1 + i % 5, rank=3 + 20 * i) for i, s in enumerate((3, 4, 8, 11, 32, 60, 128, 200, 300, 600))], width=64, vocab=200)
# latents, heads and rotated parts beyond the matrix-core forms; more than 64 experts
WIDE = config([attn(heads=2, dim=150, rot=96, vdim=140, rank=520, q_rank=200, mlp=moe(70, 5, 16, 24)), attn(heads=2, dim=40, rot=96, vdim=30, rank=520, q_rank=40, src=0)], width=100)
# every latent size of the matrix-core forms
SIZES = config([attn(heads=h, dim=d, rot=r, vdim=v, rank=k, q_rank=q) for h, d, r, v, k, q in
                ((2, 16, 16, 20, 32, 30), (3, 32, 32, 32, 64, 64), (17, 50, 24, 50, 90, 33), (2, 128, 64, 128, 128, 100), (2, 64, 48, 100, 190, 64), (4, 128, 64, 32, 256, 128),
                 (2, 30, 64, 64, 300, 50), (2, 100, 20, 120, 512, 70))], width=64, vocab=200)
CONFIGS = {"mixed": MIXED, "even": EVEN, "one": ONE, "state": STATE, "wide": WIDE, "sizes": SIZES}


def clear_choices(cfg, w, seed=0):
    """router scores far apart for every token: the residual's first channels hold a spaced permutation that no layer changes and that
    the routers read"""
    n = max([l["mlp"]["router"]["experts"] for l in cfg["layers"] if l.get("mlp") and l["mlp"]["kind"] == "moe"], default=0)
    if n < 2:
        return w
    rng = np.random.default_rng(seed + 77)
    w["embed"][:, :n] = np.stack([rng.permutation(n) for _ in range(cfg["vocab"])]) * (3.0 / n) - 1.5
    for i, l in enumerate(cfg["layers"]):
        w[f"l{i}.norm1"][:n] = 1.0
        w[f"l{i}.mix.o"][:n] = 0.0
        for k in w:
            if k.startswith(f"l{i}.mlp.") and k.endswith("down"):
                w[k][:n] = 0.0
        if l.get("mlp") and l["mlp"]["kind"] == "moe":
            e = l["mlp"]["router"]["experts"]
            w[f"l{i}.mlp.router"][:] = 0.0
            # expert j reads channel pi(j): every layer another choice; half of the scores on either side of one half
            for j, c in enumerate(rng.permutation(n)[:e]):
                w[f"l{i}.mlp.router"][j, c] = 1.5
    return w


def weights(cfg, seed=0, gain=2.0):
    """random weights with peaked attention and clear choices of experts"""
    w = T.random_weights(cfg, seed)
    for k in w:
        if k.endswith("dq.norm"):
            w[k] *= gain
    w = clear_choices(cfg, w, seed)
    return {k: bf16(v).astype(np.float64) for k, v in w.items()}


BEACON = config([attn(heads=4, dim=32, rot=16, vdim=24, rank=48, q_rank=24, scale=0.5)], vocab=64)


def beacon_weights(cfg, token, seed=0):
    """`token` is a key that every head of attention layer 0 rests on wherever it is: residual channel 0 marks it, latent 0 and key
    dimension 0 carry the mark, channel 1 (the same for every token) makes query dimension 0 large"""
    w = T.random_weights(cfg, seed)
    m, p = cfg["layers"][0]["mixer"], "l0.mix."
    w["embed"][:, 0], w["embed"][token, 0], w["embed"][:, 1] = 0.0, 6.0, 5.0
    w[p + "dkv"][0, :], w[p + "dkv"][0, 0] = 0.0, 4.0
    w[p + "dq"][0, :], w[p + "dq"][0, 1] = 0.0, 6.0
    w[p + "dkv.norm"][0] = w[p + "dq.norm"][0] = 1.0
    for h in range(m["heads"]):
        k, q = h * m["dim"], h * (m["dim"] + m["rot_dim"])
        w[p + "uk"][k, :], w[p + "uk"][k, 0] = 0.0, 4.0
        w[p + "uq"][q, :], w[p + "uq"][q, 0] = 0.0, 4.0
    return {k: bf16(v).astype(np.float64) for k, v in w.items()}
