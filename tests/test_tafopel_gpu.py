"""Tafopel on the GPU against the plain CPU restatement (oracle/tafopel_oracle.py): layer by layer, every mechanism alone, prompts,
portions, decoding, batches, far keys and block borders, slot and block reuse, greedy generation through the engine -- in both
precisions."""
import functools
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import tafopel_oracle as T
from tests.berevik_util import row_err
from tests.tafopel_util import BEACON, CONFIGS, EVEN, MIXED, STATE, TOL, YARN, attn, beacon_weights, bf16, config, dense, mamba, moe, weights
from tests.util import write_checkpoint

pytestmark = pytest.mark.gpu
DTYPES = ("bfloat16", "float32")


def make(cfg, w, dtype, blocks=24, max_seqs=6, rows=512, ctx=None):
    import nano_vllm_candle_amd as pkg

    m = pkg.TafopelForCausalLM.from_state_dict(pkg.TafopelConfig.from_dict(cfg), w, ctx=ctx, dtype=dtype)
    m.kv_alloc(blocks, max_seqs, max_batched_tokens=rows)
    return m


def tokens(n, vocab, seed=0):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


@functools.lru_cache(maxsize=None)
def case(name, seed, n, token_seed):
    """(weights, tokens, reference logits, residual after every layer), shared by the precisions"""
    cfg = CONFIGS[name]
    w, toks = weights(cfg, seed), tokens(n, cfg["vocab"], token_seed)
    return (w, toks) + T.run(cfg, w, toks)


def decode(m, sid, toks, first):
    """logits of positions first.. of toks, one token a step"""
    return np.concatenate([m.step_score([sid], [toks[:i + 1]], False, [[i]]) for i in range(first, len(toks))])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_layer_outputs_and_logits(name, dtype):
    cfg = CONFIGS[name]
    w, toks, ref, taps = case(name, 0, 150, 0)
    m = make(cfg, w, dtype, max_seqs=256)
    m.enable_taps()
    got = m.step_score([0], [toks], True, [list(range(len(toks)))])
    for l, r in enumerate(taps):
        e = row_err(m.layer_tap(l, 1, len(toks)), r)
        assert e < TOL[dtype], (name, dtype, l, e)
    assert row_err(got, ref) < TOL[dtype]
    m.enable_taps(False)
    assert row_err(m.step_score([1], [toks], True, [list(range(len(toks)))]), ref) < TOL[dtype]


ALONE = {
    "attention": [attn()],
    "attention, plain rotation": [attn(yarn=None)],
    "attention, one shared cache": [attn(), attn(heads=2, dim=11, vdim=40, q_rank=7, src=0)],
    "scan": [mamba()],
    "scan, one tap, one state": [mamba(conv=1, state=1, rank=1)],
    "scan, sixteen taps": [mamba(conv=16, state=5)],
    "gated feed-forward": [mamba(mlp=dense(200))],
    "experts": [mamba(mlp=moe(7, 3, 20, 0))],
    "experts, one chosen": [mamba(mlp=moe(7, 1, 20, 31))],
    "experts, all chosen": [mamba(mlp=moe(3, 3, 20, 300))],
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("what", sorted(ALONE))
def test_one_mechanism(what, dtype):
    cfg = config(ALONE[what], vocab=100, eps=0.01)
    w = weights(cfg, 3)
    if cfg["layers"][0]["mlp"]:
        w["l0.mix.o"][:] = 0
    toks = tokens(70, 100, 1)
    ref, _ = T.run(cfg, w, toks)
    m = make(cfg, w, dtype, max_seqs=80)
    assert row_err(m.step_score([0], [toks], True, [list(range(70))]), ref) < TOL[dtype]
    m.step_score([1], [toks[:9]], True, [[]])
    assert row_err(decode(m, 1, toks, 9), ref[9:]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_router_without_help(dtype):
    # random scores, not the spread ones of the other tests: the seed leaves no close call
    cfg = config([mamba(mlp=moe(8, 3, 24, 16))], vocab=40)
    w = T.random_weights(cfg, 19)
    toks = tokens(40, 40, 2)
    ref, _ = T.run(cfg, w, toks)
    z = np.sort(T.layer_norm(w["embed"][toks], w["l0.norm1"], 1e-5) @ w["l0.mlp.router"].T, axis=1)
    assert (z[:, -3] - z[:, -4]).min() > 2e-3
    m = make(cfg, w, dtype, max_seqs=40)
    assert row_err(m.step_score([0], [toks], True, [list(range(40))]), ref) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "even", "wide", "one", "sizes", "state"])
def test_portions_and_decoding_equal_the_whole_prompt(name, dtype):
    cfg = CONFIGS[name]
    w, toks, ref, _ = case(name, 1, 330, 2)
    m = make(cfg, w, dtype)
    cuts = {"twos": [2] * 165, "odd": [11, 2, 37, 64, 3, 120, 1, 1, 91], "page": [255, 2, 73], "decode": [250] + [1] * 80, "short": [1, 1, 2, 1, 3, 1, 321]}
    for sid, (what, parts) in enumerate(cuts.items()):
        at, got = 0, []
        for n in parts:
            got.append(m.step_score([sid], [toks[:at + n]], False, [list(range(at, at + n))]))
            at += n
        assert at == len(toks)
        worst = np.abs(np.concatenate(got) - ref).max(1) / np.abs(ref).max()
        # latents of one element are normed to a sign: what rounding does to the smallest ones shows
        assert worst.max() < TOL[dtype] * (5 if name == "one" else 1), (name, dtype, what, int(worst.argmax()), worst.max())
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [16, 100])
def test_small_row_buffers_cut_prompts_inside(rows, dtype):
    w = weights(MIXED, 4)
    a, b = tokens(200, MIXED["vocab"], 5), tokens(31, MIXED["vocab"], 6)
    m = make(MIXED, w, dtype, max_seqs=3, rows=rows)
    want = [[0, 7, 57, 150, 199], [3, 30]]
    got = m.step_score([5, 9], [a, b], True, want)
    assert row_err(got, np.concatenate([T.run(MIXED, w, a)[0][want[0]], T.run(MIXED, w, b)[0][want[1]]])) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("form", ["absorbed", "expanded", "plain"])
def test_one_far_key_is_seen_from_everywhere(dtype, form):
    # one token outweighs every other: at the ends of 16-, 32- and 256-token tiles, right before the query and a thousand tokens back,
    # in prompts, in portions and decoded
    w = beacon_weights(BEACON, 63)
    m = make(BEACON, w, dtype, rows=1200)
    m.set_option("latent_plain" if form == "plain" else "latent_absorb", {"plain": 1, "absorbed": 1, "expanded": -1}[form])
    for sid, at in enumerate((0, 15, 16, 31, 47, 255, 256, 700)):
        n = 1100 if at in (0, 255, 700) else at + 90
        toks = tokens(n, 60, sid)
        toks[at] = 63
        ask = sorted({max(at - 1, 0), at, at + 1, at + 31, at + 64, n - 3, n - 2, n - 1})
        ref = T.run(BEACON, w, toks)[0][ask]
        assert row_err(m.step_score([sid], [toks], True, [ask]), ref) < TOL[dtype], ("prompt", at)
        cut = max(1, at - 1)
        got = [m.step_score([sid], [toks[:cut]], True, [[p for p in ask if p < cut]])]
        got.append(m.step_score([sid], [toks[:n - 3]], False, [[p for p in ask if cut <= p < n - 3]]))
        got.append(decode(m, sid, toks, n - 3))
        assert row_err(np.concatenate(got), ref) < TOL[dtype], ("portions", at)
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("form", ["absorbed", "expanded", "plain"])
@pytest.mark.parametrize("sinks", ["weak", "even", "strong", "extreme"])
def test_sinks(dtype, form, sinks):
    # the sink weighs most at the start; sinks far above and below every score, and one head's sink next to another's
    cfg = config([attn(heads=6, dim=32, rot=32, vdim=32, rank=64, q_rank=48)], vocab=60)
    w = weights(cfg, 2)
    w["l0.mix.sink"][:] = {"weak": [-6, -5, -4, -3, -2, -1], "even": [0, 1, 2, 3, 4, 5], "strong": [5, 6, 7, 8, 9, 10], "extreme": [-120, 120, -60, 60, 0, 30]}[sinks]
    toks = tokens(420, 60, 3)
    ref, _ = T.run(cfg, w, toks)
    m = make(cfg, w, dtype)
    m.set_option("latent_plain" if form == "plain" else "latent_absorb", {"plain": 1, "absorbed": 1, "expanded": -1}[form])
    assert row_err(m.step_score([0], [toks[:400]], True, [[0, 1, 2, 31, 397, 398]]), ref[[0, 1, 2, 31, 397, 398]]) < TOL[dtype]
    assert row_err(decode(m, 0, toks, 400), ref[400:]) < TOL[dtype]
    for r in (0, 1, 2, 5):
        assert row_err(m.step_score([1], [toks[:r + 1]], True, [[r]]), ref[[r]]) < TOL[dtype]
    assert row_err(np.concatenate([m.step_score([2], [toks[:1]], True, [[0]]), decode(m, 2, toks[:40], 1)]), ref[:40]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rot, base, yarn", [(8, 20.0, None), (64, 1e6, None), (40, 500.0, YARN), (64, 1e4, {"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 1.0}),
                                             (16, 1e5, {"factor": 1.0, "original": 64, "fast": 4.0, "slow": 0.5}), (2, 10.0, {"factor": 4.0, "original": 512, "fast": 2.0, "slow": 2.0})])
def test_rotation_up_to_far_positions(dtype, rot, base, yarn):
    # the rotated part alone decides the scores
    cfg = config([attn(heads=3, dim=8, rot=rot, base=base, yarn=yarn, scale=rot ** -0.5)], vocab=60)
    w = weights(cfg, 6, gain=3.0)
    w["l0.mix.uk"] *= 0.0
    toks = tokens(1100, 60, rot)
    ref, _ = T.run(cfg, w, toks)
    m = make(cfg, w, dtype, rows=1200)
    ask = [0, 1, 100, 600, 1090, 1094]
    assert row_err(m.step_score([0], [toks[:1095]], True, [ask]), ref[ask]) < TOL[dtype]
    assert row_err(decode(m, 0, toks, 1095), ref[1095:]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_state_carries_far(dtype):
    # decays so slow that the first tokens still count after a thousand
    cfg = config([mamba(inner=48, state=8, conv=4, rank=4)], vocab=40)
    w = weights(cfg, 9)
    w["l0.mix.A_log"][:] = -9.0
    w["l0.mix.conv.b"][:] = 0.0
    w["l0.mix.dt"][:] = 0.0
    w["l0.mix.dt.b"][:] = -3.0
    w["embed"][39] *= 4
    w = {k: bf16(v).astype(np.float64) for k, v in w.items()}
    toks = [39] * 30 + tokens(1030, 39, 1)
    ref = T.run(cfg, w, toks)[0][1030:]
    lost = T.run(cfg, w, toks[31:])[0][999:]
    assert row_err(lost, ref) > 10 * TOL["bfloat16"]
    m = make(cfg, w, dtype, rows=1200)
    at = 0
    for n in (3, 500, 2, 255, 270):
        at += n
        m.step_score([0], [toks[:at]], False, [[]])
    assert at == 1030
    assert row_err(decode(m, 0, toks, 1030), ref) < TOL[dtype]
    # in one chunk of several pieces
    assert row_err(m.step_score([1], [toks], True, [list(range(1030, 1036))]), ref[:6]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_decays_of_every_strength(dtype):
    # rates from exp(-12) to exp(6) and strongly varying step sizes: decays that underflow within a token beside some that never do
    cfg = config([mamba(inner=64, state=16, conv=2, rank=6)], vocab=60)
    w = weights(cfg, 5)
    w["l0.mix.A_log"][:] = np.linspace(-12, 6, 16)
    w["l0.mix.dt.b"][:] = np.random.default_rng(0).integers(-64, 49, 64) / 8
    w["l0.mix.dt"] *= 2
    w = {k: bf16(v).astype(np.float64) for k, v in w.items()}
    toks = tokens(400, 60, 2)
    ref, _ = T.run(cfg, w, toks)
    m = make(cfg, w, dtype, max_seqs=400)
    assert row_err(m.step_score([0], [toks], True, [list(range(400))]), ref) < TOL[dtype]
    m.step_score([1], [toks[:61]], True, [[]])
    assert row_err(decode(m, 1, toks[:90], 61), ref[61:90]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["even", "mixed", "state"])
def test_batches_equal_each_request_alone(name, dtype):
    cfg = CONFIGS[name]
    w = weights(cfg, 7)
    m = make(cfg, w, dtype, blocks=32, max_seqs=6)
    lens = [1, 5, 17, 64, 259, 130]
    reqs = [tokens(n + 6, cfg["vocab"], 20 + n) for n in lens]
    refs = [T.run(cfg, w, r)[0] for r in reqs]
    # prompts of all lengths, then portions and decoding rows side by side, then decoding alone
    got = m.step_score(range(6), [r[:n] for r, n in zip(reqs, lens)], True, [[n - 1] for n in lens])
    assert row_err(got, np.array([f[n - 1] for f, n in zip(refs, lens)])) < TOL[dtype]
    at = [n + s for n, s in zip(lens, [1, 3, 1, 2, 1, 3])]
    got = m.step_score(range(6), [r[:n] for r, n in zip(reqs, at)], False, [[n - 1] for n in at])
    assert row_err(got, np.array([f[n - 1] for f, n in zip(refs, at)])) < TOL[dtype]
    for order in ((5, 0, 3, 1, 4, 2), (0, 1, 2, 3, 4, 5), (2, 4)):
        at = [n + (i in order) for i, n in enumerate(at)]
        got = m.step_score(order, [reqs[i][:at[i]] for i in order], False, [[at[i] - 1] for i in order])
        assert row_err(got, np.array([refs[i][at[i] - 1] for i in order])) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_blocks_and_slots_are_reused(dtype):
    w = weights(MIXED, 8)
    m = make(MIXED, w, dtype, blocks=4, max_seqs=2)
    free = m.free_blocks()
    rng = np.random.default_rng(0)
    for i in range(6):
        a, b = tokens(int(rng.integers(260, 500)), MIXED["vocab"], 50 + i), tokens(int(rng.integers(1, 400)), MIXED["vocab"], 90 + i)
        m.step_score([2 * i, 2 * i + 1], [a[:-1], b[:max(1, len(b) - 2)]], False, [[], []])
        got = m.step_score([2 * i, 2 * i + 1], [a, b], False, [[len(a) - 1], [len(b) - 1]])
        assert row_err(got, np.stack([T.run(MIXED, w, a)[0][-1], T.run(MIXED, w, b)[0][-1]])) < TOL[dtype], i
        for s in ((2 * i, 2 * i + 1) if i % 2 else (2 * i + 1, 2 * i)):
            m.seq_free(s)
        assert m.free_blocks() == free


@pytest.mark.parametrize("dtype", DTYPES)
def test_stepping_back_starts_the_sequence_again(dtype):
    # carried state cannot be undone: the same length again, a shorter prefix, another prompt under the same id
    w = weights(STATE, 11)
    toks, other = tokens(90, STATE["vocab"], 1), tokens(50, STATE["vocab"], 2)
    ref, ref2 = T.run(STATE, w, toks)[0], T.run(STATE, w, other)[0]
    m = make(STATE, w, dtype, blocks=3, max_seqs=2)
    for n in (90, 90, 40, 41, 60, 1, 2):
        assert row_err(m.step_score([0], [toks[:n]], False, [[n - 1]]), ref[[n - 1]]) < TOL[dtype], n
    assert row_err(m.step_score([0], [other], True, [[49]]), ref2[[49]]) < TOL[dtype]


def test_long_decoding():
    cfg = config([mamba(), attn(mlp=moe()), mamba(state=16, mlp=dense()), attn(src=1)], vocab=96)
    w = weights(cfg, 9)
    toks = tokens(620, 96, 3)
    ref, _ = T.run(cfg, w, toks)
    for dtype in DTYPES:
        m = make(cfg, w, dtype)
        got = np.concatenate([m.step_score([0], [toks[:3]], True, [[2]]), decode(m, 0, toks, 3)])
        assert row_err(got, ref[2:]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_engine(dtype):
    from nano_vllm_candle_amd.engine import CausalLMRunner, LLMEngine, SamplingParams, Scheduler, SchedulerConfig

    w = weights(EVEN, 10)
    m = make(EVEN, w, dtype, max_seqs=5)  # the scheduler admits prompts while others decode: a slot for each
    prompts = [tokens(n, EVEN["vocab"], n) for n in (1, 33, 70, 300, 2)]
    eng = LLMEngine(Scheduler(SchedulerConfig(max_num_seqs=3, eos=None)), CausalLMRunner(m, greedy=True))
    outs = eng.generate(prompts, SamplingParams(max_tokens=6))
    assert len(outs) == 5 and m.free_blocks() == 24
    for p, (_, got) in zip(prompts, outs):
        want, rows = T.greedy(EVEN, w, p, 6)
        assert len(got) == 6
        for g, t, r in zip(got, want, rows):
            if g != t:  # only a near-tie may flip, and everything after it then differs
                assert (r.max() - r[g]) / np.abs(r).max() < 2 * TOL[dtype], (g, t)
                break


def test_decode_fast_path_and_sampling_follow_the_step_call():
    w = weights(EVEN, 11)
    m = make(EVEN, w, "bfloat16", max_seqs=4)
    prompts = [tokens(n, EVEN["vocab"], n) for n in (40, 3, 258)]
    ids = [0, 1, 2]
    seqs = [list(p) for p in prompts]
    nxt, lg = m.step(ids, seqs, True, want_logits=True)
    assert row_err(lg, np.array([T.run(EVEN, w, p)[0][-1] for p in prompts])) < TOL["bfloat16"]
    by_step = []
    for _ in range(5):
        for s, t in zip(seqs, nxt):
            s.append(int(t))
        nxt, _ = m.step(ids, seqs, False)
        by_step.append(nxt.tolist())
    m.step(ids, prompts, True)
    assert [m.decode_next()[:3].tolist() for _ in range(5)] == by_step
    m.step(ids, prompts, True)
    m.decode_enqueue()
    m.decode_enqueue()
    assert [m.decode_collect()[:3].tolist() for _ in range(2)] == by_step[:2]
    a, _ = m.step_sample(ids, prompts, True, [1.0] * 3, seed=5)
    b, _ = m.step_sample(ids, prompts, True, [1.0] * 3, seed=5)
    cold, _ = m.step_sample(ids, prompts, True, [1e-4] * 3, seed=5)
    assert a.tolist() == b.tolist()
    assert cold.tolist() == m.step(ids, prompts, True)[0].tolist()


@functools.lru_cache(maxsize=None)
def real_size():
    # wide enough for the register-direct, streaming, tile and grouped tile products
    cfg = config([mamba(inner=2048, state=16, conv=4, rank=64, mlp=dense(3072)), attn(heads=8, dim=128, rot=64, vdim=128, rank=512, q_rank=768, mlp=moe(8, 2, 768, 768)),
                  attn(heads=8, dim=128, rot=64, vdim=128, rank=512, q_rank=768, src=1, mlp=moe(4, 1, 512, 256))], width=1024, vocab=4096)
    return cfg, weights(cfg, 12, gain=1.5)


@pytest.mark.parametrize("rows", [1, 16, 64, 130, 700])
def test_layers_of_a_real_size_take_the_fused_products(rows):
    cfg, w = real_size()
    m = make(cfg, w, "bfloat16", blocks=160, max_seqs=64, rows=1024)
    m.set_option("tile_min_wgs", 1)  # the tile products whenever the shape fits
    f = {k: v.astype(np.float32) for k, v in w.items()}
    if rows in (16, 64):  # a decode batch of that many sequences, each a few tokens long
        reqs = [tokens(4, 4096, i) for i in range(rows)]
        m.step_score(range(rows), [r[:3] for r in reqs], True, [[]] * rows)
        got = m.step_score(range(rows), reqs, False, [[3]] * rows)
        ref = np.array([T.run(cfg, f, r)[0][3] for r in reqs])
    else:
        t = tokens(rows, 4096, 1)
        ask = sorted({0, rows // 2, rows - 1})
        got, ref = m.step_score([0], [t], True, [ask]), T.run(cfg, f, t)[0][ask]
    assert row_err(got, ref) < TOL["bfloat16"]
    if rows > 128:
        assert m.counter("tile_gemm_launches") > 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_two_ranks_match_one(dtype):
    import threading

    import nano_vllm_candle_amd as pkg

    cfg = config([mamba(inner=40, mlp=dense()), attn(heads=4, mlp=moe()), attn(heads=2, src=1), mamba(inner=70, state=9, rank=33, mlp=moe(5, 2, 18, 0))], vocab=128)
    w = weights(cfg, 13)
    toks = tokens(90, 128, 1)
    res, errs = [None, None], []

    def rank(r):
        try:
            m = make(cfg, w, dtype, 8, 2, 128, ctx=pkg.Context(0, r, 2, loopback_group=f"tafopel-{dtype}"))
            _, a = m.step([0], [toks[:80]], True, want_logits=True)
            nxt, b = m.step([0], [toks[:81]], False, want_logits=True)
            nxt, c = m.step([0], [toks], False, want_logits=True)
            res[r] = (np.concatenate([a, b, c]), int(nxt[0]))
        except Exception as e:  # noqa: BLE001
            errs.append(e)

    ts = [threading.Thread(target=rank, args=(r,)) for r in range(2)]
    [t.start() for t in ts]
    [t.join(100) for t in ts]
    assert not errs, errs
    ref = T.run(cfg, w, toks)[0][[79, 80, 89]]
    for lg, nxt in res:
        assert row_err(lg, ref) < TOL[dtype]
        assert nxt == int(ref[2].argmax())


@pytest.mark.parametrize("dtype", DTYPES)
def test_programs_on_a_checkpoint(tmp_path, dtype):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = MIXED
    w = weights(cfg, 14)
    write_checkpoint(tmp_path, cfg, w)
    a, b = tokens(30, cfg["vocab"], 1), tokens(12, cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:20], "want": [19, 4]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b, "want": []}, {"id": "x", "tokens": a[20:29], "want": [8]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": a[29:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "x", "tokens": b, "want": [11]}], "end": []}]
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "64"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.split() == "done 0 done 1 done 2 done 3".split()
    ra, rb = T.run(cfg, w, a)[0], T.run(cfg, w, b)[0]
    for step, ref in ((0, ra[[19, 4]]), (1, ra[[28]]), (2, ra[[29]]), (3, rb[[11]])):
        got = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert row_err(got, ref) < TOL[dtype], step
    if dtype == "bfloat16":
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), "--model", str(tmp_path), "--prompt", ",".join(map(str, a)), "--max-tokens", "3"],
                           capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        want, rows = T.greedy(cfg, w, a, 1)
        first = int(r.stdout.split(",")[0])
        assert first == want[0] or (rows[0].max() - rows[0][first]) / np.abs(rows[0]).max() < 2 * TOL[dtype]


def test_what_the_library_refuses():
    import nano_vllm_candle_amd as pkg

    good = config([attn(mlp=moe()), attn(src=0), mamba(mlp=dense())])
    w = weights(good, 1)
    for layers in ([attn(rot=7)], [mamba(conv=17)], [mamba(state=1025)], [mamba(mlp=moe(4, 5))], [mamba(mlp=moe(1025, 1))], [mamba(mlp=moe(100, 65))]):
        with pytest.raises(pkg._lib.NvllmError, match="layer"):
            pkg.TafopelForCausalLM(pkg.TafopelConfig.from_dict(config(layers)))
    c = pkg.TafopelConfig.from_dict(good)
    for missing in ("l0.mix.sink", "l0.mlp.e3.down", "l2.mix.A_log", "l1.mix.uq", "l0.mlp.shared.sg"):
        with pytest.raises(pkg._lib.NvllmError, match="missing tensor " + missing):
            pkg.TafopelForCausalLM.from_state_dict(c, {k: v for k, v in w.items() if k != missing})
    for short in ("l0.mix.dq", "l0.mlp.e0.up", "l2.mix.x", "l2.mix.conv", "l0.mlp.router"):
        with pytest.raises(pkg._lib.NvllmError, match="shape mismatch"):
            pkg.TafopelForCausalLM.from_state_dict(c, dict(w, **{short: w[short][:-1]}))
    for name in ("l0.mix.nope", "l1.mix.dkv", "l0.mlp.e6.up", "l0.norm2", "l2.mix.sink"):
        with pytest.raises(pkg._lib.NvllmError, match="unknown tensor"):
            pkg.TafopelForCausalLM.from_state_dict(c, dict(w, **{name: w["l0.norm1"]}))
