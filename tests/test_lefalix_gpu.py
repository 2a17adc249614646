"""Lefalix on the GPU against the plain CPU restatement (oracle/lefalix_oracle.py): layer by layer, every mechanism alone, prompts,
portions, decoding, batches, far keys, block borders and window edges, slot and block reuse, greedy generation through the engine -- in both
precisions."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import lefalix_oracle as L
from tests.berevik_util import row_err
from tests.lefalix_util import CONFIGS, EVEN, MIXED, STATE, TOL, beacon_config, beacon_weights, config, delta, dense, moe, par, rule, weights, win
from tests.util import write_checkpoint

pytestmark = pytest.mark.gpu
DTYPES = ("bfloat16", "float32")


def f32(w):
    return {k: np.asarray(v, np.float32) for k, v in w.items()}


def make(cfg, w, dtype, blocks=24, max_seqs=6, rows=512, ctx=None):
    import nano_vllm_candle_amd as pkg

    c = pkg.LefalixConfig.from_dict(cfg, {k: np.shape(v) for k, v in w.items()})
    m = pkg.LefalixForCausalLM.from_state_dict(c, f32(w), ctx=ctx, dtype=dtype)
    m.kv_alloc(blocks, max_seqs, max_batched_tokens=rows)
    return m


def tokens(n, vocab, seed=0):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


def logits(cfg, w, toks, want=None):
    r = L.run(cfg, w, toks)[0]
    return r if want is None else r[want]


def decode(m, sid, toks, first):
    """logits of positions first.. of toks, one token a step"""
    return np.concatenate([m.step_score([sid], [toks[:i + 1]], False, [[i]]) for i in range(first, len(toks))])


def portions(m, sid, toks, parts):
    at, got = 0, []
    for n in parts:
        got.append(m.step_score([sid], [toks[:at + n]], False, [list(range(at, at + n))]))
        at += n
    assert at == len(toks)
    return np.concatenate(got)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_layer_outputs_and_logits(name, dtype):
    cfg = CONFIGS[name]
    w = weights(cfg)
    toks = tokens(150, cfg["vocab"])
    ref, taps = L.run(cfg, w, toks)
    m = make(cfg, w, dtype, max_seqs=256)
    m.enable_taps()
    got = m.step_score([0], [toks], True, [list(range(len(toks)))])
    # heads of one to three elements are normed to a direction: what rounding does to the smallest ones shows; ten layers in a row
    tol = TOL[dtype] * {"one": 10 if dtype == "bfloat16" else 4, "sizes": 4}.get(name, 1)
    for l, r in enumerate(taps):
        e = row_err(m.layer_tap(l, 1, len(toks)), r)
        assert e < tol, (name, dtype, l, e)
    assert row_err(got, ref) < tol
    m.enable_taps(False)
    assert row_err(m.step_score([1], [toks], True, [list(range(len(toks)))]), ref) < tol


ALONE = {
    "two mixers": [par()],
    "one tap": [par(win(conv=1), rule(conv=1))],
    "many taps": [par(win(conv=7), rule(conv=9))],
    "partial rotation": [par(win(dim=40, rot=6))],
    "whole rotation": [par(win(dim=16, rot=16, yarn=None))],
    "one key head": [par(win(heads=5, kv=1), rule(heads=6, kv=1))],
    "window of one": [par(win(window=1))],
    "window beyond the prompt": [par(win(window=5000))],
    "decay per channel": [delta()],
    "gelu": [delta(dense(200))],
    "experts": [delta(moe(8, 3, 40, (4, 2)))],
    "all experts": [delta(moe(5, 5, 16, (5, 5)))],
    "many experts": [delta(moe(96, 7, 8, (24, 11)), heads=1, kv=1)],
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("what", sorted(ALONE))
def test_one_mechanism(what, dtype):
    cfg = config(ALONE[what], vocab=100, eps=0.01, width=200 if what == "many experts" else 72)
    w = weights(cfg, 3)
    if cfg["layers"][0]["mlp"]:
        w["l0.mix.o"][:] = 0
    toks = tokens(90, 100, 1)
    ref = logits(cfg, w, toks)
    m = make(cfg, w, dtype, max_seqs=100)
    assert row_err(m.step_score([0], [toks], True, [list(range(90))]), ref) < TOL[dtype]
    m.step_score([1], [toks[:9]], True, [[]])
    assert row_err(decode(m, 1, toks, 9), ref[9:]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("side", ["left", "right"])
def test_one_side_alone(side, dtype):
    # the other side's output norm is zero, so this one is half of the sum
    cfg = config([par(win(window=33))], vocab=100)
    w = weights(cfg, 4)
    w[f"l0.mix.{'left' if side == 'right' else 'right'}.out"][:] = 0
    toks = tokens(80, 100, 2)
    ref = logits(cfg, w, toks)
    m = make(cfg, w, dtype, max_seqs=80)
    assert row_err(m.step_score([0], [toks], True, [list(range(80))]), ref) < TOL[dtype]
    assert row_err(portions(m, 1, toks, [30] + [2, 1] * 10 + [20]), ref) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "even", "wide", "one", "sizes", "state"])
def test_portions_and_decoding_equal_the_whole_prompt(name, dtype):
    cfg = CONFIGS[name]
    w = weights(cfg, 1)
    toks = tokens(330, cfg["vocab"], 2)
    ref = logits(cfg, w, toks)
    m = make(cfg, w, dtype)
    cuts = {"twos": [2] * 165, "odd": [11, 2, 37, 64, 3, 120, 1, 1, 91], "page": [255, 2, 73], "decode": [250] + [1] * 80, "short": [1, 1, 2, 1, 3, 1, 321]}
    for sid, (what, parts) in enumerate(cuts.items()):
        worst = np.abs(portions(m, sid, toks, parts) - ref).max(1) / np.abs(ref).max()
        assert worst.max() < TOL[dtype] * (5 if name in ("one", "sizes") else 1), (name, dtype, what, int(worst.argmax()), worst.max())
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [16, 100])
def test_small_row_buffers_cut_prompts_inside(rows, dtype):
    w = weights(MIXED, 4)
    a, b = tokens(200, MIXED["vocab"], 5), tokens(31, MIXED["vocab"], 6)
    m = make(MIXED, w, dtype, max_seqs=3, rows=rows)
    want = [[0, 7, 57, 150, 199], [3, 30]]
    got = m.step_score([5, 9], [a, b], True, want)
    assert row_err(got, np.concatenate([logits(MIXED, w, a, want[0]), logits(MIXED, w, b, want[1])])) < TOL[dtype]


@pytest.mark.parametrize("dtype, plain", [("bfloat16", 0), ("bfloat16", 1), ("float32", 0)])  # 32-bit mode has the plain kernel alone
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 100, 256, 300])
def test_a_key_just_inside_and_just_outside_the_window(window, plain, dtype):
    # one token outweighs every other while it is seen: right at the query, at the window's last place, one behind it; in prompts (a query
    # at every place of a tile and of a block), in portions, decoded one by one
    cfg = beacon_config(window)
    w = beacon_weights(cfg, 63)
    m = make(cfg, w, dtype, rows=700)
    m.set_option("bias_attn_plain", plain)
    for sid, at in enumerate((0, 15, 31, 250, 255, 256)):
        n = at + window + 3
        toks = tokens(n, 60, 10 * window + sid)
        toks[at] = 63
        edges = sorted({at, at + 1, at + window - 1, at + window, at + window + 1} | ({at + window // 2} if window > 3 else set()))
        ref = logits(cfg, w, toks, edges)
        got = m.step_score([sid], [toks], True, [edges])
        assert row_err(got, ref) < TOL[dtype], ("prompt", at)
        m.seq_free(sid)
        cut = max(1, at + window - 2)
        got = [m.step_score([sid], [toks[:cut]], True, [[p for p in edges if p < cut]]), decode(m, sid, toks, cut)[[p - cut for p in edges if p >= cut]]]
        assert row_err(np.concatenate(got), ref) < TOL[dtype], ("decoded", at)
        m.seq_free(sid)
        got = [m.step_score([sid], [toks[:at + 1]], True, [[at]]), m.step_score([sid], [toks], False, [edges[1:]])]
        assert row_err(np.concatenate(got), ref) < TOL[dtype], ("portions", at)
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_inside_a_wide_window(dtype):
    cfg = beacon_config(1024)
    w = beacon_weights(cfg, 63)
    m = make(cfg, w, dtype, rows=1300)
    for sid, at in enumerate((0, 47, 255, 256)):
        n = at + 1030
        toks = tokens(n, 60, sid)
        toks[at] = 63
        ask = sorted({at, at + 1, at + 500, at + 1022, at + 1023, at + 1024, n - 1})
        ref = logits(cfg, w, toks, ask)
        assert row_err(m.step_score([sid], [toks], True, [ask]), ref) < TOL[dtype], ("prompt", at)
        m.seq_free(sid)
        m.step_score([sid], [toks[:at + 1020]], True, [[]])
        late = [p for p in ask if p >= at + 1020]
        assert row_err(decode(m, sid, toks, at + 1020)[[p - at - 1020 for p in late]], ref[-len(late):]) < TOL[dtype], ("decoded", at)
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_and_sinks(dtype):
    # sinks of every strength weigh most where few keys are seen; the convolutions reach before the start
    cfg = config([par(win(heads=4, kv=4, conv=6, window=3), rule(conv=5)), par(win(heads=4, kv=2, window=40))], vocab=50)
    w = weights(cfg, 7)
    for i in range(2):
        w[f"l{i}.mix.left.sink"][:] = [-60.0, 0.0, 4.0, 60.0]
    toks = tokens(50, 50, 3)
    ref = logits(cfg, w, toks)
    m = make(cfg, w, dtype, max_seqs=60)
    assert row_err(m.step_score([0], [toks], True, [list(range(50))]), ref) < TOL[dtype]
    m.seq_free(0)
    assert row_err(decode(m, 0, toks, 0), ref) < TOL[dtype]
    for n in (1, 2, 3, 6):
        assert row_err(m.step_score([1], [toks[:n]], True, [list(range(n))]), ref[:n]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_state_carries_far(dtype):
    # almost no decay: the first token still counts after a thousand
    cfg = config([par(win(window=5), rule(heads=2, kv=1, dim=48)), delta(heads=2, kv=2, dim=40)], vocab=40, loop=(0, 2, 2))
    w = weights(cfg, 9)
    w["l0.mix.right.A_log"][:] = w["l1.mix.A_log"][:] = -9.0
    w["l0.mix.right.b"] *= 0.05  # rows small: half of what a key holds is overwritten only
    w["embed"][39] *= 8
    toks = [39] + tokens(1059, 39, 1)
    ref = logits(cfg, w, toks, list(range(1030, 1060)))
    lost = logits(cfg, w, toks[3:], list(range(1027, 1057)))
    assert row_err(lost, ref) > 5 * TOL["float32"]
    m = make(cfg, w, dtype)
    at = 0
    for n in (3, 500, 2, 255, 270):
        at += n
        m.step_score([0], [toks[:at]], False, [[]])
    assert at == 1030
    assert row_err(decode(m, 0, toks, 1030), ref) < TOL[dtype]
    assert row_err(m.step_score([1], [toks], True, [list(range(1030, 1034))]), ref[:4]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "even", "wide", "state"])
def test_recurrences_token_by_token_and_in_pieces(name, dtype):
    # prompt portions in pieces of 16 tokens and by the scan, each continuing from the state the other left
    cfg = CONFIGS[name]
    w = weights(cfg, 17)
    toks = tokens(260, cfg["vocab"], 3)
    ref = logits(cfg, w, toks)
    m = make(cfg, w, dtype)
    for sid, scans in enumerate(([1] * 6, [0] * 6, [0, 1, 0, 1, 0, 1])):
        at, got = 0, []
        for n, scan in zip((17, 64, 33, 5, 80, 61), scans):
            m.set_option("recur_scan", scan)
            got.append(m.step_score([sid], [toks[:at + n]], False, [list(range(at, at + n))]))
            at += n
        assert at == 260 and row_err(np.concatenate(got), ref) < TOL[dtype], scans
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_decays_of_every_strength(dtype):
    # rates from exp(-12) to exp(6) and strongly varying steps: decays that underflow within a token beside some that never do
    cfg = config([par(win(), rule(heads=8, kv=4, dim=32, vdim=32)), delta(heads=8, kv=4, dim=32, vdim=32)], vocab=60)
    w = weights(cfg, 5)
    rng = np.random.default_rng(0)
    for p, n in (("l0.mix.right.", 8), ("l1.mix.", 256)):
        w[p + "A_log"] = np.linspace(-12, 6, 8).astype(np.float32)
        w[p + "dt_bias"] = (rng.integers(-64, 65, n) / 8).astype(np.float32)
    toks = tokens(200, 60, 2)
    w = {k: L.bf16(v).astype(np.float64) for k, v in w.items()}
    ref = logits(cfg, w, toks)
    m = make(cfg, w, dtype, max_seqs=200)
    assert row_err(m.step_score([0], [toks], True, [list(range(200))]), ref) < TOL[dtype]
    m.step_score([1], [toks[:61]], True, [[]])
    assert row_err(decode(m, 1, toks[:90], 61), ref[61:90]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["even", "mixed"])
def test_batches_equal_each_request_alone(name, dtype):
    cfg = CONFIGS[name]
    w = weights(cfg, 7)
    m = make(cfg, w, dtype, blocks=32, max_seqs=6)
    lens = [1, 5, 17, 64, 259, 130]
    reqs = [tokens(n + 6, cfg["vocab"], 20 + n) for n in lens]
    refs = [logits(cfg, w, r) for r in reqs]
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
    for i in range(5):
        a, b = tokens(int(rng.integers(260, 500)), MIXED["vocab"], 50 + i), tokens(int(rng.integers(1, 400)), MIXED["vocab"], 90 + i)
        m.step_score([2 * i, 2 * i + 1], [a[:-1], b[:max(1, len(b) - 2)]], False, [[], []])
        got = m.step_score([2 * i, 2 * i + 1], [a, b], False, [[len(a) - 1], [len(b) - 1]])
        assert row_err(got, np.concatenate([logits(MIXED, w, a, [-1]), logits(MIXED, w, b, [-1])])) < TOL[dtype], i
        for s in ((2 * i, 2 * i + 1) if i % 2 else (2 * i + 1, 2 * i)):
            m.seq_free(s)
        assert m.free_blocks() == free


@pytest.mark.parametrize("dtype", DTYPES)
def test_blocks_no_window_reaches_are_given_back(dtype):
    # every window is shorter than a block: two sequences that outgrow the pool several times over, decoding while their old blocks serve
    # the other one
    cfg = config([par(win(window=60)), delta(), par(win(window=90), rule(heads=2, kv=2))], vocab=60)
    w = weights(cfg, 6)
    m = make(cfg, w, dtype, blocks=5, max_seqs=2)
    a, b = tokens(1100, 60, 1), tokens(1100, 60, 2)
    ra, rb = logits(cfg, w, a), logits(cfg, w, b)
    for at in (200, 450, 700, 950, 1090):
        got = m.step_score([0], [a[:at]], False, [[at - 1]])
        assert row_err(got, ra[[at - 1]]) < TOL[dtype], at
        got = m.step_score([1], [b[:at]], False, [[at - 1]])
        assert row_err(got, rb[[at - 1]]) < TOL[dtype], at
        got = m.step_score([0, 1], [a[:at + 1], b[:at + 1]], False, [[at], [at]])
        assert row_err(got, np.stack([ra[at], rb[at]])) < TOL[dtype], at
    m.seq_free(0)
    m.seq_free(1)
    assert m.free_blocks() == 5


@pytest.mark.parametrize("dtype", DTYPES)
def test_stepping_back_starts_the_sequence_again(dtype):
    # carried state cannot be undone: the same length again, a shorter prefix, another prompt under the same id
    for cfg in (STATE, config([par()], vocab=80)):
        w = weights(cfg, 11)
        toks, other = tokens(90, cfg["vocab"], 1), tokens(50, cfg["vocab"], 2)
        ref, ref2 = logits(cfg, w, toks), logits(cfg, w, other)
        m = make(cfg, w, dtype, blocks=3, max_seqs=2)
        for n in (90, 90, 40, 41, 60, 1, 2):
            assert row_err(m.step_score([0], [toks[:n]], False, [[n - 1]]), ref[[n - 1]]) < TOL[dtype], n
        assert row_err(m.step_score([0], [other], True, [[49]]), ref2[[49]]) < TOL[dtype]


def test_long_decoding():
    cfg = config([par(win(window=200), mlp=dense()), delta(moe())], vocab=96, loop=(0, 1, 2))
    w = weights(cfg, 9)
    toks = tokens(620, 96, 3)
    ref = logits(cfg, w, toks)
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
    outs = eng.generate(prompts, SamplingParams(max_tokens=5))
    assert len(outs) == 5 and m.free_blocks() == 24
    for p, (_, got) in zip(prompts, outs):
        want, rows = L.greedy(EVEN, w, p, 5)
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
    assert row_err(lg, np.array([logits(EVEN, w, p, -1) for p in prompts])) < TOL["bfloat16"]
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


@pytest.mark.parametrize("rows", [1, 16, 64, 130, 520])
def test_layers_of_a_real_size_take_the_fused_products(rows):
    # wide enough for the register-direct, streaming and tile products and their epilogues, plain and over groups of experts
    cfg = config([par(win(heads=8, kv=4, dim=128, vdim=128, window=100, rot=64, scale=0.2), rule(heads=8, kv=4, dim=128, vdim=128), dense(3072)),
                  delta(moe(8, 2, 512, (4, 2)), heads=8, kv=8, dim=128, vdim=128)], width=1024, vocab=4096)
    w = weights(cfg, 12)
    m = make(cfg, w, "bfloat16", blocks=160, max_seqs=64, rows=1024)
    m.set_option("tile_min_wgs", 1)  # the tile products whenever the shape fits
    if rows in (16, 64):  # a decode batch of that many sequences, each a few tokens long
        reqs = [tokens(4, 4096, i) for i in range(rows)]
        m.step_score(range(rows), [r[:3] for r in reqs], True, [[]] * rows)
        got = m.step_score(range(rows), reqs, False, [[3]] * rows)
        some = range(0, rows, 5)
        got, ref = got[list(some)], np.array([logits(cfg, w, reqs[i], 3) for i in some])
    else:
        t = tokens(rows, 4096, 1)
        ask = sorted({0, rows // 2, rows - 1})
        got, ref = m.step_score([0], [t], True, [ask]), logits(cfg, w, t, ask)
    assert row_err(got, ref) < TOL["bfloat16"]
    if rows > 128:
        assert m.counter("tile_gemm_launches") > 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_two_ranks_match_one(dtype):
    import threading

    import nano_vllm_candle_amd as pkg

    cfg = config([par(win(heads=4, kv=2), rule(heads=4, kv=2), dense()), delta(moe(), heads=4, kv=2), par(win(heads=2, kv=2), rule(heads=2, kv=2))], vocab=128, loop=(0, 2, 2))
    w = weights(cfg, 13)
    toks = tokens(90, 128, 1)
    ref, taps = L.run(cfg, w, toks)
    res, errs = [None, None], []

    def rank(r):
        try:
            m = make(cfg, w, dtype, 8, 2, 128, ctx=pkg.Context(0, r, 2, loopback_group=f"lefalix-{dtype}"))
            m.enable_taps()
            _, a = m.step([0], [toks[:80]], True, want_logits=True)
            tap = [m.layer_tap(i, 1, 80) for i in range(len(taps))]
            m.enable_taps(False)
            nxt, b = m.step([0], [toks[:81]], False, want_logits=True)
            nxt, c = m.step([0], [toks], False, want_logits=True)
            res[r] = (np.concatenate([a, b, c]), int(nxt[0]), tap)
        except Exception as e:  # noqa: BLE001
            errs.append(e)

    ts = [threading.Thread(target=rank, args=(r,)) for r in range(2)]
    [t.start() for t in ts]
    [t.join(100) for t in ts]
    assert not errs, errs
    for lg, nxt, tap in res:
        assert row_err(lg, ref[[79, 80, 89]]) < TOL[dtype]
        assert nxt == int(ref[89].argmax())
        assert max(row_err(a, b[:80]) for a, b in zip(tap, taps)) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_programs_on_a_checkpoint(tmp_path, dtype):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = MIXED
    w = weights(cfg, 14)
    write_checkpoint(tmp_path, cfg, f32(w))
    a, b = tokens(30, cfg["vocab"], 1), tokens(12, cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:20], "want": [19, 4]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b, "want": []}, {"id": "x", "tokens": a[20:29], "want": [8]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": a[29:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "x", "tokens": b, "want": [11]}], "end": []}]
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "64"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.split() == "done 0 done 1 done 2 done 3".split()
    ra, rb = logits(cfg, w, a), logits(cfg, w, b)
    for step, ref in ((0, ra[[19, 4]]), (1, ra[[28]]), (2, ra[[29]]), (3, rb[[11]])):
        got = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert row_err(got, ref) < TOL[dtype], step
    if dtype == "bfloat16":
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), "--model", str(tmp_path), "--prompt", ",".join(map(str, a)), "--max-tokens", "3"],
                           capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        want, rows = L.greedy(cfg, w, a, 1)
        first = int(r.stdout.split(",")[0])
        assert first == want[0] or (rows[0].max() - rows[0][first]) / np.abs(rows[0]).max() < 2 * TOL[dtype]


def test_what_the_library_refuses():
    import nano_vllm_candle_amd as pkg

    for layers in ([par(win(heads=5, kv=2))], [par(win(dim=514, rot=4))], [par(win(conv=17))], [par(win(rot=22))], [par(win(rot=5))], [delta(conv=17)], [par(right=rule(dim=513))],
                   [delta(moe(6, 3, 8, (3, 1)))], [delta(moe(6, 2, 8, (4, 2)))], [delta(moe(6, 7, 8, (1, 1)))]):
        cfg = config(layers)
        c = pkg.LefalixConfig.from_dict(cfg, {k: np.shape(v) for k, v in L.random_weights(cfg).items()})
        with pytest.raises(pkg._lib.NvllmError, match="layer"):
            pkg.LefalixForCausalLM(c)
    good = config([par(mlp=dense()), delta(moe())])
    w = f32(weights(good, 1))
    shapes = {k: np.shape(v) for k, v in w.items()}
    c = pkg.LefalixConfig.from_dict(good, shapes)
    with pytest.raises(pkg._lib.NvllmError, match="loop"):
        pkg.LefalixForCausalLM(pkg.LefalixConfig.from_dict(dict(good, loop={"start": 1, "stop": 3, "times": 2}), shapes))
    for name in ("l0.mix.left.sink", "l0.mix.right.out", "l0.norm1b", "l1.mlp.e3.gate", "l0.mix.left.o.b", "l0.mix.right.g", "l1.mix.g2"):
        with pytest.raises(pkg._lib.NvllmError, match="missing tensor " + name):
            pkg.LefalixForCausalLM.from_state_dict(c, {k: v for k, v in w.items() if k != name})
        with pytest.raises(pkg._lib.NvllmError, match="shape mismatch"):
            pkg.LefalixForCausalLM.from_state_dict(c, dict(w, **{name: w[name][:-1]}))
    for name in ("l0.mix.nope", "l0.mix.left.rel", "l0.mix.q", "l1.mix.left.q", "l1.mix.a", "l0.mlp.gate", "l1.mlp.e6.up"):
        with pytest.raises(pkg._lib.NvllmError, match="unknown tensor"):
            pkg.LefalixForCausalLM.from_state_dict(c, dict(w, **{name: w["l0.norm1"]}))


@pytest.mark.parametrize("width", [1024, 2048, 4096])
def test_wide_rows_of_long_prompts(width):
    # the two-branch norm of every width it has a form for, over whole and partly filled blocks of rows
    cfg = config([par(win(heads=2, kv=1, dim=16, vdim=16, rot=8), rule(heads=2, kv=1, dim=16, vdim=16), dense(64)), par(win(heads=2, kv=2), rule(heads=2, kv=2))], width=width, vocab=64, loop=(0, 1, 2))
    w = weights(cfg, 6)
    m = make(cfg, w, "bfloat16", rows=1024)
    for n in (528, 601):
        toks = tokens(n, 64, n)
        ask = [0, 15, 16, 300, n - 1]
        assert row_err(m.step_score([n], [toks], True, [ask]), logits(cfg, w, toks, ask)) < TOL["bfloat16"]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank", [1, 33, 150])
def test_ranks_of_the_two_step_gates(rank, dtype):
    cfg = config([delta(heads=3, kv=3, dim=40, vdim=24), par()], vocab=64)
    w = {k: L.bf16(v).astype(np.float64) for k, v in L.random_weights(cfg, 3, rank=rank).items()}
    toks = tokens(100, 64, 1)
    ref = logits(cfg, w, toks)
    m = make(cfg, w, dtype)
    assert row_err(portions(m, 0, toks, [70, 1, 1, 28]), ref) < TOL[dtype]
