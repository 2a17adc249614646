"""Berevik on the GPU against the plain CPU restatement (oracle/berevik_oracle.py): layer by layer, prompts, portions, decoding,
batches, window edges, block and slot reuse, greedy generation through the engine -- in both precisions."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import berevik_oracle as B
from tests.berevik_util import CONFIGS, EVEN, MIXED, TOL, beacon_weights, config, layer, row_err, sharp_weights
from tests.util import write_checkpoint

pytestmark = pytest.mark.gpu
DTYPES = ("bfloat16", "float32")


def make(cfg, w, dtype, blocks=24, max_seqs=6, rows=512):
    import nano_vllm_candle_amd as pkg

    m = pkg.BerevikForCausalLM.from_state_dict(pkg.BerevikConfig.from_dict(cfg), w, dtype=dtype)
    m.kv_alloc(blocks, max_seqs, max_batched_tokens=rows)
    return m


def tokens(n, vocab, seed=0):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_layer_outputs_and_logits(name, dtype):
    cfg = CONFIGS[name]
    w = sharp_weights(cfg)
    toks = tokens(150, cfg["vocab"])
    outs = []
    ref = B.forward(cfg, w, toks, layer_outputs=outs)
    m = make(cfg, w, dtype, max_seqs=256)
    m.enable_taps()
    got = m.step_score([0], [toks], True, [list(range(len(toks)))])
    for run, r in enumerate(outs):
        e = row_err(m.layer_tap(run, 1, len(toks)), r)
        assert e < TOL[dtype], (name, dtype, run, e)
    e = row_err(got, ref)
    assert e < TOL[dtype], (name, dtype, e)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("part", ["attention", "feed_forward", "embedding_and_head"])
def test_one_mechanism(part, dtype):
    cfg = config([layer(heads=4, window=9)], vocab=100, embed=0.7, cap=2.0, eps=0.01)
    w = sharp_weights(cfg, 3)
    if part != "attention":
        w["l0.mix.o"][:] = 0
    if part != "feed_forward":
        w["l0.mlp.down"][:] = 0
    for k in ("l0.mlp.gate", "l0.mlp.up"):  # well past the clamps on both sides
        w[k] *= 4
    toks = tokens(40, 100, 1)
    m = make(cfg, w, dtype, max_seqs=64)
    assert row_err(m.step_score([0], [toks], True, [list(range(40))]), B.forward(cfg, w, toks)) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "even", "wide"])
def test_portions_and_decoding_equal_the_whole_prompt(name, dtype):
    cfg = CONFIGS[name]
    w = sharp_weights(cfg, 1)
    toks = tokens(330, cfg["vocab"], 2)
    ref = B.forward(cfg, w, toks)
    m = make(cfg, w, dtype)
    cuts = {"twos": [2] * 165, "odd": [11, 2, 37, 64, 3, 120, 1, 1, 91], "page": [255, 2, 73], "decode": [250] + [1] * 80}
    for sid, (what, parts) in enumerate(cuts.items()):
        at, got = 0, []
        for n in parts:
            got.append(m.step_score([sid], [toks[:at + n]], False, [list(range(at, at + n))]))
            at += n
        assert at == len(toks)
        got = np.concatenate(got)
        worst = np.abs(got - ref).max(1) / np.abs(ref).max()
        assert worst.max() < TOL[dtype], (name, dtype, what, int(worst.argmax()), worst.max())
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [16, 100])
def test_small_row_buffers_cut_prompts_inside(rows, dtype):
    cfg = MIXED
    w = sharp_weights(cfg, 4)
    a, b = tokens(200, cfg["vocab"], 5), tokens(31, cfg["vocab"], 6)
    m = make(cfg, w, dtype, max_seqs=3, rows=rows)
    want = [[0, 7, 57, 150, 199], [3, 30]]
    got = m.step_score([5, 9], [a, b], True, want)
    ref = np.concatenate([B.forward(cfg, w, a, want[0]), B.forward(cfg, w, b, want[1])])
    assert row_err(got, ref) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 200, 257])
def test_window_edges(window, dtype):
    # one token dominates every query that sees it: the last position inside its window and the first outside, decoded and in
    # prompt portions, with the token at several places of its 16-, 32- and 256-token tiles
    cfg = config([layer(heads=3, window=window, ff=0)], vocab=64)
    w = beacon_weights(cfg, 63)
    wrong = [dict(cfg, layers=[layer(heads=3, window=window + d, ff=0)]) for d in (1, -1) if window + d > 0]
    m = make(cfg, w, dtype)
    for sid, at in enumerate((0, 15, 47, 255, 256)):
        n = at + window + 3
        toks = tokens(n, 60, sid)
        toks[at] = 63
        ask = [at, at + window - 1, at + window, at + window + 1]
        ask = sorted(set(ask))
        ref = B.forward(cfg, w, toks, ask)
        for c in wrong:  # the weights make a window one token off show
            assert row_err(B.forward(c, w, toks, ask), ref) > 0.05
        got = m.step_score([sid], [toks], True, [ask])
        assert row_err(got, ref) < TOL[dtype], ("prompt", window, at)
        cut = max(1, at + window - 2)
        m.set_option("latent_absorb", -1 if sid % 2 else 1)  # alternately the expanded and the absorbed form for the prompt part
        parts = [m.step_score([sid], [toks[:cut]], True, [[p for p in ask if p < cut]])]
        for i in range(cut, n):
            parts.append(m.step_score([sid], [toks[:i + 1]], False, [[i] if i in ask else []]))
        assert row_err(np.concatenate(parts), ref) < TOL[dtype], ("decoded", window, at)
        m.seq_free(sid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_batches_equal_each_request_alone(dtype):
    cfg = EVEN
    w = sharp_weights(cfg, 7)
    m = make(cfg, w, dtype, blocks=32, max_seqs=6)
    lens = [1, 5, 17, 64, 259, 130]
    reqs = [tokens(n + 6, cfg["vocab"], 20 + n) for n in lens]
    refs = [B.forward(cfg, w, r) for r in reqs]
    # mixed step: prompts of all lengths, then prompts and decoding rows side by side, then decoding alone
    got = m.step_score(range(6), [r[:n] for r, n in zip(reqs, lens)], True, [[n - 1] for n in lens])
    assert row_err(got, np.array([f[n - 1] for f, n in zip(refs, lens)])) < TOL[dtype]
    step = [1, 3, 1, 2, 1, 3]
    at = [n + s for n, s in zip(lens, step)]
    got = m.step_score(range(6), [r[:n] for r, n in zip(reqs, at)], False, [[n - 1] for n in at])
    assert row_err(got, np.array([f[n - 1] for f, n in zip(refs, at)])) < TOL[dtype]
    for _ in range(3):
        at = [n + 1 for n in at]
        got = m.step_score(range(6), [r[:n] for r, n in zip(reqs, at)], False, [[n - 1] for n in at])
        assert row_err(got, np.array([f[n - 1] for f, n in zip(refs, at)])) < TOL[dtype]


@pytest.mark.parametrize("form", [1, -1])
@pytest.mark.parametrize("name", ["mixed", "even", "ranks"])
def test_absorbed_and_expanded_prompt_attention(name, form):
    # both forms on whole prompts, on portions with context in the cache and on batches of unequal portions
    cfg = CONFIGS[name]
    w = sharp_weights(cfg, 15)
    m = make(cfg, w, "bfloat16", rows=256)
    m.set_option("latent_absorb", form)
    toks = tokens(420, cfg["vocab"], 3)
    ref = B.forward(cfg, w, toks)
    at = 0
    for n in (3, 130, 2, 200, 85):
        got = m.step_score([0], [toks[:at + n]], False, [sorted({at, at + n // 2, at + n - 1})])
        at += n
        assert row_err(got, ref[sorted({at - n, at - n + n // 2, at - 1})]) < TOL["bfloat16"], (n, at)
    m.step_score([1, 2], [toks[:100], toks[:7]], True, [[], []])
    got = m.step_score([1, 2, 3], [toks[:350], toks[:9], toks[:40]], False, [[100, 349], [7, 8], [39]])
    assert row_err(got, ref[[100, 349, 7, 8, 39]]) < TOL["bfloat16"]
    assert (m.counter("latent_expanded") > 0) == (form == -1)


@pytest.mark.parametrize("dtype", DTYPES)
def test_blocks_and_slots_are_reused(dtype):
    cfg = MIXED
    w = sharp_weights(cfg, 8)
    m = make(cfg, w, dtype, blocks=4, max_seqs=2)
    free = m.free_blocks()
    rng = np.random.default_rng(0)
    for i in range(6):
        a, b = tokens(int(rng.integers(260, 500)), cfg["vocab"], 50 + i), tokens(int(rng.integers(1, 400)), cfg["vocab"], 90 + i)
        got = m.step_score([2 * i, 2 * i + 1], [a, b], False, [[len(a) - 1], [len(b) - 1]])
        ref = np.concatenate([B.forward(cfg, w, a, [-1]), B.forward(cfg, w, b, [-1])])
        assert row_err(got, ref) < TOL[dtype], i
        for s in ((2 * i, 2 * i + 1) if i % 2 else (2 * i + 1, 2 * i)):
            m.seq_free(s)
        assert m.free_blocks() == free


@pytest.mark.parametrize("dtype", DTYPES)
def test_blocks_behind_every_window_are_given_back(dtype):
    cfg = config([layer(window=40), layer(window=300, heads=2)], vocab=96)
    w = sharp_weights(cfg, 16)
    toks, other = tokens(1100, 96, 4), tokens(700, 96, 5)
    ref, ref2 = B.forward(cfg, w, toks), B.forward(cfg, w, other)
    m = make(cfg, w, dtype, blocks=6, max_seqs=2)
    got = m.step_score([0], [toks[:1000]], True, [[999]])
    assert row_err(got, ref[[999]]) < TOL[dtype]
    assert m.free_blocks() == 4  # positions 701.. stay visible: blocks 2 and 3
    # another sequence on the returned blocks, the first one decoding beside it
    got = m.step_score([0, 1], [toks[:1001], other[:600]], False, [[1000], [599]])
    assert row_err(got, np.concatenate([ref[[1000]], ref2[[599]]])) < TOL[dtype]
    for i in range(1001, 1100):
        n2 = 600 + i - 1000
        got = m.step_score([0, 1], [toks[:i + 1], other[:n2]], False, [[i], [n2 - 1]])
        assert row_err(got, np.concatenate([ref[[i]], ref2[[n2 - 1]]])) < TOL[dtype], i
    assert m.free_blocks() == 6 - 2 - 2
    m.seq_free(1)
    # stepping back: within the kept blocks the last token alone, further back the whole sequence again
    for n in (1100, 1050, 500):
        assert row_err(m.step_score([0], [toks[:n]], False, [[n - 1]]), ref[[n - 1]]) < TOL[dtype]
    m.seq_free(0)
    assert m.free_blocks() == 6


def test_long_decoding_keeps_the_window():
    cfg = config([layer(window=40), layer(window=300, heads=2)], vocab=96)
    w = sharp_weights(cfg, 9)
    toks = tokens(620, 96, 3)
    ref = B.forward(cfg, w, toks)
    for dtype in DTYPES:
        m = make(cfg, w, dtype)
        got = [m.step_score([0], [toks[:3]], True, [[2]])]
        for i in range(3, len(toks)):
            got.append(m.step_score([0], [toks[:i + 1]], False, [[i]]))
        assert row_err(np.concatenate(got), ref[2:]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_engine(dtype):
    from nano_vllm_candle_amd.engine import CausalLMRunner, LLMEngine, SamplingParams, Scheduler, SchedulerConfig

    cfg = EVEN
    w = sharp_weights(cfg, 10)
    m = make(cfg, w, dtype, max_seqs=5)  # the scheduler admits prompts while others decode: a slot for each
    prompts = [tokens(n, cfg["vocab"], n) for n in (1, 33, 70, 300, 2)]
    eng = LLMEngine(Scheduler(SchedulerConfig(max_num_seqs=3, eos=None)), CausalLMRunner(m, greedy=True))
    outs = eng.generate(prompts, SamplingParams(max_tokens=6))
    assert len(outs) == 5 and m.free_blocks() == 24
    for p, (_, got) in zip(prompts, outs):
        want, rows = B.greedy(cfg, w, p, 6)
        for g, t, r in zip(got, want, rows):
            if g != t:  # only a near-tie may flip, and everything after it then differs
                assert (r.max() - r[g]) / np.abs(r).max() < 2 * TOL[dtype], (g, t)
                break


def test_decode_fast_path_and_sampling_follow_the_step_call():
    cfg = EVEN
    w = sharp_weights(cfg, 11)
    m = make(cfg, w, "bfloat16", max_seqs=4)
    prompts = [tokens(n, cfg["vocab"], n) for n in (40, 3, 258)]
    ids = [0, 1, 2]
    seqs = [list(p) for p in prompts]
    nxt, lg = m.step(ids, seqs, True, want_logits=True)
    assert row_err(lg, np.array([B.forward(cfg, w, p, [-1])[0] for p in prompts])) < TOL["bfloat16"]
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
    # wide enough for the register-direct, streaming and tile products and their gated epilogue
    cfg = config([layer(heads=16, dim=64, rot=64, vdim=128, rank=256, window=400, ff=3072, limit=1.2)], width=1024, vocab=4096, cap=15.0)
    w = sharp_weights(cfg, 12, gain=1.5)
    m = make(cfg, w, "bfloat16", blocks=160, max_seqs=64, rows=1024)
    m.set_option("tile_min_wgs", 1)  # the tile products whenever the shape fits
    if rows in (16, 64):  # a decode batch of that many sequences, each a few tokens long
        reqs = [tokens(4, 4096, i) for i in range(rows)]
        m.step_score(range(rows), [r[:3] for r in reqs], True, [[]] * rows)
        got = m.step_score(range(rows), reqs, False, [[3]] * rows)
        ref = np.array([B.forward(cfg, w, r, [3], dtype=np.float32)[0] for r in reqs])
    else:
        t = tokens(rows, 4096, 1)
        ask = sorted({0, rows // 2, rows - 1})
        got, ref = m.step_score([0], [t], True, [ask]), B.forward(cfg, w, t, ask, dtype=np.float32)
    assert row_err(got, ref) < TOL["bfloat16"]
    if rows > 128:
        assert m.counter("tile_gemm_launches") > 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_two_ranks_match_one(dtype):
    import threading

    import nano_vllm_candle_amd as pkg

    cfg = config([layer(heads=4, ff=80), layer(heads=2, dim=16, ff=0)], vocab=128, loop={"start": 0, "stop": 2, "times": 2})
    w = sharp_weights(cfg, 13)
    toks = tokens(90, 128, 1)
    res, errs = [None, None], []

    def rank(r):
        try:
            c = pkg.Context(0, r, 2, loopback_group=f"berevik-{dtype}")
            m = pkg.BerevikForCausalLM.from_state_dict(pkg.BerevikConfig.from_dict(cfg), w, ctx=c, dtype=dtype)
            m.kv_alloc(8, 2, max_batched_tokens=128)
            _, a = m.step([0], [toks[:80]], True, want_logits=True)
            nxt, b = m.step([0], [toks], False, want_logits=True)
            res[r] = (np.concatenate([a, b]), int(nxt[0]))
        except Exception as e:  # noqa: BLE001
            errs.append(e)

    ts = [threading.Thread(target=rank, args=(r,)) for r in range(2)]
    [t.start() for t in ts]
    [t.join(100) for t in ts]
    assert not errs, errs
    ref = B.forward(cfg, w, toks, [79, 89])
    for lg, nxt in res:
        assert row_err(lg, ref) < TOL[dtype]
        assert nxt == int(ref[1].argmax())


@pytest.mark.parametrize("dtype", DTYPES)
def test_programs_on_a_checkpoint(tmp_path, dtype):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = MIXED
    w = sharp_weights(cfg, 14)
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
    ra, rb = B.forward(cfg, w, a), B.forward(cfg, w, b)
    for step, ref in ((0, ra[[19, 4]]), (1, ra[[28]]), (2, ra[[29]]), (3, rb[[11]])):
        got = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert row_err(got, ref) < TOL[dtype], step
    if dtype == "bfloat16":
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), "--model", str(tmp_path), "--prompt", ",".join(map(str, a)), "--max-tokens", "3"],
                           capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        want, rows = B.greedy(cfg, w, a, 1)
        first = int(r.stdout.split(",")[0])
        assert first == want[0] or (rows[0].max() - rows[0][first]) / np.abs(rows[0]).max() < 2 * TOL[dtype]


@pytest.mark.parametrize("rows", [64, 512])
def test_scoring_serves_qwen3_too(rows, tmp_path):
    # the same call on the other model class: chosen positions of a prompt, of portions and of decoded tokens equal the logits the
    # sampling step returns for each prefix
    import nano_vllm_candle_amd as pkg

    m = pkg.Qwen3ForCausalLM.from_synthetic(pkg.Qwen3Config.tiny(), seed=1)
    m.kv_alloc(8, 3, max_batched_tokens=rows)
    toks = tokens(300, 512, 2)
    ask = [0, 5, 17, 63, 64, 130, 255, 256, 299]
    ref = np.concatenate([m.step([i], [toks[:p + 1]], True, want_logits=True)[1] for i, p in enumerate(ask) if not m.seq_free(i - 1)])
    for i in range(len(ask)):
        m.seq_free(i)
    assert row_err(m.step_score([50], [toks], True, [ask]), ref) < 1e-3
    got, at = [], 0
    for n in (64, 1, 66, 125, 1, 43):
        at += n
        got.append(m.step_score([51], [toks[:at]], False, [[p for p in ask if at - n <= p < at]]))
    assert at == 300 and row_err(np.concatenate(got), ref) < 1e-3
    with pytest.raises(pkg._lib.NvllmError, match="wanted position"):
        m.step_score([51], [toks], False, [[3]])  # cached already
