"""What every decoder behind the C ABI shares on the host side: checkpoint reading, the block pool, the step / score / decode
calls, profiling and taps.  A model class supplies its configuration (`cfg`, with vocab_size and hidden_size) and creates the
native handle `h` on a Context `ctx`."""
import ctypes as C
import json
import os
import struct
from dataclasses import dataclass

import numpy as np

from . import _lib
from .context import Context


def _safetensors_header(path):
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        header = json.loads(f.read(n))
    header.pop("__metadata__", None)
    return header, 8 + n


def tensor_shapes(model_dir):
    """name -> shape of every tensor of a checkpoint directory"""
    return {name: tuple(meta["shape"]) for path in checkpoint_files(model_dir) for name, meta in _safetensors_header(path)[0].items()}


def read_safetensors(path):
    """Minimal safetensors reader (header JSON + raw little-endian data, memory-mapped): yields
    (name, np.ndarray view, dtype code).  Executes nothing from the file.  BF16 tensors come back as uint16."""
    header, start = _safetensors_header(path)
    data = np.memmap(path, dtype=np.uint8, mode="r", offset=start)
    for name, meta in header.items():
        b, e = meta["data_offsets"]
        dt = meta["dtype"]
        if dt == "BF16":
            arr, code = data[b:e].view(np.uint16), _lib.DTYPE_BF16
        elif dt == "F32":
            arr, code = data[b:e].view(np.float32), _lib.DTYPE_F32
        elif dt == "F16":
            arr, code = data[b:e].view(np.float16).astype(np.float32), _lib.DTYPE_F32
        else:
            raise ValueError(f"{path}: tensor {name} has unsupported dtype {dt}")
        yield name, arr.reshape(meta["shape"]), code


def checkpoint_files(model_dir):
    """safetensors files of an HF model directory: the shards named by model.safetensors.index.json (each once, in
    name order) or the single model.safetensors the reference expects (qwen3.rs:517-521; same error text)"""
    idx = os.path.join(model_dir, "model.safetensors.index.json")
    single = os.path.join(model_dir, "model.safetensors")
    if os.path.exists(idx):
        with open(idx) as f:
            names = sorted(set(json.load(f)["weight_map"].values()))
        return [os.path.join(model_dir, x) for x in names]
    if os.path.exists(single):
        return [single]
    raise RuntimeError(f"mmap {single}: no such file")


class CausalLM:
    """Base of the model classes: a native model handle and the calls on it"""

    cfg = None
    ctx = None
    h = None

    @property
    def vocab_size(self):
        return self.cfg.vocab_size

    def load_tensor(self, name, arr, code=None):
        if code is None:
            code = _lib.DTYPE_BF16 if arr.dtype == np.uint16 else _lib.DTYPE_F32
            if code == _lib.DTYPE_F32:
                arr = np.ascontiguousarray(arr, np.float32)
        arr = np.ascontiguousarray(arr).reshape(arr.shape)  # ascontiguousarray makes a scalar one-dimensional
        shape = (C.c_int64 * arr.ndim)(*arr.shape)
        _lib.check(_lib.lib().nvllm_model_load_tensor(self.h, name.encode(), arr.ctypes.data_as(C.c_void_p), code, shape,
                                                      arr.ndim), self.ctx.h)

    def finalize(self):
        _lib.check(_lib.lib().nvllm_model_finalize(self.h), self.ctx.h)

    # ---- KV pool ----
    def kv_alloc(self, num_blocks, max_seqs, max_batched_tokens=4096, block_size=256):
        _lib.check(_lib.lib().nvllm_kv_alloc(self.h, num_blocks, block_size, max_seqs, max_batched_tokens), self.ctx.h)
        self._kv = True
        self.max_seqs = max_seqs

    def free_blocks(self):
        return _lib.lib().nvllm_kv_num_free_blocks(self.h)

    def seq_free(self, seq_id):
        _lib.check(_lib.lib().nvllm_seq_free(self.h, int(seq_id)), self.ctx.h)

    @property
    def weight_bytes(self):
        return _lib.lib().nvllm_model_weight_bytes(self.h)

    @property
    def kv_bytes_per_token(self):
        return _lib.lib().nvllm_kv_bytes_per_token(self.h)

    @property
    def last_step_bytes(self):
        return _lib.lib().nvllm_last_step_bytes(self.h)

    # ---- the hot path ----
    @staticmethod
    def _step_args(seq_ids, token_lists):
        n = len(seq_ids)
        arrs = [np.ascontiguousarray(t, dtype=np.uint32) for t in token_lists]
        u32p = C.POINTER(C.c_uint32)
        return (u32p, (C.c_int64 * n)(*[int(s) for s in seq_ids]), (u32p * n)(*[a.ctypes.data_as(u32p) for a in arrs]),
                (C.c_int32 * n)(*[len(a) for a in arrs]), arrs)

    def step_score(self, seq_ids, token_lists, is_prefill, wanted):
        """Process the tokens not cached yet (all of them when is_prefill) without sampling; wanted[i]: ascending positions
        of sequence i among them.  -> float32 [sum of wanted, vocab] in that order"""
        n = len(seq_ids)
        if len(wanted) != n:
            raise ValueError("one list of wanted positions per sequence")
        flat = [int(p) for w in wanted for p in w]
        out = np.empty((len(flat), self.cfg.vocab_size), np.float32)
        if n == 0:
            return out
        u32p, ids, ptrs, lens, _keep = self._step_args(seq_ids, token_lists)
        nw = (C.c_int32 * n)(*[len(w) for w in wanted])
        pos = (C.c_int32 * max(len(flat), 1))(*flat)
        _lib.check(_lib.lib().nvllm_step_score(self.h, n, ids, ptrs, lens, int(bool(is_prefill)), nw, pos,
                                               out.ctypes.data_as(C.POINTER(C.c_float))), self.ctx.h)
        return out

    def step(self, seq_ids, token_lists, is_prefill, want_logits=False):
        """ModelRunner::run: -> (next_ids uint32[n], last_logits float32[n,V] or None)"""
        n = len(seq_ids)
        if n == 0:
            return np.empty(0, np.uint32), None
        u32p, ids, ptrs, lens, _keep = self._step_args(seq_ids, token_lists)
        nxt = np.empty(n, np.uint32)
        lg = np.empty((n, self.cfg.vocab_size), np.float32) if want_logits else None
        _lib.check(_lib.lib().nvllm_step(self.h, n, ids, ptrs, lens, int(bool(is_prefill)), nxt.ctypes.data_as(u32p),
                                         lg.ctypes.data_as(C.POINTER(C.c_float)) if lg is not None else None), self.ctx.h)
        return nxt, lg

    def step_sample(self, seq_ids, token_lists, is_prefill, temperatures, seed, want_logits=False):
        """ModelRunner::run with sample_token on the device (llm_engine.rs:97-133): -> (sampled ids, last_logits or None)"""
        n = len(seq_ids)
        if n == 0:
            return np.empty(0, np.uint32), None
        u32p, ids, ptrs, lens, _keep = self._step_args(seq_ids, token_lists)
        temps = np.ascontiguousarray(temperatures, np.float32)
        if temps.shape != (n,):
            raise ValueError("one temperature per sequence")
        nxt = np.empty(n, np.uint32)
        lg = np.empty((n, self.cfg.vocab_size), np.float32) if want_logits else None
        _lib.check(_lib.lib().nvllm_step_sample(self.h, n, ids, ptrs, lens, int(bool(is_prefill)),
                                                temps.ctypes.data_as(C.POINTER(C.c_float)), int(seed) & (2**64 - 1), nxt.ctypes.data_as(u32p),
                                                lg.ctypes.data_as(C.POINTER(C.c_float)) if lg is not None else None), self.ctx.h)
        return nxt, lg

    def decode_next(self, want_ids=True):
        n = getattr(self, "max_seqs", 0)
        buf = np.empty(max(n, 1), np.uint32)
        _lib.check(_lib.lib().nvllm_decode_next(self.h, buf.ctypes.data_as(C.POINTER(C.c_uint32)) if want_ids else None),
                   self.ctx.h)
        return buf

    def decode_enqueue(self):
        """put one more decode step on the stream without waiting (pipelined decode)"""
        _lib.check(_lib.lib().nvllm_decode_enqueue(self.h), self.ctx.h)

    def decode_collect(self):
        """ids of the oldest enqueued decode step"""
        buf = np.empty(max(getattr(self, "max_seqs", 1), 1), np.uint32)
        _lib.check(_lib.lib().nvllm_decode_collect(self.h, buf.ctypes.data_as(C.POINTER(C.c_uint32))), self.ctx.h)
        return buf

    PROF_KINDS = {"attn": 1, "gemm": 2, "norm": 3, "qk": 4, "silu": 5, "lm_head": 6, "empty": 7, "recur": 8}

    def profile_kernel(self, kind):
        """HIP-event bracketing of one kernel class on the library stream (None/0 = off)"""
        k = self.PROF_KINDS.get(kind, kind) if kind else 0
        _lib.check(_lib.lib().nvllm_profile_kernel(self.h, int(k)), self.ctx.h)

    def profile_read(self):
        ms, n = C.c_double(), C.c_int64()
        _lib.check(_lib.lib().nvllm_profile_read(self.h, C.byref(ms), C.byref(n)), self.ctx.h)
        return ms.value, n.value

    def set_option(self, name, value):
        """tuning switch of the model (include/nvllm_amd_debug.h nvllm_debug_set_option)"""
        _lib.check(_lib.lib().nvllm_debug_set_option(self.h, name.encode(), int(value)), self.ctx.h)

    def counter(self, name):
        """debug counter of the model (include/nvllm_amd_debug.h nvllm_debug_get_counter)"""
        v = C.c_int64()
        _lib.check(_lib.lib().nvllm_debug_get_counter(self.h, name.encode(), C.byref(v)), self.ctx.h)
        return int(v.value)

    def enable_taps(self, on=True):
        _lib.check(_lib.lib().nvllm_debug_enable_taps(self.h, int(on)), self.ctx.h)

    def layer_tap(self, layer, what, rows):
        out = np.empty((rows, self.cfg.hidden_size), np.float32)
        _lib.check(_lib.lib().nvllm_debug_layer_tap(self.h, layer, what, out.ctypes.data_as(C.POINTER(C.c_float)), out.size),
                   self.ctx.h)
        return out

    def close(self):
        if getattr(self, "h", None):
            _lib.lib().nvllm_model_destroy(self.h)
            self.h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass


class LayeredCausalLM(CausalLM):
    """Base of the models built from layer descriptions.  dtype "bfloat16": products on bf16 hi + lo activation planes, f16 cache (the
    serving mode); "float32": every product and the cache in f32.  A subclass names its CONFIG (with from_dir, tensor_shapes and
    random_tensor) and creates the native handle from it."""

    DTYPES = ("bfloat16", "float32")
    CONFIG = None

    def __init__(self, cfg, ctx=None, dtype="bfloat16"):
        if dtype not in self.DTYPES:
            raise ValueError(f"dtype {dtype!r} unsupported ({', '.join(self.DTYPES)})")
        self.cfg, self.dtype = cfg, dtype
        self.ctx = ctx or Context(0)
        h = C.c_void_p()
        _lib.check(self._create(cfg, dtype == "float32", C.byref(h)), self.ctx.h)
        self.h = h

    def _create(self, cfg, f32, out):
        raise NotImplementedError

    @classmethod
    def from_dir(cls, model_dir, ctx=None, dtype="bfloat16"):
        m = cls(cls.CONFIG.from_dir(model_dir), ctx, dtype)
        for path in checkpoint_files(model_dir):
            for name, arr, code in read_safetensors(path):
                m.load_tensor(name, arr, code)
        m.finalize()
        return m

    @classmethod
    def from_state_dict(cls, cfg, tensors, ctx=None, dtype="bfloat16"):
        """tensors: name -> ndarray, float32 or bf16 bits as uint16 (full shapes)"""
        m = cls(cfg, ctx, dtype)
        for name, arr in tensors.items():
            m.load_tensor(name, np.asarray(arr))
        m.finalize()
        return m

    @classmethod
    def from_random(cls, cfg, seed=0, ctx=None, dtype="bfloat16"):
        """random weights of the configured shapes (benchmarks)"""
        rng = np.random.default_rng(seed)
        m = cls(cfg, ctx, dtype)
        for name, shape in cfg.tensor_shapes().items():
            m.load_tensor(name, cfg.random_tensor(name, shape, rng))
        m.finalize()
        return m


def random_matrix(shape, rng):
    """bf16 bits of unit output variance: random sign and mantissa, exponent of 1 / sqrt(fan-in)"""
    e = 127 - max(1, int(round(0.5 * np.log2(shape[1]))))
    return (rng.integers(0, 1 << 16, shape, dtype=np.uint16) & np.uint16(0x807F)) | np.uint16(e << 7)


@dataclass
class Yarn:
    """YaRN scaling of a rotation"""
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def from_dict(cls, d):
        return cls(*(float(d[k]) for k in ("factor", "original", "fast", "slow"))) if d else None
