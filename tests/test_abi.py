"""CPU: the C-ABI library loads and exports every symbol include/nvllm_amd.h declares; failures are loud."""
import os
import re

import pytest

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
HEADER = os.path.join(ROOT, "include", "nvllm_amd.h")              # the boundary a maintainer binds
DEBUG_HEADER = os.path.join(ROOT, "include", "nvllm_amd_debug.h")  # profiling / parity-debug / tuning exports


def header_functions(paths=(HEADER, DEBUG_HEADER)):
    names = set()
    for path in paths:
        src = open(path).read()
        src = re.sub(r"/\*.*?\*/", "", src, flags=re.S)
        names.update(re.findall(r"\b(nvllm_[a-z0-9_]+)\s*\(", src))
    return sorted(names)


def test_boundary_header_holds_no_debug_or_tuning_exports():
    names = header_functions((HEADER,))
    assert not [n for n in names if "_debug_" in n or "_profile_" in n], names


def test_library_exports_every_header_symbol():
    import ctypes

    import nano_vllm_candle_amd as pkg

    lib = ctypes.CDLL(pkg._lib.LIB_PATH)
    names = header_functions()
    assert len(names) >= 40
    for n in names:
        assert hasattr(lib, n), f"{n} declared in include/nvllm_amd.h but not exported"


def test_python_binding_covers_the_header():
    import nano_vllm_candle_amd as pkg

    assert sorted(pkg._lib.EXPORTED_SYMBOLS) == header_functions()


def test_library_is_in_tree_and_no_cpu_fallback():
    import nano_vllm_candle_amd as pkg

    assert os.path.dirname(pkg._lib.LIB_PATH).endswith("nano-vllm-candle_amd")
    # the product never imports the oracle
    for root, _, files in os.walk(os.path.join(ROOT, "nano-vllm-candle_amd")):
        for f in files:
            if f.endswith((".py", ".cpp", ".hip", ".h")):
                txt = open(os.path.join(root, f)).read()
                assert "import oracle" not in txt and "from oracle" not in txt and "qwen3_oracle" not in txt, f


@pytest.mark.skipif(os.path.exists("/dev/kfd"), reason="a GPU is present")
def test_context_creation_fails_loudly_without_a_gpu():
    import nano_vllm_candle_amd as pkg

    with pytest.raises(pkg._lib.NvllmError):
        pkg.Context(0)


def test_missing_library_raises(monkeypatch, tmp_path):
    import nano_vllm_candle_amd as pkg

    monkeypatch.setattr(pkg._lib, "_lib", None)
    monkeypatch.setattr(pkg._lib, "LIB_PATH", str(tmp_path / "nope.so"))
    with pytest.raises(pkg._lib.NvllmLibraryMissing):
        pkg._lib.lib()


def _kernel_resources():
    out = {}
    for name in ("kernel_resources.txt", "kernel_resources_tile.txt", "kernel_resources_latent.txt", "kernel_resources_latent_prefill.txt", "kernel_resources_bias_attn.txt",
                 "kernel_resources_recurrent.txt", "kernel_resources_recurrent_chunk.txt", "kernel_resources_scan.txt", "kernel_resources_moe.txt",
                 "kernel_resources_conv_attn.txt"):
        path = os.path.join(ROOT, "nano-vllm-candle_amd", name)
        if not os.path.exists(path):
            pytest.skip(name + " missing: rebuild the library (make -C nano-vllm-candle_amd/csrc)")
        for blk in open(path).read().split("Function Name: ")[1:]:
            lines = blk.strip().splitlines()
            out[lines[0].strip()] = {k.strip(): int(v) for k, v in (l.split(":", 1) for l in lines[1:])}
    return out


def test_hot_kernels_keep_their_register_budget():
    # hipcc's own per-kernel report, written beside the library by the build.  The decode path is tuned to exact wave
    # counts per SIMD: the decode attention kernel at 2 waves (<= 256 registers; at 269 it silently ran at 1 wave per
    # SIMD and the whole step lost 12 %), the register-direct GEMMs of the 0.6B layer at >= 4 (16-wave workgroups),
    # none of them with scratch in its inner loop.
    res = _kernel_resources()
    want = {  # mangled-name prefix -> minimum waves per SIMD
        "_ZN5nvllm17attn_paged_kernelILi128ELi1ELi4ELb1ELi0EEE": 2,   # fused decode attention, head_dim 128
        "_ZN5nvllm17attn_paged_kernelILi128ELi1ELi4ELb0ELi0EEE": 2,
        "_ZN5nvllm17attn_paged_kernelILi128ELi1ELi4ELb1ELi1EEE": 2,   # ... with the 24-bit V cache (one tile set per wave)
        "_ZN5nvllm17attn_paged_kernelILi128ELi1ELi4ELb1ELi2EEE": 2,   # ... with 24-bit K and V
        "_ZN5nvllm18gemm_rowdir_kernelILi4ELi16ELi2ELi2EEE": 4,   # QKV        (0.6B: N 4096, K 1024)
        "_ZN5nvllm18gemm_rowdir_kernelILi1ELi16ELi4ELi0EEE": 4,   # o_proj     (N 1024, K 2048)
        "_ZN5nvllm18gemm_rowdir_kernelILi6ELi16ELi2ELi1EEE": 4,   # gate/up    (N 6144, K 1024)
        "_ZN5nvllm18gemm_rowdir_kernelILi1ELi16ELi6ELi0EEE": 4,   # down_proj  (N 1024, K 3072)
        "_ZN5nvllm13lmhead_kernelILi4ELi5ELi4EEE": 2,             # LM head, 64 rows, vocabulary 151936, K 1024
        "_ZN5nvllm16gemm_tile_kernelILi8ELi2ELi0EEE": 2,              # prefill tile GEMM: 8-wave workgroups, two waves per SIMD
        "_ZN5nvllm16gemm_tile_kernelILi6ELi2ELi2EEE": 2,
        "_ZN5nvllm16gemm_tile_kernelILi8ELi2ELi3EEE": 2,              # ... with the q/k-norm + RoPE + KV-write epilogue
    }
    # without packed fp32 instructions the fused attention kernels spill a few prologue values (outside the K/V loop)
    scratch = {"_ZN5nvllm17attn_paged_kernelILi128ELi1ELi4ELb1ELi0EEE": 16, "_ZN5nvllm17attn_paged_kernelILi128ELi1ELi4ELb1ELi1EEE": 96,
               "_ZN5nvllm17attn_paged_kernelILi128ELi1ELi4ELb1ELi2EEE": 144}
    for prefix, min_waves in want.items():
        hits = [(n, r) for n, r in res.items() if n.startswith(prefix)]
        assert len(hits) == 1, (prefix, [n for n, _ in hits])
        r = hits[0][1]
        assert r["Occupancy [waves/SIMD]"] >= min_waves, (prefix, r)
        assert r["ScratchSize [bytes/lane]"] <= scratch.get(prefix, 0), (prefix, r)


def test_latent_attention_kernels_stay_in_registers():
    # attention over the latent cache, the expansion and the prompt kernel: no scratch in any instance; two waves per SIMD for the
    # attention kernels (their LDS allows two workgroups per CU, or one of eight waves)
    res = {n: r for n, r in _kernel_resources().items() if "latent" in n}
    assert len([n for n in res if "latent_attn_kernel" in n]) == 16
    for n, r in res.items():
        assert r["ScratchSize [bytes/lane]"] == 0, (n, r)
        if "latent_attn_kernel" in n or "latent_prefill_kernel" in n:
            assert r["Occupancy [waves/SIMD]"] >= 2, (n, r)


def test_bias_attention_and_recurrence_kernels_stay_in_registers():
    # prompt kernels read LDS by inline asm: a destination spilled while its read is in flight would lose the data, so no instance may
    # use scratch; the token-by-token scan may for key sizes above 256
    res = _kernel_resources()
    for part, count in (("bias_prefill_kernel", 20), ("bias_decode_kernel", 20), ("piece_scan_kernel", 24), ("delta_pieces_kernel", 8)):
        hits = {n: r for n, r in res.items() if part in n}
        assert len(hits) == count, (part, len(hits))
        for n, r in hits.items():
            assert r["ScratchSize [bytes/lane]"] == 0, (n, r)
    for n, r in res.items():
        if "bias_prefill_kernelILi4ELi8" in n or "bias_decode_kernelILi4ELi8" in n:
            assert r["Occupancy [waves/SIMD]"] >= 2, (n, r)
        if "recurrence_decode_kernelILi2" in n:
            assert r["Occupancy [waves/SIMD]"] >= 4 and r["ScratchSize [bytes/lane]"] == 0, (n, r)


def test_scan_and_expert_kernels_stay_in_registers():
    res = _kernel_resources()
    for part, count in (("scan_prompt_kernel", 18), ("scan_decode_kernel", 9), ("conv_rows16_kernel", 3), ("group_gemm_kernel", 8), ("gemm_tile_kernelILi8ELi2ELi5", 1), ("gemm_tile_kernelILi8ELi2ELi6", 1),
                        ("gemm_tile_kernelILi8ELi2ELi7", 1), ("gemm_tile_kernelILi6ELi2ELi8", 1), ("conv_attn_rows16_kernel", 12), ("conv_attn_decode_kernel", 12)):
        hits = {n: r for n, r in res.items() if part in n and "piece_scan" not in n}
        assert len(hits) == count, (part, len(hits))
        for n, r in hits.items():
            assert r["ScratchSize [bytes/lane]"] == 0, (n, r)
    for n, r in res.items():
        if "scan_prompt_kernelILi4ELi4E" in n or "scan_decode_kernelILi4ELi4E" in n:
            assert r["Occupancy [waves/SIMD]"] >= 4, (n, r)
