// Device-side helpers shared by the .hip translation units of libnvllm_amd.so (kernels.hip, stream_gemm.hip):
// MFMA fragment types, bf16 hi/lo split, deferred-RMSNorm helpers, the LDS-DMA publish barrier, diagnostic stamps.
#pragma once
#include <hip/hip_runtime.h>

#include <atomic>
#include <type_traits>

#include "kernels.h"

namespace nvllm {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(8))) _Float16 f16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

// ---------------------------------------------------------------------------------------------------
// small helpers
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ uint16_t bf16_bits_of(float x) { return __builtin_bit_cast(uint16_t, (__bf16)x); }
__device__ __forceinline__ float bf16_to_f32(uint16_t b) { return __builtin_bit_cast(float, (uint32_t)b << 16); }
__device__ __forceinline__ void split_bf16(float x, uint16_t& hi, uint16_t& lo) {
    const __bf16 h = (__bf16)x;
    hi = __builtin_bit_cast(uint16_t, h);
    lo = __builtin_bit_cast(uint16_t, (__bf16)(x - (float)h));
}
__device__ __forceinline__ _Float16 f16_sat(float x) { return (_Float16)fminf(fmaxf(x, -65504.f), 65504.f); }

// 24-bit V (opt-in): beside the f16 value the cache keeps the rounding residual r = x - f16(x) as the TOP BYTE
// of f16(r) -- an e5m2 number (sign, 5 exponent bits, 2 mantissa bits), rounded to nearest even.  |r| <= ulp/2, so the pair
// carries 13..14 significant bits, and the reader rebuilds r's f16 by a byte shift (no arithmetic).
__device__ __forceinline__ void store_v24(_Float16* v, uint8_t* vlo, int t_in_block, int d, int hd, float x);

// max of three without the canonicalising v_max_f32 x, x that fmaxf() adds per operand (operands here are MFMA results
// and finite constants: no signalling NaN to quiet)
__device__ __forceinline__ float max3_raw(float a, float b, float c) {
    float r;
    asm("v_max3_f32 %0, %1, %2, %3" : "=v"(r) : "v"(a), "v"(b), "v"(c));
    return r;
}

// SiluAndMul (src/layers/activation.rs:13-18) in the GEMM epilogues: x * sigmoid(x) * up with v_rcp_f32 (1 ulp) instead
// of an IEEE division (a dozen instructions per element: 1.5 us of a 256 x 192 tile's epilogue).  exp overflow gives
// rcp(inf) = 0, i.e. -0 for very negative gates; no NaN.  The fine-seam op keeps the division.
__device__ __forceinline__ float silu_mul(float g, float u) { return (g * __builtin_amdgcn_rcpf(1.0f + __expf(-g))) * u; }

__device__ __forceinline__ float relu2(float x) {
    x = fmaxf(x, 0.f);
    return x * x;
}

// x / 2 (1 + erf(x / sqrt 2)) with erfc by formula 7.1.26 of Abramowitz and Stegun, "Handbook of Mathematical Functions" (absolute error
// 1.5e-7): for f16 and bf16 hi + lo consumers
__device__ __forceinline__ float gelu_erf_fast(float x) {
    const float z = fabsf(x) * 0.7071067811865476f, t = __builtin_amdgcn_rcpf(1.0f + 0.3275911f * z);
    const float p = ((((1.061405429f * t - 1.453152027f) * t + 1.421413741f) * t - 0.284496736f) * t + 0.254829592f) * t;
    const float c = p * __expf(-z * z);  // erfc(z)
    return 0.5f * x * (x < 0.f ? c : 2.0f - c);
}
template <int ACT>
__device__ __forceinline__ float act_of(float x) {
    return ACT == ACT_GELU ? gelu_erf_fast(x) : relu2(x);
}

// 1 / 2 (1 + tanh a) = 1 / (1 + e^-2a): -2a of the tanh form of GELU
__device__ __forceinline__ float gelu_arg(float g) { return -1.5957691216057308f * (g + 0.044715f * g * g * g); }

// any GluSpec (uniform branch: the plain form costs nothing extra)
__device__ __forceinline__ float glu_mul(float g, float u, const GluSpec& s) {
    if (s.limit <= 0.f) {
        if (!s.gelu) return silu_mul(g, u);
        return g * __builtin_amdgcn_rcpf(1.0f + __expf(gelu_arg(g))) * u;
    }
    g = fminf(g, s.limit);
    u = fminf(fmaxf(u, -s.limit), s.limit);
    return (g * __builtin_amdgcn_rcpf(1.0f + __expf(-s.alpha * g))) * (u + s.shift);
}

// cap * tanh(v / cap) in the LM-head epilogues: tanh z = 1 - 2 / (exp(2z) + 1), absolute error about 1e-7 of the cap; an
// overflowing exponential gives 1, a vanishing one -1
__device__ __forceinline__ float soft_cap(float v, float cap) {
    const float z = v * __builtin_amdgcn_rcpf(cap);
    return cap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(__expf(2.0f * z) + 1.0f));
}

// log(1 + e^x) without overflow
__device__ __forceinline__ float softplusf(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// 16 bytes of a stream that THIS CU reads once per launch (a sequence's K/V in decode): non-temporal, so the lines do not
// displace what other kernels re-read from L2 / Infinity Cache (`global_load_dwordx4 ... nt`; guide, nt-weights row)
__device__ __forceinline__ uint4 ld_stream16(const void* p) {
    typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
    const u32x4 v = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p));
    return make_uint4(v[0], v[1], v[2], v[3]);
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
    return v;
}

// sum over the 16 lanes of a DPP row, in every lane
__device__ __forceinline__ float row16_sum(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x128, 0xf, 0xf, false));  // row_ror:8
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x124, 0xf, 0xf, false));  // row_ror:4
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x122, 0xf, 0xf, false));  // row_ror:2
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x121, 0xf, 0xf, false));  // row_ror:1
    return v;
}
// sum over the wave without LDS traffic, as a uniform value
__device__ __forceinline__ float wave_sum_uniform(float v) {
    const int x = __builtin_bit_cast(int, row16_sum(v));
    return (__builtin_bit_cast(float, __builtin_amdgcn_readlane(x, 0)) + __builtin_bit_cast(float, __builtin_amdgcn_readlane(x, 16))) +
           (__builtin_bit_cast(float, __builtin_amdgcn_readlane(x, 32)) + __builtin_bit_cast(float, __builtin_amdgcn_readlane(x, 48)));
}

// rinv[row] of a deferred RMSNorm (see RowNorm); 1 when the activations were normalised by the producer
__device__ __forceinline__ float rownorm_rinv(const RowNorm& rn, int row) {
    if (!rn.ssq) return 1.0f;
    float t = 0.f;
    for (int g = 0; g < rn.groups; ++g) t += rn.ssq[(size_t)g * rn.stride + row];
    return 1.0f / sqrtf(t * rn.inv_h + rn.eps);
}

// Workgroup-cooperative form for kernels whose epilogue needs rinv of up to NR rows: every thread sums a
// strided quarter of the groups of one row with independent (unrollable) loads and parks it in LDS;
// after any later barrier rownorm_rinv_lds() finishes the sum.  groups <= 64.
template <int NR>
__device__ __forceinline__ void rownorm_partials(const RowNorm& rn, int m0, int M, float* lds_part) {
    if (!rn.ssq) return;
    // every thread runs the loads (index clamped, only the LDS store is predicated): loads under a divergent branch
    // are serialised by the compiler, one vmcnt(0) round trip each
    for (int i0 = 0; i0 < 4 * NR; i0 += blockDim.x) {
        const int idx = i0 + (int)threadIdx.x;
        const int ic = min(idx, 4 * NR - 1);
        const int r = ic % NR, part = ic / NR;
        int row = min(m0 + r, M - 1);
        if (rn.row_idx) row = rn.row_idx[row];
        float v[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) v[i] = rn.ssq[(size_t)min(part + 4 * i, rn.groups - 1) * rn.stride + row];
        float t = 0.f;
#pragma unroll
        for (int i = 0; i < 16; ++i) t += (part + 4 * i) < rn.groups ? v[i] : 0.f;
        if (idx < 4 * NR) lds_part[part * NR + r] = t;
    }
}
template <int NR>
__device__ __forceinline__ float rownorm_rinv_lds(const RowNorm& rn, const float* lds_part, int r) {
    if (!rn.ssq) return 1.0f;
    const float t = lds_part[r] + lds_part[NR + r] + lds_part[2 * NR + r] + lds_part[3 * NR + r];
    return 1.0f / sqrtf(t * rn.inv_h + rn.eps);
}
// one row, one wave: lane g loads group g (groups <= 64)
__device__ __forceinline__ float rownorm_rinv_wave(const RowNorm& rn, int row, int lane) {
    if (!rn.ssq) return 1.0f;
    float t = lane < rn.groups ? rn.ssq[(size_t)lane * rn.stride + row] : 0.f;
    t = wave_sum(t);
    return 1.0f / sqrtf(t * rn.inv_h + rn.eps);
}

// hipFuncSetAttribute is per device: remember on which devices a kernel's dynamic-LDS limit has been raised
// (one bit per device ordinal; idempotent, so a race between two host threads only repeats the call)
static inline void ensure_dyn_lds(const void* fn, size_t lds, std::atomic<uint64_t>& done) {
    int dev = 0;
    (void)hipGetDevice(&dev);
    const uint64_t bit = 1ull << (dev & 63);
    if (!(done.load(std::memory_order_acquire) & bit)) {
        (void)hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        done.fetch_or(bit, std::memory_order_release);
    }
}

// KV-cache element offsets inside one (block, kv head) slab of kBlockTokens x hd f16:
// V in PV A-fragment order: token tt (0..31) of a 32-token tile sits in k-slot (g, j): tt<16: g=tt>>2, j=tt&3;
//   else g=(tt-16)>>2, j=4+(tt&3); element (tt, d) -> (((tile*(hd/16) + d/16)*64 + g*16 + d%16)*8 + j
// K in QK^T A-fragment order: 16-token tiles, each hd/32 chunks of 1 KiB: lane (g*16 + r) holds token r, dims 32c+8g..+7
__device__ __forceinline__ size_t k_packed_offset(int t_in_block, int d, int hd) {
    const int tt = t_in_block >> 4, r = t_in_block & 15;
    const int c = d >> 5, g = (d & 31) >> 3, j = d & 7;
    return ((size_t)(tt * (hd >> 5) + c) * 64 + (g << 4) + r) * 8 + j;
}

__device__ __forceinline__ size_t v_packed_offset(int t_in_block, int d, int hd) {
    const int tile = t_in_block >> 5, tt = t_in_block & 31;
    const int g = (tt & 15) >> 2, j = ((tt >> 4) << 2) | (tt & 3);
    return ((size_t)(tile * (hd >> 4) + (d >> 4)) * 64 + (g << 4) + (d & 15)) * 8 + j;
}

// 24-bit V: the residual bytes of TWO neighbouring PV fragments (features 32p..32p+15 and 32p+16..32p+31) share one 16-byte
// lane slot, [8 bytes of the even fragment][8 of the odd one], so the attention kernels fetch them with full 1 KiB wave-loads
// (512-byte loads cost the memory pipe as much per instruction as 1 KiB ones: measured +48 % kernel time for +25 % bytes).
// Byte offset inside one (block, kv head) slab of kBlockTokens x hd bytes:
__device__ __forceinline__ size_t vlo_packed_offset(int t_in_block, int d, int hd) {
    const int tile = t_in_block >> 5, tt = t_in_block & 31;
    const int g = (tt & 15) >> 2, j = ((tt >> 4) << 2) | (tt & 3);
    return ((size_t)(tile * (hd >> 5) + (d >> 5)) * 64 + (g << 4) + (d & 15)) * 16 + (size_t)(((d >> 4) & 1) << 3) + j;
}
__device__ __forceinline__ void store_v24(_Float16* v, uint8_t* vlo, int t_in_block, int d, int hd, float x) {
    const _Float16 h = f16_sat(x);
    v[v_packed_offset(t_in_block, d, hd)] = h;
    if (vlo) {
        const float xc = fminf(fmaxf(x, -65504.f), 65504.f);
        const uint32_t b = __builtin_bit_cast(uint16_t, (_Float16)(xc - (float)h));
        vlo[vlo_packed_offset(t_in_block, d, hd)] = (uint8_t)((b + 0x7Fu + ((b >> 8) & 1u)) >> 8);
    }
}

// 24-bit K (KvLayout::klo): the same residual byte per K element, two QK^T fragments (head-dim chunks c, c+1 of one 16-token
// tile) per 16-byte lane slot.  Byte offset inside one (block, kv head) slab of kBlockTokens x hd bytes:
__device__ __forceinline__ size_t klo_packed_offset(int t_in_block, int d, int hd) {
    const int tt = t_in_block >> 4, r = t_in_block & 15;
    const int c = d >> 5, g = (d & 31) >> 3, j = d & 7;
    return ((size_t)(tt * (hd >> 6) + (c >> 1)) * 64 + (g << 4) + r) * 16 + (size_t)((c & 1) << 3) + j;
}
__device__ __forceinline__ void store_k24(_Float16* k, uint8_t* klo, int t_in_block, int d, int hd, float x) {
    const _Float16 h = f16_sat(x);
    k[k_packed_offset(t_in_block, d, hd)] = h;
    if (klo) {
        const float xc = fminf(fmaxf(x, -65504.f), 65504.f);
        const uint32_t b = __builtin_bit_cast(uint16_t, (_Float16)(xc - (float)h));
        klo[klo_packed_offset(t_in_block, d, hd)] = (uint8_t)((b + 0x7Fu + ((b >> 8) & 1u)) >> 8);
    }
}

// eight consecutive elements summed over the slabs of a split-K product (only the first `left` exist, the others are 0);
// vector loads when the address allows
__device__ __forceinline__ void load_slabs8(float (&x)[8], const float* p, int left, int n_slabs, int64_t stride) {
    if (left >= 8 && ((reinterpret_cast<uintptr_t>(p) & 15) | (stride & 3)) == 0) {
        float4 u = *reinterpret_cast<const float4*>(p), v = *reinterpret_cast<const float4*>(p + 4);
        for (int sl0 = 1; sl0 < n_slabs; sl0 += 4) {  // independent loads (clamped index, masked sum)
            float4 a[4], b[4];
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const float* ps = p + (size_t)min(sl0 + q, n_slabs - 1) * stride;
                a[q] = *reinterpret_cast<const float4*>(ps);
                b[q] = *reinterpret_cast<const float4*>(ps + 4);
            }
#pragma unroll
            for (int q = 0; q < 4; ++q)
                if (sl0 + q < n_slabs) {
                    u.x += a[q].x; u.y += a[q].y; u.z += a[q].z; u.w += a[q].w;
                    v.x += b[q].x; v.y += b[q].y; v.z += b[q].z; v.w += b[q].w;
                }
        }
        x[0] = u.x; x[1] = u.y; x[2] = u.z; x[3] = u.w; x[4] = v.x; x[5] = v.y; x[6] = v.z; x[7] = v.w;
        return;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        x[j] = 0.f;
        if (j < left)
            for (int sl = 0; sl < n_slabs; ++sl) x[j] += p[(size_t)sl * stride + j];
    }
}

// s += the n partial sums of one float4, four independent loads per trip (clamped index, masked sum)
__device__ __forceinline__ void add_slabs(float4& s, const float* p, int n, int64_t stride) {
    if (n == 1) {
        const float4 t = *reinterpret_cast<const float4*>(p);
        s.x += t.x; s.y += t.y; s.z += t.z; s.w += t.w;
        return;
    }
    for (int sl0 = 0; sl0 < n; sl0 += 4) {
        float4 t[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) t[u] = *reinterpret_cast<const float4*>(p + (size_t)min(sl0 + u, n - 1) * stride);
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (sl0 + u < n) { s.x += t[u].x; s.y += t[u].y; s.z += t[u].z; s.w += t[u].w; }
    }
}
// one element of them
__device__ __forceinline__ float slab_elem(const float* p, int n_slabs, int64_t stride) {
    float v = p[0];
    for (int sl0 = 1; sl0 < n_slabs; sl0 += 4) {  // four independent loads per trip (clamped index, masked sum)
        float t[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) t[u] = p[(size_t)min(sl0 + u, n_slabs - 1) * stride];
#pragma unroll
        for (int u = 0; u < 4; ++u) v += sl0 + u < n_slabs ? t[u] : 0.f;
    }
    return v;
}

// four consecutive columns of one row (only the first `left` exist) as bf16 hi / lo, row-major or fragment order
__device__ __forceinline__ void put_planes4(uint16_t* ph, uint16_t* pl, int row, int col, int left, int ld, int packed, const f32x4& v) {
    uint16_t h[4], l[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) split_bf16(v[r], h[r], l[r]);
    if (left >= 4 && (col & 3) == 0) {
        const size_t o = packed ? xpack_off(row, col, ld >> 5) : (size_t)row * ld + col;
        *reinterpret_cast<uint2*>(ph + o) = make_uint2(h[0] | ((uint32_t)h[1] << 16), h[2] | ((uint32_t)h[3] << 16));
        *reinterpret_cast<uint2*>(pl + o) = make_uint2(l[0] | ((uint32_t)l[1] << 16), l[2] | ((uint32_t)l[3] << 16));
        return;
    }
    for (int r = 0; r < 4 && r < left; ++r) {
        const size_t o = packed ? xpack_off(row, col + r, ld >> 5) : (size_t)row * ld + col + r;
        ph[o] = h[r];
        pl[o] = l[r];
    }
}

// sum over the workgroup; red: one float per wave
__device__ __forceinline__ float block_sum(float v, float* red, int n_waves) {
    v = wave_sum(v);
    __syncthreads();  // red may still be read from an earlier sum
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    v = 0.f;
    for (int q = 0; q < n_waves; ++q) v += red[q];
    return v;
}

typedef const __attribute__((address_space(1))) void* gptr_t;
typedef __attribute__((address_space(3))) void* lptr_t;

// Diagnostic build (make stamps, -DNVLLM_STAMPS): in-kernel time stamps of the 100 MHz constant clock, one slot per
// (workgroup, wave, point); tools/stamp_timeline.py reads them.  Compiled out of the product library.
#ifdef NVLLM_STAMPS
#define NVLLM_STAMP(args_, idx_)                                                                                          \
    do {                                                                                                                  \
        if ((args_).stamps && (threadIdx.x & 63) == 0)                                                                    \
            (args_).stamps[(((size_t)blockIdx.x + (size_t)gridDim.x * (blockIdx.y + (size_t)gridDim.y * blockIdx.z)) * 16 + (threadIdx.x >> 6)) * 8 + (idx_)] = \
                __builtin_amdgcn_s_memrealtime();                                                                         \
    } while (0)
#else
#define NVLLM_STAMP(args_, idx_) do { } while (0)
#endif

// LDS reads beside an LDS-DMA in flight: hipcc waits for every outstanding global_load_lds before an ordinary LDS read (it cannot
// tell the buffers apart), which serialises the copy with the compute it should hide behind.  These reads are inline asm with counted
// waits: LDS returns in order, so LDS_WAIT(n) leaves at most the n youngest outstanding (anything else in flight only makes it wait longer).
#define NVLLM_LDS_READ128(DST_, ADDR_, OFF_) asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(DST_) : "v"(ADDR_), "n"(OFF_))
#define NVLLM_LDS_READ32(DST_, ADDR_) asm volatile("ds_read_b32 %0, %1" : "=v"(DST_) : "v"(ADDR_))
#define NVLLM_LDS_WAIT(N_)                                             \
    do {                                                               \
        asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(N_) : "memory");    \
        __builtin_amdgcn_sched_barrier(0);                             \
    } while (0)
__device__ __forceinline__ uint32_t lds_address(const void* p) { return (uint32_t)(uintptr_t)(lptr_t)p; }

// Barrier that PUBLISHES LDS-DMA data (global_load_lds): every wave first waits for its own DMA to land, then joins the
// barrier; only then may any wave ds_read fragments another wave staged.  __syncthreads() alone is not enough: hipcc
// (ROCm 7.2) emitted the loop-header barrier of gemm_kernel's chunk loop as `s_waitcnt lgkmcnt(0); s_barrier` with
// the vmcnt(0) AFTER the barrier -- each wave then waits for its own DMA only, and reads of another wave's still-in-
// flight fragments returned old LDS bytes (no stall, no fault): wrong sums under memory load (several contexts on one
// GPU), clean on a quiet chip.  The asm wait is invisible to the compiler's waitcnt pass and cannot be moved.
__device__ __forceinline__ void dma_publish_barrier() {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
}

}  // namespace nvllm
