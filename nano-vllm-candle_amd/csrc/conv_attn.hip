// gfx950 row kernels of attention with short convolutions: between the fused q / k / v projection and the attention kernels (bias_attn.hip).
// One wave per unit of a row -- a query head, a key head or a value head -- lane d % 64 holds channel d: causal convolution over the
// biased projections, rotation of neighbouring channels (neighbouring lanes), RMS norm over the head, then the query buffer or the cache.
#include <algorithm>

#include "device_common.h"
#include "hybrid.h"
#include "short_conv.h"

namespace nvllm {

typedef __attribute__((ext_vector_type(4))) _Float16 f16x4;

struct Unit {
    int kind, head, c0, n;  // kind: 0 query, 1 key, 2 value; first channel and number of channels
};
__device__ __forceinline__ Unit unit_of(const ConvAttnRowsArgs& a, int u) {
    const int kv = a.kv.kv;
    if (u < a.heads) return {0, u, u * a.kv.dim, a.kv.dim};
    if (u < a.heads + kv) return {1, u - a.heads, u * a.kv.dim, a.kv.dim};
    const int h = u - a.heads - kv;
    return {2, h, (a.heads + kv) * a.kv.dim + h * a.kv.vdim, a.kv.vdim};
}
__device__ __forceinline__ float neighbour(float v) {  // lane ^ 1
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xb1, 0xf, 0xf, false));  // quad_perm [1, 0, 3, 2]
}
__device__ __forceinline__ size_t kv_block(const ConvAttnRowsArgs& a, int slot, int pos, int head) {
    return (size_t)a.block_tables[(size_t)slot * a.max_blocks + pos / kBlockTokens] * a.kv.kv + head;
}
__device__ __forceinline__ void put(void* base, int f32, size_t o, float v) {
    if (f32) reinterpret_cast<float*>(base)[o] = v;
    else reinterpret_cast<_Float16*>(base)[o] = f16_sat(v);
}
// rotation and norm of a query or key head
template <int NE>
__device__ __forceinline__ void turn(const ConvAttnRowsArgs& a, int pos, int lane, float (&y)[NE], float scale) {
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < NE; ++e) {
        const int d = e * 64 + lane;
        const float other = neighbour(y[e]);
        if (d < a.rot) {
            const size_t t = (size_t)pos * (a.rot >> 1) + (d >> 1);
            const float s = a.sin[t];
            y[e] = y[e] * a.cos[t] + (d & 1 ? other : -other) * s;
        }
        ss += y[e] * y[e];
    }
    const float f = scale / sqrtf(wave_sum_uniform(ss) / (float)a.kv.dim + a.eps);
#pragma unroll
    for (int e = 0; e < NE; ++e) y[e] *= f;
}
// a finished unit of one row (channels past the head are 0)
template <int NE>
__device__ __forceinline__ void finish(const ConvAttnRowsArgs& a, const Unit& u, int row, int slot, int pos, int lane, float (&y)[NE]) {
    if (u.kind < 2) turn<NE>(a, pos, lane, y, u.kind ? 1.f : a.q_scale);
    if (u.kind == 0) {
        float* q = a.q + ((size_t)row * a.heads + u.head) * a.kv.dim_p;
#pragma unroll
        for (int e = 0; e < NE; ++e)
            if (e * 64 + lane < a.kv.dim_p) q[e * 64 + lane] = y[e];
        return;
    }
    const size_t blk = kv_block(a, slot, pos, u.head) * kBlockTokens;
    const int t = pos & (kBlockTokens - 1);
#pragma unroll
    for (int e = 0; e < NE; ++e) {
        const int d = e * 64 + lane;
        if (d >= u.n) continue;
        if (u.kind == 1) put(a.kv.k, a.kv.f32, blk * a.kv.dim_p + k_packed_offset(t, d, a.kv.dim_p), y[e]);
        else put(a.kv.v, a.kv.f32, blk * a.kv.vdim_p + v_packed_offset(t, d, a.kv.vdim_p), y[e]);
    }
}

// decode rows (TAPS known): every input is read once, for the convolution and for the history's next half
template <int TAPS, int NE>
__global__ void __launch_bounds__(256) conv_attn_decode_kernel(ConvAttnRowsArgs a) {
    const int lane = threadIdx.x & 63, row = blockIdx.x, unit = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    if (unit >= a.units()) return;
    const Unit u = unit_of(a, unit);
    const int channels = a.channels(), slot = a.slot[row], pos = a.pos[row];
    const float* in = a.in + (size_t)row * a.ld + u.c0;
    const float* past = a.history + ((size_t)(pos & 1) * a.slots + slot) * (TAPS - 1) * channels + u.c0;
    float* next = a.history + ((size_t)((pos + 1) & 1) * a.slots + slot) * (TAPS - 1) * channels + u.c0;
    float x[TAPS][NE], y[NE];
#pragma unroll
    for (int e = 0; e < NE; ++e) {
        const int d = min(e * 64 + lane, u.n - 1);
        x[TAPS - 1][e] = slab_elem(in + d, a.n_slabs, a.slab_stride) + (a.in_bias ? a.in_bias[u.c0 + d] : 0.f);
#pragma unroll
        for (int i = 0; i < TAPS - 1; ++i) {
            const float h = past[(size_t)i * channels + d];
            x[i][e] = pos >= TAPS - 1 - i ? h : 0.f;
        }
    }
#pragma unroll
    for (int e = 0; e < NE; ++e) {
        const int d = e * 64 + lane, dc = min(d, u.n - 1);
        float t = 0.f;
#pragma unroll
        for (int i = 0; i < TAPS; ++i) t += x[i][e] * a.conv[(size_t)i * channels + u.c0 + dc];
        y[e] = d < u.n ? t : 0.f;
        if (d < u.n) {
#pragma unroll
            for (int i = 0; i < TAPS - 1; ++i) next[(size_t)i * channels + d] = x[i + 1][e];
        }
    }
    finish<NE>(a, u, row, slot, pos, lane, y);
}

// any rows and taps; decode rows leave the next history too
template <int NE>
__global__ void __launch_bounds__(256) conv_attn_rows_kernel(ConvAttnRowsArgs a) {
    const int lane = threadIdx.x & 63, row = blockIdx.x, unit = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    if (unit >= a.units()) return;
    const Unit u = unit_of(a, unit);
    const int channels = a.channels();
    RowPast p;
    if (a.seg.single) {
        p.slot = a.slot[row];
        p.pos0 = a.pos[row];
    } else {
        p = row_past(a, row);
    }
    float y[NE];
#pragma unroll
    for (int e = 0; e < NE; ++e) {
        const int d = e * 64 + lane, c = u.c0 + min(d, u.n - 1);
        float t = 0.f;
        for (int i = 0; i < a.taps; ++i) t += past_input(a, p, row, a.taps - 1 - i, c, channels) * a.conv[(size_t)i * channels + c];
        y[e] = d < u.n ? t : 0.f;
    }
    if (a.seg.single) {
        float* next = a.history + ((size_t)((p.pos0 + 1) & 1) * a.slots + p.slot) * (a.taps - 1) * channels;
        for (int i = 0; i < a.taps - 1; ++i)
            for (int d = lane; d < u.n; d += 64) next[(size_t)i * channels + u.c0 + d] = past_input(a, p, row, a.taps - 2 - i, u.c0 + d, channels);
    }
    finish<NE>(a, u, row, p.slot, a.pos[row], lane, y);
}

// prompt chunks: one wave per (16 rows, unit), the inputs of the block and of the tokens before it in registers.  Values of four
// consecutive tokens are neighbours in the cache.
template <int TAPS, int NE>
__global__ void __launch_bounds__(256) conv_attn_rows16_kernel(ConvAttnRowsArgs a, int rows) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int row0 = blockIdx.x * 16, row1 = min(row0 + 16, rows);
    if (unit >= a.units()) return;
    const Unit u = unit_of(a, unit);
    const int channels = a.channels();
    float w[TAPS][NE], bias[NE];
#pragma unroll
    for (int e = 0; e < NE; ++e) {
        const int c = u.c0 + min(e * 64 + lane, u.n - 1);
        const bool in = e * 64 + lane < u.n;
        bias[e] = in && a.in_bias ? a.in_bias[c] : 0.f;
#pragma unroll
        for (int i = 0; i < TAPS; ++i) w[i][e] = in ? a.conv[(size_t)i * channels + c] : 0.f;
    }
    bool plain = row0 + 16 <= rows && row0 >= TAPS - 1 && a.n_slabs == 1;  // one sequence, its window inside the chunk
    if (plain)
        for (int r = -(TAPS - 1); r < 15; ++r) plain &= a.slot[row0 + r] == a.slot[row0 + 15];
    if (plain) {
        float z[15 + TAPS][NE];
        const float* in = a.in + (size_t)(row0 - (TAPS - 1)) * a.ld + u.c0;
#pragma unroll
        for (int r = 0; r < 15 + TAPS; ++r)
#pragma unroll
            for (int e = 0; e < NE; ++e) z[r][e] = in[(size_t)r * a.ld + min(e * 64 + lane, u.n - 1)] + bias[e];
        const int slot = a.slot[row0], pos0 = a.pos[row0];
        if (u.kind == 2 && !a.kv.f32 && (pos0 & 3) == 0) {
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const int pos = pos0 + g * 4;
                const size_t blk = kv_block(a, slot, pos, u.head) * kBlockTokens * a.kv.vdim_p;
#pragma unroll
                for (int e = 0; e < NE; ++e) {
                    float v[4];
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        v[r] = 0.f;
#pragma unroll
                        for (int i = 0; i < TAPS; ++i) v[r] += z[g * 4 + r + i][e] * w[i][e];
                    }
                    if (e * 64 + lane < u.n)
                        *reinterpret_cast<f16x4*>(reinterpret_cast<_Float16*>(a.kv.v) + blk + v_packed_offset(pos & (kBlockTokens - 1), e * 64 + lane, a.kv.vdim_p)) =
                            f16x4{f16_sat(v[0]), f16_sat(v[1]), f16_sat(v[2]), f16_sat(v[3])};
                }
            }
            return;
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            float y[NE];
#pragma unroll
            for (int e = 0; e < NE; ++e) {
                y[e] = 0.f;
#pragma unroll
                for (int i = 0; i < TAPS; ++i) y[e] += z[r + i][e] * w[i][e];
            }
            finish<NE>(a, u, row0 + r, slot, pos0 + r, lane, y);
        }
        return;
    }
    float x[TAPS][NE];
    for (int row = row0; row < row1; ++row) {
        const int slot = a.slot[row];
        if (row == row0 || a.slot[row - 1] != slot) {
            const RowPast p = row_past(a, row);
#pragma unroll
            for (int j = 1; j < TAPS; ++j)
#pragma unroll
                for (int e = 0; e < NE; ++e) x[TAPS - 1 - j][e] = past_input(a, p, row, j, u.c0 + min(e * 64 + lane, u.n - 1), channels);
        } else {
#pragma unroll
            for (int i = 0; i < TAPS - 1; ++i)
#pragma unroll
                for (int e = 0; e < NE; ++e) x[i][e] = x[i + 1][e];
        }
        float y[NE];
#pragma unroll
        for (int e = 0; e < NE; ++e) {
            x[TAPS - 1][e] = slab_elem(a.in + (size_t)row * a.ld + u.c0 + min(e * 64 + lane, u.n - 1), a.n_slabs, a.slab_stride) + bias[e];
            y[e] = 0.f;
#pragma unroll
            for (int i = 0; i < TAPS; ++i) y[e] += x[i][e] * w[i][e];
        }
        finish<NE>(a, u, row, slot, a.pos[row], lane, y);
    }
}

template <int NE>
static hipError_t conv_attn_t(const ConvAttnRowsArgs& a, int rows, hipStream_t s) {
    const int wgs = (a.units() + 3) / 4;
#define NVLLM_CA(T_)                                                                                                                  \
    case T_:                                                                                                                          \
        if (a.seg.single) conv_attn_decode_kernel<T_, NE><<<dim3(rows, wgs), 256, 0, s>>>(a);                                         \
        else conv_attn_rows16_kernel<T_, NE><<<dim3((rows + 15) / 16, wgs), 256, 0, s>>>(a, rows);                                    \
        return hipGetLastError();
    if (a.seg.single || (rows >= 64 && NE <= 4)) {
        if constexpr (NE <= 4) {
            switch (a.taps) { NVLLM_CA(1) NVLLM_CA(2) NVLLM_CA(3) NVLLM_CA(4) }
        }
    }
#undef NVLLM_CA
    conv_attn_rows_kernel<NE><<<dim3(rows, wgs), 256, 0, s>>>(a);
    return hipGetLastError();
}
hipError_t launch_conv_attn_rows(const ConvAttnRowsArgs& a, int rows, hipStream_t s) {
    const int widest = std::max(a.kv.dim_p, a.kv.vdim);
    if (a.heads < 1 || a.kv.kv < 1 || a.heads % a.kv.kv || a.kv.dim_p % 32 || a.kv.vdim_p % 16 || a.taps < 1 || a.taps > kMaxTaps || a.channels() > a.ld || a.rot % 2 || a.rot > a.kv.dim ||
        (a.rot && (!a.cos || !a.sin)) || (a.taps > 1 && !a.history))
        return hipErrorInvalidValue;
    if (widest > kConvAttnDim) return hipErrorNotSupported;
    if (rows <= 0) return hipSuccess;
    if (widest <= 64) return conv_attn_t<1>(a, rows, s);
    if (widest <= 128) return conv_attn_t<2>(a, rows, s);
    if (widest <= 256) return conv_attn_t<4>(a, rows, s);
    return conv_attn_t<8>(a, rows, s);
}
hipError_t launch_conv_attn_history(const ConvAttnRowsArgs& a, hipStream_t s) {
    if (a.seg.single || a.taps > kMaxTaps) return hipErrorInvalidValue;
    if (a.taps < 2 || a.seg.count <= 0) return hipSuccess;
    conv_history_kernel<<<dim3((a.channels() + 255) / 256, a.seg.count), 256, 0, s>>>(a, a.channels());
    return hipGetLastError();
}

}  // namespace nvllm
