// gfx950 kernels of the selective-scan mixer: short convolution rows, the scan of a decode step, the scan of prompt chunks.
#include <algorithm>

#include "device_common.h"
#include "scan.h"
#include "short_conv.h"

namespace nvllm {

// x / (1 + e^-x) with the hardware exponential and reciprocal (an ulp each): the argument's rounding costs |x| 2^-24 of e^-x
__device__ __forceinline__ float silu_fast(float x) { return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x * -1.4426950408889634f)); }

// ---------------------------------------------------------------------------------------------------
// convolution rows: four channels per thread
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ float4 conv_input4(const ConvRowsArgs& a, int row, int c) {
    const float* p = a.in + (size_t)row * a.ld + c;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c + 4 <= a.channels && ((a.ld | a.slab_stride) & 3) == 0) {
        add_slabs(v, p, a.n_slabs, a.slab_stride);
    } else {
        float t[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (c + e < a.channels) t[e] = slab_elem(p + e, a.n_slabs, a.slab_stride);
        v = make_float4(t[0], t[1], t[2], t[3]);
    }
    return v;
}
__device__ __forceinline__ float4 row4(const float* p, int c, int channels) {
    float t[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) t[e] = c + e < channels ? p[c + e] : 0.f;
    return make_float4(t[0], t[1], t[2], t[3]);
}
__device__ __forceinline__ void fma4(float4& y, const float4& x, const float4& w) { y.x += x.x * w.x; y.y += x.y * w.y; y.z += x.z * w.z; y.w += x.w * w.w; }
__device__ __forceinline__ void conv_out(const ConvRowsArgs& a, int row, int c, const float4& y) {
    const f32x4 v = {silu_fast(y.x), silu_fast(y.y), silu_fast(y.z), silu_fast(y.w)};
    const int left = a.channels - c;
    float* o = a.x + (size_t)row * a.ldx + c;
    if (left >= 4) *reinterpret_cast<float4*>(o) = make_float4(v[0], v[1], v[2], v[3]);
    else
        for (int e = 0; e < left; ++e) o[e] = v[e];
    if (a.xh) put_planes4(a.xh, a.xl, row, c, left, a.ldx, a.packed, v);
}

// any taps, any rows
__global__ void __launch_bounds__(256) conv_rows_kernel(ConvRowsArgs a) {
    const int row = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (c >= a.channels) return;
    const RowPast p = row_past(a, row);
    float4 y = row4(a.bias, c, a.channels);
    for (int i = 0; i < a.taps; ++i) {
        float t[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) t[e] = c + e < a.channels ? past_input(a, p, row, a.taps - 1 - i, c + e, a.channels) : 0.f;
        fma4(y, make_float4(t[0], t[1], t[2], t[3]), row4(a.conv + (size_t)i * a.channels, c, a.channels));
    }
    conv_out(a, row, c, y);
}
// decode: the window moves on by one token (this half of the history to the other one)
__global__ void __launch_bounds__(256) conv_decode_kernel(ConvRowsArgs a) {
    const int row = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (c >= a.channels) return;
    const int slot = a.slot[row], pos = a.pos[row], H = a.taps - 1;
    const float* past = a.history + ((size_t)(pos & 1) * a.slots + slot) * H * a.channels;
    float* next = a.history + ((size_t)((pos + 1) & 1) * a.slots + slot) * H * a.channels;
    const float4 cur = conv_input4(a, row, c);
    float4 y = row4(a.bias, c, a.channels);
    for (int i = 0; i < H; ++i) {
        float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
        if (pos >= H - i) x = row4(past + (size_t)i * a.channels, c, a.channels);
        fma4(y, x, row4(a.conv + (size_t)i * a.channels, c, a.channels));
        if (i > 0) {
            const float t[4] = {x.x, x.y, x.z, x.w};
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (c + e < a.channels) next[(size_t)(i - 1) * a.channels + c + e] = t[e];
        }
    }
    if (H > 0) {
        const float t[4] = {cur.x, cur.y, cur.z, cur.w};
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (c + e < a.channels) next[(size_t)(H - 1) * a.channels + c + e] = t[e];
    }
    fma4(y, cur, row4(a.conv + (size_t)H * a.channels, c, a.channels));
    conv_out(a, row, c, y);
}
// prompt chunks: a wave owns 16 rows x 32 channels, lane (grp, l15) row l15's eight consecutive channels: its plane stores in fragment
// order are one contiguous KiB
template <int TAPS>
__global__ void __launch_bounds__(256) conv_rows16_kernel(ConvRowsArgs a, int rows) {
    const int lane = threadIdx.x & 63, l15 = lane & 15, grp = lane >> 4;
    const int row0 = blockIdx.y * 16, row = min(row0 + l15, rows - 1), kt = blockIdx.x * 4 + (threadIdx.x >> 6), c = kt * 32 + grp * 8;
    if (kt * 32 >= a.channels) return;
    float y[8], w[8];
    auto eight = [&](float (&v)[8], const float* p, bool whole) {
        if (whole) {
            *reinterpret_cast<float4*>(&v[0]) = *reinterpret_cast<const float4*>(p);
            *reinterpret_cast<float4*>(&v[4]) = *reinterpret_cast<const float4*>(p + 4);
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = c + e < a.channels ? p[e] : 0.f;
        }
    };
    const bool whole = (a.channels & 7) == 0 && c < a.channels;
    eight(y, a.bias + c, whole);
    // the window of every row of the wave inside this chunk (a sequence's rows are consecutive)
    const int far = row - (TAPS - 1);
    const bool inside = far >= 0 && a.slot[max(far, 0)] == a.slot[row];
    if (__all(inside) && a.n_slabs == 1 && whole && (a.ld & 3) == 0) {
        float x[TAPS][8];
#pragma unroll
        for (int i = 0; i < TAPS; ++i) eight(x[i], a.in + (size_t)(far + i) * a.ld + c, true);
#pragma unroll
        for (int i = 0; i < TAPS; ++i) {
            eight(w, a.conv + (size_t)i * a.channels + c, true);
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] += x[i][e] * w[e];
        }
    } else {
        const RowPast p = row_past(a, row);
        for (int i = 0; i < TAPS; ++i) {
            eight(w, a.conv + (size_t)i * a.channels + c, whole);
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (c + e < a.channels) y[e] += past_input(a, p, row, TAPS - 1 - i, c + e, a.channels) * w[e];
        }
    }
    if (row0 + l15 >= rows) return;
#pragma unroll
    for (int e = 0; e < 8; ++e) y[e] = silu_fast(y[e]);
    float* o = a.x + (size_t)row * a.ldx + c;
    if (whole) {
        *reinterpret_cast<float4*>(o) = make_float4(y[0], y[1], y[2], y[3]);
        *reinterpret_cast<float4*>(o + 4) = make_float4(y[4], y[5], y[6], y[7]);
    } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
            if (c + e < a.channels) o[e] = y[e];
    }
    if (!a.xh) return;
    uint16_t h[8], l[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) split_bf16(c + e < a.channels ? y[e] : 0.f, h[e], l[e]);
    const size_t at = a.packed ? xpack_off(row, c, a.ldx >> 5) : (size_t)row * a.ldx + c;  // ldx is a multiple of 32: padding columns exist
    *reinterpret_cast<uint4*>(a.xh + at) = make_uint4(h[0] | ((uint32_t)h[1] << 16), h[2] | ((uint32_t)h[3] << 16), h[4] | ((uint32_t)h[5] << 16), h[6] | ((uint32_t)h[7] << 16));
    *reinterpret_cast<uint4*>(a.xl + at) = make_uint4(l[0] | ((uint32_t)l[1] << 16), l[2] | ((uint32_t)l[3] << 16), l[4] | ((uint32_t)l[5] << 16), l[6] | ((uint32_t)l[7] << 16));
}
hipError_t launch_conv_rows(const ConvRowsArgs& a, int rows, hipStream_t s) {
    if (a.taps < 1 || a.taps > kMaxTaps || a.channels > a.ld || a.channels > a.ldx || a.ldx % 32 || (a.taps > 1 && !a.history)) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const int bx = (a.channels + 1023) / 1024;
    if (a.seg.single) {
        conv_decode_kernel<<<dim3(bx, rows), 256, 0, s>>>(a);
        return hipGetLastError();
    }
    const dim3 grid((a.channels + 127) / 128, (rows + 15) / 16);
    if (rows >= 64 && a.taps == 4) conv_rows16_kernel<4><<<grid, 256, 0, s>>>(a, rows);
    else if (rows >= 64 && a.taps == 3) conv_rows16_kernel<3><<<grid, 256, 0, s>>>(a, rows);
    else if (rows >= 64 && a.taps == 2) conv_rows16_kernel<2><<<grid, 256, 0, s>>>(a, rows);
    else conv_rows_kernel<<<dim3(bx, rows), 256, 0, s>>>(a);
    return hipGetLastError();
}
hipError_t launch_conv_history(const ConvRowsArgs& a, hipStream_t s) {
    if (a.seg.single || a.taps > kMaxTaps) return hipErrorInvalidValue;
    if (a.taps < 2 || a.seg.count <= 0) return hipSuccess;
    conv_history_kernel<<<dim3((a.channels + 255) / 256, a.seg.count), 256, 0, s>>>(a, a.channels);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// scan: a lane holds NS states of one channel, NL neighbouring lanes the channel
// ---------------------------------------------------------------------------------------------------
template <int NL>
__device__ __forceinline__ float lanes_sum(float v) {
#define NVLLM_DPP(C_) v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), C_, 0xf, 0xf, false))
    if constexpr (NL >= 2) NVLLM_DPP(0xB1);   // quad_perm 1,0,3,2
    if constexpr (NL >= 4) NVLLM_DPP(0x4E);   // quad_perm 2,3,0,1
    if constexpr (NL >= 8) NVLLM_DPP(0x141);  // row_half_mirror
    if constexpr (NL >= 16) NVLLM_DPP(0x140); // row_mirror
#undef NVLLM_DPP
    if constexpr (NL >= 32) v += __shfl_xor(v, 16);
    if constexpr (NL >= 64) v += __shfl_xor(v, 32);
    return v;
}
template <int NS>
__device__ __forceinline__ void load_states(float (&v)[NS], const float* p) {
#pragma unroll
    for (int i = 0; i < NS; i += 4) {
        const float4 t = *reinterpret_cast<const float4*>(p + i);
        v[i] = t.x; v[i + 1] = t.y; v[i + 2] = t.z; v[i + 3] = t.w;
    }
}
template <int NS>
__device__ __forceinline__ void store_states(float* p, const float (&v)[NS]) {
#pragma unroll
    for (int i = 0; i < NS; i += 4) *reinterpret_cast<float4*>(p + i) = make_float4(v[i], v[i + 1], v[i + 2], v[i + 3]);
}
__device__ __forceinline__ void put_row4(const ScanArgs& a, int row, int c, const f32x4& v) {
    const int left = a.channels - c;
    if (left <= 0) return;
    if (a.oh) put_planes4(a.oh, a.ol, row, c, left, a.ld, a.packed, v);
    if (a.of)
        for (int e = 0; e < min(4, left); ++e) a.of[(size_t)row * a.ld + c + e] = v[e];
}

template <int NS, int NL>
__global__ void __launch_bounds__(256) scan_decode_kernel(ScanArgs a) {
    constexpr int CH = 256 / NL;
    __shared__ float ys[CH < 4 ? 4 : CH];
    const int row = blockIdx.y, q = threadIdx.x % NL, lc = threadIdx.x / NL, c = blockIdx.x * CH + lc;
    const size_t at = (size_t)c * a.states + q * NS;
    float* st = a.state + (size_t)a.slot[row] * a.channels_p * a.states + at;
    float S[NS], A[NS], B[NS], C[NS];
    load_states(S, st);
    load_states(A, a.A + at);
    const float* bc = a.bc + (size_t)row * a.ldbc + q * NS;
    load_states(B, bc + a.b0);
    load_states(C, bc + a.c0);
    const int cc = min(c, a.channels - 1);
    const float x = a.x[(size_t)row * a.ldx + cc], dt = a.dt[(size_t)row * a.channels_p + c];
    const float z = slab_elem(a.z + (size_t)row * a.ldz + cc, a.z_slabs, a.z_stride);
    const bool fresh = a.pos[row] == 0;
    const float dx = dt * x;
    float y = 0.f;
#pragma unroll
    for (int i = 0; i < NS; ++i) {
        S[i] = (fresh ? 0.f : S[i]) * __builtin_amdgcn_exp2f(dt * A[i]) + dx * B[i];
        y += S[i] * C[i];
    }
    store_states(st, S);
    y = lanes_sum<NL>(y);
    if (q == 0) ys[lc] = (y + a.D[c] * x) * silu_fast(z);
    __syncthreads();
    if ((int)threadIdx.x * 4 < CH) put_row4(a, row, blockIdx.x * CH + threadIdx.x * 4, f32x4{ys[threadIdx.x * 4], ys[threadIdx.x * 4 + 1], ys[threadIdx.x * 4 + 2], ys[threadIdx.x * 4 + 3]});
}

// one workgroup: CH channels of one piece, TB tokens at a time staged through LDS, the next TB on their way in registers
template <int NS, int NL, int TB, bool CARRY>
__global__ void __launch_bounds__(256) scan_prompt_kernel(ScanArgs a) {
    constexpr int CH = 256 / NL, ST = NS * NL, NX = (TB * CH + 255) / 256, NB = (TB * 2 * ST + 255) / 256;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float *bcs = sm, *xs = bcs + TB * 2 * ST, *dts = xs + TB * CH, *zs = dts + TB * CH;  // zs becomes the output
    const int tid = threadIdx.x, q = tid % NL, lc = tid / NL, c0 = blockIdx.x * CH, c = c0 + lc;
    const int piece = blockIdx.y, k = a.piece_at[piece], of = a.piece_of[piece];
    const int row0 = a.piece_row0[piece], n = a.piece_n[piece];
    const size_t at = (size_t)c * a.states + q * NS, per = (size_t)a.channels_p * a.states;
    float* st = a.state + (size_t)a.piece_slot[piece] * per + at;
    float S[NS], A[NS];
    if (CARRY && k == 0 && of > 1) {  // the state before the segment, out of the last piece's way
        load_states(S, st);
        if (a.pos[row0] == 0) {
#pragma unroll
            for (int i = 0; i < NS; ++i) S[i] = 0.f;
        }
        store_states(a.carry + (size_t)piece * per + at, S);
    }
    if (CARRY && k == of - 1) return;
    load_states(A, a.A + at);
    [[maybe_unused]] float D = 0.f;
    if constexpr (!CARRY) D = a.D[c];
#pragma unroll
    for (int i = 0; i < NS; ++i) S[i] = 0.f;
    float total = 0.f;
    if constexpr (!CARRY) {
        if (of == 1) {
            if (a.pos[row0] != 0) load_states(S, st);
        } else {
            load_states(S, a.carry + (size_t)(piece - k) * per + at);
            for (int j = 1; j <= k; ++j) {
                float E[NS];
                load_states(E, a.carry + (size_t)(piece - k + j) * per + at);
                const float d = a.carry_dt[(size_t)(piece - k + j) * a.channels_p + c];
#pragma unroll
                for (int i = 0; i < NS; ++i) S[i] = S[i] * __builtin_amdgcn_exp2f(d * A[i]) + E[i];
            }
        }
    }
    float rx[NX], rd[NX], rz[NX], rb[NB];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NX; ++i) {
            const int e = tid + i * 256, t = min(t0 + e / CH, n - 1), ch = min(c0 + e % CH, a.channels - 1);
            const size_t row = row0 + t;
            rx[i] = a.x[row * a.ldx + ch];
            rd[i] = a.dt[row * a.channels_p + ch];
            if constexpr (!CARRY) rz[i] = slab_elem(a.z + row * a.ldz + ch, a.z_slabs, a.z_stride);
        }
#pragma unroll
        for (int i = 0; i < NB; ++i) {
            const int e = tid + i * 256, t = min(t0 + e / (2 * ST), n - 1), j = e % (2 * ST);
            rb[i] = a.bc[(size_t)(row0 + t) * a.ldbc + (j < ST ? a.b0 + j : a.c0 + j - ST)];
        }
    };
    fetch(0);
    for (int t0 = 0; t0 < n; t0 += TB) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < NX; ++i) {
            const int e = tid + i * 256;
            if (TB * CH % 256 && e >= TB * CH) continue;
            xs[e] = rx[i];
            dts[e] = rd[i];
            if constexpr (!CARRY) zs[e] = rz[i];
        }
#pragma unroll
        for (int i = 0; i < NB; ++i) {
            const int e = tid + i * 256;
            if (TB * 2 * ST % 256 == 0 || e < TB * 2 * ST) bcs[e] = rb[i];
        }
        __syncthreads();
        if (t0 + TB < n) fetch(t0 + TB);
        const int m = min(TB, n - t0);
        // U tokens at a time: everything but the state's own chain is independent.  Tokens past the end have dt = 0: the state stays.
        constexpr int U = NS == 4 ? 4 : 1;
        for (int t = 0; t < m; t += U) {
            float dt[U], x[U], dx[U], B[U][NS], C[U][NS], y[U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int tt = t + u;
                dt[u] = tt < m ? dts[tt * CH + lc] : 0.f;
                x[u] = xs[tt * CH + lc];
                dx[u] = dt[u] * x[u];
                load_states(B[u], bcs + tt * 2 * ST + q * NS);
                if constexpr (!CARRY) load_states(C[u], bcs + tt * 2 * ST + ST + q * NS);
            }
#pragma unroll
            for (int u = 0; u < U; ++u) {
                y[u] = 0.f;
#pragma unroll
                for (int i = 0; i < NS; ++i) {
                    S[i] = S[i] * __builtin_amdgcn_exp2f(dt[u] * A[i]) + dx[u] * B[u][i];
                    if constexpr (!CARRY) y[u] += S[i] * C[u][i];
                }
                if constexpr (CARRY) total += dt[u];
            }
            if constexpr (!CARRY) {
#pragma unroll
                for (int u = 0; u < U; ++u) {
                    y[u] = lanes_sum<NL>(y[u]);
                    if (q == 0) xs[(t + u) * CH + lc] = y[u] + D * x[u];  // this channel's x there has been read by its lanes' wave
                }
            }
        }
        if constexpr (!CARRY) {
            __syncthreads();
            for (int e = tid * 4; e < m * CH; e += 1024) {
                const int t = e / CH, ch = e % CH;
                const size_t row = row0 + t0 + t;
                f32x4 v;
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = xs[e + r] * silu_fast(zs[e + r]);
                put_row4(a, (int)row, c0 + ch, v);
            }
        }
    }
    if constexpr (CARRY) {
        store_states(a.carry + (size_t)(piece + 1) * per + at, S);
        if (q == 0) a.carry_dt[(size_t)(piece + 1) * a.channels_p + c] = total;
    } else {
        if (k == of - 1) store_states(st, S);
    }
}

static bool scan_args_ok(const ScanArgs& a) {
    return a.states >= 4 && a.states <= kMaxScanStates && (a.states & (a.states - 1)) == 0 && a.channels_p % scan_channels(a.states) == 0 && a.channels <= a.channels_p && a.channels <= a.ldx &&
           (a.oh || a.of) && a.ld >= a.channels && a.b0 % 4 == 0 && a.c0 % 4 == 0 && a.ldbc % 4 == 0 && a.ldbc >= std::max(a.b0, a.c0) + a.states;
}
#define NVLLM_SCAN_SIZES(X_) X_(4, 1, 32) X_(4, 2, 32) X_(4, 4, 32) X_(4, 8, 32) X_(4, 16, 32) X_(4, 32, 16) X_(4, 64, 16) X_(8, 64, 8) X_(16, 64, 8)
hipError_t launch_scan_decode(const ScanArgs& a, int rows, hipStream_t s) {
    if (!scan_args_ok(a)) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
#define NVLLM_SD(NS_, NL_, TB_) \
    if (a.states == NS_ * NL_) scan_decode_kernel<NS_, NL_><<<dim3(a.channels_p / (256 / NL_), rows), 256, 0, s>>>(a);
    NVLLM_SCAN_SIZES(NVLLM_SD)
#undef NVLLM_SD
    return hipGetLastError();
}
template <int NS, int NL, int TB>
static void scan_prompt(const ScanArgs& a, hipStream_t s) {
    constexpr int CH = 256 / NL;
    const size_t lds = (size_t)TB * (2 * NS * NL + 3 * CH) * 4;
    static std::atomic<uint64_t> set0{0}, set1{0};
    ensure_dyn_lds(reinterpret_cast<const void*>(scan_prompt_kernel<NS, NL, TB, true>), lds, set0);
    ensure_dyn_lds(reinterpret_cast<const void*>(scan_prompt_kernel<NS, NL, TB, false>), lds, set1);
    const dim3 grid(a.channels_p / CH, a.pieces);
    if (a.several) scan_prompt_kernel<NS, NL, TB, true><<<grid, 256, lds, s>>>(a);
    scan_prompt_kernel<NS, NL, TB, false><<<grid, 256, lds, s>>>(a);
}
hipError_t launch_scan_prompt(const ScanArgs& a, hipStream_t s) {
    if (!scan_args_ok(a) || (a.several && (!a.carry || !a.carry_dt)) || a.pieces > 65535) return hipErrorInvalidValue;
    if (a.pieces <= 0) return hipSuccess;
#define NVLLM_SP(NS_, NL_, TB_) if (a.states == NS_ * NL_) scan_prompt<NS_, NL_, TB_>(a, s);
    NVLLM_SCAN_SIZES(NVLLM_SP)
#undef NVLLM_SP
    return hipGetLastError();
}

}  // namespace nvllm
