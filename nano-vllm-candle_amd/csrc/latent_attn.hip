// Matrix-core attention over the latent cache, absorbed form (gfx950): the query has been carried into latent space, so one cached
// vector per token serves every head, as key (latent and rotated part) and as value (latent part).
//
// One workgroup = 16 (token, head) query rows of one sequence (sub-tile of a q-tile) x a range of 32-token tiles of the cache; four
// waves (S = 1) or four pairs of waves (S = 2) take alternate tiles and are combined through LDS at the end.
//   S^T[token][row] = K[token][:] . q[row][:]        A = cache fragment as stored, B = q fragment (f16 hi + lo, from LDS)
//   O^T[d][row]    += C^T[d][token] . P[token][row]  A = the SAME cache fragment, transposed by the matrix core, B = P (hi + lo)
// Transposing: (16 tokens x 32 d) . (selection of 16 of the 32 d) leaves D[token 4g + r][d l15] in lane (g, l15) -- the A-fragment
// order of C^T for those tokens, exact since a product with 1 changes nothing.  The cache is read once and stored once; a value
// copy in transposed order would nearly double the bytes a decode step reads.
// S = 2 (latents above 256): each wave of a pair owns half of the latent's chunks, for scores (partial sums exchanged through LDS)
// and for values; a single wave would keep 128 accumulators and a 36 KiB tile and spend its time moving them to and from AGPRs.
#include <algorithm>

#include "device_common.h"
#include "latent.h"

namespace nvllm {

__device__ __forceinline__ f16x8 selection_frag(int grp, int l15, int half) {
    f16x8 s;
#pragma unroll
    for (int j = 0; j < 8; ++j) s[j] = (_Float16)(8 * grp + j == l15 + 16 * half ? 1.f : 0.f);
    return s;
}

// KW: latent chunks (32 elements) per wave, RC: rotated chunks of the cache row, S: waves sharing a tile
template <int KW, int RC, int S>
__global__ void __launch_bounds__(256 * S, 2) latent_attn_kernel(LatentAttnArgs a) {
    constexpr int KC = KW * S, DC = KC + RC;          // chunks of a cache row
    constexpr int RW = (RC + S - 1) / S, QW = KW + RW;  // rotated / all chunks a wave works on
    constexpr int G = 8 / S;                            // output tiles per wave and combine pass
    constexpr int kQ = 2 * S * QW * 64, kO = 4 * S * G * 64;
    __shared__ __attribute__((aligned(16))) uint4 lds[kQ > kO ? kQ : kO];
    __shared__ __attribute__((aligned(16))) f32x4 xch[S == 2 ? 2 * 8 * 2 * 64 : 1];
    __shared__ float ml[4][2][16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int pair = wave / S, part = wave % S;
    const int l15 = lane & 15, grp = lane >> 4;
    // decode: q-tile i is row i (no tile list to wait for)
    const int tile = blockIdx.x, row0 = a.single ? tile : a.tile_row0[tile], total = (a.single ? 1 : a.tile_nrows[tile]) * a.heads;
    const int slot = a.single ? a.slot[tile] : a.tile_slot[tile];
    const int f0 = blockIdx.y * 16;
    if (f0 >= total) return;
    const int pos0 = a.pos[row0];
    const int flat = min(f0 + l15, total - 1);
    const int tok = flat / a.heads, head = flat - tok * a.heads;
    const bool valid = f0 + l15 < total;
    const int my_pos = valid ? pos0 + tok : -1;
    const int my_first = a.window > 0 ? my_pos - a.window + 1 : 0;
    const int pmin = pos0 + f0 / a.heads, pmax = pos0 + min(f0 + 15, total - 1) / a.heads;
    const int t_lo = a.window > 0 ? max(0, pmin - a.window + 1) >> 5 : 0, t_hi = (pmax >> 5) + 1;
    const int t_begin = a.part_tiles ? t_lo + (int)blockIdx.z * a.part_tiles : t_lo;
    const int t_end = a.part_tiles ? min(t_hi, t_begin + a.part_tiles) : t_hi;
    if (t_begin >= t_hi) return;
    const int* bt = a.block_tables + (size_t)slot * a.max_blocks;
    const _Float16* data = reinterpret_cast<const _Float16*>(a.cache.data);
    constexpr size_t kBlockElems = (size_t)kBlockTokens * DC * 32;
    // chunk i of this wave in the cache row; a pair's second wave has no rotated chunk when RC is 1: it re-reads the first (q is zero)
    auto chunk = [&](int i) { return i < KW ? part * KW + i : KC + min(part * RW + (i - KW), RC - 1); };
    // the two 16-token fragment sets of 32-token tile t: 2 * DC contiguous KiB
    auto tile_ptr = [&](int t) { return data + (size_t)bt[t >> 3] * kBlockElems + (size_t)(t & 7) * (2 * DC * 512) + lane * 8; };
    // loads in the order they are needed: the query (split to f16 hi + lo and shared through LDS), then this wave's first tile
    constexpr int QI = (S * QW + 4 * S - 1) / (4 * S);
    float qx[QI][8];
    {
        const float* ql = a.qlat + ((size_t)(row0 + tok) * a.heads + head) * (KC * 32) + grp * 8;
        const float* qr = a.qrot + (size_t)(row0 + tok) * a.qrot_row + (size_t)head * a.qrot_head + grp * 8;
#pragma unroll
        for (int i = 0; i < QI; ++i) {
            const int c = min(wave + i * 4 * S, S * QW - 1), r = min(c - KC, RC - 1);  // slot order: latent chunks, then rotated ones
            const float* p = c < KC ? ql + c * 32 : qr + r * 32;
            *reinterpret_cast<float4*>(&qx[i][0]) = *reinterpret_cast<const float4*>(p);
            *reinterpret_cast<float4*>(&qx[i][4]) = *reinterpret_cast<const float4*>(p + 4);
        }
    }
    uint4 ka[QW], kb[QW];
    int kt = t_begin + pair;
    {
        const _Float16* p = tile_ptr(min(kt, t_end - 1));
#pragma unroll
        for (int i = 0; i < QW; ++i) {
            ka[i] = *reinterpret_cast<const uint4*>(p + chunk(i) * 512);
            kb[i] = *reinterpret_cast<const uint4*>(p + (DC + chunk(i)) * 512);
        }
    }
#pragma unroll
    for (int i = 0; i < QI; ++i) {
        const int c = wave + i * 4 * S;
        f16x8 h, l;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float v = valid && c < DC ? qx[i][j] : 0.f;
            h[j] = f16_sat(v);
            l[j] = f16_sat(v - (float)h[j]);
        }
        if (c < S * QW) {
            lds[c * 64 + lane] = __builtin_bit_cast(uint4, h);
            lds[(S * QW + c) * 64 + lane] = __builtin_bit_cast(uint4, l);
        }
    }
    const f16x8 sel0 = selection_frag(grp, l15, 0), sel1 = selection_frag(grp, l15, 1);
    f32x4 o[2 * KW];
#pragma unroll
    for (int d = 0; d < 2 * KW; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -1e30f, lsum = 0.f;
    __syncthreads();
    const int rounds = (t_end - t_begin + 3) >> 2;  // the same for every wave: pairs meet at barriers
    for (int it = 0; it < rounds; ++it, kt += 4) {
        f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < QW; ++i) {
            // keep the scheduler from hoisting every chunk's LDS reads (register spills otherwise)
            if constexpr (KW >= 6) { if (i % 4 == 0) __builtin_amdgcn_sched_barrier(0); }
            const int c = i < KW ? part * KW + i : KC + part * RW + (i - KW);
            const f16x8 qh = __builtin_bit_cast(f16x8, lds[c * 64 + lane]), ql = __builtin_bit_cast(f16x8, lds[(S * QW + c) * 64 + lane]);
            const f16x8 fa = __builtin_bit_cast(f16x8, ka[i]), fb = __builtin_bit_cast(f16x8, kb[i]);
            sa = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, qh, sa, 0, 0, 0);
            sb = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, qh, sb, 0, 0, 0);
            sa = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, ql, sa, 0, 0, 0);
            sb = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, ql, sb, 0, 0, 0);
        }
        if constexpr (S == 2) {
            // add the other wave's half of every score; two buffers: a wave two rounds ahead has passed the barrier in between
            f32x4* x = xch + (size_t)(it & 1) * 8 * 2 * 64;
            x[(wave * 2 + 0) * 64 + lane] = sa;
            x[(wave * 2 + 1) * 64 + lane] = sb;
            __syncthreads();
            const f32x4 xa = x[((wave ^ 1) * 2 + 0) * 64 + lane], xb = x[((wave ^ 1) * 2 + 1) * 64 + lane];
#pragma unroll
            for (int r = 0; r < 4; ++r) { sa[r] += xa[r]; sb[r] += xb[r]; }
        }
        const int last = kt < t_end ? my_pos : -1;  // a round past the range sees nothing
        const int tokA = (kt << 5) + grp * 4, tokB = tokA + 16;
        float mt = -1e30f;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            if (tokA + r <= last && tokA + r >= my_first) mt = fmaxf(mt, sa[r]);
            if (tokB + r <= last && tokB + r >= my_first) mt = fmaxf(mt, sb[r]);
        }
        mt = fmaxf(mt, __shfl_xor(mt, 16));
        mt = fmaxf(mt, __shfl_xor(mt, 32));
        const float mn = fmaxf(m, mt), alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        f16x8 P, Pl;
        float ps = 0.f;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float pa = (tokA + r <= last && tokA + r >= my_first) ? __builtin_amdgcn_exp2f(sa[r] - mn) : 0.f;
            const float pb = (tokB + r <= last && tokB + r >= my_first) ? __builtin_amdgcn_exp2f(sb[r] - mn) : 0.f;
            ps += pa + pb;
            P[r] = (_Float16)pa;
            P[4 + r] = (_Float16)pb;
            Pl[r] = (_Float16)(pa - (float)P[r]);
            Pl[4 + r] = (_Float16)(pb - (float)P[4 + r]);
        }
        lsum = lsum * alpha + ps;
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int d = 0; d < 2 * KW; ++d) { o[d][0] *= alpha; o[d][1] *= alpha; o[d][2] *= alpha; o[d][3] *= alpha; }
        }
        // values, refilling each fragment register for this wave's next tile once it has been used
        const _Float16* next = tile_ptr(min(kt + 4, t_end - 1));
#pragma unroll
        for (int i = 0; i < KW; ++i) {
            if constexpr (KW >= 6) { if (i % 2 == 0) __builtin_amdgcn_sched_barrier(0); }
            const f16x8 fa = __builtin_bit_cast(f16x8, ka[i]), fb = __builtin_bit_cast(f16x8, kb[i]);
            const f32x4 z = {0.f, 0.f, 0.f, 0.f};
            const f32x4 a0 = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, sel0, z, 0, 0, 0), b0 = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, sel0, z, 0, 0, 0);
            const f32x4 a1 = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, sel1, z, 0, 0, 0), b1 = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, sel1, z, 0, 0, 0);
            ka[i] = *reinterpret_cast<const uint4*>(next + chunk(i) * 512);
            kb[i] = *reinterpret_cast<const uint4*>(next + (DC + chunk(i)) * 512);
            f16x8 v0, v1;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                v0[r] = (_Float16)a0[r]; v0[4 + r] = (_Float16)b0[r];
                v1[r] = (_Float16)a1[r]; v1[4 + r] = (_Float16)b1[r];
            }
            o[2 * i] = __builtin_amdgcn_mfma_f32_16x16x32_f16(v0, P, o[2 * i], 0, 0, 0);
            o[2 * i + 1] = __builtin_amdgcn_mfma_f32_16x16x32_f16(v1, P, o[2 * i + 1], 0, 0, 0);
            o[2 * i] = __builtin_amdgcn_mfma_f32_16x16x32_f16(v0, Pl, o[2 * i], 0, 0, 0);
            o[2 * i + 1] = __builtin_amdgcn_mfma_f32_16x16x32_f16(v1, Pl, o[2 * i + 1], 0, 0, 0);
        }
#pragma unroll
        for (int i = KW; i < QW; ++i) {
            ka[i] = *reinterpret_cast<const uint4*>(next + chunk(i) * 512);
            kb[i] = *reinterpret_cast<const uint4*>(next + (DC + chunk(i)) * 512);
        }
    }
    // combine the four waves (pairs); both waves of a pair hold the same m and lsum
    lsum += __shfl_xor(lsum, 16);
    lsum += __shfl_xor(lsum, 32);
    if (grp == 0 && part == 0) { ml[pair][0][l15] = m; ml[pair][1][l15] = lsum; }
    __syncthreads();
    float ms = -1e30f, lt = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) ms = fmaxf(ms, ml[w][0][l15]);
#pragma unroll
    for (int w = 0; w < 4; ++w) lt += ml[w][1][l15] * __builtin_amdgcn_exp2f(ml[w][0][l15] - ms);
    const int n_parts = a.part_tiles ? (t_hi - t_lo + a.part_tiles - 1) / a.part_tiles : 1;
    if (a.sink && n_parts == 1) {  // parts: the sink joins where they are combined
        const float sk = a.sink[head], mn = fmaxf(ms, sk);
        lt = lt * __builtin_amdgcn_exp2f(ms - mn) + __builtin_amdgcn_exp2f(sk - mn);
        ms = mn;
    }
    const float f = __builtin_amdgcn_exp2f(m - ms);
    const float scale = n_parts > 1 ? 1.0f : 1.0f / lt;
    const size_t rh = (size_t)(row0 + tok) * a.heads + head;
    float* dst = n_parts > 1 ? a.part_o + (rh * a.max_parts + blockIdx.z) * (KC * 32) : a.out + rh * (KC * 32);
    f32x4* obuf = reinterpret_cast<f32x4*>(lds);
#pragma unroll
    for (int g = 0; g < (2 * KW + G - 1) / G; ++g) {
        if (g) __syncthreads();
#pragma unroll
        for (int i = 0; i < G; ++i)
            if (g * G + i < 2 * KW) obuf[(wave * G + i) * 64 + lane] = f32x4{o[g * G + i][0] * f, o[g * G + i][1] * f, o[g * G + i][2] * f, o[g * G + i][3] * f};
        __syncthreads();
#pragma unroll
        for (int i = 0; i < G / 4; ++i) {
            const int t = pair + i * 4, d = g * G + t;
            if (d >= 2 * KW) continue;
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int w = 0; w < 4; ++w) {
                const f32x4 v = obuf[((w * S + part) * G + t) * 64 + lane];
                acc[0] += v[0]; acc[1] += v[1]; acc[2] += v[2]; acc[3] += v[3];
            }
            if (valid) *reinterpret_cast<float4*>(dst + (part * 2 * KW + d) * 16 + grp * 4) = make_float4(acc[0] * scale, acc[1] * scale, acc[2] * scale, acc[3] * scale);
        }
    }
    if (n_parts > 1 && wave == 0 && grp == 0 && valid) {
        float* pm = a.part_ml + (rh * a.max_parts + blockIdx.z) * 2;
        pm[0] = ms;
        pm[1] = lt;
    }
}

static const int kChunkSizes[] = {1, 2, 3, 4, 6, 8, 12, 16};
int latent_rank_padded(int rank) {
    for (int c : kChunkSizes)
        if (rank <= c * 32) return c * 32;
    return (rank + 31) / 32 * 32;
}
bool latent_attn_ok(const LatentCache& c) { return !c.f32 && c.rank_p <= 512 && c.rank_p == latent_rank_padded(c.rank) && c.rot_p >= 32 && c.rot_p <= 64; }

hipError_t launch_latent_attn(const LatentAttnArgs& a, int n_tiles, int tile_rows, int n_parts_max, hipStream_t s) {
    if (!latent_attn_ok(a.cache) || n_parts_max > a.max_parts || (n_parts_max > 1 && (tile_rows != 1 || a.part_tiles < 1 || !a.part_o || !a.part_ml)))
        return hipErrorInvalidValue;
    if (n_tiles <= 0) return hipSuccess;
    const dim3 grid(n_tiles, (tile_rows * a.heads + 15) / 16, n_parts_max);
    const int kc = a.cache.rank_p / 32, rc = a.cache.rot_p / 32;
#define NVLLM_LA(K_)                                                                                      \
    if (kc == K_) {                                                                                       \
        constexpr int S_ = K_ > 8 ? 2 : 1;                                                                \
        if (rc == 1) latent_attn_kernel<K_ / S_, 1, S_><<<grid, 256 * S_, 0, s>>>(a);                     \
        else latent_attn_kernel<K_ / S_, 2, S_><<<grid, 256 * S_, 0, s>>>(a);                             \
    }
    NVLLM_LA(1) NVLLM_LA(2) NVLLM_LA(3) NVLLM_LA(4) NVLLM_LA(6) NVLLM_LA(8) NVLLM_LA(12) NVLLM_LA(16)
#undef NVLLM_LA
    return hipGetLastError();
}

}  // namespace nvllm
