// gfx950 grouped-query attention over the paged cache with an optional distance bias, window and sink term in the denominator:
//   s = q . k (scaled) + bias[head][min(i - j, n_bias - 1)],  p_j = exp(s_j) / ([exp(sink_h)] + sum exp(s_j)),  i - window < j <= i.
// Scores, weights and sums are f32, in units of log2.  Query rows are (token, head of the group) pairs, so one cached key serves every
// head of its group.  Matrix-core kernels (f16 cache): A = K (or V) fragment as stored, B = q (or P) as f16 hi + lo, the accumulator
// layout of the scores is the B-fragment order of P.
#include <algorithm>

#include "device_common.h"
#include "hybrid.h"

namespace nvllm {

__device__ __forceinline__ int first_seen(int pos, int window) { return window > 0 ? max(0, pos - window + 1) : 0; }

static const int kDimChunks[] = {1, 2, 3, 4, 8};   // of 32
static const int kVdimTiles[] = {2, 4, 8, 16};     // of 16
int bias_attn_dim(int dim) {
    for (int c : kDimChunks) if (dim <= c * 32) return c * 32;
    return 0;
}
int bias_attn_vdim(int vdim) {
    for (int c : kVdimTiles) if (vdim <= c * 16) return c * 16;
    return 0;
}

// ---------------------------------------------------------------------------------------------------
// plain form: one workgroup per (row, head); a wave takes 64 tokens at a time, one per lane for the scores, then one value
// dimension per lane
// ---------------------------------------------------------------------------------------------------
template <typename T>
__device__ __forceinline__ void load8(float (&x)[8], const T* p) {
    if constexpr (sizeof(T) == 4) {
        *reinterpret_cast<float4*>(&x[0]) = *reinterpret_cast<const float4*>(p);
        *reinterpret_cast<float4*>(&x[4]) = *reinterpret_cast<const float4*>(p + 4);
    } else {
        const f16x8 v = *reinterpret_cast<const f16x8*>(p);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] = (float)v[j];
    }
}
template <typename T, int NE>
__global__ void __launch_bounds__(256) bias_attn_plain_kernel(BiasAttnArgs a) {
    extern __shared__ float sh[];
    __shared__ float pw[4][64];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int row = blockIdx.x, head = blockIdx.y;
    const PagedKV& c = a.kv;
    const int kvh = head / (a.heads / c.kv), pos = a.pos[row];
    float* q = sh;                      // [dim_p]
    float* acc = sh + c.dim_p;          // [4][vdim_p + 2]
    for (int d = threadIdx.x; d < c.dim_p; d += 256) q[d] = a.q[((size_t)row * a.heads + head) * c.dim_p + d];
    __syncthreads();
    const int* bt = a.block_tables + (size_t)a.slot[row] * a.max_blocks;
    const float* bias = a.bias + (size_t)head * a.n_bias;
    float o[NE], m = -1e30f, l = 0.f;
#pragma unroll
    for (int e = 0; e < NE; ++e) o[e] = 0.f;
    const int first = first_seen(pos, a.window);
    for (int j0 = (first & ~63) + wave * 64; j0 <= pos; j0 += 256) {
        const int j = j0 + lane;
        const size_t blk = (size_t)bt[j0 / kBlockTokens] * c.kv + kvh;
        const T* kp = reinterpret_cast<const T*>(c.k) + blk * kBlockTokens * c.dim_p + k_packed_offset(j & (kBlockTokens - 1), 0, c.dim_p);
        float s = -1e30f;
        const bool seen = j >= first && j <= pos;
        if (seen) {
            s = 0.f;
            for (int d = 0; d < c.dim_p; d += 8) {
                float k[8];
                load8(k, kp + (size_t)(d >> 5) * 512 + ((d & 31) >> 3) * 128);
#pragma unroll
                for (int i = 0; i < 8; ++i) s += q[d + i] * k[i];
            }
            if (a.n_bias) s += bias[min(pos - j, a.n_bias - 1)];
        }
        float mt = s;
#pragma unroll
        for (int x = 32; x > 0; x >>= 1) mt = fmaxf(mt, __shfl_xor(mt, x));
        const float mn = fmaxf(m, mt), al = exp2f(m - mn), p = seen ? exp2f(s - mn) : 0.f;
        m = mn;
        l = l * al + wave_sum(p);
        pw[wave][lane] = p;  // read by this wave alone
        __builtin_amdgcn_wave_barrier();
        const T* vp = reinterpret_cast<const T*>(c.v) + blk * kBlockTokens * c.vdim_p;
#pragma unroll
        for (int e = 0; e < NE; ++e) {
            const int d = lane + e * 64;
            if (d >= c.vdim_p) continue;
            float t = o[e] * al;
            for (int x = 0; x < 64; x += 32)
                for (int g = 0; g < 4; ++g) {
                    float v[8];
                    load8(v, vp + v_packed_offset((j0 & (kBlockTokens - 1)) + x + g * 4, d, c.vdim_p));
#pragma unroll
                    for (int i = 0; i < 8; ++i) t += pw[wave][x + (i >> 2) * 16 + g * 4 + (i & 3)] * v[i];
                }
            o[e] = t;
        }
        __builtin_amdgcn_wave_barrier();
    }
    float* mine = acc + (size_t)wave * (c.vdim_p + 2);
    if (lane == 0) { mine[0] = m; mine[1] = l; }
#pragma unroll
    for (int e = 0; e < NE; ++e)
        if (lane + e * 64 < c.vdim_p) mine[2 + lane + e * 64] = o[e];
    __syncthreads();
    const float sink = a.sink ? a.sink[head] : 0.f;
    float ms = a.sink ? sink : -1e30f, f[4];
    for (int w = 0; w < 4; ++w) ms = fmaxf(ms, acc[(size_t)w * (c.vdim_p + 2)]);
    float lt = a.sink ? exp2f(sink - ms) : 0.f;
    for (int w = 0; w < 4; ++w) {
        f[w] = exp2f(acc[(size_t)w * (c.vdim_p + 2)] - ms);
        lt += f[w] * acc[(size_t)w * (c.vdim_p + 2) + 1];
    }
    const float inv = 1.0f / lt;
    for (int d = threadIdx.x; d < c.vdim; d += 256) {
        float v = 0.f;
        for (int w = 0; w < 4; ++w) v += f[w] * acc[(size_t)w * (c.vdim_p + 2) + 2 + d];
        v *= inv;
        const int col = head * c.vdim + d;
        if (a.of) a.of[(size_t)row * a.ld + col] = v;
        if (a.oh) {
            const size_t x = a.packed ? xpack_off(row, col, a.ld >> 5) : (size_t)row * a.ld + col;
            split_bf16(v, a.oh[x], a.ol[x]);
        }
    }
}
template <typename T>
static hipError_t plain_t(const BiasAttnArgs& a, int rows, hipStream_t s) {
    const dim3 grid(rows, a.heads);
    const size_t lds = ((size_t)a.kv.dim_p + 4 * (a.kv.vdim_p + 2)) * 4;
    if (a.kv.vdim_p <= 64) bias_attn_plain_kernel<T, 1><<<grid, 256, lds, s>>>(a);
    else if (a.kv.vdim_p <= 128) bias_attn_plain_kernel<T, 2><<<grid, 256, lds, s>>>(a);
    else if (a.kv.vdim_p <= 256) bias_attn_plain_kernel<T, 4><<<grid, 256, lds, s>>>(a);
    else if (a.kv.vdim_p <= 1024) bias_attn_plain_kernel<T, 16><<<grid, 256, lds, s>>>(a);
    else return hipErrorNotSupported;
    return hipGetLastError();
}
hipError_t launch_bias_attn_plain(const BiasAttnArgs& a, int rows, hipStream_t s) {
    if (a.heads % a.kv.kv || a.kv.dim_p % 32 || a.kv.vdim_p % 16 || (!a.of && !a.oh)) return hipErrorInvalidValue;
    if (a.kv.dim_p > 4096) return hipErrorNotSupported;
    if (rows <= 0) return hipSuccess;
    return a.kv.f32 ? plain_t<float>(a, rows, s) : plain_t<_Float16>(a, rows, s);
}

// ---------------------------------------------------------------------------------------------------
// pieces of the matrix-core kernels
// ---------------------------------------------------------------------------------------------------
// a query row's 8 elements of one fragment as f16 hi + lo
__device__ __forceinline__ void q_frag(const float* p, bool valid, f16x8& h, f16x8& l) {
    float x[8];
    *reinterpret_cast<float4*>(&x[0]) = *reinterpret_cast<const float4*>(p);
    *reinterpret_cast<float4*>(&x[4]) = *reinterpret_cast<const float4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const float v = valid ? x[j] : 0.f;
        h[j] = f16_sat(v);
        l[j] = f16_sat(v - (float)h[j]);
    }
}

// weights of eight tokens as f16 hi (rounded towards zero) + lo: 21 bits together
__device__ __forceinline__ void split_weights(const float (&pa)[4], const float (&pb)[4], f16x8& h, f16x8& l) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float x = i < 2 ? pa[2 * i] : pb[2 * i - 4], y = i < 2 ? pa[2 * i + 1] : pb[2 * i - 3];
        const auto hi = __builtin_amdgcn_cvt_pkrtz(x, y);
        const auto lo = __builtin_amdgcn_cvt_pkrtz(x - (float)hi[0], y - (float)hi[1]);
        h[2 * i] = (_Float16)hi[0];
        h[2 * i + 1] = (_Float16)hi[1];
        l[2 * i] = (_Float16)lo[0];
        l[2 * i + 1] = (_Float16)lo[1];
    }
}

// ---------------------------------------------------------------------------------------------------
// decode: one workgroup = one token x up to 16 heads of one group x a range of 32-token tiles; four waves take alternate tiles
// ---------------------------------------------------------------------------------------------------
template <int DC, int VC>
__global__ void __launch_bounds__(256) bias_decode_kernel(BiasAttnArgs a) {
    constexpr int G = 4;  // value tiles per combine pass
    __shared__ __attribute__((aligned(16))) f32x4 obuf[4 * G * 64];
    __shared__ float ml[4][2][16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l15 = lane & 15, grp = lane >> 4;
    const int row = blockIdx.x, pos = a.pos[row];
    const int gqa = a.heads / a.kv.kv, hb = (gqa + 15) / 16, kvh = blockIdx.y / hb, h0 = (blockIdx.y % hb) * 16;
    const bool valid = h0 + l15 < gqa;
    const int head = kvh * gqa + min(h0 + l15, gqa - 1);
    const int first = first_seen(pos, a.window), t_lo = first >> 5;
    const int t_hi = (pos >> 5) + 1, t_begin = t_lo + (a.part_tiles ? (int)blockIdx.z * a.part_tiles : 0);
    const int t_end = a.part_tiles ? min(t_hi, t_begin + a.part_tiles) : t_hi;
    if (t_begin >= t_hi) return;
    const int* bt = a.block_tables + (size_t)a.slot[row] * a.max_blocks;
    const _Float16* kd = reinterpret_cast<const _Float16*>(a.kv.k);
    const _Float16* vd = reinterpret_cast<const _Float16*>(a.kv.v);
    auto k_ptr = [&](int t) { return kd + ((size_t)bt[t >> 3] * a.kv.kv + kvh) * (kBlockTokens * DC * 32) + (size_t)(t & 7) * (2 * DC * 512) + lane * 8; };
    auto v_ptr = [&](int t) { return vd + ((size_t)bt[t >> 3] * a.kv.kv + kvh) * (kBlockTokens * VC * 16) + (size_t)(t & 7) * (VC * 512) + lane * 8; };
    int t = t_begin + wave;
    uint4 kf[2 * DC], vf[VC];
    {
        const _Float16* p = k_ptr(min(t, t_end - 1));
#pragma unroll
        for (int i = 0; i < 2 * DC; ++i) kf[i] = ld_stream16(p + i * 512);
    }
    f16x8 qh[DC], ql[DC];
    const float* qp = a.q + ((size_t)row * a.heads + head) * (DC * 32) + grp * 8;
#pragma unroll
    for (int c = 0; c < DC; ++c) q_frag(qp + c * 32, valid, qh[c], ql[c]);
    const float* bias = a.bias + (size_t)head * a.n_bias;
    const int far = a.n_bias - 1;
    const float b_far = a.n_bias ? bias[far] : 0.f;
    f32x4 o[VC];
#pragma unroll
    for (int d = 0; d < VC; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -1e30f, lsum = 0.f;
    for (; t < t_end; t += 4) {
        {
            const _Float16* p = v_ptr(t);
#pragma unroll
            for (int i = 0; i < VC; ++i) vf[i] = ld_stream16(p + i * 512);
        }
        const int tokA = (t << 5) + grp * 4, tokB = tokA + 16;
        float ba[4], bb[4];
        const bool near = a.n_bias && pos - (t << 5) - 31 < far;
        if (near) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                ba[r] = bias[max(0, min(pos - tokA - r, far))];
                bb[r] = bias[max(0, min(pos - tokB - r, far))];
            }
        } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) ba[r] = bb[r] = b_far;
        }
        f32x4 sa = {ba[0], ba[1], ba[2], ba[3]}, sb = {bb[0], bb[1], bb[2], bb[3]};
#pragma unroll
        for (int c = 0; c < DC; ++c) {
            const f16x8 fa = __builtin_bit_cast(f16x8, kf[c]), fb = __builtin_bit_cast(f16x8, kf[DC + c]);
            sa = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, qh[c], sa, 0, 0, 0);
            sb = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, qh[c], sb, 0, 0, 0);
            sa = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, ql[c], sa, 0, 0, 0);
            sb = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, ql[c], sb, 0, 0, 0);
        }
        {
            const _Float16* p = k_ptr(min(t + 4, t_end - 1));
#pragma unroll
            for (int i = 0; i < 2 * DC; ++i) kf[i] = ld_stream16(p + i * 512);
        }
        auto seen = [&](int j) { return j <= pos && j >= first; };
        float mt = -1e30f;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            if (seen(tokA + r)) mt = fmaxf(mt, sa[r]);
            if (seen(tokB + r)) mt = fmaxf(mt, sb[r]);
        }
        mt = fmaxf(mt, __shfl_xor(mt, 16));
        mt = fmaxf(mt, __shfl_xor(mt, 32));
        const float mn = fmaxf(m, mt), alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        f16x8 P, Pl;
        float ps = 0.f, pa[4], pb[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            pa[r] = seen(tokA + r) ? __builtin_amdgcn_exp2f(sa[r] - mn) : 0.f;
            pb[r] = seen(tokB + r) ? __builtin_amdgcn_exp2f(sb[r] - mn) : 0.f;
            ps += pa[r] + pb[r];
        }
        split_weights(pa, pb, P, Pl);
        lsum = lsum * alpha + ps;
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int d = 0; d < VC; ++d) { o[d][0] *= alpha; o[d][1] *= alpha; o[d][2] *= alpha; o[d][3] *= alpha; }
        }
#pragma unroll
        for (int d = 0; d < VC; ++d) {
            const f16x8 v = __builtin_bit_cast(f16x8, vf[d]);
            o[d] = __builtin_amdgcn_mfma_f32_16x16x32_f16(v, P, o[d], 0, 0, 0);
            o[d] = __builtin_amdgcn_mfma_f32_16x16x32_f16(v, Pl, o[d], 0, 0, 0);
        }
    }
    lsum += __shfl_xor(lsum, 16);
    lsum += __shfl_xor(lsum, 32);
    if (grp == 0) { ml[wave][0][l15] = m; ml[wave][1][l15] = lsum; }
    __syncthreads();
    const int n_parts = a.part_tiles ? (t_hi - t_lo + a.part_tiles - 1) / a.part_tiles : 1;
    const bool sinks = a.sink && n_parts == 1;
    const float sink = sinks ? a.sink[head] : 0.f;
    float ms = sinks ? sink : -1e30f;
#pragma unroll
    for (int w = 0; w < 4; ++w) ms = fmaxf(ms, ml[w][0][l15]);
    float lt = sinks ? __builtin_amdgcn_exp2f(sink - ms) : 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) lt += ml[w][1][l15] * __builtin_amdgcn_exp2f(ml[w][0][l15] - ms);
    const float f = __builtin_amdgcn_exp2f(m - ms), scale = n_parts > 1 ? 1.0f : 1.0f / lt;
    const size_t rp = ((size_t)row * a.heads + head) * a.max_parts + blockIdx.z;
#pragma unroll
    for (int g = 0; g < (VC + G - 1) / G; ++g) {
        if (g) __syncthreads();
#pragma unroll
        for (int i = 0; i < G; ++i)
            if (g * G + i < VC) obuf[(wave * G + i) * 64 + lane] = f32x4{o[g * G + i][0] * f, o[g * G + i][1] * f, o[g * G + i][2] * f, o[g * G + i][3] * f};
        __syncthreads();
        const int d = g * G + wave;
        if (d >= VC || !valid) continue;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const f32x4 v = obuf[(w * G + wave) * 64 + lane];
            acc[0] += v[0]; acc[1] += v[1]; acc[2] += v[2]; acc[3] += v[3];
        }
        const int e = d * 16 + grp * 4;
        if (n_parts > 1) *reinterpret_cast<float4*>(a.part_o + rp * (VC * 16) + e) = make_float4(acc[0], acc[1], acc[2], acc[3]);
        else if (e < a.kv.vdim) put_planes4(a.oh, a.ol, row, head * a.kv.vdim + e, a.kv.vdim - e, a.ld, a.packed, f32x4{acc[0] * scale, acc[1] * scale, acc[2] * scale, acc[3] * scale});
    }
    if (n_parts > 1 && wave == 0 && grp == 0 && valid) {
        a.part_ml[rp * 2] = ms;
        a.part_ml[rp * 2 + 1] = lt;
    }
}

// one wave per (row, head): parts merged, four value dimensions per lane
__global__ void __launch_bounds__(256) bias_combine_kernel(BiasAttnArgs a, int items) {
    const int lane = threadIdx.x & 63, it = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (it >= items) return;
    const int row = it / a.heads, head = it % a.heads;
    const int pos = a.pos[row], n = ((pos >> 5) + 1 - (first_seen(pos, a.window) >> 5) + a.part_tiles - 1) / a.part_tiles;
    if (n <= 1) return;  // written by the attention kernel
    const float* pm = a.part_ml + (size_t)it * a.max_parts * 2;
    const float sink = a.sink ? a.sink[head] : 0.f;
    float ms = a.sink ? sink : -1e30f, mine = -1e30f, l = 0.f;
    if (lane < n) { mine = pm[2 * lane]; l = pm[2 * lane + 1]; }  // at most kBiasMaxParts = 64 parts
    ms = fmaxf(ms, mine);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) ms = fmaxf(ms, __shfl_xor(ms, o));
    const float w = lane < n ? exp2f(mine - ms) : 0.f;
    const float inv = 1.0f / (wave_sum(w * l) + (a.sink ? exp2f(sink - ms) : 0.f));
    for (int e0 = 0; e0 < a.kv.vdim_p; e0 += 256) {  // every lane stays for the shuffles
        const int e = e0 + lane * 4;
        const float* po = a.part_o + (size_t)it * a.max_parts * a.kv.vdim_p + min(e, a.kv.vdim_p - 4);
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        for (int p0 = 0; p0 < n; p0 += 4) {
            float4 v[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) v[u] = *reinterpret_cast<const float4*>(po + (size_t)min(p0 + u, n - 1) * a.kv.vdim_p);
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const float f = p0 + u < n ? __shfl(w, p0 + u) * inv : 0.f;
                acc[0] += f * v[u].x; acc[1] += f * v[u].y; acc[2] += f * v[u].z; acc[3] += f * v[u].w;
            }
        }
        if (e < a.kv.vdim) put_planes4(a.oh, a.ol, row, head * a.kv.vdim + e, a.kv.vdim - e, a.ld, a.packed, acc);
    }
}

static bool matrix_core_ok(const BiasAttnArgs& a) {
    return !a.kv.f32 && a.kv.kv > 0 && a.heads % a.kv.kv == 0 && a.oh && a.kv.dim_p == bias_attn_dim(a.kv.dim) && a.kv.vdim_p == bias_attn_vdim(a.kv.vdim) &&
           a.heads * a.kv.vdim <= a.ld && (!a.packed || a.ld % 32 == 0) && (!a.n_bias || a.bias);
}
#define NVLLM_BA_V(K_, LAUNCH_) \
    switch (a.kv.vdim_p / 16) { case 2: LAUNCH_(K_, 2) break; case 4: LAUNCH_(K_, 4) break; case 8: LAUNCH_(K_, 8) break; default: LAUNCH_(K_, 16) break; }
#define NVLLM_BA(LAUNCH_)                              \
    switch (a.kv.dim_p / 32) {                         \
        case 1: NVLLM_BA_V(1, LAUNCH_) break;          \
        case 2: NVLLM_BA_V(2, LAUNCH_) break;          \
        case 3: NVLLM_BA_V(3, LAUNCH_) break;          \
        case 4: NVLLM_BA_V(4, LAUNCH_) break;          \
        default: NVLLM_BA_V(8, LAUNCH_) break;         \
    }

hipError_t launch_bias_decode(const BiasAttnArgs& a, int rows, int parts, hipStream_t s) {
    if (!matrix_core_ok(a) || (parts > 1 && (parts > a.max_parts || a.max_parts > kBiasMaxParts || a.part_tiles < 1 || !a.part_o || !a.part_ml))) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const int gqa = a.heads / a.kv.kv;
    const dim3 grid(rows, a.kv.kv * ((gqa + 15) / 16), std::max(1, parts));
#define NVLLM_BA_D(K_, V_) bias_decode_kernel<K_, V_><<<grid, 256, 0, s>>>(a);
    NVLLM_BA(NVLLM_BA_D)
#undef NVLLM_BA_D
    if (parts > 1) bias_combine_kernel<<<(rows * a.heads + 3) / 4, 256, 0, s>>>(a, rows * a.heads);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// prompt chunks: one workgroup = 128 (token, head of the group) rows of one sequence (64 for the widest heads, whose accumulators
// would not stay in registers: a fragment spilled while its read is in flight would be lost); four waves of MT 16-row tiles share the
// 32-token K and V tiles, copied straight into LDS (two buffers, the next tile in flight)
// ---------------------------------------------------------------------------------------------------
template <int DC, int VC, int MT>
__global__ void __launch_bounds__(256, 2) bias_prefill_kernel(BiasAttnArgs a, int bias_lds) {
    constexpr int RW = 64 * MT, F = 2 * DC + VC, NL = (F + 3) / 4;  // fragments per tile, per wave
    __shared__ __attribute__((aligned(16))) uint4 buf[2][F * 64];
    extern __shared__ float tab[];  // [gqa][n_bias] when bias_lds
    const int lane = threadIdx.x & 63, l15 = lane & 15, grp = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int tile = a.tile_order ? a.tile_order[blockIdx.y] : blockIdx.y;  // every head's longest tiles start first
    const int gqa = a.heads / a.kv.kv, per = gqa * (kBiasTileRows / RW), kvh = blockIdx.x / per, f0 = (blockIdx.x % per) * RW;
    const int row0 = a.tile_row0[tile], total = a.tile_nrows[tile] * gqa, slot = a.tile_slot[tile];
    if (f0 >= total) return;
    const int pos0 = a.pos[row0];
    const int pmin = pos0 + f0 / gqa, pmax = pos0 + min(f0 + RW - 1, total - 1) / gqa;
    const int nt = (pmax >> 5) + 1, t0 = first_seen(pmin, a.window) >> 5;
    const int low = a.window > 0 ? pmax - a.window + 1 : 0;  // some row does not see the tokens before
    const int* bt = a.block_tables + (size_t)slot * a.max_blocks;
    const _Float16* kd = reinterpret_cast<const _Float16*>(a.kv.k);
    const _Float16* vd = reinterpret_cast<const _Float16*>(a.kv.v);
    const int far = a.n_bias - 1;
    // fragments of tile t straight into LDS, a KiB per wave and copy
    auto stage = [&](int t, uint4* b) {
        const size_t blk = (size_t)bt[t >> 3] * a.kv.kv + kvh;
        const uint4* kp = reinterpret_cast<const uint4*>(kd + blk * (kBlockTokens * DC * 32) + (size_t)(t & 7) * (2 * DC * 512));
        const uint4* vp = reinterpret_cast<const uint4*>(vd + blk * (kBlockTokens * VC * 16) + (size_t)(t & 7) * (VC * 512)) - 2 * DC * 64;
#pragma unroll
        for (int i = 0; i < NL; ++i) {
            const int f = wave + i * 4;
            if (F % 4 == 0 || f < F) __builtin_amdgcn_global_load_lds((gptr_t)((f < 2 * DC ? kp : vp) + f * 64 + lane), (lptr_t)(b + f * 64), 16, 0, 0);
        }
    };
    stage(t0, buf[t0 & 1]);
    if (bias_lds)
        for (int i = threadIdx.x; i < gqa * a.n_bias; i += 256) tab[i] = a.bias[(size_t)kvh * gqa * a.n_bias + i];
    int my_pos[MT];
    bool valid[MT];
    int tok[MT], hd[MT];
    f16x8 qh[MT][DC], ql[MT][DC];
    const float* bias[MT];
    float b_far[MT];
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        const int flat = f0 + (wave * MT + u) * 16 + l15;
        valid[u] = flat < total;
        const int fc = min(flat, total - 1);
        tok[u] = fc / gqa;
        hd[u] = fc - tok[u] * gqa;
        my_pos[u] = pos0 + tok[u];
        const float* qp = a.q + ((size_t)(row0 + tok[u]) * a.heads + kvh * gqa + hd[u]) * (DC * 32) + grp * 8;
#pragma unroll
        for (int c = 0; c < DC; ++c) q_frag(qp + c * 32, valid[u], qh[u][c], ql[u][c]);
        bias[u] = a.bias + (size_t)(kvh * gqa + hd[u]) * a.n_bias;
        b_far[u] = a.n_bias ? bias[u][far] : 0.f;
    }
    f32x4 o[MT][VC];
    float m[MT], lsum[MT];
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        m[u] = -1e30f;
        lsum[u] = 0.f;
#pragma unroll
        for (int d = 0; d < VC; ++d) o[u][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    dma_publish_barrier();
    const uint32_t tab0 = lds_address(tab);
    for (int t = t0; t < nt; ++t) {
        const uint32_t b = lds_address(buf[t & 1]) + lane * 16;
        if (t + 1 < nt) stage(t + 1, buf[(t + 1) & 1]);  // its last readers have passed the barrier of the previous tile
        const int tokA = (t << 5) + grp * 4, tokB = tokA + 16;
        f32x4 sa[MT], sb[MT];
        constexpr int KG = DC < 4 ? DC : 4;  // chunks of K in flight
        f16x8 ka[KG], kb[KG];
        auto read_k = [&](int c0) {
#pragma unroll
            for (int c = 0; c < KG; ++c)
                if (c0 + c < DC) {
                    NVLLM_LDS_READ128(ka[c], b + c0 * 1024, c * 1024);
                    NVLLM_LDS_READ128(kb[c], b + c0 * 1024, (DC + c) * 1024);
                }
        };
        if (a.n_bias && pmin - (t << 5) - 31 < far) {  // some distance below the last bucket
#pragma unroll
            for (int u = 0; u < MT; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int na = max(0, min(my_pos[u] - tokA - r, far)), nb = max(0, min(my_pos[u] - tokB - r, far));
                    float xa, xb;
                    if (bias_lds) {
                        NVLLM_LDS_READ32(xa, tab0 + (uint32_t)(hd[u] * a.n_bias + na) * 4u);
                        NVLLM_LDS_READ32(xb, tab0 + (uint32_t)(hd[u] * a.n_bias + nb) * 4u);
                    } else {
                        xa = bias[u][na];
                        xb = bias[u][nb];
                    }
                    sa[u][r] = xa;
                    sb[u][r] = xb;
                }
            read_k(0);
            NVLLM_LDS_WAIT(2 * KG - 2);
        } else {
            read_k(0);
#pragma unroll
            for (int u = 0; u < MT; ++u) sa[u] = sb[u] = f32x4{b_far[u], b_far[u], b_far[u], b_far[u]};
            NVLLM_LDS_WAIT(2 * KG - 2);
        }
#pragma unroll
        for (int c = 0; c < DC; ++c) {
            if (c % KG == 0 && c) { read_k(c); NVLLM_LDS_WAIT(2 * KG - 2); }
            if (c % KG == 1) NVLLM_LDS_WAIT(KG > 2 ? 2 * KG - 4 : 0);
            if (c % KG == 2) NVLLM_LDS_WAIT(KG > 3 ? 2 * KG - 6 : 0);
            if (c % KG == 3) NVLLM_LDS_WAIT(0);
            const f16x8 fa = ka[c % KG], fb = kb[c % KG];
#pragma unroll
            for (int u = 0; u < MT; ++u) {
                sa[u] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, qh[u][c], sa[u], 0, 0, 0);
                sb[u] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, qh[u][c], sb[u], 0, 0, 0);
                sa[u] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, ql[u][c], sa[u], 0, 0, 0);
                sb[u] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, ql[u][c], sb[u], 0, 0, 0);
            }
            __builtin_amdgcn_sched_barrier(0);
        }
        constexpr int VG = VC < 8 ? VC : 8;  // value tiles in flight
        f16x8 vf[VG];
        auto read_v = [&](int d0) {
#pragma unroll
            for (int d = 0; d < VG; ++d) NVLLM_LDS_READ128(vf[d], b + d0 * 1024, (2 * DC + d) * 1024);
        };
        read_v(0);
        const bool edge = (t << 5) + 31 > pmin || (t << 5) < low;  // some row does not see the whole tile
        f16x8 P[MT], Pl[MT];
#pragma unroll
        for (int u = 0; u < MT; ++u) {
            // distances 0 .. span - 1 are seen
            const uint32_t span = a.window > 0 ? (uint32_t)a.window : 0x7fffffffu;
            auto hidden = [&](int j) { return (uint32_t)(my_pos[u] - j) >= span; };
            if (edge) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    if (hidden(tokA + r)) sa[u][r] = -1e30f;
                    if (hidden(tokB + r)) sb[u][r] = -1e30f;
                }
            }
            float mt = fmaxf(max3_raw(sa[u][0], sa[u][1], sa[u][2]), max3_raw(sa[u][3], sb[u][0], sb[u][1]));
            mt = max3_raw(mt, sb[u][2], sb[u][3]);
            mt = fmaxf(mt, __shfl_xor(mt, 16));
            mt = fmaxf(mt, __shfl_xor(mt, 32));
            const float mn = fmaxf(m[u], mt), alpha = __builtin_amdgcn_exp2f(m[u] - mn);
            m[u] = mn;
            float ps = 0.f, pa[4], pb[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                // a row that sees nothing of any tile so far has mn = -1e30: its masked scores would count as exp2(0)
                pa[r] = edge && hidden(tokA + r) ? 0.f : __builtin_amdgcn_exp2f(sa[u][r] - mn);
                pb[r] = edge && hidden(tokB + r) ? 0.f : __builtin_amdgcn_exp2f(sb[u][r] - mn);
                ps += pa[r] + pb[r];
            }
            split_weights(pa, pb, P[u], Pl[u]);
            lsum[u] = lsum[u] * alpha + ps;
            if (__any(alpha != 1.0f)) {
#pragma unroll
                for (int d = 0; d < VC; ++d) { o[u][d][0] *= alpha; o[u][d][1] *= alpha; o[u][d][2] *= alpha; o[u][d][3] *= alpha; }
            }
        }
#pragma unroll
        for (int d0 = 0; d0 < VC; d0 += VG) {
            if (d0) read_v(d0);
#pragma unroll
            for (int d = 0; d < VG; ++d) {
                if (d == 0) NVLLM_LDS_WAIT(VG / 2);
                if (d == VG / 2) NVLLM_LDS_WAIT(0);
#pragma unroll
                for (int u = 0; u < MT; ++u) {
                    o[u][d0 + d] = __builtin_amdgcn_mfma_f32_16x16x32_f16(vf[d], P[u], o[u][d0 + d], 0, 0, 0);
                    o[u][d0 + d] = __builtin_amdgcn_mfma_f32_16x16x32_f16(vf[d], Pl[u], o[u][d0 + d], 0, 0, 0);
                }
            }
            __builtin_amdgcn_sched_barrier(0);
        }
        dma_publish_barrier();
    }
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        float l = lsum[u];
        l += __shfl_xor(l, 16);
        l += __shfl_xor(l, 32);
        const float sink = a.sink ? a.sink[kvh * gqa + hd[u]] : 0.f, ms = a.sink ? fmaxf(m[u], sink) : m[u];
        float f = __builtin_amdgcn_exp2f(m[u] - ms);
        f = f / (l * f + (a.sink ? __builtin_amdgcn_exp2f(sink - ms) : 0.f));
        if (!valid[u]) continue;
        const int col = (kvh * gqa + hd[u]) * a.kv.vdim;
#pragma unroll
        for (int d = 0; d < VC; ++d) {
            const int e = d * 16 + grp * 4;
            if (e < a.kv.vdim) put_planes4(a.oh, a.ol, row0 + tok[u], col + e, a.kv.vdim - e, a.ld, a.packed, f32x4{o[u][d][0] * f, o[u][d][1] * f, o[u][d][2] * f, o[u][d][3] * f});
        }
    }
}

hipError_t launch_bias_prefill(const BiasAttnArgs& a, int n_tiles, hipStream_t s) {
    if (!matrix_core_ok(a)) return hipErrorInvalidValue;
    if (n_tiles > 65535) return hipErrorNotSupported;
    if (n_tiles <= 0) return hipSuccess;
    const int gqa = a.heads / a.kv.kv;
    const int bias_lds = a.n_bias && (size_t)gqa * a.n_bias <= 6144;
    const size_t lds = bias_lds ? (size_t)gqa * a.n_bias * 4 : 0;
#define NVLLM_BA_P(K_, V_)                                                                                           \
    {                                                                                                                \
        constexpr int MT_ = K_ > 4 || V_ > 8 ? 1 : 2;                                                                \
        const dim3 grid(a.kv.kv * gqa * (kBiasTileRows / (64 * MT_)), n_tiles);                                      \
        if (lds + 2 * (2 * K_ + V_) * 1024 > 64 * 1024) {                                                            \
            static std::atomic<uint64_t> done{0};                                                                    \
            ensure_dyn_lds(reinterpret_cast<const void*>(bias_prefill_kernel<K_, V_, MT_>), 24 * 1024, done);             \
        }                                                                                                            \
        bias_prefill_kernel<K_, V_, MT_><<<grid, 256, lds, s>>>(a, bias_lds);                                             \
    }
    NVLLM_BA(NVLLM_BA_P)
#undef NVLLM_BA_P
    return hipGetLastError();
}

}  // namespace nvllm
