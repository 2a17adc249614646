// gfx950 row kernels of the hybrid decoders: activations, the steps between a mixer's input projection and its attention or
// recurrence (biases, norms, value mixing, cache write; convolution, unit norms, gates), the gated output norm.
#include <algorithm>

#include "device_common.h"
#include "hybrid.h"
#include "short_conv.h"

namespace nvllm {

__device__ __forceinline__ float sigmoidf(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---------------------------------------------------------------------------------------------------
// activation of summed slabs
// ---------------------------------------------------------------------------------------------------
template <int ACT>
__global__ void __launch_bounds__(256) act_kernel(const float* __restrict__ in, int n_slabs, int64_t slab_stride, int rows, int F,
                                                    uint16_t* __restrict__ hi, uint16_t* __restrict__ lo, int packed, float* __restrict__ y) {
    const int64_t total = (int64_t)rows * (F >> 2);
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
        const int r = (int)(i / (F >> 2)), c = (int)(i % (F >> 2)) * 4;
        float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
        add_slabs(s, in + (size_t)r * F + c, n_slabs, slab_stride);
        const float x[4] = {s.x, s.y, s.z, s.w};
        f32x4 v;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = ACT == ACT_GELU ? 0.5f * x[e] * (1.0f + erff(x[e] * 0.7071067811865476f)) : relu2(x[e]);
        if (y) *reinterpret_cast<float4*>(y + (size_t)r * F + c) = make_float4(v[0], v[1], v[2], v[3]);
        if (hi) put_planes4(hi, lo, r, c, 4, F, packed, v);
    }
}
hipError_t launch_act(Act act, const float* in, int n_slabs, int64_t slab_stride, int rows, int F, bf16_bits* hi, bf16_bits* lo, int packed, float* y,
                      hipStream_t s) {
    if (F % 32 || n_slabs < 1) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const int64_t wgs = ((int64_t)rows * (F / 4) + 255) / 256;
    auto* const kernel = act == ACT_GELU ? act_kernel<ACT_GELU> : act_kernel<ACT_RELU2>;
    kernel<<<(int)std::min<int64_t>(wgs, 8192), 256, 0, s>>>(in, n_slabs, slab_stride, rows, F, hi, lo, packed, y);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// attention rows: one workgroup per row; the summed projection stays in LDS between the norms and the stores
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ void kv_put(void* base, int f32, size_t o, float v) {
    if (f32) reinterpret_cast<float*>(base)[o] = v;
    else reinterpret_cast<_Float16*>(base)[o] = f16_sat(v);
}
// sums columns [0, n) of a row of slabs (+ bias) into LDS
__device__ __forceinline__ void sum_row(float* x, const float* in, int n, int n_slabs, int64_t stride, const float* bias) {
    if (((n | (int)stride) & 3) == 0 && (reinterpret_cast<uintptr_t>(in) & 15) == 0) {
        for (int c = threadIdx.x * 4; c < n; c += blockDim.x * 4) {
            float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
            if (bias) s = *reinterpret_cast<const float4*>(bias + c);
            add_slabs(s, in + c, n_slabs, stride);
            *reinterpret_cast<float4*>(x + c) = s;
        }
    } else {
        for (int c = threadIdx.x; c < n; c += blockDim.x) x[c] = slab_elem(in + c, n_slabs, stride) + (bias ? bias[c] : 0.f);
    }
}

// BS = 1024 for the few rows of a decode step: every thread's loads are in flight at once
template <int BS>
__global__ void __launch_bounds__(BS) attn_rows_kernel(AttnRowsArgs a) {
    extern __shared__ __attribute__((aligned(16))) float xr[];
    __shared__ float red[2 * BS / 64];
    const int row = blockIdx.x;
    const int nq = a.heads * a.kv.dim, nk = a.kv.kv * a.kv.dim, nv = a.kv.kv * a.kv.vdim;
    sum_row(xr, a.in + (size_t)row * a.ld, (nq + nk + nv + 3) & ~3, a.n_slabs, a.slab_stride, a.bias);
    __syncthreads();
    float sq = 0.f, sk = 0.f;
    if (a.ssq) {
        sq = a.ssq[row * 2];
        sk = a.ssq[row * 2 + 1];
    } else {
        for (int c = threadIdx.x; c < nq; c += BS) sq += xr[c] * xr[c];
        for (int c = threadIdx.x; c < nk; c += BS) sk += xr[nq + c] * xr[nq + c];
        sq = wave_sum_uniform(sq);
        sk = wave_sum_uniform(sk);
        if ((threadIdx.x & 63) == 0) { red[threadIdx.x >> 6] = sq; red[BS / 64 + (threadIdx.x >> 6)] = sk; }
        __syncthreads();
        sq = sk = 0.f;
#pragma unroll
        for (int w = 0; w < BS / 64; ++w) { sq += red[w]; sk += red[BS / 64 + w]; }
    }
    const float rq = 1.0f / sqrtf(sq / (float)a.q_all + a.eps), rk = 1.0f / sqrtf(sk / (float)a.k_all + a.eps);
    float* q = a.q + (size_t)row * a.heads * a.kv.dim_p;
    const int pos = a.pos[row], t = pos & (kBlockTokens - 1);
    const size_t blk = (size_t)a.block_tables[(size_t)a.slot[row] * a.max_blocks + pos / kBlockTokens] * a.kv.kv;
    if (((a.kv.dim | a.kv.vdim) & 3) == 0) {  // four columns of one head per thread
        const int d4 = a.kv.dim_p >> 2, k4 = a.kv.dim >> 2, v4 = a.kv.vdim >> 2;
        for (int i = threadIdx.x; i < a.heads * d4; i += BS) {
            const int h = i / d4, d = (i - h * d4) * 4, c = h * a.kv.dim + d;
            float4 y = make_float4(0.f, 0.f, 0.f, 0.f);
            if (d < a.kv.dim) {
                const float4 x = *reinterpret_cast<const float4*>(xr + c), w = *reinterpret_cast<const float4*>(a.qn + c);
                y = make_float4((x.x * rq) * w.x * a.q_scale, (x.y * rq) * w.y * a.q_scale, (x.z * rq) * w.z * a.q_scale, (x.w * rq) * w.w * a.q_scale);
            }
            reinterpret_cast<float4*>(q)[i] = y;
        }
        for (int i = threadIdx.x; i < a.kv.kv * k4; i += BS) {
            const int h = i / k4, d = (i - h * k4) * 4, c = h * a.kv.dim + d;
            const float4 x = *reinterpret_cast<const float4*>(xr + nq + c), w = *reinterpret_cast<const float4*>(a.kn + c);
            const float y[4] = {(x.x * rk) * w.x, (x.y * rk) * w.y, (x.z * rk) * w.z, (x.w * rk) * w.w};
            const size_t o = (blk + h) * kBlockTokens * a.kv.dim_p + k_packed_offset(t, d, a.kv.dim_p);
            if (a.kv.f32) *reinterpret_cast<float4*>(reinterpret_cast<float*>(a.kv.k) + o) = make_float4(y[0], y[1], y[2], y[3]);
            else {
                typedef __attribute__((ext_vector_type(4))) _Float16 f16x4;
                *reinterpret_cast<f16x4*>(reinterpret_cast<_Float16*>(a.kv.k) + o) = f16x4{f16_sat(y[0]), f16_sat(y[1]), f16_sat(y[2]), f16_sat(y[3])};
            }
        }
        const float lam = a.mix == 2 ? a.lambda[0] : 0.f;
        for (int i = threadIdx.x; i < a.kv.kv * v4; i += BS) {
            const int h = i / v4, d = (i - h * v4) * 4, c = h * a.kv.vdim + d;
            float4 x = *reinterpret_cast<const float4*>(xr + nq + nk + c);
            float4* vf = reinterpret_cast<float4*>(a.v_first + (size_t)row * nv + c);
            if (a.mix == 1) *vf = x;
            if (a.mix == 2) {
                const float4 f = *vf;
                x = make_float4((1.0f - lam) * x.x + lam * f.x, (1.0f - lam) * x.y + lam * f.y, (1.0f - lam) * x.z + lam * f.z, (1.0f - lam) * x.w + lam * f.w);
            }
            const size_t o = (blk + h) * kBlockTokens * a.kv.vdim_p + v_packed_offset(t, d, a.kv.vdim_p);  // neighbouring dimensions are 8 apart
            kv_put(a.kv.v, a.kv.f32, o, x.x);
            kv_put(a.kv.v, a.kv.f32, o + 8, x.y);
            kv_put(a.kv.v, a.kv.f32, o + 16, x.z);
            kv_put(a.kv.v, a.kv.f32, o + 24, x.w);
        }
        return;
    }
    for (int i = threadIdx.x; i < a.heads * a.kv.dim_p; i += BS) {
        const int h = i / a.kv.dim_p, d = i - h * a.kv.dim_p, c = h * a.kv.dim + d;
        q[i] = d < a.kv.dim ? (xr[c] * rq) * a.qn[c] * a.q_scale : 0.f;
    }
    for (int c = threadIdx.x; c < nk; c += BS) {
        const int h = c / a.kv.dim, d = c - h * a.kv.dim;
        kv_put(a.kv.k, a.kv.f32, (blk + h) * kBlockTokens * a.kv.dim_p + k_packed_offset(t, d, a.kv.dim_p), (xr[nq + c] * rk) * a.kn[c]);
    }
    const float lam = a.mix == 2 ? a.lambda[0] : 0.f;
    for (int c = threadIdx.x; c < nv; c += BS) {
        const int h = c / a.kv.vdim, d = c - h * a.kv.vdim;
        float v = xr[nq + nk + c];
        if (a.mix == 1) a.v_first[(size_t)row * nv + c] = v;
        if (a.mix == 2) v = (1.0f - lam) * v + lam * a.v_first[(size_t)row * nv + c];
        kv_put(a.kv.v, a.kv.f32, (blk + h) * kBlockTokens * a.kv.vdim_p + v_packed_offset(t, d, a.kv.vdim_p), v);
    }
}
// prompt chunks: a wave per row, four rows per workgroup, the row in registers; values meet in LDS, so that four consecutive tokens of
// one dimension, neighbours in the cache, are one store
template <int NI>
__global__ void __launch_bounds__(256) attn_rows4_kernel(AttnRowsArgs a, int rows) {
    extern __shared__ __attribute__((aligned(16))) float vs[];  // [4][nv]
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int row0 = blockIdx.x * 4, row = min(row0 + wave, rows - 1);
    const int nq = a.heads * a.kv.dim, nk = a.kv.kv * a.kv.dim, nv = a.kv.kv * a.kv.vdim, n = nq + nk + nv;
    const float* in = a.in + (size_t)row * a.ld;
    float4 x[NI];
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int c = (lane + i * 64) * 4;
        x[i] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (c < n) {
            if (a.bias) x[i] = *reinterpret_cast<const float4*>(a.bias + c);
            add_slabs(x[i], in + c, a.n_slabs, a.slab_stride);
        }
        const float ss = x[i].x * x[i].x + x[i].y * x[i].y + x[i].z * x[i].z + x[i].w * x[i].w;
        if (c < nq) sq += ss;
        else if (c < nq + nk) sk += ss;
    }
    sq = a.ssq ? a.ssq[row * 2] : wave_sum_uniform(sq);
    sk = a.ssq ? a.ssq[row * 2 + 1] : wave_sum_uniform(sk);
    const float rq = 1.0f / sqrtf(sq / (float)a.q_all + a.eps), rk = 1.0f / sqrtf(sk / (float)a.k_all + a.eps);
    const int pos = a.pos[row], t = pos & (kBlockTokens - 1);
    const int* bt = a.block_tables + (size_t)a.slot[row] * a.max_blocks;
    const size_t blk = (size_t)bt[pos / kBlockTokens] * a.kv.kv;
    const float lam = a.mix == 2 ? a.lambda[0] : 0.f;
    const bool live = row0 + wave < rows;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int c = (lane + i * 64) * 4;
        if (!live || c >= n) continue;
        if (c < nq) {
            const float4 w = *reinterpret_cast<const float4*>(a.qn + c);
            const int h = c / a.kv.dim, d = c - h * a.kv.dim;
            *reinterpret_cast<float4*>(a.q + ((size_t)row * a.heads + h) * a.kv.dim_p + d) =
                make_float4((x[i].x * rq) * w.x * a.q_scale, (x[i].y * rq) * w.y * a.q_scale, (x[i].z * rq) * w.z * a.q_scale, (x[i].w * rq) * w.w * a.q_scale);
        } else if (c < nq + nk) {
            const float4 w = *reinterpret_cast<const float4*>(a.kn + c - nq);
            const int h = (c - nq) / a.kv.dim, d = c - nq - h * a.kv.dim;
            typedef __attribute__((ext_vector_type(4))) _Float16 f16x4;
            *reinterpret_cast<f16x4*>(reinterpret_cast<_Float16*>(a.kv.k) + (blk + h) * kBlockTokens * a.kv.dim_p + k_packed_offset(t, d, a.kv.dim_p)) =
                f16x4{f16_sat((x[i].x * rk) * w.x), f16_sat((x[i].y * rk) * w.y), f16_sat((x[i].z * rk) * w.z), f16_sat((x[i].w * rk) * w.w)};
        } else {
            float4 v = x[i];
            float4* vf = reinterpret_cast<float4*>(a.v_first + (size_t)row * nv + c - nq - nk);
            if (a.mix == 1) *vf = v;
            if (a.mix == 2) {
                const float4 f = *vf;
                v = make_float4((1.0f - lam) * v.x + lam * f.x, (1.0f - lam) * v.y + lam * f.y, (1.0f - lam) * v.z + lam * f.z, (1.0f - lam) * v.w + lam * f.w);
            }
            *reinterpret_cast<float4*>(vs + (size_t)wave * nv + c - nq - nk) = v;
        }
    }
    for (int d = a.kv.dim + lane; d < a.kv.dim_p; d += 64)
        if (live)
            for (int h = 0; h < a.heads; ++h) a.q[((size_t)row * a.heads + h) * a.kv.dim_p + d] = 0.f;
    __syncthreads();
    const int p0 = a.pos[row0], s0 = a.slot[row0];
    bool together = row0 + 4 <= rows && (p0 & 3) == 0;
    for (int r = 1; r < 4; ++r) together = together && a.slot[min(row0 + r, rows - 1)] == s0;
    _Float16* v = reinterpret_cast<_Float16*>(a.kv.v);
    if (together) {
        typedef __attribute__((ext_vector_type(4))) _Float16 f16x4;
        const size_t b0 = (size_t)a.block_tables[(size_t)s0 * a.max_blocks + p0 / kBlockTokens] * a.kv.kv;
        for (int c = threadIdx.x; c < nv; c += 256) {
            const int h = c / a.kv.vdim, d = c - h * a.kv.vdim;
            *reinterpret_cast<f16x4*>(v + (b0 + h) * kBlockTokens * a.kv.vdim_p + v_packed_offset(p0 & (kBlockTokens - 1), d, a.kv.vdim_p)) =
                f16x4{f16_sat(vs[c]), f16_sat(vs[nv + c]), f16_sat(vs[2 * nv + c]), f16_sat(vs[3 * nv + c])};
        }
    } else if (live) {
        for (int c = lane; c < nv; c += 64) {
            const int h = c / a.kv.vdim, d = c - h * a.kv.vdim;
            v[(blk + h) * kBlockTokens * a.kv.vdim_p + v_packed_offset(t, d, a.kv.vdim_p)] = f16_sat(vs[(size_t)wave * nv + c]);
        }
    }
}

hipError_t launch_attn_rows(const AttnRowsArgs& a, int rows, hipStream_t s) {
    const int n = a.heads * a.kv.dim + a.kv.kv * (a.kv.dim + a.kv.vdim);
    if (a.kv.dim_p % 32 || a.kv.vdim_p % 16 || n > a.ld || a.ld % 4 || (a.mix && !a.v_first) || (a.mix == 2 && !a.lambda)) return hipErrorInvalidValue;
    const size_t lds = ((size_t)n + 4) * 4;
    if (lds > 64 * 1024) return hipErrorNotSupported;
    if (rows <= 0) return hipSuccess;
    const size_t lds4 = (size_t)4 * a.kv.kv * a.kv.vdim * 4;
    if (rows > 128 && !a.kv.f32 && ((a.kv.dim | a.kv.vdim) & 3) == 0 && (a.slab_stride & 3) == 0 && n <= 24 * 256 && lds4 <= 64 * 1024) {
        const int wgs = (rows + 3) / 4;
        if (n <= 8 * 256) attn_rows4_kernel<8><<<wgs, 256, lds4, s>>>(a, rows);
        else if (n <= 16 * 256) attn_rows4_kernel<16><<<wgs, 256, lds4, s>>>(a, rows);
        else attn_rows4_kernel<24><<<wgs, 256, lds4, s>>>(a, rows);
        return hipGetLastError();
    }
    if (rows <= 128 && n > 1024) attn_rows_kernel<1024><<<rows, 1024, lds, s>>>(a);
    else attn_rows_kernel<256><<<rows, 256, lds, s>>>(a);
    return hipGetLastError();
}

__global__ void __launch_bounds__(256) rows_ssq_kernel(const float* __restrict__ in, int n_slabs, int64_t slab_stride, int ld, const float* __restrict__ bias,
                                                       int c0, int n0, int c1, int n1, float* __restrict__ out) {
    __shared__ float red[4];
    const int row = blockIdx.x, first = blockIdx.y ? c1 : c0, n = blockIdx.y ? n1 : n0;
    float ss = 0.f;
    for (int c = threadIdx.x; c < n; c += 256) {
        const float v = slab_elem(in + (size_t)row * ld + first + c, n_slabs, slab_stride) + (bias ? bias[first + c] : 0.f);
        ss += v * v;
    }
    ss = block_sum(ss, red, 4);
    if (threadIdx.x == 0) out[row * 2 + blockIdx.y] = ss;
}
hipError_t launch_rows_ssq(const float* in, int n_slabs, int64_t slab_stride, int ld, const float* bias, const int c0[2], const int n[2], int rows,
                           float* out, hipStream_t s) {
    if (rows <= 0) return hipSuccess;
    rows_ssq_kernel<<<dim3(rows, 2), 256, 0, s>>>(in, n_slabs, slab_stride, ld, bias, c0[0], n[0], c0[1], n[1], out);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// constant-decay recurrence: silu(q, k, v), sigmoid(gate); four consecutive padded columns per thread
// ---------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256) linear_rows_kernel(LinearRowsArgs a, int rows) {
    const int qk = a.heads * (a.dim_p >> 2), vg = a.heads * (a.vdim_p >> 2), per = 2 * (qk + vg);
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= (int64_t)rows * per) return;
    const int row = (int)(i / per);
    int c = (int)(i - (int64_t)row * per), which = 0, col0 = 0;  // which: q, k, v, gate
    if (c >= qk) { c -= qk; which = 1; }
    if (which == 1 && c >= qk) { c -= qk; which = 2; }
    if (which == 2 && c >= vg) { c -= vg; which = 3; }
    const int p4 = (which < 2 ? a.dim_p : a.vdim_p) >> 2, n = which < 2 ? a.dim : a.vdim;
    const int h = c / p4, d = (c - h * p4) * 4;
    if (which == 1) col0 = a.heads * a.dim;
    if (which >= 2) col0 = 2 * a.heads * a.dim + (which - 2) * a.heads * a.vdim;
    const float* in = a.in + (size_t)row * a.ld + col0 + h * n + d;
    float x[4];
    if (d + 4 <= n && ((reinterpret_cast<uintptr_t>(in) & 15) | (a.slab_stride & 3)) == 0) {
        float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
        add_slabs(s, in, a.n_slabs, a.slab_stride);
        x[0] = s.x; x[1] = s.y; x[2] = s.z; x[3] = s.w;
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = d + e < n ? slab_elem(in + e, a.n_slabs, a.slab_stride) : 0.f;
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const float sg = sigmoidf(x[e]);
        x[e] = which == 3 ? sg : x[e] * sg;
    }
    float* o = which == 0 ? a.q : which == 1 ? a.k : which == 2 ? a.v : a.gate;
    *reinterpret_cast<float4*>(o + ((size_t)row * a.heads + h) * (p4 * 4) + d) = make_float4(x[0], x[1], x[2], x[3]);
}
hipError_t launch_linear_rows(const LinearRowsArgs& a, int rows, hipStream_t s) {
    if (a.dim_p % 4 || a.vdim_p % 4 || 2 * a.heads * (a.dim + a.vdim) > a.ld) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const int64_t n = (int64_t)rows * a.heads * 2 * (a.dim_p / 4 + a.vdim_p / 4);
    linear_rows_kernel<<<(int)((n + 255) / 256), 256, 0, s>>>(a, rows);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// delta rule: one wave per (row, unit); units = q heads, k heads, v heads, then those of delta_extra.  The form for any size of prompt
// chunk first, then those of decode and of long chunks.
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ float conv_silu(const DeltaRowsArgs& a, const RowPast& p, int row, int c, int channels) {
    float y = 0.f;
    for (int i = 0; i < a.taps; ++i) y += past_input(a, p, row, a.taps - 1 - i, c, channels) * a.conv[(size_t)i * channels + c];
    return y * sigmoidf(y);
}

// column i behind the convolved ones: write strengths, then what the decays come from, or the decays of the heads
__device__ __forceinline__ void delta_extra(const DeltaRowsArgs& a, int row, int i, float x) {
    if (i < a.heads) a.beta[(size_t)row * a.heads + i] = sigmoidf(x);
    else if (a.rate) a.decay[(size_t)row * a.heads + i - a.heads] = expf(-a.rate[i - a.heads] * softplusf(x + a.dt[i - a.heads]));
    else a.gate_in[(size_t)row * 2 * a.rank_p + i - a.heads] = x;
}

template <int NE>
__global__ void __launch_bounds__(256) delta_rows_kernel(DeltaRowsArgs a) {
    const int lane = threadIdx.x & 63, row = blockIdx.x, unit = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int channels = 2 * a.kv * a.dim + a.heads * a.vdim;
    if (unit > 2 * a.kv + a.heads) return;
    const RowPast p = row_past(a, row);
    if (unit < 2 * a.kv) {
        const int h = unit % a.kv, c0 = unit * a.dim;
        float x[NE], ss = 0.f;
#pragma unroll
        for (int e = 0; e < NE; ++e) {
            const int d = lane + e * 64;
            x[e] = d < a.dim ? conv_silu(a, p, row, c0 + d, channels) : 0.f;
            ss += x[e] * x[e];
        }
        const float f = (unit < a.kv ? a.q_scale : 1.f) / sqrtf(wave_sum(ss) + kUnitNormEps);
        float* o = (unit < a.kv ? a.q : a.k) + ((size_t)row * a.kv + h) * a.dim_p;
#pragma unroll
        for (int e = 0; e < NE; ++e)
            if (lane + e * 64 < a.dim_p) o[lane + e * 64] = x[e] * f;
    } else if (unit < 2 * a.kv + a.heads) {
        const int h = unit - 2 * a.kv, c0 = 2 * a.kv * a.dim + h * a.vdim;
        float* o = a.v + ((size_t)row * a.heads + h) * a.vdim_p;
        for (int d = lane; d < a.vdim_p; d += 64) o[d] = d < a.vdim ? conv_silu(a, p, row, c0 + d, channels) : 0.f;
    } else {
        for (int i = lane; i < a.extras(); i += 64) delta_extra(a, row, i, slab_elem(a.in + (size_t)row * a.ld + channels + i, a.n_slabs, a.slab_stride));
    }
}

// decode: every input is read once, for the convolution and for the history's next half (this half moved on by one token)
template <int TAPS, int NE>
__global__ void __launch_bounds__(256) delta_rows_decode_kernel(DeltaRowsArgs a) {
    const int lane = threadIdx.x & 63, row = blockIdx.x, unit = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int channels = 2 * a.kv * a.dim + a.heads * a.vdim;
    if (unit > 2 * a.kv + a.heads) return;
    if (unit == 2 * a.kv + a.heads) {
        for (int i = lane; i < a.extras(); i += 64) delta_extra(a, row, i, slab_elem(a.in + (size_t)row * a.ld + channels + i, a.n_slabs, a.slab_stride));
        return;
    }
    const int slot = a.slot[row], pos = a.pos[row];
    const bool qk = unit < 2 * a.kv;
    const int n = qk ? a.dim : a.vdim, n_p = qk ? a.dim_p : a.vdim_p;
    const int c0 = qk ? unit * a.dim : 2 * a.kv * a.dim + (unit - 2 * a.kv) * a.vdim;
    const int hd = qk ? unit % a.kv : unit - 2 * a.kv, hs = qk ? a.kv : a.heads;
    float* out = (qk ? (unit < a.kv ? a.q : a.k) : a.v) + ((size_t)row * hs + hd) * n_p;
    const float* in = a.in + (size_t)row * a.ld + c0;
    const float* past = a.history + ((size_t)(pos & 1) * a.slots + slot) * (TAPS - 1) * channels + c0;
    float* next = a.history + ((size_t)((pos + 1) & 1) * a.slots + slot) * (TAPS - 1) * channels + c0;
    for (int d0 = 0; d0 < n_p; d0 += 64 * NE) {  // once for q and k (dim_p <= 64 NE): their norm needs the whole head
        float x[TAPS][NE], y[NE], ss = 0.f;
#pragma unroll
        for (int e = 0; e < NE; ++e) {
            const int d = min(d0 + e * 64 + lane, n - 1);
            x[TAPS - 1][e] = slab_elem(in + d, a.n_slabs, a.slab_stride);
#pragma unroll
            for (int i = 0; i < TAPS - 1; ++i) {
                const float h = past[(size_t)i * channels + d];
                x[i][e] = pos >= TAPS - 1 - i ? h : 0.f;
            }
        }
#pragma unroll
        for (int e = 0; e < NE; ++e) {
            const int d = d0 + e * 64 + lane;
            float t = 0.f;
#pragma unroll
            for (int i = 0; i < TAPS; ++i) t += x[i][e] * a.conv[(size_t)i * channels + c0 + min(d, n - 1)];
            y[e] = d < n ? t * sigmoidf(t) : 0.f;
            ss += y[e] * y[e];
            if (d < n) {
#pragma unroll
                for (int i = 0; i < TAPS - 1; ++i) next[(size_t)i * channels + d] = x[i + 1][e];
            }
        }
        const float f = qk ? (unit < a.kv ? a.q_scale : 1.f) / sqrtf(wave_sum_uniform(ss) + kUnitNormEps) : 1.f;
#pragma unroll
        for (int e = 0; e < NE; ++e)
            if (d0 + e * 64 + lane < n_p) out[d0 + e * 64 + lane] = y[e] * f;
    }
}
template <int NE>
static bool delta_rows_decode(const DeltaRowsArgs& a, int rows, hipStream_t s) {
    const dim3 grid(rows, (2 * a.kv + a.heads + 1 + 3) / 4);
    switch (a.taps) {
#define NVLLM_DD(T_) case T_: delta_rows_decode_kernel<T_, NE><<<grid, 256, 0, s>>>(a); return true;
        NVLLM_DD(1) NVLLM_DD(2) NVLLM_DD(3) NVLLM_DD(4) NVLLM_DD(5) NVLLM_DD(6) NVLLM_DD(7) NVLLM_DD(8)
        NVLLM_DD(9) NVLLM_DD(10) NVLLM_DD(11) NVLLM_DD(12) NVLLM_DD(13) NVLLM_DD(14) NVLLM_DD(15) NVLLM_DD(16)
#undef NVLLM_DD
    }
    return false;
}

// prompt chunks: one wave per (16 rows, unit), the convolution's window in registers
template <int TAPS, int NE>
__global__ void __launch_bounds__(256) delta_rows16_kernel(DeltaRowsArgs a, int rows) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int row0 = blockIdx.x * 16, row1 = min(row0 + 16, rows);
    const int channels = 2 * a.kv * a.dim + a.heads * a.vdim;
    if (unit > 2 * a.kv + a.heads) return;
    if (unit == 2 * a.kv + a.heads) {
        const int per = a.extras(), n = (row1 - row0) * per;
        for (int i0 = lane; i0 < n; i0 += 256) {  // four loads in flight
            float x[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int i = min(i0 + u * 64, n - 1);
                x[u] = slab_elem(a.in + (size_t)(row0 + i / per) * a.ld + channels + i % per, a.n_slabs, a.slab_stride);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u)
                if (i0 + u * 64 < n) delta_extra(a, row0 + (i0 + u * 64) / per, (i0 + u * 64) % per, x[u]);
        }
        return;
    }
    const bool qk = unit < 2 * a.kv;
    const int n = qk ? a.dim : a.vdim, n_p = qk ? a.dim_p : a.vdim_p;
    const int c0 = qk ? unit * a.dim : 2 * a.kv * a.dim + (unit - 2 * a.kv) * a.vdim;
    const int hd = qk ? unit % a.kv : unit - 2 * a.kv, hs = qk ? a.kv : a.heads;
    float* out = (qk ? (unit < a.kv ? a.q : a.k) : a.v) + (size_t)hd * n_p;
    const float unit_scale = unit < a.kv ? a.q_scale : 1.f;
    bool plain = row0 + 16 <= rows && row0 >= TAPS - 1 && a.n_slabs == 1;
    if (plain)
        for (int r = -(TAPS - 1); r < 15; ++r) plain &= a.slot[row0 + r] == a.slot[row0 + 15];
    for (int d0 = 0; d0 < n_p; d0 += 64 * NE) {  // once for q and k (dim_p = 64 NE): their norm needs the whole head
        float w[TAPS][NE], x[TAPS][NE];
#pragma unroll
        for (int e = 0; e < NE; ++e) {
            const int d = d0 + e * 64 + lane;
#pragma unroll
            for (int i = 0; i < TAPS; ++i) w[i][e] = d < n ? a.conv[(size_t)i * channels + c0 + d] : 0.f;
        }
        if (plain) {  // one sequence, its window inside the chunk: every load of the block is in flight at once
            float z[15 + TAPS][NE];
            const float* in = a.in + (size_t)(row0 - (TAPS - 1)) * a.ld + c0;
#pragma unroll
            for (int r = 0; r < 15 + TAPS; ++r)
#pragma unroll
                for (int e = 0; e < NE; ++e) {
                    const int d = d0 + e * 64 + lane;
                    z[r][e] = d < n ? in[(size_t)r * a.ld + d] : 0.f;
                }
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                float y[NE], ss = 0.f;
#pragma unroll
                for (int e = 0; e < NE; ++e) {
                    float t = 0.f;
#pragma unroll
                    for (int i = 0; i < TAPS; ++i) t += z[r + i][e] * w[i][e];
                    y[e] = t * sigmoidf(t);
                    ss += y[e] * y[e];
                }
                const float f = qk ? unit_scale / sqrtf(wave_sum_uniform(ss) + kUnitNormEps) : 1.f;
#pragma unroll
                for (int e = 0; e < NE; ++e)
                    if (d0 + e * 64 + lane < n_p) out[(size_t)(row0 + r) * hs * n_p + d0 + e * 64 + lane] = y[e] * f;
            }
            continue;
        }
        for (int row = row0; row < row1; ++row) {
            const int slot = a.slot[row];
            const bool start = row == 0 || a.slot[row - 1] != slot;
            if (row == row0 || start) {
                const RowPast p = row_past(a, row);
#pragma unroll
                for (int j = 1; j < TAPS; ++j)
#pragma unroll
                    for (int e = 0; e < NE; ++e) {
                        const int d = d0 + e * 64 + lane;
                        x[TAPS - 1 - j][e] = d < n ? past_input(a, p, row, j, c0 + d, channels) : 0.f;
                    }
            } else {
#pragma unroll
                for (int i = 0; i < TAPS - 1; ++i)
#pragma unroll
                    for (int e = 0; e < NE; ++e) x[i][e] = x[i + 1][e];
            }
            const float* in = a.in + (size_t)row * a.ld + c0;
            float y[NE], ss = 0.f;
#pragma unroll
            for (int e = 0; e < NE; ++e) {
                const int d = d0 + e * 64 + lane;
                x[TAPS - 1][e] = d < n ? slab_elem(in + d, a.n_slabs, a.slab_stride) : 0.f;
                float t = 0.f;
#pragma unroll
                for (int i = 0; i < TAPS; ++i) t += x[i][e] * w[i][e];
                y[e] = t * sigmoidf(t);
                ss += y[e] * y[e];
            }
            const float f = qk ? unit_scale / sqrtf(wave_sum_uniform(ss) + kUnitNormEps) : 1.f;
#pragma unroll
            for (int e = 0; e < NE; ++e)
                if (d0 + e * 64 + lane < n_p) out[(size_t)row * hs * n_p + d0 + e * 64 + lane] = y[e] * f;
        }
    }
}
template <int NE>
static bool delta_rows16(const DeltaRowsArgs& a, int rows, hipStream_t s) {
    const dim3 grid((rows + 15) / 16, (2 * a.kv + a.heads + 1 + 3) / 4);
    if (a.taps == 4) delta_rows16_kernel<4, NE><<<grid, 256, 0, s>>>(a, rows);
    else if (a.taps == 3) delta_rows16_kernel<3, NE><<<grid, 256, 0, s>>>(a, rows);
    else if (a.taps == 2) delta_rows16_kernel<2, NE><<<grid, 256, 0, s>>>(a, rows);
    else return false;
    return true;
}
hipError_t launch_delta_rows(const DeltaRowsArgs& a, int rows, hipStream_t s) {
    if (a.dim_p % 64 || a.vdim_p % 4 || a.taps < 1 || a.channels() + a.extras() > a.ld || (a.rate ? !a.dt || !a.decay : !a.gate_in)) return hipErrorInvalidValue;
    if (a.dim_p > 512) return hipErrorNotSupported;
    if (rows <= 0) return hipSuccess;
    if (!a.seg.single && rows >= 64) {
        const bool done = a.dim_p == 64 ? delta_rows16<1>(a, rows, s) : a.dim_p == 128 ? delta_rows16<2>(a, rows, s) : a.dim_p == 256 ? delta_rows16<4>(a, rows, s) : false;
        if (done) return hipGetLastError();
    }
    if (a.seg.single) {
        const bool done = a.dim_p <= 64 ? delta_rows_decode<1>(a, rows, s) : a.dim_p <= 128 ? delta_rows_decode<2>(a, rows, s)
                        : a.dim_p <= 256 ? delta_rows_decode<4>(a, rows, s) : delta_rows_decode<8>(a, rows, s);
        return done ? hipGetLastError() : hipErrorNotSupported;
    }
    const dim3 grid(rows, (2 * a.kv + a.heads + 1 + 3) / 4);
    if (a.dim_p <= 64) delta_rows_kernel<1><<<grid, 256, 0, s>>>(a);
    else if (a.dim_p <= 128) delta_rows_kernel<2><<<grid, 256, 0, s>>>(a);
    else if (a.dim_p <= 256) delta_rows_kernel<4><<<grid, 256, 0, s>>>(a);
    else delta_rows_kernel<8><<<grid, 256, 0, s>>>(a);
    return hipGetLastError();
}

hipError_t launch_delta_history(const DeltaRowsArgs& a, hipStream_t s) {
    if (a.seg.single || a.taps > kMaxTaps) return hipErrorInvalidValue;
    if (a.taps < 2 || a.seg.count <= 0) return hipSuccess;
    const int channels = 2 * a.kv * a.dim + a.heads * a.vdim;
    conv_history_kernel<<<dim3((channels + 255) / 256, a.seg.count), 256, 0, s>>>(a, channels);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// second step of the gate projections over prompt chunks: one workgroup = 64 rows x a slice of one gate's features; the rows' operand
// is built once in LDS as bf16 hi + lo fragments, each wave streams its share of the weight fragments
// ---------------------------------------------------------------------------------------------------
// exp(x) for decays and gates: the argument's rounding costs |x| 2^-24 of the result
__device__ __forceinline__ float exp_fast(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
// log(1 + e^z) = max(z, 0) + log1p(e^-|z|) with log1p(t) = log(u) t / (u - 1), u = 1 + t rounded: the quotient undoes u's rounding
__device__ __forceinline__ float softplus_fast(float z) {
    const float t = exp_fast(-fabsf(z)), u = 1.0f + t, d = u - 1.0f;
    const float l = __builtin_amdgcn_logf(u) * 0.6931471805599453f;
    return fmaxf(z, 0.f) + (d == 0.f ? t : l * (t * __builtin_amdgcn_rcpf(d)));
}
__device__ __forceinline__ float sigmoid_fast(float x) { return __builtin_amdgcn_rcpf(1.0f + exp_fast(-x)); }

// STEP: one head of softplus(v + bias) alone (step sizes of a scan)
template <int KT, bool STEP>
__global__ void __launch_bounds__(256) delta_gates_kernel(HeadGemmArgs a) {
    __shared__ __attribute__((aligned(16))) uint4 xs[2 * 4 * KT * 64];  // [plane][row tile][k-tile][lane]
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l15 = lane & 15, grp = lane >> 4;
    const int row0 = blockIdx.x * 64, head = blockIdx.y;
    const uint4* w = a.w + (size_t)head * a.w_head;
    const int ntiles = a.N >> 4;
    uint4 wn[KT];  // the next tile's weights
    auto fetch = [&](int nt) {
#pragma unroll
        for (int k = 0; k < KT; ++k) wn[k] = w[((size_t)min(nt, ntiles - 1) * KT + k) * 64 + lane];
    };
    fetch(blockIdx.z * 4 + wave);
    for (int i = wave; i < 4 * KT; i += 4) {
        const int row = min(row0 + (i / KT) * 16 + l15, a.M - 1);
        const float* p = a.x + (size_t)row * a.x_row + (size_t)head * a.x_head + (i % KT) * 32 + grp * 8;
        float x[8];
        *reinterpret_cast<float4*>(&x[0]) = *reinterpret_cast<const float4*>(p);
        *reinterpret_cast<float4*>(&x[4]) = *reinterpret_cast<const float4*>(p + 4);
        bf16x8 h, l;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            h[j] = (__bf16)x[j];
            l[j] = (__bf16)(x[j] - (float)h[j]);
        }
        xs[i * 64 + lane] = __builtin_bit_cast(uint4, h);
        xs[(4 * KT + i) * 64 + lane] = __builtin_bit_cast(uint4, l);
    }
    __syncthreads();
    for (int nt = blockIdx.z * 4 + wave; nt < ntiles; nt += 4 * gridDim.z) {
        uint4 wf[KT];
#pragma unroll
        for (int k = 0; k < KT; ++k) wf[k] = wn[k];
        fetch(nt + 4 * gridDim.z);
        f32x4 acc[4];
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < KT; ++k) {
                const bf16x8 wv = __builtin_bit_cast(bf16x8, wf[k]);
                acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, __builtin_bit_cast(bf16x8, xs[(b * KT + k) * 64 + lane]), acc[b], 0, 0, 0);
                acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, __builtin_bit_cast(bf16x8, xs[((4 + b) * KT + k) * 64 + lane]), acc[b], 0, 0, 0);
            }
        }
        const int f0 = nt * 16 + grp * 4;
        float4 rate = make_float4(0.f, 0.f, 0.f, 0.f), dt = rate;
        if (STEP || head == 0) {
            if constexpr (!STEP) rate = *reinterpret_cast<const float4*>(a.decay_rate + f0);
            dt = *reinterpret_cast<const float4*>(a.decay_bias + f0);
        }
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            const int row = row0 + b * 16 + l15;
            const f32x4 v = acc[b];
            float4 o;
            if constexpr (STEP) o = make_float4(softplus_fast(v[0] + dt.x), softplus_fast(v[1] + dt.y), softplus_fast(v[2] + dt.z), softplus_fast(v[3] + dt.w));
            else if (head == 0) o = make_float4(exp_fast(-rate.x * softplus_fast(v[0] + dt.x)), exp_fast(-rate.y * softplus_fast(v[1] + dt.y)),
                                           exp_fast(-rate.z * softplus_fast(v[2] + dt.z)), exp_fast(-rate.w * softplus_fast(v[3] + dt.w)));
            else o = make_float4(sigmoid_fast(v[0]), sigmoid_fast(v[1]), sigmoid_fast(v[2]), sigmoid_fast(v[3]));
            if (row < a.M) *reinterpret_cast<float4*>(a.y + (size_t)row * a.y_row + (size_t)head * a.y_head + f0) = o;
        }
    }
}
hipError_t launch_delta_gates(const HeadGemmArgs& a, hipStream_t s) {
    const int kt = a.K / 32;
    const bool step = a.decay_bias && !a.decay_rate && a.heads == 1;
    if (a.exact || kt > 4 + 4 * step || a.N % 16 || a.K % 32 || a.x_row % 4 || a.x_head % 4 || a.y_row % 4 || a.y_head % 4 || a.n_valid != a.N || (!a.decay_rate && !step))
        return launch_head_gemm(a, s);
    if (a.M <= 0) return hipSuccess;
    // eight slices per row block for prompt chunks, for few rows one tile per wave
    const int blocks = (a.M + 63) / 64, tiles = a.N / 16;
    const dim3 grid(blocks, a.heads, std::max(1, std::min((tiles + 3) / 4, std::max(8, 256 / (blocks * a.heads)))));
    switch (step ? kt + 8 : kt) {
        case 1: delta_gates_kernel<1, false><<<grid, 256, 0, s>>>(a); break;
        case 2: delta_gates_kernel<2, false><<<grid, 256, 0, s>>>(a); break;
        case 3: delta_gates_kernel<3, false><<<grid, 256, 0, s>>>(a); break;
        case 4: delta_gates_kernel<4, false><<<grid, 256, 0, s>>>(a); break;
#define NVLLM_ST(K_) case K_ + 8: delta_gates_kernel<K_, true><<<grid, 256, 0, s>>>(a); break;
        NVLLM_ST(1) NVLLM_ST(2) NVLLM_ST(3) NVLLM_ST(4) NVLLM_ST(5) NVLLM_ST(6) NVLLM_ST(7) NVLLM_ST(8)
#undef NVLLM_ST
        default: return hipErrorInvalidValue;
    }
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// gated output norm: one wave per (row, head), or one workgroup per row when the norm runs over all heads
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ float gate_factor(const GatedNormArgs& a, const float* p) {
    if (!a.gate_slabs) return *p;
    const float z = slab_elem(p, a.gate_slabs, a.gate_stride);
    return z * sigmoidf(z);
}
template <bool WHOLE>
__global__ void __launch_bounds__(256) gated_norm_kernel(GatedNormArgs a, int rows) {
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int row = WHOLE ? blockIdx.x : (blockIdx.x * 4 + wave) / a.heads, head0 = WHOLE ? 0 : (blockIdx.x * 4 + wave) % a.heads;
    if (row >= rows) return;  // WHOLE: one row per workgroup, never taken
    const float* o = a.o + ((size_t)row * a.heads + head0) * a.vdim_p;
    const float* gate = a.gate + (size_t)row * a.gate_row + (size_t)head0 * a.gate_head;
    constexpr int step = WHOLE ? 256 : 64;
    const int t0 = WHOLE ? threadIdx.x : lane;
    const float n = WHOLE ? (float)a.all : (float)a.vdim;
    if ((a.vdim & 3) == 0 && ((a.gate_head | a.gate_row | a.gate_stride) & 3) == 0 && (reinterpret_cast<uintptr_t>(a.gate) & 15) == 0) {  // four values of one head per thread; padding columns of o are zero
        const int n4 = WHOLE ? a.heads * (a.vdim_p >> 2) : a.vdim_p >> 2;
        float ss = 0.f;
        if (WHOLE && a.ssq) {
            ss = a.ssq[row * 2];
        } else {
            for (int i = t0; i < n4; i += step) {
                const float4 x = reinterpret_cast<const float4*>(o)[i];
                ss += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
            }
            ss = WHOLE ? block_sum(ss, red, 4) : wave_sum_uniform(ss);
        }
        const float rinv = 1.0f / sqrtf(ss / n + a.eps);
        for (int i = t0; i < n4; i += step) {
            const int h = WHOLE ? i * 4 / a.vdim_p : 0, e = i * 4 - h * a.vdim_p, col = (head0 + h) * a.vdim + e;
            if (e >= a.vdim) continue;
            const float4 x = reinterpret_cast<const float4*>(o)[i];
            float4 g = make_float4(0.f, 0.f, 0.f, 0.f);
            add_slabs(g, gate + (size_t)h * a.gate_head + e, max(a.gate_slabs, 1), a.gate_stride);
            if (a.gate_slabs) g = make_float4(g.x * sigmoidf(g.x), g.y * sigmoidf(g.y), g.z * sigmoidf(g.z), g.w * sigmoidf(g.w));
            const float4 w = *reinterpret_cast<const float4*>(a.weight + (WHOLE ? col : e));
            const f32x4 v = {(x.x * rinv) * w.x * g.x, (x.y * rinv) * w.y * g.y, (x.z * rinv) * w.z * g.z, (x.w * rinv) * w.w * g.w};
            if (a.of) *reinterpret_cast<float4*>(a.of + (size_t)row * a.ld + col) = make_float4(v[0], v[1], v[2], v[3]);
            if (a.oh) put_planes4(a.oh, a.ol, row, col, 4, a.ld, a.packed, v);
        }
        return;
    }
    const int cnt = WHOLE ? a.heads * a.vdim : a.vdim;
    float ss = 0.f;
    if (WHOLE && a.ssq) {
        ss = a.ssq[row * 2];
    } else {
        for (int i = t0; i < cnt; i += step) {
            const int h = WHOLE ? i / a.vdim : 0, e = i - h * a.vdim;
            const float v = o[h * a.vdim_p + e];
            ss += v * v;
        }
        ss = WHOLE ? block_sum(ss, red, 4) : wave_sum_uniform(ss);
    }
    const float rinv = 1.0f / sqrtf(ss / n + a.eps);
    for (int i = t0; i < cnt; i += step) {
        const int h = WHOLE ? i / a.vdim : 0, e = i - h * a.vdim, col = (head0 + h) * a.vdim + e;
        const float v = (o[h * a.vdim_p + e] * rinv) * a.weight[i] * gate_factor(a, gate + (size_t)h * a.gate_head + e);
        if (a.of) a.of[(size_t)row * a.ld + col] = v;
        if (a.oh) {
            const size_t x = a.packed ? xpack_off(row, col, a.ld >> 5) : (size_t)row * a.ld + col;
            split_bf16(v, a.oh[x], a.ol[x]);
        }
    }
}
hipError_t launch_gated_norm(const GatedNormArgs& a, int rows, hipStream_t s) {
    if (a.heads * a.vdim > a.ld || (!a.oh && !a.of) || (a.whole && a.all < 1) || a.vdim_p % 4) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    if (a.whole) gated_norm_kernel<true><<<rows, 256, 0, s>>>(a, rows);
    else gated_norm_kernel<false><<<(rows * a.heads + 3) / 4, 256, 0, s>>>(a, rows);
    return hipGetLastError();
}

}  // namespace nvllm
