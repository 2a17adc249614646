// gfx950 row kernels of the hybrid decoders: squared-ReLU activation, the steps between a mixer's input projection and its attention or
// recurrence (biases, norms, value mixing, cache write; convolution, unit norms, gates), the gated output norm.
#include <algorithm>

#include "device_common.h"
#include "hybrid.h"

namespace nvllm {

__device__ __forceinline__ float sigmoidf(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---------------------------------------------------------------------------------------------------
// squared ReLU
// ---------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256) relu2_kernel(const float* __restrict__ in, int n_slabs, int64_t slab_stride, int rows, int F,
                                                    uint16_t* __restrict__ hi, uint16_t* __restrict__ lo, int packed, float* __restrict__ y) {
    const int64_t total = (int64_t)rows * (F >> 2);
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
        const int r = (int)(i / (F >> 2)), c = (int)(i % (F >> 2)) * 4;
        float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
        add_slabs(s, in + (size_t)r * F + c, n_slabs, slab_stride);
        const f32x4 v = {relu2(s.x), relu2(s.y), relu2(s.z), relu2(s.w)};
        if (y) *reinterpret_cast<float4*>(y + (size_t)r * F + c) = make_float4(v[0], v[1], v[2], v[3]);
        if (hi) put_planes4(hi, lo, r, c, 4, F, packed, v);
    }
}
hipError_t launch_relu2(const float* in, int n_slabs, int64_t slab_stride, int rows, int F, bf16_bits* hi, bf16_bits* lo, int packed, float* y,
                        hipStream_t s) {
    if (F % 32 || n_slabs < 1) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const int64_t wgs = ((int64_t)rows * (F / 4) + 255) / 256;
    relu2_kernel<<<(int)std::min<int64_t>(wgs, 8192), 256, 0, s>>>(in, n_slabs, slab_stride, rows, F, hi, lo, packed, y);
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

__global__ void __launch_bounds__(256) attn_rows_kernel(AttnRowsArgs a) {
    extern __shared__ __attribute__((aligned(16))) float xr[];
    __shared__ float red[4];
    const int row = blockIdx.x;
    const int nq = a.heads * a.kv.dim, nk = a.kv.kv * a.kv.dim, nv = a.kv.kv * a.kv.vdim;
    sum_row(xr, a.in + (size_t)row * a.ld, (nq + nk + nv + 3) & ~3, a.n_slabs, a.slab_stride, a.bias);
    __syncthreads();
    float sq = 0.f, sk = 0.f;
    if (a.ssq) {
        sq = a.ssq[row * 2];
        sk = a.ssq[row * 2 + 1];
    } else {
        for (int c = threadIdx.x; c < nq; c += 256) sq += xr[c] * xr[c];
        for (int c = threadIdx.x; c < nk; c += 256) sk += xr[nq + c] * xr[nq + c];
        sq = block_sum(sq, red, 4);
        sk = block_sum(sk, red, 4);
    }
    const float rq = 1.0f / sqrtf(sq / (float)a.q_all + a.eps), rk = 1.0f / sqrtf(sk / (float)a.k_all + a.eps);
    float* q = a.q + (size_t)row * a.heads * a.kv.dim_p;
    for (int i = threadIdx.x; i < a.heads * a.kv.dim_p; i += 256) {
        const int h = i / a.kv.dim_p, d = i - h * a.kv.dim_p, c = h * a.kv.dim + d;
        q[i] = d < a.kv.dim ? (xr[c] * rq) * a.qn[c] * a.q_scale : 0.f;
    }
    const int pos = a.pos[row], t = pos & (kBlockTokens - 1);
    const size_t blk = (size_t)a.block_tables[(size_t)a.slot[row] * a.max_blocks + pos / kBlockTokens] * a.kv.kv;
    for (int c = threadIdx.x; c < nk; c += 256) {
        const int h = c / a.kv.dim, d = c - h * a.kv.dim;
        kv_put(a.kv.k, a.kv.f32, (blk + h) * kBlockTokens * a.kv.dim_p + k_packed_offset(t, d, a.kv.dim_p), (xr[nq + c] * rk) * a.kn[c]);
    }
    const float lam = a.mix == 2 ? a.lambda[0] : 0.f;
    for (int c = threadIdx.x; c < nv; c += 256) {
        const int h = c / a.kv.vdim, d = c - h * a.kv.vdim;
        float v = xr[nq + nk + c];
        if (a.mix == 1) a.v_first[(size_t)row * nv + c] = v;
        if (a.mix == 2) v = (1.0f - lam) * v + lam * a.v_first[(size_t)row * nv + c];
        kv_put(a.kv.v, a.kv.f32, (blk + h) * kBlockTokens * a.kv.vdim_p + v_packed_offset(t, d, a.kv.vdim_p), v);
    }
}
hipError_t launch_attn_rows(const AttnRowsArgs& a, int rows, hipStream_t s) {
    const int n = a.heads * a.kv.dim + a.kv.kv * (a.kv.dim + a.kv.vdim);
    if (a.kv.dim_p % 32 || a.kv.vdim_p % 16 || n > a.ld || a.ld % 4 || (a.mix && !a.v_first) || (a.mix == 2 && !a.lambda)) return hipErrorInvalidValue;
    const size_t lds = ((size_t)n + 4) * 4;
    if (lds > 64 * 1024) return hipErrorNotSupported;
    if (rows <= 0) return hipSuccess;
    attn_rows_kernel<<<rows, 256, lds, s>>>(a);
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
// delta rule: one wave per (row, unit); units = q heads, k heads, v heads, then one for beta and the gate inputs
// ---------------------------------------------------------------------------------------------------
// what a row sees of the tokens before its chunk: rows back to its segment's start, then the slot's history
struct RowPast {
    int in_chunk = 0;  // earlier rows of the same sequence in this chunk, at most taps - 1
    int pos0 = 0;      // position of the segment's first row (valid when in_chunk < taps - 1)
    int slot = 0;
};
__device__ __forceinline__ RowPast row_past(const DeltaRowsArgs& a, int row) {
    RowPast p;
    p.slot = a.slot[row];
    const int pos = a.pos[row];
    if (!a.seg.single)
        while (p.in_chunk < a.taps - 1 && row - p.in_chunk - 1 >= 0 && a.slot[row - p.in_chunk - 1] == p.slot) ++p.in_chunk;
    p.pos0 = pos - p.in_chunk;
    return p;
}
// raw input of channel c, j tokens before the row
__device__ __forceinline__ float past_input(const DeltaRowsArgs& a, const RowPast& p, int row, int j, int c, int channels) {
    if (j <= p.in_chunk) return slab_elem(a.in + (size_t)(row - j) * a.ld + c, a.n_slabs, a.slab_stride);
    const int back = j - p.in_chunk;  // tokens before the segment
    if (back > p.pos0) return 0.f;
    return a.history[((((size_t)(p.pos0 & 1) * a.slots + p.slot) * (a.taps - 1)) + (a.taps - 1 - back)) * channels + c];
}
__device__ __forceinline__ float conv_silu(const DeltaRowsArgs& a, const RowPast& p, int row, int c, int channels) {
    float y = 0.f;
    for (int i = 0; i < a.taps; ++i) y += past_input(a, p, row, a.taps - 1 - i, c, channels) * a.conv[(size_t)i * channels + c];
    return y * sigmoidf(y);
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
        const float* in = a.in + (size_t)row * a.ld + channels;
        for (int h = lane; h < a.heads; h += 64) a.beta[(size_t)row * a.heads + h] = sigmoidf(slab_elem(in + h, a.n_slabs, a.slab_stride));
        for (int i = lane; i < 2 * a.rank_p; i += 64) a.gate_in[(size_t)row * 2 * a.rank_p + i] = slab_elem(in + a.heads + i, a.n_slabs, a.slab_stride);
    }
    if (!a.seg.single || a.taps < 2) return;
    // decode: the next half of the history = this half moved on by one token
    const int pos = a.pos[row];
    const int c0 = unit < 2 * a.kv ? unit * a.dim : 2 * a.kv * a.dim + (unit - 2 * a.kv) * a.vdim;
    const int n = unit < 2 * a.kv ? a.dim : unit < 2 * a.kv + a.heads ? a.vdim : 0;
    float* next = a.history + ((size_t)((pos + 1) & 1) * a.slots + p.slot) * (a.taps - 1) * channels;
    for (int d = lane; d < n; d += 64)
        for (int i = 0; i < a.taps - 1; ++i) next[(size_t)i * channels + c0 + d] = past_input(a, p, row, a.taps - 2 - i, c0 + d, channels);
}
hipError_t launch_delta_rows(const DeltaRowsArgs& a, int rows, hipStream_t s) {
    if (a.dim_p % 4 || a.vdim_p % 4 || a.taps < 1 || 2 * a.kv * a.dim + a.heads * (a.vdim + 1) + 2 * a.rank_p > a.ld) return hipErrorInvalidValue;
    if (a.dim_p > 512) return hipErrorNotSupported;
    if (rows <= 0) return hipSuccess;
    const dim3 grid(rows, (2 * a.kv + a.heads + 1 + 3) / 4);
    if (a.dim_p <= 64) delta_rows_kernel<1><<<grid, 256, 0, s>>>(a);
    else if (a.dim_p <= 128) delta_rows_kernel<2><<<grid, 256, 0, s>>>(a);
    else if (a.dim_p <= 256) delta_rows_kernel<4><<<grid, 256, 0, s>>>(a);
    else delta_rows_kernel<8><<<grid, 256, 0, s>>>(a);
    return hipGetLastError();
}

// one thread per (segment, channel): everything the segment leaves behind is read before it is written
constexpr int kMaxTaps = 16;
__global__ void __launch_bounds__(256) delta_history_kernel(DeltaRowsArgs a) {
    const int channels = 2 * a.kv * a.dim + a.heads * a.vdim;
    const int c = blockIdx.x * 256 + threadIdx.x, sg = blockIdx.y;
    if (c >= channels) return;
    const int row = a.seg.row0[sg] + a.seg.n[sg] - 1;
    RowPast p;
    p.slot = a.seg.slot[sg];
    p.in_chunk = a.seg.n[sg] - 1;
    p.pos0 = a.pos[a.seg.row0[sg]];
    float x[kMaxTaps - 1];
#pragma unroll
    for (int i = 0; i < kMaxTaps - 1; ++i)
        if (i < a.taps - 1) x[i] = past_input(a, p, row, a.taps - 2 - i, c, channels);
    float* next = a.history + ((size_t)((a.pos[row] + 1) & 1) * a.slots + p.slot) * (a.taps - 1) * channels;
#pragma unroll
    for (int i = 0; i < kMaxTaps - 1; ++i)
        if (i < a.taps - 1) next[(size_t)i * channels + c] = x[i];
}
hipError_t launch_delta_history(const DeltaRowsArgs& a, hipStream_t s) {
    if (a.seg.single || a.taps > kMaxTaps) return hipErrorInvalidValue;
    if (a.taps < 2 || a.seg.count <= 0) return hipSuccess;
    const int channels = 2 * a.kv * a.dim + a.heads * a.vdim;
    delta_history_kernel<<<dim3((channels + 255) / 256, a.seg.count), 256, 0, s>>>(a);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// gated output norm: one wave per (row, head), or one workgroup per row when the norm runs over all heads
// ---------------------------------------------------------------------------------------------------
template <bool WHOLE>
__global__ void __launch_bounds__(256) gated_norm_kernel(GatedNormArgs a, int rows) {
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int row = WHOLE ? blockIdx.x : (blockIdx.x * 4 + wave) / a.heads, head0 = WHOLE ? 0 : (blockIdx.x * 4 + wave) % a.heads;
    if (row >= rows) return;  // WHOLE: one row per workgroup, never taken
    const float* o = a.o + (size_t)row * a.heads * a.vdim_p;
    const int n = WHOLE ? a.heads * a.vdim : a.vdim, t0 = WHOLE ? threadIdx.x : lane;
    constexpr int step = WHOLE ? 256 : 64;
    float ss = 0.f;
    if (WHOLE && a.ssq) {
        ss = a.ssq[row * 2];
    } else {
        for (int i = t0; i < n; i += step) {
            const int h = WHOLE ? i / a.vdim : 0, e = i - h * a.vdim;
            const float v = o[(head0 + h) * a.vdim_p + e];
            ss += v * v;
        }
        ss = WHOLE ? block_sum(ss, red, 4) : wave_sum(ss);
    }
    const float rinv = 1.0f / sqrtf(ss / (float)(WHOLE ? a.all : n) + a.eps);
    const float* gate = a.gate + (size_t)row * a.gate_row;
    for (int i = t0; i < n; i += step) {
        const int h = head0 + (WHOLE ? i / a.vdim : 0), e = WHOLE ? i - h * a.vdim : i, col = h * a.vdim + e;
        const float v = (o[h * a.vdim_p + e] * rinv) * a.weight[i] * gate[h * a.gate_head + e];
        if (a.of) a.of[(size_t)row * a.ld + col] = v;
        if (a.oh) {
            const size_t x = a.packed ? xpack_off(row, col, a.ld >> 5) : (size_t)row * a.ld + col;
            split_bf16(v, a.oh[x], a.ol[x]);
        }
    }
}
hipError_t launch_gated_norm(const GatedNormArgs& a, int rows, hipStream_t s) {
    if (a.heads * a.vdim > a.ld || (!a.oh && !a.of) || (a.whole && a.all < 1)) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    if (a.whole) gated_norm_kernel<true><<<rows, 256, 0, s>>>(a, rows);
    else gated_norm_kernel<false><<<(rows * a.heads + 3) / 4, 256, 0, s>>>(a, rows);
    return hipGetLastError();
}

}  // namespace nvllm
