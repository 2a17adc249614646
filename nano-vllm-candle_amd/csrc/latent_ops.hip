// gfx950 kernels of the latent-attention decoders: row kernels (residual + norms, query split / rotation / cache write),
// per-head and 32-bit matrix products, the plain attention kernel (any size, f16 or f32 cache), the logits finish.
#include <algorithm>

#include "device_common.h"
#include "latent.h"

namespace nvllm {

// ---------------------------------------------------------------------------------------------------
// residual add + up to two norms of the same row; one workgroup per row, 4 columns per thread and step
// ---------------------------------------------------------------------------------------------------
constexpr int kAddNormMax = 8192;  // widest row

enum { NORM_PLAIN, NORM_POST, NORM_CENTER, NORM_BRANCH };  // NORM_BRANCH: two normed branches, then as NORM_POST

// BS = 256, or 1024 for few wide rows (decode): every thread's loads are then in flight at once
template <int BS, int KIND>
__global__ void __launch_bounds__(BS) add_norm_kernel(AddNormArgs a) {
    constexpr bool POST = KIND == NORM_POST || KIND == NORM_BRANCH;
    constexpr int NV = kAddNormMax / 4 / BS;
    __shared__ float red[BS / 64];
    float4 other[KIND == NORM_BRANCH ? NV : 1];
    float so = 0.f;
    const int r = blockIdx.x;
    const int src = a.row_idx ? a.row_idx[r] : r;
    const int nv4 = a.ldr >> 2;
    float4 cache[NV], res[POST ? NV : 1];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < NV; ++c) {
        const int i = threadIdx.x + c * BS;
        if (i < nv4) {
            float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
            if (!POST && a.ids) {
                const uint2 e = *reinterpret_cast<const uint2*>(a.embed + (size_t)a.ids[src] * a.ldr + (size_t)i * 4);
                s = make_float4(bf16_to_f32(e.x & 0xffff) * a.embed_scale, bf16_to_f32(e.x >> 16) * a.embed_scale,
                                bf16_to_f32(e.y & 0xffff) * a.embed_scale, bf16_to_f32(e.y >> 16) * a.embed_scale);
            } else {
                if (a.in) add_slabs(s, a.in + (size_t)src * a.ldr + (size_t)i * 4, a.n_slabs, a.slab_stride);
                if (POST && a.in_bias) {
                    const float4 b = *reinterpret_cast<const float4*>(a.in_bias + (size_t)i * 4);
                    s.x += b.x; s.y += b.y; s.z += b.z; s.w += b.w;
                }
                if constexpr (KIND == NORM_BRANCH) {
                    float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
                    add_slabs(t, a.in2 + (size_t)src * a.ldr + (size_t)i * 4, a.n_slabs2, a.slab_stride2);
                    other[c] = t;
                    so += t.x * t.x + t.y * t.y + t.z * t.z + t.w * t.w;
                } else if (a.in2) {
                    float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
                    add_slabs(t, a.in2 + (size_t)src * a.ldr + (size_t)i * 4, a.n_slabs2, a.slab_stride2);
                    const float f = a.in2_scale ? a.in2_scale[src] : 1.f;
                    s.x += t.x * f; s.y += t.y * f; s.z += t.z * f; s.w += t.w * f;
                }
                for (int k = 0; k < a.n_gather; ++k) {
                    const float4 t = *reinterpret_cast<const float4*>(a.gather + (size_t)a.gather_row[(size_t)src * a.n_gather + k] * a.ldr + (size_t)i * 4);
                    s.x += t.x; s.y += t.y; s.z += t.z; s.w += t.w;
                }
            }
            float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
            if (a.residual_in) t = *reinterpret_cast<const float4*>(a.residual_in + (size_t)src * a.ldr + (size_t)i * 4);
            if constexpr (POST) {
                res[c] = t;
            } else {
                if (a.residual_in) { s.x += t.x; s.y += t.y; s.z += t.z; s.w += t.w; }
                if (a.residual_out) *reinterpret_cast<float4*>(a.residual_out + (size_t)src * a.ldr + (size_t)i * 4) = s;
            }
            cache[c] = s;
            ss += KIND == NORM_CENTER ? (s.x + s.y) + (s.z + s.w) : s.x * s.x + s.y * s.y + s.z * s.z + s.w * s.w;
        }
    }
    if constexpr (KIND == NORM_CENTER) {
        if (!a.w[0] && !a.w[1]) return;
        const float mean = block_sum(ss, red, BS / 64) / (float)a.W;
        ss = 0.f;
#pragma unroll
        for (int c = 0; c < NV; ++c) {
            const int i = threadIdx.x + c * BS;
            if (i >= nv4) continue;
            float4 s = cache[c];
            s.x = i * 4 < a.W ? s.x - mean : 0.f; s.y = i * 4 + 1 < a.W ? s.y - mean : 0.f;
            s.z = i * 4 + 2 < a.W ? s.z - mean : 0.f; s.w = i * 4 + 3 < a.W ? s.w - mean : 0.f;
            cache[c] = s;
            ss += s.x * s.x + s.y * s.y + s.z * s.z + s.w * s.w;
        }
    }
    if constexpr (KIND == NORM_BRANCH) {
        const float f = 0.5f / sqrtf(block_sum(ss, red, BS / 64) / (float)a.W + a.eps), fo = 0.5f / sqrtf(block_sum(so, red, BS / 64) / (float)a.W + a.eps);
        ss = 0.f;
#pragma unroll
        for (int c = 0; c < NV; ++c) {
            const int i = threadIdx.x + c * BS;
            if (i >= nv4) continue;
            const float4 w = *reinterpret_cast<const float4*>(a.branch_w[0] + (size_t)i * 4), v = *reinterpret_cast<const float4*>(a.branch_w[1] + (size_t)i * 4);
            float4 s = cache[c];
            const float4 t = other[c];
            s.x = (s.x * f) * w.x + (t.x * fo) * v.x; s.y = (s.y * f) * w.y + (t.y * fo) * v.y;
            s.z = (s.z * f) * w.z + (t.z * fo) * v.z; s.w = (s.w * f) * w.w + (t.w * fo) * v.w;
            cache[c] = s;
            ss += s.x * s.x + s.y * s.y + s.z * s.z + s.w * s.w;
        }
    }
    if constexpr (POST) {
        const float f = a.post_mult / sqrtf(block_sum(ss, red, BS / 64) / (float)a.W + a.eps);
        ss = 0.f;
#pragma unroll
        for (int c = 0; c < NV; ++c) {
            const int i = threadIdx.x + c * BS;
            if (i >= nv4) continue;
            const float4 w = *reinterpret_cast<const float4*>(a.post_w + (size_t)i * 4);
            float4 s = cache[c];
            s.x = res[c].x + (s.x * f) * w.x; s.y = res[c].y + (s.y * f) * w.y; s.z = res[c].z + (s.z * f) * w.z; s.w = res[c].w + (s.w * f) * w.w;
            if (a.again) {
                const uint2 e = *reinterpret_cast<const uint2*>(a.embed + (size_t)a.ids[src] * a.ldr + (size_t)i * 4);
                s.x += bf16_to_f32(e.x & 0xffff) * a.embed_scale; s.y += bf16_to_f32(e.x >> 16) * a.embed_scale;
                s.z += bf16_to_f32(e.y & 0xffff) * a.embed_scale; s.w += bf16_to_f32(e.y >> 16) * a.embed_scale;
            }
            if (a.residual_out) *reinterpret_cast<float4*>(a.residual_out + (size_t)src * a.ldr + (size_t)i * 4) = s;
            cache[c] = s;
            ss += s.x * s.x + s.y * s.y + s.z * s.z + s.w * s.w;
        }
    }
    if (!a.w[0] && !a.w[1] && !a.raw) return;
    const float rinv = a.w[0] || a.w[1] ? 1.0f / sqrtf(block_sum(ss, red, BS / 64) / (float)a.W + a.eps) : 1.f;
    const int no4 = a.ldx >> 2;
#pragma unroll
    for (int c = 0; c < NV; ++c) {
        const int i = threadIdx.x + c * BS;
        if (i >= no4) continue;
        const float4 s = i < nv4 ? cache[c] : make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const bool raw = k == 0 && a.raw;
            if (!a.w[k] && !raw) continue;
            float y0 = s.x, y1 = s.y, y2 = s.z, y3 = s.w;
            if (!raw) {
                const float4 w = *reinterpret_cast<const float4*>(a.w[k] + (size_t)i * 4);
                y0 = (s.x * rinv) * w.x; y1 = (s.y * rinv) * w.y; y2 = (s.z * rinv) * w.z; y3 = (s.w * rinv) * w.w;
            }
            if (a.y[k]) *reinterpret_cast<float4*>(a.y[k] + (size_t)r * a.ldx + (size_t)i * 4) = make_float4(y0, y1, y2, y3);
            if (a.xh[k]) {
                uint16_t h0, h1, h2, h3, l0, l1, l2, l3;
                split_bf16(y0, h0, l0); split_bf16(y1, h1, l1); split_bf16(y2, h2, l2); split_bf16(y3, h3, l3);
                const size_t xo = a.packed[k] ? xpack_off(r, i * 4, a.ldx >> 5) : (size_t)r * a.ldx + (size_t)i * 4;
                *reinterpret_cast<uint2*>(a.xh[k] + xo) = make_uint2(h0 | ((uint32_t)h1 << 16), h2 | ((uint32_t)h3 << 16));
                *reinterpret_cast<uint2*>(a.xl[k] + xo) = make_uint2(l0 | ((uint32_t)l1 << 16), l2 | ((uint32_t)l3 << 16));
            }
        }
    }
}

// prompt chunks whose outputs are planes in fragment order: one workgroup = 16 rows, lane (grp, l15) owns row l15's eight consecutive
// columns of k-tiles wave, wave + 16, ...  Reads are whole 128-byte lines, every plane store one contiguous KiB per wave.
template <int IT, int KIND>
__global__ void __launch_bounds__(1024) add_norm_rows16_kernel(AddNormArgs a, int rows) {
    constexpr int NW = 16;
    constexpr bool POST = KIND == NORM_POST || KIND == NORM_BRANCH;
    __shared__ float red[KIND == NORM_PLAIN ? 1 : KIND == NORM_BRANCH ? 4 : 2][NW][16];
    constexpr bool HOLD = KIND == NORM_BRANCH && IT <= 4;  // the second branch in registers; the widest rows read it again
    float o[HOLD ? IT : 1][8];
    float so = 0.f;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l15 = lane & 15, grp = lane >> 4;
    const int KT = a.ldr >> 5, row = blockIdx.x * 16 + l15, rowc = min(row, rows - 1);
    float v[IT][8];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < IT; ++i) {
        const int kt = wave + i * NW;
        if (kt >= KT) continue;
        const size_t col = (size_t)kt * 32 + grp * 8, off = (size_t)rowc * a.ldr + col;
        float4 s0 = make_float4(0.f, 0.f, 0.f, 0.f), s1 = s0;
        if (!POST && a.ids) {
            const uint4 e = *reinterpret_cast<const uint4*>(a.embed + (size_t)a.ids[rowc] * a.ldr + col);
            const float f = a.embed_scale;
            s0 = make_float4(bf16_to_f32(e.x & 0xffff) * f, bf16_to_f32(e.x >> 16) * f, bf16_to_f32(e.y & 0xffff) * f, bf16_to_f32(e.y >> 16) * f);
            s1 = make_float4(bf16_to_f32(e.z & 0xffff) * f, bf16_to_f32(e.z >> 16) * f, bf16_to_f32(e.w & 0xffff) * f, bf16_to_f32(e.w >> 16) * f);
        } else {
            auto add = [&](const float* p, float f = 1.f) {
                const float4 t0 = *reinterpret_cast<const float4*>(p), t1 = *reinterpret_cast<const float4*>(p + 4);
                s0.x += t0.x * f; s0.y += t0.y * f; s0.z += t0.z * f; s0.w += t0.w * f;
                s1.x += t1.x * f; s1.y += t1.y * f; s1.z += t1.z * f; s1.w += t1.w * f;
            };
            const size_t off_in = a.ld_in ? (size_t)rowc * a.ld_in + col : off;
            if (a.in) for (int sl = 0; sl < a.n_slabs; ++sl) add(a.in + (size_t)sl * a.slab_stride + off_in);
            if (POST && a.in_bias) add(a.in_bias + col);
            if constexpr (KIND == NORM_BRANCH) {
                const float4 k0 = s0, k1 = s1;
                s0 = s1 = make_float4(0.f, 0.f, 0.f, 0.f);
                for (int sl = 0; sl < a.n_slabs2; ++sl) add(a.in2 + (size_t)sl * a.slab_stride2 + off);
                so += s0.x * s0.x + s0.y * s0.y + s0.z * s0.z + s0.w * s0.w + s1.x * s1.x + s1.y * s1.y + s1.z * s1.z + s1.w * s1.w;
                if constexpr (HOLD) {
                    o[i][0] = s0.x; o[i][1] = s0.y; o[i][2] = s0.z; o[i][3] = s0.w;
                    o[i][4] = s1.x; o[i][5] = s1.y; o[i][6] = s1.z; o[i][7] = s1.w;
                }
                s0 = k0; s1 = k1;
            } else if (a.in2) {
                const float f = a.in2_scale ? a.in2_scale[rowc] : 1.f;
                for (int sl = 0; sl < a.n_slabs2; ++sl) add(a.in2 + (size_t)sl * a.slab_stride2 + off, f);
            }
            for (int k = 0; k < a.n_gather; ++k) add(a.gather + (size_t)a.gather_row[(size_t)rowc * a.n_gather + k] * a.ldr + col);
            if (!POST && a.residual_in) add(a.residual_in + off);
        }
        if (!POST && a.residual_out && row < rows) {
            *reinterpret_cast<float4*>(a.residual_out + off) = s0;
            *reinterpret_cast<float4*>(a.residual_out + off + 4) = s1;
        }
        v[i][0] = s0.x; v[i][1] = s0.y; v[i][2] = s0.z; v[i][3] = s0.w;
        v[i][4] = s1.x; v[i][5] = s1.y; v[i][6] = s1.z; v[i][7] = s1.w;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += KIND == NORM_CENTER ? v[i][e] : v[i][e] * v[i][e];
    }
    auto row_sum = [&](float (&rd)[NW][16]) {
        ss += __shfl_xor(ss, 16);
        ss += __shfl_xor(ss, 32);
        if (grp == 0) rd[wave][l15] = ss;
        __syncthreads();
        ss = 0.f;
#pragma unroll
        for (int q = 0; q < NW; ++q) ss += rd[q][l15];
        return ss;
    };
    auto row_rinv = [&](float (&rd)[NW][16]) { return 1.0f / sqrtf(row_sum(rd) / (float)a.W + a.eps); };
    if constexpr (KIND == NORM_CENTER) {
        const float mean = row_sum(red[1]) / (float)a.W;
        ss = 0.f;
#pragma unroll
        for (int i = 0; i < IT; ++i) {
            const int kt = wave + i * NW;
            if (kt >= KT) continue;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                v[i][e] = kt * 32 + grp * 8 + e < a.W ? v[i][e] - mean : 0.f;
                ss += v[i][e] * v[i][e];
            }
        }
    }
    if constexpr (KIND == NORM_BRANCH) {
        const float f = 0.5f * row_rinv(red[2]);
        ss = so;
        const float fo = 0.5f * row_rinv(red[3]);
        ss = 0.f;
#pragma unroll
        for (int i = 0; i < IT; ++i) {
            const int kt = wave + i * NW;
            if (kt >= KT) continue;
            const float *w = a.branch_w[0] + kt * 32 + grp * 8, *u = a.branch_w[1] + kt * 32 + grp * 8;
            float4 x0 = make_float4(0.f, 0.f, 0.f, 0.f), x1 = x0;
            if constexpr (HOLD) {
                x0 = make_float4(o[i][0], o[i][1], o[i][2], o[i][3]);
                x1 = make_float4(o[i][4], o[i][5], o[i][6], o[i][7]);
            } else {
                const float* p = a.in2 + (size_t)rowc * a.ldr + kt * 32 + grp * 8;
                add_slabs(x0, p, a.n_slabs2, a.slab_stride2);
                add_slabs(x1, p + 4, a.n_slabs2, a.slab_stride2);
            }
            const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                v[i][e] = (v[i][e] * f) * w[e] + (x[e] * fo) * u[e];
                ss += v[i][e] * v[i][e];
            }
        }
    }
    if constexpr (POST) {
        const float f = row_rinv(red[1]) * a.post_mult;
        ss = 0.f;
#pragma unroll
        for (int i = 0; i < IT; ++i) {
            const int kt = wave + i * NW;
            if (kt >= KT) continue;
            const size_t col = (size_t)kt * 32 + grp * 8, off = (size_t)rowc * a.ldr + col;
            float4 s0 = *reinterpret_cast<const float4*>(a.residual_in + off), s1 = *reinterpret_cast<const float4*>(a.residual_in + off + 4);
            const float4 w0 = *reinterpret_cast<const float4*>(a.post_w + col), w1 = *reinterpret_cast<const float4*>(a.post_w + col + 4);
            s0.x += (v[i][0] * f) * w0.x; s0.y += (v[i][1] * f) * w0.y; s0.z += (v[i][2] * f) * w0.z; s0.w += (v[i][3] * f) * w0.w;
            s1.x += (v[i][4] * f) * w1.x; s1.y += (v[i][5] * f) * w1.y; s1.z += (v[i][6] * f) * w1.z; s1.w += (v[i][7] * f) * w1.w;
            if (a.again) {
                const uint4 e = *reinterpret_cast<const uint4*>(a.embed + (size_t)a.ids[rowc] * a.ldr + col);
                const float fe = a.embed_scale;
                s0.x += bf16_to_f32(e.x & 0xffff) * fe; s0.y += bf16_to_f32(e.x >> 16) * fe; s0.z += bf16_to_f32(e.y & 0xffff) * fe; s0.w += bf16_to_f32(e.y >> 16) * fe;
                s1.x += bf16_to_f32(e.z & 0xffff) * fe; s1.y += bf16_to_f32(e.z >> 16) * fe; s1.z += bf16_to_f32(e.w & 0xffff) * fe; s1.w += bf16_to_f32(e.w >> 16) * fe;
            }
            if (a.residual_out && row < rows) {
                *reinterpret_cast<float4*>(a.residual_out + off) = s0;
                *reinterpret_cast<float4*>(a.residual_out + off + 4) = s1;
            }
            v[i][0] = s0.x; v[i][1] = s0.y; v[i][2] = s0.z; v[i][3] = s0.w;
            v[i][4] = s1.x; v[i][5] = s1.y; v[i][6] = s1.z; v[i][7] = s1.w;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss += v[i][e] * v[i][e];
        }
    }
    const float rinv = a.w[0] || a.w[1] ? row_rinv(red[0]) : 1.f;
#pragma unroll
    for (int i = 0; i < IT; ++i) {
        const int kt = wave + i * NW;
        if (kt >= KT) continue;
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const bool raw = k == 0 && a.raw;
            if (!a.w[k] && !raw) continue;
            float wv[8];
            if (!raw) {
                const float4 w0 = *reinterpret_cast<const float4*>(a.w[k] + kt * 32 + grp * 8), w1 = *reinterpret_cast<const float4*>(a.w[k] + kt * 32 + grp * 8 + 4);
                wv[0] = w0.x; wv[1] = w0.y; wv[2] = w0.z; wv[3] = w0.w; wv[4] = w1.x; wv[5] = w1.y; wv[6] = w1.z; wv[7] = w1.w;
            }
            uint16_t h[8], l[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) split_bf16(raw ? v[i][e] : (v[i][e] * rinv) * wv[e], h[e], l[e]);
            if (!a.packed[k] && row >= rows) continue;
            const size_t o = a.packed[k] ? ((size_t)blockIdx.x * KT + kt) * 64 + lane : (((size_t)row * a.ldx) >> 3) + kt * 4 + grp;
            reinterpret_cast<uint4*>(a.xh[k])[o] = make_uint4(h[0] | ((uint32_t)h[1] << 16), h[2] | ((uint32_t)h[3] << 16), h[4] | ((uint32_t)h[5] << 16), h[6] | ((uint32_t)h[7] << 16));
            reinterpret_cast<uint4*>(a.xl[k])[o] = make_uint4(l[0] | ((uint32_t)l[1] << 16), l[2] | ((uint32_t)l[3] << 16), l[4] | ((uint32_t)l[5] << 16), l[6] | ((uint32_t)l[7] << 16));
        }
    }
}

hipError_t launch_add_norm(const AddNormArgs& a, int rows, hipStream_t s) {
    if (a.ldr % 16 || a.ldr > kAddNormMax || ((a.w[0] || a.w[1] || a.raw) && (a.ldx % 16 || a.ldx < a.ldr || a.ldx > kAddNormMax)))
        return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const bool post = a.post_w != nullptr, any = a.w[0] || a.w[1] || a.raw;
    const bool branch = a.branch_w[0] != nullptr;
    if (a.raw && a.w[0]) return hipErrorInvalidValue;
    if ((a.again && (!post || !a.ids || !a.embed)) || (a.in_bias && !post) || (branch && (!post || !a.branch_w[1] || !a.in || !a.in2 || a.in2_scale || a.n_gather))) return hipErrorInvalidValue;
    bool packed = any && a.ldr == a.ldx && a.ldr % 32 == 0 && !a.row_idx && (!post || a.residual_in);
    for (int k = 0; k < 2; ++k) packed &= !(a.w[k] || (k == 0 && a.raw)) || ((a.packed[k] || (k == 1 && a.w[0])) && a.xh[k] && !a.y[k]);
    if ((a.center && (post || a.raw)) || (a.ld_in && (!packed || a.ldr > 4096 || a.ld_in % 4 || a.slab_stride % 4))) return hipErrorInvalidValue;
    auto launch = [&](auto P) {
        constexpr int KIND = decltype(P)::value;
        if (packed && (rows >= 512 || a.ld_in) && a.ldr <= 4096) {
            const int kt = a.ldr / 32, tiles = (rows + 15) / 16;
            if (kt <= 32) add_norm_rows16_kernel<2, KIND><<<tiles, 1024, 0, s>>>(a, rows);
            else if (kt <= 64) add_norm_rows16_kernel<4, KIND><<<tiles, 1024, 0, s>>>(a, rows);
            else add_norm_rows16_kernel<8, KIND><<<tiles, 1024, 0, s>>>(a, rows);
        } else if (rows <= 128 && a.ldr >= 2048) {
            add_norm_kernel<1024, KIND><<<rows, 1024, 0, s>>>(a);
        } else {
            add_norm_kernel<256, KIND><<<rows, 256, 0, s>>>(a);
        }
    };
    if (branch) launch(std::integral_constant<int, NORM_BRANCH>{});
    else if (post) launch(std::integral_constant<int, NORM_POST>{});
    else if (a.center) launch(std::integral_constant<int, NORM_CENTER>{});
    else launch(std::integral_constant<int, NORM_PLAIN>{});
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// rows of the q / latent projection: one wave per (row, head); head index `heads` = the latent part
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ void cache_put(const LatentCache& c, size_t block_base, int t, int d, float v) {
    const size_t o = block_base + k_packed_offset(t, d, c.D());
    if (c.f32) reinterpret_cast<float*>(c.data)[o] = v;
    else reinterpret_cast<_Float16*>(c.data)[o] = f16_sat(v);
}

// one wave: the row's latent (RMS norm over `rank`) and rotated key part into the cache
__device__ __forceinline__ void latent_to_cache(const LatentRowsArgs& a, int row, int lane) {
    const LatentCache& c = a.cache;
    const int half = c.rot >> 1, pos = a.pos[row];
    const float* in = a.kv + (size_t)row * a.ldkv;
    const float* cs = a.cos + (size_t)pos * half;
    const float* sn = a.sin + (size_t)pos * half;
    const int blk = a.block_tables[(size_t)a.slot[row] * a.max_blocks + (pos / kBlockTokens)];
    const size_t base = (size_t)blk * kBlockTokens * c.D();
    const int t = pos & (kBlockTokens - 1);
    if (c.rank <= 512) {  // the whole latent in registers: one pass, independent loads
        float v[8], w[8], ss = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int d = min(lane + i * 64, c.rank - 1);
            v[i] = in[d];
            w[i] = a.norm_w[d];
        }
        for (int sl0 = 1; sl0 < a.kv_slabs; sl0 += 4) {
            float t[4][8];
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int i = 0; i < 8; ++i) t[u][i] = in[(size_t)min(sl0 + u, a.kv_slabs - 1) * a.kv_stride + min(lane + i * 64, c.rank - 1)];
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int i = 0; i < 8; ++i) v[i] += sl0 + u < a.kv_slabs ? t[u][i] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += lane + i * 64 < c.rank ? v[i] * v[i] : 0.f;
        const float rinv = 1.0f / sqrtf(wave_sum(ss) / (float)c.rank + a.eps);
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (lane + i * 64 < c.rank) cache_put(c, base, t, lane + i * 64, v[i] * rinv * w[i]);
    } else {
        float ss = 0.f;
        for (int d = lane; d < c.rank; d += 64) {
            const float v = slab_elem(in + d, a.kv_slabs, a.kv_stride);
            ss += v * v;
        }
        const float rinv = 1.0f / sqrtf(wave_sum(ss) / (float)c.rank + a.eps);
        for (int d = lane; d < c.rank; d += 64) cache_put(c, base, t, d, slab_elem(in + d, a.kv_slabs, a.kv_stride) * rinv * a.norm_w[d]);
    }
    for (int i = lane; i < half; i += 64) {
        const float u = slab_elem(in + c.rank + i, a.kv_slabs, a.kv_stride), v = slab_elem(in + c.rank + half + i, a.kv_slabs, a.kv_stride);
        cache_put(c, base, t, c.rank_p + i, u * cs[i] - v * sn[i]);
        cache_put(c, base, t, c.rank_p + half + i, v * cs[i] + u * sn[i]);
    }
}

__global__ void __launch_bounds__(256) latent_rows_kernel(LatentRowsArgs a) {
    const int lane = threadIdx.x & 63;
    const int row = blockIdx.x, head = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (head > a.heads || (head == a.heads && !a.kv)) return;
    const LatentCache& c = a.cache;
    const int rot = c.rot, half = rot >> 1, pos = a.pos[row];
    const float* in = a.qkv + (size_t)row * a.ldq + (size_t)head * (a.dim + rot);
    const float* cs = a.cos + (size_t)pos * half;
    const float* sn = a.sin + (size_t)pos * half;
    if (head < a.heads) {
        const int dq = a.dim_p + c.rot_p;
        float* q = a.q + ((size_t)row * a.heads + head) * dq;
        if (((a.dim | half | a.ldq) & 3) == 0 && (a.slab_stride & 3) == 0) {  // four elements per lane
            auto sum4 = [&](const float* p) {
                float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
                add_slabs(v, p, a.n_slabs, a.slab_stride);
                return v;
            };
            const int n4 = a.dim_p >> 2, h4 = half >> 2, z4 = (c.rot_p - rot) >> 2;
            for (int i = lane; i < n4 + h4 + z4; i += 64) {
                if (i < n4) {
                    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
                    if (i * 4 < a.dim) v = sum4(in + i * 4);
                    *reinterpret_cast<float4*>(q + i * 4) = make_float4(v.x * a.scale, v.y * a.scale, v.z * a.scale, v.w * a.scale);
                } else if (i < n4 + h4) {
                    const int k = (i - n4) * 4;
                    const float4 u = sum4(in + a.dim + k), v = sum4(in + a.dim + half + k);
                    const float4 co = *reinterpret_cast<const float4*>(cs + k), si = *reinterpret_cast<const float4*>(sn + k);
                    float* o = q + a.dim_p + k;
                    *reinterpret_cast<float4*>(o) = make_float4((u.x * co.x - v.x * si.x) * a.scale, (u.y * co.y - v.y * si.y) * a.scale,
                                                                (u.z * co.z - v.z * si.z) * a.scale, (u.w * co.w - v.w * si.w) * a.scale);
                    *reinterpret_cast<float4*>(o + half) = make_float4((v.x * co.x + u.x * si.x) * a.scale, (v.y * co.y + u.y * si.y) * a.scale,
                                                                       (v.z * co.z + u.z * si.z) * a.scale, (v.w * co.w + u.w * si.w) * a.scale);
                } else {
                    *reinterpret_cast<float4*>(q + a.dim_p + rot + (i - n4 - h4) * 4) = make_float4(0.f, 0.f, 0.f, 0.f);
                }
            }
            return;
        }
        for (int d = lane; d < a.dim_p; d += 64) q[d] = d < a.dim ? slab_elem(in + d, a.n_slabs, a.slab_stride) * a.scale : 0.f;
        float* qr = q + a.dim_p;
        for (int i = lane; i < half; i += 64) {
            const float u = slab_elem(in + a.dim + i, a.n_slabs, a.slab_stride), v = slab_elem(in + a.dim + half + i, a.n_slabs, a.slab_stride);
            qr[i] = (u * cs[i] - v * sn[i]) * a.scale;
            qr[i + half] = (v * cs[i] + u * sn[i]) * a.scale;
        }
        for (int d = rot + lane; d < c.rot_p; d += 64) qr[d] = 0.f;
        return;
    }
    latent_to_cache(a, row, lane);
}

__global__ void __launch_bounds__(256) latent_cache_kernel(LatentRowsArgs a, int rows) {
    const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row < rows) latent_to_cache(a, row, threadIdx.x & 63);
}
hipError_t launch_latent_cache(const LatentRowsArgs& a, int rows, hipStream_t s) {
    if (a.cache.rot % 2 || a.cache.rank_p % 32 || a.cache.rot_p % 32) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    latent_cache_kernel<<<(rows + 3) / 4, 256, 0, s>>>(a, rows);
    return hipGetLastError();
}

__global__ void __launch_bounds__(256) query_latent_kernel(QueryLatentArgs a, LatentRowsArgs kv) {
    __shared__ float red[4];
    const int row = blockIdx.x;
    if (blockIdx.y) {
        if (threadIdx.x < 64) latent_to_cache(kv, row, threadIdx.x);
        return;
    }
    const float* in = a.in + (size_t)row * a.ld;
    auto four = [&](int c) {
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (c + 4 <= a.rank && ((a.ld | a.slab_stride) & 3) == 0) {
            float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
            add_slabs(t, in + c, a.n_slabs, a.slab_stride);
            v = f32x4{t.x, t.y, t.z, t.w};
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (c + e < a.rank) v[e] = slab_elem(in + c + e, a.n_slabs, a.slab_stride);
        }
        return v;
    };
    auto put = [&](int c, f32x4 v, float rinv) {
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = c + e < a.rank ? (v[e] * rinv) * a.norm_w[c + e] : 0.f;
        if (a.y) *reinterpret_cast<float4*>(a.y + (size_t)row * a.ldx + c) = make_float4(v[0], v[1], v[2], v[3]);
        if (a.xh) put_planes4(a.xh, a.xl, row, c, 4, a.ldx, a.packed, v);
    };
    constexpr int NV = 4;  // ranks up to 4096 stay in registers
    f32x4 v[NV];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (threadIdx.x + i * 256) * 4;
        v[i] = c < a.rank ? four(c) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += v[i][e] * v[i][e];
    }
    for (int c = (threadIdx.x + NV * 256) * 4; c < a.rank; c += 1024) {
        const f32x4 t = four(c);
        ss += (t[0] * t[0] + t[1] * t[1]) + (t[2] * t[2] + t[3] * t[3]);
    }
    const float rinv = 1.0f / sqrtf(block_sum(ss, red, 4) / (float)a.rank + a.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if ((int)(threadIdx.x + i * 256) * 4 < a.ldx) put((threadIdx.x + i * 256) * 4, v[i], rinv);
    for (int c = (threadIdx.x + NV * 256) * 4; c < a.ldx; c += 1024) put(c, c < a.rank ? four(c) : f32x4{0.f, 0.f, 0.f, 0.f}, rinv);
}
hipError_t launch_query_latent(const QueryLatentArgs& a, const LatentRowsArgs& kv, int rows, hipStream_t s) {
    if (a.rank < 1 || a.rank > a.ld || a.ldx < a.rank || a.ldx % 32 || (!a.xh && !a.y) || kv.cache.rot % 2 || kv.cache.rank_p % 32 || kv.cache.rot_p % 32) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    if (rows >= 512 && a.packed && a.xh && !a.y && a.rank == a.ldx && a.rank <= 4096 && a.ld % 4 == 0 && a.slab_stride % 4 == 0) {
        AddNormArgs n;
        n.in = a.in; n.n_slabs = a.n_slabs; n.slab_stride = a.slab_stride; n.ld_in = a.ld; n.W = n.ldr = n.ldx = a.rank; n.eps = a.eps;
        n.w[0] = a.norm_w; n.xh[0] = a.xh; n.xl[0] = a.xl; n.packed[0] = 1;
        hipError_t e = launch_add_norm(n, rows, s);
        if (e != hipSuccess || !kv.kv) return e;
        return launch_latent_cache(kv, rows, s);
    }
    query_latent_kernel<<<dim3(rows, kv.kv ? 2 : 1), 256, 0, s>>>(a, kv);
    return hipGetLastError();
}

hipError_t launch_latent_rows(const LatentRowsArgs& a, int rows, hipStream_t s) {
    if (a.cache.rot % 2 || a.cache.rank_p % 32 || a.cache.rot_p % 32) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    latent_rows_kernel<<<dim3(rows, (a.heads + 1 + 3) / 4), 256, 0, s>>>(a);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// per-head products: wave = NT n-tiles x MT m-tiles of one head, fragments straight from memory
// ---------------------------------------------------------------------------------------------------
template <int MT, int NT, bool EXACT>
__global__ void __launch_bounds__(256) head_gemm_kernel(HeadGemmArgs a) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int l15 = lane & 15, grp = lane >> 4;
    const int ntiles = a.N >> 4, KT = a.K >> 5;
    const int nt0 = (blockIdx.x * 4 + wave) * NT;
    if (nt0 >= ntiles) return;
    const int head = blockIdx.y, m0 = blockIdx.z * (MT * 16);
    const uint4* wp = a.w + (size_t)head * a.w_head;
    const float* xp[MT];
#pragma unroll
    for (int b = 0; b < MT; ++b) xp[b] = a.x + (size_t)min(m0 + b * 16 + l15, a.M - 1) * a.x_row + (size_t)head * a.x_head + grp * 8;
    f32x4 acc[NT][MT];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int b = 0; b < MT; ++b) acc[n][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int kt = 0; kt < KT; ++kt) {
        uint4 wf[NT];
        float xv[MT][8];
#pragma unroll
        for (int n = 0; n < NT; ++n) wf[n] = wp[((size_t)min(nt0 + n, ntiles - 1) * KT + kt) * 64 + lane];
#pragma unroll
        for (int b = 0; b < MT; ++b) {
            *reinterpret_cast<float4*>(&xv[b][0]) = *reinterpret_cast<const float4*>(xp[b] + kt * 32);
            *reinterpret_cast<float4*>(&xv[b][4]) = *reinterpret_cast<const float4*>(xp[b] + kt * 32 + 4);
        }
        if constexpr (EXACT) {
            // step j multiplies the k = 32 kt + 8 grp + j of every lane group: the weight widened to f32 is exact
#pragma unroll
            for (int n = 0; n < NT; ++n) {
                const uint32_t wd[4] = {wf[n].x, wf[n].y, wf[n].z, wf[n].w};
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const float wv = (j & 1) ? __builtin_bit_cast(float, wd[j >> 1] & 0xffff0000u) : __builtin_bit_cast(float, wd[j >> 1] << 16);
#pragma unroll
                    for (int b = 0; b < MT; ++b) acc[n][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(wv, xv[b][j], acc[n][b], 0, 0, 0);
                }
            }
        } else {
#pragma unroll
            for (int b = 0; b < MT; ++b) {
                bf16x8 h, l;
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    h[j] = (__bf16)xv[b][j];
                    l[j] = (__bf16)(xv[b][j] - (float)h[j]);
                }
#pragma unroll
                for (int n = 0; n < NT; ++n) {
                    const bf16x8 wv = __builtin_bit_cast(bf16x8, wf[n]);
                    acc[n][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, h, acc[n][b], 0, 0, 0);
                    acc[n][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, l, acc[n][b], 0, 0, 0);
                }
            }
        }
    }
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        const int f0 = (nt0 + n) * 16 + grp * 4;
        if (f0 >= a.n_valid || nt0 + n >= ntiles) continue;
        const bool whole = f0 + 4 <= a.n_valid;
#pragma unroll
        for (int b = 0; b < MT; ++b) {
            const int row = m0 + b * 16 + l15;
            if (row >= a.M) continue;
            f32x4 v = acc[n][b];
            if (a.decay_bias) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int f = min(f0 + r, a.n_valid - 1);
                    if (!a.decay_rate) {
                        v[r] = softplusf(v[r] + a.decay_bias[f]);
                    } else if (head == 0) {
                        v[r] = expf(-a.decay_rate[f] * softplusf(v[r] + a.decay_bias[f]));
                    } else {
                        v[r] = 1.0f / (1.0f + expf(-v[r]));
                    }
                }
            }
            if (a.y) {
                float* o = a.y + (size_t)row * a.y_row + (size_t)head * a.y_head + f0;
                if (whole && ((a.y_row | a.y_head) & 3) == 0) *reinterpret_cast<float4*>(o) = make_float4(v[0], v[1], v[2], v[3]);
                else
                    for (int r = 0; r < 4; ++r)
                        if (f0 + r < a.n_valid) o[r] = v[r];
            }
            if (a.yh) put_planes4(a.yh, a.yl, row, head * a.n_valid + f0, a.n_valid - f0, a.ld, a.packed, v);
        }
    }
}

template <int MT, int NT>
static hipError_t head_gemm_launch(const HeadGemmArgs& a, hipStream_t s) {
    const dim3 grid((a.N / 16 + 4 * NT - 1) / (4 * NT), a.heads, (a.M + MT * 16 - 1) / (MT * 16));
    if (a.exact) head_gemm_kernel<MT, NT, true><<<grid, 256, 0, s>>>(a);
    else head_gemm_kernel<MT, NT, false><<<grid, 256, 0, s>>>(a);
    return hipGetLastError();
}
hipError_t launch_head_gemm(const HeadGemmArgs& a, hipStream_t s) {
    if (a.N % 16 || a.K % 32 || a.x_row % 4 || a.x_head % 4 || a.n_valid > a.N || (!a.y && !a.yh)) return hipErrorInvalidValue;
    if (a.M <= 0) return hipSuccess;
    if (a.M <= 16) return head_gemm_launch<1, 1>(a, s);
    if (a.M <= 64) return head_gemm_launch<2, 1>(a, s);
    return head_gemm_launch<4, 2>(a, s);
}

// ---------------------------------------------------------------------------------------------------
// decode: fused neighbours of the attention kernel.  One workgroup = 16 rows x one head x a slice of the output features; the rows'
// operand is built once in LDS as bf16 hi + lo fragments, then each wave streams its share of the head's weight fragments.
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ void put_hilo_frag(uint4* lds, int KT, int slot, const float (&x)[8]) {
    bf16x8 h, l;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        h[j] = (__bf16)x[j];
        l[j] = (__bf16)(x[j] - (float)h[j]);
    }
    lds[slot] = __builtin_bit_cast(uint4, h);
    lds[KT * 64 + slot] = __builtin_bit_cast(uint4, l);
}
// D[feature 4g + r][row l15] of two n-tiles over KT k-tiles from the LDS operand (both tiles' fragments in flight)
__device__ __forceinline__ void frag_product2(const uint4* __restrict__ w0, const uint4* __restrict__ w1, const uint4* lds, int KT, int lane, f32x4 (&acc)[2]) {
    acc[0] = f32x4{0.f, 0.f, 0.f, 0.f};
    acc[1] = acc[0];
    for (int k0 = 0; k0 < KT; k0 += 4) {
        uint4 wf[2][4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const size_t k = (size_t)min(k0 + u, KT - 1) * 64 + lane;
            wf[0][u] = w0[k];
            wf[1][u] = w1[k];
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (k0 + u < KT) {
                const bf16x8 h = __builtin_bit_cast(bf16x8, lds[(k0 + u) * 64 + lane]), l = __builtin_bit_cast(bf16x8, lds[(KT + k0 + u) * 64 + lane]);
#pragma unroll
                for (int n = 0; n < 2; ++n) {
                    const bf16x8 wv = __builtin_bit_cast(bf16x8, wf[n][u]);
                    acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, h, acc[n], 0, 0, 0);
                    acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, l, acc[n], 0, 0, 0);
                }
            }
    }
}

__global__ void __launch_bounds__(256) latent_query_kernel(LatentRowsArgs a, const uint4* __restrict__ w, float* __restrict__ y, int rows) {
    extern __shared__ __attribute__((aligned(16))) char smem_q[];
    uint4* lds = reinterpret_cast<uint4*>(smem_q);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int r0 = blockIdx.x * 16, head = blockIdx.y, nr = min(16, rows - r0);
    const LatentCache& c = a.cache;
    if (head >= a.heads) {  // the rest of the rows' work, once: four workgroups for the latents (a row per wave), then the rotated parts
        if (blockIdx.z) return;
        const int q = head - a.heads;
        if (q < 4) {
            if (a.kv && q * 4 + wave < nr) latent_to_cache(a, r0 + q * 4 + wave, lane);
            return;
        }
        const int half = c.rot >> 1, per = c.rot_p - half, i = (q - 4) * 256 + (int)threadIdx.x;  // one pair (or one padding zero) per thread
        if (i >= nr * a.heads * per) return;
        const int k = i % per, hd = (i / per) % a.heads, row = r0 + i / (per * a.heads);
        float* o = a.q + ((size_t)row * a.heads + hd) * (a.dim_p + c.rot_p) + a.dim_p;
        if (k < half) {
            const float* in = a.qkv + (size_t)row * a.ldq + (size_t)hd * (a.dim + c.rot) + a.dim;
            const float u = slab_elem(in + k, a.n_slabs, a.slab_stride), v = slab_elem(in + half + k, a.n_slabs, a.slab_stride);
            const float cs = a.cos[(size_t)a.pos[row] * half + k], sn = a.sin[(size_t)a.pos[row] * half + k];
            o[k] = (u * cs - v * sn) * a.scale;
            o[k + half] = (v * cs + u * sn) * a.scale;
        } else {
            o[half + k] = 0.f;
        }
        return;
    }
    const int KT = a.dim_p >> 5, NT = c.rank_p >> 4;
    const size_t col = (size_t)head * (a.dim + c.rot);
    for (int slot = threadIdx.x; slot < KT * 64; slot += 256) {
        const int l = slot & 63, d0 = (slot >> 6) * 32 + (l >> 4) * 8;
        const float* in = a.qkv + (size_t)(r0 + min(l & 15, nr - 1)) * a.ldq + col + d0;
        float x[8];
        load_slabs8(x, in, a.dim - d0, a.n_slabs, a.slab_stride);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] *= a.scale;
        put_hilo_frag(lds, KT, slot, x);
    }
    __syncthreads();
    const uint4* wh = w + (size_t)head * NT * KT * 64;
    const int row = r0 + (lane & 15);
    const int step = 4 * gridDim.z;
    for (int nt = blockIdx.z * 4 + wave; nt < NT; nt += 2 * step) {
        const bool two = nt + step < NT;
        f32x4 v[2];
        frag_product2(wh + (size_t)nt * KT * 64, wh + (size_t)(two ? nt + step : nt) * KT * 64, lds, KT, lane, v);
        if (row >= rows) continue;
        float* o = y + ((size_t)row * a.heads + head) * c.rank_p + nt * 16 + (lane >> 4) * 4;
        *reinterpret_cast<float4*>(o) = make_float4(v[0][0], v[0][1], v[0][2], v[0][3]);
        if (two) *reinterpret_cast<float4*>(o + step * 16) = make_float4(v[1][0], v[1][1], v[1][2], v[1][3]);
    }
}

// output slices: enough workgroups for the chip, at least one n-tile per wave
static int head_slices(int base, int ntiles) { return std::max(1, std::min((ntiles + 3) / 4, 512 / std::max(base, 1))); }

hipError_t launch_latent_query(const LatentRowsArgs& a, const uint4* w, float* y, int rows, hipStream_t s) {
    if (a.cache.rot % 2 || a.cache.rank_p % 32 || a.cache.rot_p % 32 || a.dim_p % 32) return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const size_t lds = (size_t)2 * (a.dim_p / 32) * 1024;
    if (lds > 64 * 1024) return hipErrorNotSupported;
    const int rb = (rows + 15) / 16;
    // every slice sums the projection's slabs again: fewer slices when there are many
    const int slices = std::max(1, head_slices(rb * a.heads, a.cache.rank_p / 16) * 4 / std::max(4, a.n_slabs));
    latent_query_kernel<<<dim3(rb, a.heads + 4 + (16 * a.heads * (a.cache.rot_p - a.cache.rot / 2) + 255) / 256, slices), 256, lds, s>>>(a, w, y, rows);
    return hipGetLastError();
}

__global__ void __launch_bounds__(256) latent_values_kernel(LatentAttnArgs a, const uint4* __restrict__ w, int vdim, int NT, uint16_t* __restrict__ oh,
                                                            uint16_t* __restrict__ ol, int ld, int packed, int rows, int split) {
    extern __shared__ __attribute__((aligned(16))) char smem_v[];
    uint4* lds = reinterpret_cast<uint4*>(smem_v);
    __shared__ float wgt[16][kLatentMaxParts];
    __shared__ int np[16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int r0 = blockIdx.x * 16, head = blockIdx.y, nr = min(16, rows - r0);
    const int R = a.cache.rank_p, KT = R >> 5;
    if (split) {
        // 16 lanes per row: the parts' weights 2^(m_p - m) / sum 2^(m_p - m) l_p
        const int r = threadIdx.x >> 4, q = threadIdx.x & 15, row = r0 + min(r, nr - 1);
        const int pos = a.pos[row];
        const int t_lo = a.window > 0 ? max(0, pos - a.window + 1) >> 5 : 0;
        const int n = ((pos >> 5) + 1 - t_lo + a.part_tiles - 1) / a.part_tiles;
        const float* pm = a.part_ml + ((size_t)row * a.heads + head) * a.max_parts * 2;
        float m[kLatentMaxParts / 16], l[kLatentMaxParts / 16], ms = -1e30f, lt = 0.f;
#pragma unroll
        for (int i = 0; i < kLatentMaxParts / 16; ++i) {
            const int p = q + i * 16;
            m[i] = -1e30f;
            l[i] = 0.f;
            if (n > 1 && p < n) { m[i] = pm[2 * p]; l[i] = pm[2 * p + 1]; }
            ms = fmaxf(ms, m[i]);
        }
#pragma unroll
        for (int o = 1; o < 16; o <<= 1) ms = fmaxf(ms, __shfl_xor(ms, o));
        if (a.sink) {
            ms = fmaxf(ms, a.sink[head]);
            if (q == 0) lt = exp2f(a.sink[head] - ms);
        }
#pragma unroll
        for (int i = 0; i < kLatentMaxParts / 16; ++i) lt += l[i] * exp2f(m[i] - ms);
#pragma unroll
        for (int o = 1; o < 16; o <<= 1) lt += __shfl_xor(lt, o);
#pragma unroll
        for (int i = 0; i < kLatentMaxParts / 16; ++i) wgt[r][q + i * 16] = n > 1 ? exp2f(m[i] - ms) / lt : 0.f;
        if (q == 0) np[r] = n;
        __syncthreads();
    }
    for (int slot = threadIdx.x; slot < KT * 64; slot += 256) {
        const int l = slot & 63, r = min(l & 15, nr - 1), d0 = (slot >> 6) * 32 + (l >> 4) * 8;
        const size_t rh = (size_t)(r0 + r) * a.heads + head;
        float x[8];
        if (split && np[r] > 1) {
#pragma unroll
            for (int j = 0; j < 8; ++j) x[j] = 0.f;
            const float* po = a.part_o + rh * a.max_parts * R + d0;
            const int n = np[r];
            for (int p0 = 0; p0 < n; p0 += 4) {  // four parts' loads in flight (clamped index, weight 0 past the end)
                float4 u[4], v[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float* p = po + (size_t)min(p0 + i, n - 1) * R;
                    u[i] = *reinterpret_cast<const float4*>(p);
                    v[i] = *reinterpret_cast<const float4*>(p + 4);
                }
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float f = p0 + i < n ? wgt[r][p0 + i] : 0.f;
                    x[0] += f * u[i].x; x[1] += f * u[i].y; x[2] += f * u[i].z; x[3] += f * u[i].w;
                    x[4] += f * v[i].x; x[5] += f * v[i].y; x[6] += f * v[i].z; x[7] += f * v[i].w;
                }
            }
        } else {
            *reinterpret_cast<float4*>(&x[0]) = *reinterpret_cast<const float4*>(a.out + rh * R + d0);
            *reinterpret_cast<float4*>(&x[4]) = *reinterpret_cast<const float4*>(a.out + rh * R + d0 + 4);
        }
        put_hilo_frag(lds, KT, slot, x);
    }
    __syncthreads();
    const uint4* wh = w + (size_t)head * NT * KT * 64;
    const int row = r0 + (lane & 15);
    const int step = 4 * gridDim.z;
    for (int nt = blockIdx.z * 4 + wave; nt < NT; nt += 2 * step) {
        const bool two = nt + step < NT;
        f32x4 v[2];
        frag_product2(wh + (size_t)nt * KT * 64, wh + (size_t)(two ? nt + step : nt) * KT * 64, lds, KT, lane, v);
#pragma unroll
        for (int n = 0; n < 2; ++n) {
            const int f0 = (nt + n * step) * 16 + (lane >> 4) * 4;
            if ((n == 0 || two) && row < rows && f0 < vdim) put_planes4(oh, ol, row, head * vdim + f0, vdim - f0, ld, packed, v[n]);
        }
    }
}

hipError_t launch_latent_values(const LatentAttnArgs& a, int n_parts_max, const uint4* w, int vdim, int vdim_p, bf16_bits* oh, bf16_bits* ol,
                                int ld, int packed, int rows, hipStream_t s) {
    if (a.cache.rank_p % 32 || vdim_p % 16 || (n_parts_max > 1 && (!a.part_o || !a.part_ml || a.part_tiles < 1 || n_parts_max > kLatentMaxParts)))
        return hipErrorInvalidValue;
    if (rows <= 0) return hipSuccess;
    const size_t lds = (size_t)2 * (a.cache.rank_p / 32) * 1024;
    if (lds > 60 * 1024) return hipErrorNotSupported;
    const int rb = (rows + 15) / 16;
    latent_values_kernel<<<dim3(rb, a.heads, head_slices(rb * a.heads, vdim_p / 16)), 256, lds, s>>>(a, w, vdim, vdim_p / 16, oh, ol, ld, packed, rows, n_parts_max > 1);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// attention, plain form: one workgroup per (row, head), each wave takes every fourth visible token; any size
// ---------------------------------------------------------------------------------------------------
template <typename T, int NE>
__global__ void __launch_bounds__(256) latent_attn_plain_kernel(LatentAttnArgs a) {
    extern __shared__ float sh[];  // 4 waves x (m, l, o[rank_p])
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int row = blockIdx.x, head = blockIdx.y;
    const LatentCache& c = a.cache;
    const int D = c.D(), pos = a.pos[row];
    const int first = a.window > 0 ? max(0, pos - a.window + 1) : 0;
    const int* bt = a.block_tables + (size_t)a.slot[row] * a.max_blocks;
    const T* data = reinterpret_cast<const T*>(c.data);
    float q[NE], o[NE];
    const float* ql = a.qlat + ((size_t)row * a.heads + head) * c.rank_p;
    const float* qr = a.qrot + (size_t)row * a.qrot_row + (size_t)head * a.qrot_head;
#pragma unroll
    for (int e = 0; e < NE; ++e) {
        const int d = lane + e * 64;
        q[e] = d < c.rank_p ? ql[d] : d < D ? qr[d - c.rank_p] : 0.f;
        o[e] = 0.f;
    }
    float m = -1e30f, l = 0.f;
    for (int j = first + wave; j <= pos; j += 4) {
        const size_t base = (size_t)bt[j / kBlockTokens] * kBlockTokens * D;
        float k[NE], s = 0.f;
#pragma unroll
        for (int e = 0; e < NE; ++e) {
            const int d = lane + e * 64;
            k[e] = d < D ? (float)data[base + k_packed_offset(j & (kBlockTokens - 1), d, D)] : 0.f;
            s += q[e] * k[e];
        }
        s = wave_sum(s);
        const float mn = fmaxf(m, s), al = exp2f(m - mn), p = exp2f(s - mn);
        m = mn;
        l = l * al + p;
#pragma unroll
        for (int e = 0; e < NE; ++e) o[e] = o[e] * al + p * k[e];
    }
    float* mine = sh + (size_t)wave * (c.rank_p + 2);
    if (lane == 0) { mine[0] = m; mine[1] = l; }
#pragma unroll
    for (int e = 0; e < NE; ++e)
        if (lane + e * 64 < c.rank_p) mine[2 + lane + e * 64] = o[e];
    __syncthreads();
    float ms = -1e30f, lt = 0.f, f[4];
    for (int w = 0; w < 4; ++w) ms = fmaxf(ms, sh[(size_t)w * (c.rank_p + 2)]);
    if (a.sink) {
        ms = fmaxf(ms, a.sink[head]);
        lt = exp2f(a.sink[head] - ms);
    }
    for (int w = 0; w < 4; ++w) {
        f[w] = exp2f(sh[(size_t)w * (c.rank_p + 2)] - ms);
        lt += f[w] * sh[(size_t)w * (c.rank_p + 2) + 1];
    }
    const float inv = 1.0f / lt;
    for (int d = threadIdx.x; d < c.rank_p; d += 256) {
        float v = 0.f;
        for (int w = 0; w < 4; ++w) v += f[w] * sh[(size_t)w * (c.rank_p + 2) + 2 + d];
        a.out[((size_t)row * a.heads + head) * c.rank_p + d] = v * inv;
    }
}

template <typename T>
static hipError_t latent_attn_plain_t(const LatentAttnArgs& a, int rows, hipStream_t s) {
    const dim3 grid(rows, a.heads);
    const size_t lds = (size_t)4 * (a.cache.rank_p + 2) * 4;
    const int D = a.cache.D();
    if (D <= 256) latent_attn_plain_kernel<T, 4><<<grid, 256, lds, s>>>(a);
    else if (D <= 640) latent_attn_plain_kernel<T, 10><<<grid, 256, lds, s>>>(a);
    else if (D <= 2560) latent_attn_plain_kernel<T, 40><<<grid, 256, lds, s>>>(a);
    else return hipErrorNotSupported;
    return hipGetLastError();
}
hipError_t launch_latent_attn_plain(const LatentAttnArgs& a, int rows, hipStream_t s) {
    if (rows <= 0) return hipSuccess;
    return a.cache.f32 ? latent_attn_plain_t<float>(a, rows, s) : latent_attn_plain_t<_Float16>(a, rows, s);
}

// ---------------------------------------------------------------------------------------------------
// logits of a product left as slabs (32-bit mode, vocabularies that are no multiple of 16)
// ---------------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256) logits_finish_kernel(const float* __restrict__ in, int n_slabs, int64_t slab_stride, int ld_in, int V,
                                                            float softcap, float* __restrict__ logits, int64_t ld_out) {
    const int row = blockIdx.y;
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= V) return;
    float v = slab_elem(in + (size_t)row * ld_in + i, n_slabs, slab_stride);
    if (softcap > 0.f) v = softcap * tanhf(v / softcap);
    logits[(size_t)row * ld_out + i] = v;
}
hipError_t launch_logits_finish(const float* in, int n_slabs, int64_t slab_stride, int ld_in, int rows, int V, float softcap,
                                float* logits, int64_t ld_out, hipStream_t s) {
    if (rows <= 0) return hipSuccess;
    logits_finish_kernel<<<dim3((V + 255) / 256, rows), 256, 0, s>>>(in, n_slabs, slab_stride, ld_in, V, softcap, logits, ld_out);
    return hipGetLastError();
}

}  // namespace nvllm
