// Prompt attention of the latent-attention decoders (gfx950), expanded form: the cached latents a chunk of rows can see are turned
// into per-head keys and values once (latent_expand_kernel), then 128-row q-tiles run windowed attention over them from LDS
// (latent_prefill_kernel).  Per visible (query, key) pair and head this costs dim + rot + vdim products instead of the absorbed
// form's 2 rank + rot, for one extra pass over the chunk's context.
#include <algorithm>

#include "device_common.h"
#include "latent.h"

namespace nvllm {

// ---------------------------------------------------------------------------------------------------
// expansion: one wave = two 32-token tiles of the cache x one head, the head's weights shared by the workgroup's four waves through
// LDS (double buffered, one 16-feature row of fragments per step).
//   keys    D[feature][token] = W_uk[feature][:] . c[token][:]    lane: 4 features of one token -> 8 bytes of a K fragment
//   values  D[token][feature] = c[token][:] . W_uv[feature][:]    lane: 4 + 4 tokens of one feature -> a 16-byte V slot
// The weights are f16 after a power-of-two scale that brings the matrix's largest entry to 2^14..2^15 (bf16 has fewer mantissa bits;
// what falls below the f16 range is 2^-38 of the largest entry), so the products with the cached f16 latents are exact.
// ---------------------------------------------------------------------------------------------------
template <int KC>
__global__ void __launch_bounds__(256, KC <= 8 ? 2 : 1) latent_expand_kernel(LatentExpandArgs a) {
    typedef __attribute__((ext_vector_type(4))) _Float16 f16x4;
    __shared__ __attribute__((aligned(16))) uint4 lds[2][KC * 64];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int l15 = lane & 15, grp = lane >> 4;
    const int head = blockIdx.y;
    const int DC = a.cache.D() >> 5;
    const int e0 = (blockIdx.x * 4 + wave) * 2;
    bool need[2];
    f16x8 cf[2][2][KC];  // [tile][half][chunk]
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const int e = min(e0 + u, a.n_tiles - 1);
        const int slot = a.exp_slot[e], t = a.exp_tile[e];
        // a tile no row of its segment sees in this layer stays unexpanded
        need[u] = e0 + u < a.n_tiles && (a.window <= 0 || t * 32 + 31 >= a.exp_pos0[e] - a.window + 1);
        const _Float16* p = reinterpret_cast<const _Float16*>(a.cache.data) +
                            (size_t)a.block_tables[(size_t)slot * a.max_blocks + (t >> 3)] * kBlockTokens * a.cache.D() + (size_t)(t & 7) * (2 * DC * 512) + lane * 8;
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int c = 0; c < KC; ++c) cf[u][s][c] = *reinterpret_cast<const f16x8*>(p + (size_t)(s * DC + c) * 512);
    }
    if (!__syncthreads_or(need[0] || need[1])) return;
    const int nk = a.dim_p / 16, nv = a.vdim_p / 16, DK = a.dim_p >> 5;
    const uint4* wk = a.uk + (size_t)head * nk * KC * 64;
    const uint4* wv = a.uv + (size_t)head * nv * KC * 64;
    auto issue = [&](int nt, int buf) {
        const uint4* src = nt < nk ? wk + (size_t)nt * KC * 64 : wv + (size_t)(nt - nk) * KC * 64;
#pragma unroll
        for (int i = 0; i < (KC + 3) / 4; ++i) {
            const int c = wave + i * 4;
            if (KC % 4 == 0 || c < KC) __builtin_amdgcn_global_load_lds((gptr_t)(src + c * 64 + lane), (lptr_t)(&lds[buf][c * 64]), 16, 0, 0);
        }
    };
    issue(0, 0);
    for (int nt = 0; nt < nk + nv; ++nt) {
        const int buf = nt & 1;
        dma_publish_barrier();  // step nt's weights have landed; every wave is done with the other buffer
        if (nt + 1 < nk + nv) issue(nt + 1, buf ^ 1);
        f32x4 acc[2][2];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int s = 0; s < 2; ++s) acc[u][s] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (nt < nk) {
#pragma unroll
            for (int c = 0; c < KC; ++c) {
                const f16x8 w = __builtin_bit_cast(f16x8, lds[buf][c * 64 + lane]);
#pragma unroll
                for (int u = 0; u < 2; ++u)
#pragma unroll
                    for (int s = 0; s < 2; ++s) acc[u][s] = __builtin_amdgcn_mfma_f32_16x16x32_f16(w, cf[u][s][c], acc[u][s], 0, 0, 0);
            }
            const int d = nt * 16 + grp * 4;
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                if (!need[u]) continue;
                _Float16* kx = reinterpret_cast<_Float16*>(a.kx) + ((size_t)head * a.cap + e0 + u) * 32 * a.dim_p;
#pragma unroll
                for (int s = 0; s < 2; ++s) {
                    f16x4 o;
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[r] = f16_sat(acc[u][s][r] * a.uk_scale);
                    *reinterpret_cast<f16x4*>(kx + ((size_t)(s * DK + (d >> 5)) * 64 + (((d & 31) >> 3) << 4) + l15) * 8 + (d & 7)) = o;
                }
            }
        } else {
#pragma unroll
            for (int c = 0; c < KC; ++c) {
                const f16x8 w = __builtin_bit_cast(f16x8, lds[buf][c * 64 + lane]);
#pragma unroll
                for (int u = 0; u < 2; ++u)
#pragma unroll
                    for (int s = 0; s < 2; ++s) acc[u][s] = __builtin_amdgcn_mfma_f32_16x16x32_f16(cf[u][s][c], w, acc[u][s], 0, 0, 0);
            }
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                if (!need[u]) continue;
                _Float16* vx = reinterpret_cast<_Float16*>(a.vx) + ((size_t)head * a.cap + e0 + u) * 32 * a.vdim_p;
                f16x8 o;
#pragma unroll
                for (int r = 0; r < 4; ++r) { o[r] = f16_sat(acc[u][0][r] * a.uv_scale); o[4 + r] = f16_sat(acc[u][1][r] * a.uv_scale); }
                *reinterpret_cast<f16x8*>(vx + ((size_t)(nt - nk) * 64 + lane) * 8) = o;
            }
        }
    }
}

hipError_t launch_latent_expand(const LatentExpandArgs& a, int heads, hipStream_t s) {
    if (a.cache.f32 || a.dim_p % 32 || a.vdim_p % 16 || a.n_tiles > a.cap) return hipErrorInvalidValue;
    if (a.n_tiles <= 0) return hipSuccess;
    const dim3 grid((a.n_tiles + 7) / 8, heads);
    switch (a.cache.rank_p / 32) {
#define NVLLM_LE(K_) case K_: latent_expand_kernel<K_><<<grid, 256, 0, s>>>(a); break;
        NVLLM_LE(1) NVLLM_LE(2) NVLLM_LE(3) NVLLM_LE(4) NVLLM_LE(6) NVLLM_LE(8) NVLLM_LE(12) NVLLM_LE(16)
#undef NVLLM_LE
        default: return hipErrorNotSupported;
    }
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// windowed attention of a q-tile (<= 128 rows of one sequence) x one head.  Four waves, 32 rows each (two 16-row B operands); the
// 32-token K / rotated-part / V fragments of a tile are staged once per workgroup by LDS-DMA, double buffered.
// ---------------------------------------------------------------------------------------------------
template <int DK, int RC, int VT>
__global__ void __launch_bounds__(256, 2) latent_prefill_kernel(LatentPrefillArgs a) {
    constexpr int QC = DK + RC, FR = 2 * QC + VT, QT = 2;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    uint4* lds = reinterpret_cast<uint4*>(smem);  // [2][FR][64]
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int l15 = lane & 15, grp = lane >> 4;
    // workgroups of one XCD (ids equal modulo 8) take neighbouring work items: tiles of one head share its keys in that L2
    const int total = a.n_tiles * a.heads, per = (total + 7) >> 3;
    const int item = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || item >= total) return;
    const int head = item / a.n_tiles;
    const int tile = a.tile_order[item - head * a.n_tiles];
    const int row0 = a.tile_row0[tile], nrows = a.tile_nrows[tile], slot = a.tile_slot[tile], ebase = a.tile_exp[tile];
    const int pos0 = a.pos[row0];
    const int t_lo = a.window > 0 ? max(0, pos0 - a.window + 1) >> 5 : 0, t_hi = ((pos0 + nrows - 1) >> 5) + 1;
    const int* bt = a.block_tables + (size_t)slot * a.max_blocks;
    const int DC = a.cache.D() >> 5;
    const _Float16* cdata = reinterpret_cast<const _Float16*>(a.cache.data);
    const _Float16* kx = reinterpret_cast<const _Float16*>(a.kx) + ((size_t)head * a.cap + ebase) * (32 * DK * 32);
    const _Float16* vx = reinterpret_cast<const _Float16*>(a.vx) + ((size_t)head * a.cap + ebase) * (32 * VT * 16);
    auto issue = [&](int t, int buf) {
        const _Float16* kt = kx + (size_t)t * (32 * DK * 32);
        const _Float16* vt = vx + (size_t)t * (32 * VT * 16);
        const _Float16* rt = cdata + (size_t)bt[t >> 3] * kBlockTokens * (DC * 32) + (size_t)(t & 7) * (2 * DC * 512);
#pragma unroll
        for (int i = 0; i < (FR + 3) / 4; ++i) {
            const int f = wave + i * 4;
            if (FR % 4 == 0 || f < FR) {
                // fragment order in LDS: K of the two 16-token halves, rotated part of the two halves, V
                const _Float16* src = f < 2 * DK ? kt + (size_t)f * 512
                                      : f < 2 * QC ? rt + (size_t)(((f - 2 * DK) / RC) * DC + (DC - RC) + (f - 2 * DK) % RC) * 512
                                                   : vt + (size_t)(f - 2 * QC) * 512;
                __builtin_amdgcn_global_load_lds((gptr_t)(src + lane * 8), (lptr_t)(lds + (size_t)(buf * FR + f) * 64), 16, 0, 0);
            }
        }
    };
    // q: split, rotated, scaled, as f16 hi + lo in registers
    f16x8 qh[QT][QC], ql[QT][QC];
    int my_pos[QT];
#pragma unroll
    for (int s = 0; s < QT; ++s) {
        const int r = wave * 32 + s * 16 + l15;
        const bool ok = r < nrows;
        my_pos[s] = ok ? pos0 + r : -1;
        const int rot = a.cache.rot, half = rot >> 1;
        const float* q = a.qkv + (size_t)(row0 + min(r, nrows - 1)) * a.ldq + (size_t)head * (a.dim + rot);
        const size_t tab = (size_t)(pos0 + min(r, nrows - 1)) * half;
#pragma unroll
        for (int c = 0; c < QC; ++c) {
            float x[8];
            if (c < DK) {
                const int d = c * 32 + grp * 8;
                load_slabs8(x, q + d, a.dim - d, a.n_slabs, a.slab_stride);
            } else {
                // rotated part: element i pairs with i + half; a lane's eight lie on one side when half % 8 == 0
                const int i0 = (c - DK) * 32 + grp * 8;
                if ((half & 7) == 0 && i0 < rot) {
                    const bool upper = i0 >= half;
                    const int k = upper ? i0 - half : i0;
                    float y[8];
                    load_slabs8(x, q + a.dim + i0, 8, a.n_slabs, a.slab_stride);
                    load_slabs8(y, q + a.dim + (upper ? k : k + half), 8, a.n_slabs, a.slab_stride);
#pragma unroll
                    for (int j = 0; j < 8; ++j) x[j] = x[j] * a.cos[tab + k + j] + (upper ? y[j] : -y[j]) * a.sin[tab + k + j];
                } else {
#pragma unroll
                    for (int j = 0; j < 8; ++j) {
                        const int i = i0 + j;
                        x[j] = 0.f;
                        if (i < rot) {
                            const bool upper = i >= half;
                            const int k = upper ? i - half : i;
                            float own = 0.f, other = 0.f;
                            for (int sl = 0; sl < a.n_slabs; ++sl) {
                                own += q[(size_t)sl * a.slab_stride + a.dim + i];
                                other += q[(size_t)sl * a.slab_stride + a.dim + (upper ? k : k + half)];
                            }
                            x[j] = own * a.cos[tab + k] + (upper ? other : -other) * a.sin[tab + k];
                        }
                    }
                }
            }
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const float v = x[j] * a.scale;
                qh[s][c][j] = f16_sat(v);
                ql[s][c][j] = f16_sat(v - (float)qh[s][c][j]);
            }
        }
    }
    f32x4 o[QT][VT];
    float m[QT], lsum[QT];
#pragma unroll
    for (int s = 0; s < QT; ++s) {
        m[s] = -1e30f;
        lsum[s] = 0.f;
#pragma unroll
        for (int d = 0; d < VT; ++d) o[s][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const int w_lo = pos0 + wave * 32, w_hi = pos0 + min(wave * 32 + 31, nrows - 1);  // this wave's positions (empty: w_hi < w_lo)
    const int w_first = a.window > 0 ? w_lo - a.window + 1 : 0;
    auto compute = [&](int t, int buf) {
        const uint4* L = lds + (size_t)buf * FR * 64 + lane;
        f32x4 sa[QT], sb[QT];
#pragma unroll
        for (int s = 0; s < QT; ++s) { sa[s] = f32x4{0.f, 0.f, 0.f, 0.f}; sb[s] = f32x4{0.f, 0.f, 0.f, 0.f}; }
#pragma unroll
        for (int c = 0; c < QC; ++c) {
            const int ia = c < DK ? c : 2 * DK + (c - DK), ib = c < DK ? DK + c : 2 * DK + RC + (c - DK);
            const f16x8 fa = __builtin_bit_cast(f16x8, L[ia * 64]), fb = __builtin_bit_cast(f16x8, L[ib * 64]);
#pragma unroll
            for (int s = 0; s < QT; ++s) {
                sa[s] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, qh[s][c], sa[s], 0, 0, 0);
                sb[s] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, qh[s][c], sb[s], 0, 0, 0);
                sa[s] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fa, ql[s][c], sa[s], 0, 0, 0);
                sb[s] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fb, ql[s][c], sb[s], 0, 0, 0);
            }
        }
        const int tokA = (t << 5) + grp * 4, tokB = tokA + 16;
        // every row of the wave sees the whole tile: no masking
        const bool inner = (t << 5) + 31 <= w_lo && (a.window <= 0 || (t << 5) >= w_hi - a.window + 1) && wave * 32 + 31 < nrows;
        f16x8 P[QT], Pl[QT];
        float al[QT];
        bool rescale = false;
#pragma unroll
        for (int s = 0; s < QT; ++s) {
            if (!inner) {
                const int first = a.window > 0 ? my_pos[s] - a.window + 1 : 0;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    if (tokA + r > my_pos[s] || tokA + r < first) sa[s][r] = -INFINITY;
                    if (tokB + r > my_pos[s] || tokB + r < first) sb[s][r] = -INFINITY;
                }
            }
            float mt = fmaxf(fmaxf(fmaxf(sa[s][0], sa[s][1]), fmaxf(sa[s][2], sa[s][3])), fmaxf(fmaxf(sb[s][0], sb[s][1]), fmaxf(sb[s][2], sb[s][3])));
            mt = fmaxf(mt, __shfl_xor(mt, 16));
            mt = fmaxf(mt, __shfl_xor(mt, 32));
            const float mn = fmaxf(m[s], mt);  // finite: m starts at -1e30
            al[s] = __builtin_amdgcn_exp2f(m[s] - mn);
            m[s] = mn;
            rescale |= al[s] != 1.0f;
            float ps = 0.f;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float pa = __builtin_amdgcn_exp2f(sa[s][r] - mn), pb = __builtin_amdgcn_exp2f(sb[s][r] - mn);
                ps += pa + pb;
                P[s][r] = (_Float16)pa;
                P[s][4 + r] = (_Float16)pb;
                Pl[s][r] = (_Float16)(pa - (float)P[s][r]);
                Pl[s][4 + r] = (_Float16)(pb - (float)P[s][4 + r]);
            }
            lsum[s] = lsum[s] * al[s] + ps;
        }
        if (__any(rescale)) {
#pragma unroll
            for (int s = 0; s < QT; ++s)
#pragma unroll
                for (int d = 0; d < VT; ++d) { o[s][d][0] *= al[s]; o[s][d][1] *= al[s]; o[s][d][2] *= al[s]; o[s][d][3] *= al[s]; }
        }
#pragma unroll
        for (int d = 0; d < VT; ++d) {
            const f16x8 fv = __builtin_bit_cast(f16x8, L[(2 * QC + d) * 64]);
#pragma unroll
            for (int s = 0; s < QT; ++s) {
                o[s][d] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fv, P[s], o[s][d], 0, 0, 0);
                o[s][d] = __builtin_amdgcn_mfma_f32_16x16x32_f16(fv, Pl[s], o[s][d], 0, 0, 0);
            }
        }
    };
    issue(t_lo, 0);
    for (int t = t_lo, buf = 0; t < t_hi; ++t, buf ^= 1) {
        dma_publish_barrier();  // tile t has landed; every wave is done with the other buffer
        if (t + 1 < t_hi) issue(t + 1, buf ^ 1);
        if ((t << 5) <= w_hi && (t << 5) + 31 >= w_first && w_lo <= w_hi) compute(t, buf);
    }
    // normalise, write the context planes at column head * vdim
#pragma unroll
    for (int s = 0; s < QT; ++s) {
        float l = lsum[s];
        l += __shfl_xor(l, 16);
        l += __shfl_xor(l, 32);
        if (my_pos[s] < 0) continue;
        float inv = 1.0f / l;
        if (a.sink) {
            const float sk = a.sink[head], mn = fmaxf(m[s], sk), f = __builtin_amdgcn_exp2f(m[s] - mn);
            inv = f / (l * f + __builtin_amdgcn_exp2f(sk - mn));
        }
        const int row = row0 + wave * 32 + s * 16 + l15;
#pragma unroll
        for (int d = 0; d < VT; ++d) {
            const int f = d * 16 + grp * 4;
            if (f >= a.vdim) continue;
            uint16_t h[4], lo[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) split_bf16(o[s][d][r] * inv, h[r], lo[r]);
            const int col = head * a.vdim + f;
            if (f + 4 <= a.vdim && (col & 3) == 0) {
                const size_t x = a.packed ? xpack_off(row, col, a.ld >> 5) : (size_t)row * a.ld + col;
                *reinterpret_cast<uint2*>(a.oh + x) = make_uint2(h[0] | ((uint32_t)h[1] << 16), h[2] | ((uint32_t)h[3] << 16));
                *reinterpret_cast<uint2*>(a.ol + x) = make_uint2(lo[0] | ((uint32_t)lo[1] << 16), lo[2] | ((uint32_t)lo[3] << 16));
            } else {
                for (int r = 0; r < 4; ++r)
                    if (f + r < a.vdim) {
                        const size_t x = a.packed ? xpack_off(row, col + r, a.ld >> 5) : (size_t)row * a.ld + col + r;
                        a.oh[x] = h[r];
                        a.ol[x] = lo[r];
                    }
            }
        }
    }
}

// instance sizes: padded query/key and value sizes an expanded layer uses (0: none, the absorbed form serves the layer)
int latent_prefill_dim(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : 0; }
int latent_prefill_vdim(int vdim) { return vdim <= 32 ? 32 : vdim <= 64 ? 64 : vdim <= 128 ? 128 : 0; }

template <int DK, int RC, int VT>
static hipError_t latent_prefill_t(const LatentPrefillArgs& a, hipStream_t s) {
    const size_t lds = (size_t)2 * (2 * (DK + RC) + VT) * 1024;
    static std::atomic<uint64_t> lds_set{0};
    ensure_dyn_lds(reinterpret_cast<const void*>(latent_prefill_kernel<DK, RC, VT>), lds, lds_set);
    latent_prefill_kernel<DK, RC, VT><<<(a.n_tiles * a.heads + 7) / 8 * 8, 256, lds, s>>>(a);
    return hipGetLastError();
}
hipError_t launch_latent_prefill(const LatentPrefillArgs& a, hipStream_t s) {
    if (a.n_tiles <= 0) return hipSuccess;
    const int rc = a.cache.rot_p / 32;
#define NVLLM_LP(D_, V_)                                                                  \
    if (a.dim_p == D_ * 32 && a.vdim_p == V_ * 16) {                                      \
        if (rc == 1) return latent_prefill_t<D_, 1, V_>(a, s);                            \
        if (rc == 2) return latent_prefill_t<D_, 2, V_>(a, s);                            \
    }
#define NVLLM_LPD(D_) NVLLM_LP(D_, 2) NVLLM_LP(D_, 4) NVLLM_LP(D_, 8)
    NVLLM_LPD(1) NVLLM_LPD(2) NVLLM_LPD(4)
#undef NVLLM_LPD
#undef NVLLM_LP
    return hipErrorNotSupported;
}

}  // namespace nvllm
