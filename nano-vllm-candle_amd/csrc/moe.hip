// gfx950 kernels of routed feed-forwards: choice of experts, grouping of rows, products over groups.
#include <algorithm>

#include "device_common.h"
#include "moe.h"

namespace nvllm {

// ---------------------------------------------------------------------------------------------------
// choice: NL lanes per row (16, 32 or a wave); lane l of them holds the logits of experts l, l + NL, ...
// ---------------------------------------------------------------------------------------------------
__device__ __forceinline__ float sigmoid_exact(float x) { return 1.0f / (1.0f + expf(-x)); }

template <int NV, int NL>
__device__ __forceinline__ void route_row(const RouteArgs& a, int row, int lane) {
    const bool in = row < a.rows;  // lanes past the last row take part in the exchanges
    const float* z = a.z + (size_t)min(row, a.rows - 1) * a.ld;
    float v[NV];
    float gate = 0.f;
    if (a.gate_col >= 0) gate = z[a.gate_col];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int e = lane + i * NL;
        const float x = z[min(e, a.experts - 1)];
        v[i] = e < a.experts ? x : -INFINITY;
    }
    if (a.gate_col >= 0 && lane == 0 && in) a.gate[row] = sigmoid_exact(gate);
    // the largest of the row and its expert, lowest index on a tie
    auto largest = [&](const float (&x)[NV], float& best, int& at) {
        best = -INFINITY;
        at = kMaxExperts;
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (x[i] > best) { best = x[i]; at = lane + i * NL; }
#pragma unroll
        for (int o = NL / 2; o > 0; o >>= 1) {
            const float b = __shfl_xor(best, o);
            const int c = __shfl_xor(at, o);
            if (b > best || (b == best && c < at)) { best = b; at = c; }
        }
        at = min(at, a.experts - 1);  // no finite logit left
    };
    float top_z = 0.f, total = 1.f;
    if (a.softmax) {
        top_z = v[0];
#pragma unroll
        for (int i = 1; i < NV; ++i) top_z = fmaxf(top_z, v[i]);
#pragma unroll
        for (int o = NL / 2; o > 0; o >>= 1) top_z = fmaxf(top_z, __shfl_xor(top_z, o));
        total = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) total += expf(v[i] - top_z);
#pragma unroll
        for (int o = NL / 2; o > 0; o >>= 1) total += __shfl_xor(total, o);
    }
    if (a.keep < a.groups) {  // the best group left holds the largest logit of the groups left
        const int per = a.experts / a.groups;
        float left[NV];
        bool kept[NV];
#pragma unroll
        for (int i = 0; i < NV; ++i) { left[i] = v[i]; kept[i] = false; }
        for (int k = 0; k < a.keep; ++k) {
            float best;
            int at;
            largest(left, best, at);
            const int g = at / per;
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if ((lane + i * NL) / per == g) { left[i] = -INFINITY; kept[i] = true; }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) v[i] = kept[i] ? v[i] : -INFINITY;
    }
    for (int k = 0; k < a.top; ++k) {
        float best;
        int at;
        largest(v, best, at);
        if (lane == 0 && in) {
            a.chosen[(size_t)row * a.top + k] = at;
            a.score[(size_t)row * a.top + k] = a.softmax ? expf(best - top_z) / total : sigmoid_exact(best);
        }
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (at == lane + i * NL) v[i] = -INFINITY;
    }
}
template <int NV, int NL>
__global__ void __launch_bounds__(256) route_kernel(RouteArgs a) {
    route_row<NV, NL>(a, blockIdx.x * (256 / NL) + threadIdx.x / NL, threadIdx.x % NL);
}

// a member's entries
__device__ __forceinline__ void place_row(const RouteArgs& a, int i, int p, float score) {
    const int row = i / a.top, k = i - row * a.top;
    a.src[p] = row;
    a.pre[p] = a.weight_in ? score : 1.f;
    a.post[p] = a.weight_in ? 1.f : score;
    a.place[(size_t)row * (a.top + a.shared_group) + k] = p;
}
__device__ __forceinline__ void place_shared(const RouteArgs& a, int row, int p) {
    a.src[p] = row;
    a.pre[p] = 1.f;
    a.post[p] = a.gate_col >= 0 ? a.gate[row] : 1.f;
    a.place[(size_t)row * (a.top + 1) + a.top] = p;
}

// one workgroup: group sizes, starts, tiles and padding.  NV > 0 (few rows): the choice and every row's position as well; else the positions
// are left to place_rows_kernel, which starts from cursor.
template <int NV, int NL>
__global__ void __launch_bounds__(1024) group_rows_kernel(RouteArgs a) {
    __shared__ int count[kMaxExperts + 1], start[kMaxExperts + 1], wave_total[16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int groups = a.experts + a.shared_group, n = a.rows * a.top;
    for (int g = tid; g <= kMaxExperts; g += 1024) count[g] = 0;
    if constexpr (NV > 0)
        for (int r0 = 0; r0 < a.rows; r0 += 1024 / NL) route_row<NV, NL>(a, r0 + tid / NL, tid % NL);
    __syncthreads();
    constexpr int U = NV > 0 ? 1 : 8;  // loads in flight
    for (int i0 = tid; i0 < n; i0 += 1024 * U) {
        int g[U];
#pragma unroll
        for (int u = 0; u < U; ++u) g[u] = a.chosen[min(i0 + u * 1024, n - 1)];
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (i0 + u * 1024 < n) atomicAdd(&count[g[u]], 1);
    }
    if (a.shared_group && tid == 0) count[a.experts] = a.rows;
    __syncthreads();
    // exclusive prefix sum of the aligned sizes, one group per thread (a shared group after 1024 experts: the first thread again)
    const int sz = tid < groups ? (count[tid] + a.align - 1) / a.align * a.align : 0;
    int inc = sz;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const int t = __shfl_up(inc, o);
        if (lane >= o) inc += t;
    }
    if (lane == 63) wave_total[wave] = inc;
    __syncthreads();
    int base = 0, all = 0;
    for (int w = 0; w < 16; ++w) {
        if (w < wave) base += wave_total[w];
        all += wave_total[w];
    }
    if (tid < groups) start[tid] = base + inc - sz;
    if (groups > 1024 && tid == 0) start[1024] = all;
    __syncthreads();
    const int end = groups > 1024 ? all + (count[1024] + a.align - 1) / a.align * a.align : all;
    for (int g = wave; g < groups; g += 16) {
        const int p0 = start[g], c = count[g], p1 = p0 + (c + a.align - 1) / a.align * a.align;
        for (int t = p0 / a.align + lane; t < p1 / a.align; t += 64) a.tile_group[t] = g;
        for (int p = p0 + c + lane; p < p1; p += 64) { a.src[p] = -1; a.pre[p] = 0.f; a.post[p] = 0.f; }
    }
    for (int t = end / a.align + tid; t < a.cap / a.align; t += 1024) a.tile_group[t] = -1;
    if constexpr (NV == 0) {
        for (int g = tid; g < groups; g += 1024) a.cursor[g] = start[g];
    } else {
        __syncthreads();
        for (int i = tid; i < n; i += 1024) place_row(a, i, atomicAdd(&start[a.chosen[i]], 1), a.score[i]);
        if (a.shared_group) {
            __syncthreads();
            for (int row = tid; row < a.rows; row += 1024) place_shared(a, row, start[a.experts] + row);
        }
    }
}
// many rows: a workgroup reserves a range of every group for its share of them.  The order of a group's members does not matter: every
// position is computed alone.
__global__ void __launch_bounds__(1024) place_rows_kernel(RouteArgs a) {
    __shared__ int count[kMaxExperts], base[kMaxExperts];
    const int tid = threadIdx.x, n = a.rows * a.top, i = blockIdx.x * 1024 + tid;
    for (int g = tid; g < a.experts; g += 1024) count[g] = 0;
    __syncthreads();
    const int g = i < n ? a.chosen[i] : 0;
    const float score = i < n ? a.score[i] : 0.f;
    const int at = i < n ? atomicAdd(&count[g], 1) : 0;
    __syncthreads();
    for (int e = tid; e < a.experts; e += 1024) base[e] = count[e] ? atomicAdd(&a.cursor[e], count[e]) : 0;
    __syncthreads();
    if (i < n) place_row(a, i, base[g] + at, score);
    if (a.shared_group && i < a.rows) place_shared(a, i, a.cursor[a.experts] + i);
}

hipError_t launch_route(const RouteArgs& a, hipStream_t s) {
    const int64_t need = (int64_t)a.rows * a.top + (int64_t)std::min(a.experts, a.rows * a.top) * (a.align - 1) + (a.shared_group ? a.rows + a.align - 1 : 0);
    if (a.experts < 1 || a.experts > kMaxExperts || a.top < 1 || a.top > std::min(a.experts, kMaxTop) || a.align < 1 || a.cap % a.align || need > a.cap ||
        a.groups < 1 || a.experts % a.groups || a.keep < 1 || (a.keep < a.groups && a.top > a.keep * (a.experts / a.groups)) || a.ld < a.experts || a.gate_col >= a.ld || (a.gate_col >= 0 && !a.gate) || !a.cursor)
        return hipErrorInvalidValue;
    if (a.rows <= 0) return hipSuccess;
    const bool one = a.rows <= 64;
    const int nv = (a.experts + 63) / 64;
#define NVLLM_RT(V_, L_)                                                                   \
    if (one) group_rows_kernel<V_, L_><<<1, 1024, 0, s>>>(a);                              \
    else {                                                                                 \
        route_kernel<V_, L_><<<(a.rows + 256 / L_ - 1) / (256 / L_), 256, 0, s>>>(a);      \
        group_rows_kernel<0, 64><<<1, 1024, 0, s>>>(a);                                    \
        place_rows_kernel<<<(a.rows * a.top + 1023) / 1024, 1024, 0, s>>>(a);              \
    }
    if (a.experts <= 16) { NVLLM_RT(1, 16) }
    else if (a.experts <= 32) { NVLLM_RT(1, 32) }
    else if (nv <= 1) { NVLLM_RT(1, 64) }
    else if (nv <= 2) { NVLLM_RT(2, 64) }
    else if (nv <= 4) { NVLLM_RT(4, 64) }
    else if (nv <= 8) { NVLLM_RT(8, 64) }
    else { NVLLM_RT(16, 64) }
#undef NVLLM_RT
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------
// products over groups: MT m-tiles (16 positions each) of one group x NT n-tiles per wave; the four waves take other n-tiles (WK = 1)
// or a quarter of K each, summed through LDS (WK = 4: few rows, many weight bytes).  GLU: n-tiles are pairs of a gate and an up tile.
// ---------------------------------------------------------------------------------------------------
template <int MT, int NT, int WK, bool EXACT, bool GLU>
__global__ void __launch_bounds__(256) group_gemm_kernel(GroupGemmArgs a) {
    __shared__ __attribute__((aligned(16))) f32x4 part[WK == 4 ? 4 * NT * MT * 64 : 1];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int l15 = lane & 15, grp = lane >> 4;
    const int tile = blockIdx.y, g = a.tile_group ? a.tile_group[tile] : 0;
    if (g < 0) return;
    const bool other = g == a.last;
    const int ntiles = (other ? a.Ns : a.N) >> 4, KT = (other ? a.Ks : a.K) >> 5;
    const int nt0 = WK == 4 ? (int)blockIdx.x * NT : ((int)blockIdx.x * 4 + wave) * NT;
    if (nt0 >= ntiles) return;  // WK = 4: the whole workgroup
    const uint4* wp = other ? a.ws : a.w + (size_t)g * a.w_group;
    const int per = WK == 4 ? (KT + 3) / 4 : KT, k0 = WK == 4 ? wave * per : 0, k1 = min(KT, k0 + per);
    const int p0 = tile * (MT * 16);
    // this lane's row of every m-tile (padding positions: row 0, result multiplied by 0 or never read)
    const int KX = a.ldx >> 5;
    size_t xo[MT], step;
#pragma unroll
    for (int b = 0; b < MT; ++b) {
        const int p = p0 + b * 16 + l15;
        int row = a.src ? a.src[p] : p;
        row = min(max(row, 0), a.x_rows - 1);
        if constexpr (EXACT) xo[b] = (size_t)row * a.ldx + grp * 8;
        else xo[b] = a.x_packed ? ((size_t)(row >> 4) * KX * 64 + (grp << 4) + (row & 15)) : ((size_t)row * a.ldx >> 3) + grp;
    }
    step = EXACT ? 32 : a.x_packed ? 64 : 4;
    f32x4 acc[NT][MT];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int b = 0; b < MT; ++b) acc[n][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint4 *xh = reinterpret_cast<const uint4*>(a.xh), *xl = reinterpret_cast<const uint4*>(a.xl);
    constexpr int U = EXACT ? 1 : MT == 1 ? 4 : 1;  // k-tiles in flight
    for (int kt0 = k0; kt0 < k1; kt0 += U) {
        uint4 wf[U][NT];
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int n = 0; n < NT; ++n) wf[u][n] = wp[((size_t)min(nt0 + n, ntiles - 1) * KT + min(kt0 + u, k1 - 1)) * 64 + lane];
        if constexpr (EXACT) {
            float xv[MT][8];
#pragma unroll
            for (int b = 0; b < MT; ++b) {
                *reinterpret_cast<float4*>(&xv[b][0]) = *reinterpret_cast<const float4*>(a.xf + xo[b] + (size_t)kt0 * step);
                *reinterpret_cast<float4*>(&xv[b][4]) = *reinterpret_cast<const float4*>(a.xf + xo[b] + (size_t)kt0 * step + 4);
            }
#pragma unroll
            for (int n = 0; n < NT; ++n) {
                const uint32_t wd[4] = {wf[0][n].x, wf[0][n].y, wf[0][n].z, wf[0][n].w};
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const float wv = (j & 1) ? __builtin_bit_cast(float, wd[j >> 1] & 0xffff0000u) : __builtin_bit_cast(float, wd[j >> 1] << 16);
#pragma unroll
                    for (int b = 0; b < MT; ++b) acc[n][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(wv, xv[b][j], acc[n][b], 0, 0, 0);
                }
            }
        } else {
            uint4 fh[U][MT], fl[U][MT];
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int b = 0; b < MT; ++b) {
                    const size_t o = xo[b] + (size_t)min(kt0 + u, k1 - 1) * step;
                    fh[u][b] = xh[o];
                    fl[u][b] = xl[o];
                }
#pragma unroll
            for (int u = 0; u < U; ++u)
                if (kt0 + u < k1) {
#pragma unroll
                    for (int n = 0; n < NT; ++n) {
                        const bf16x8 wv = __builtin_bit_cast(bf16x8, wf[u][n]);
#pragma unroll
                        for (int b = 0; b < MT; ++b) {
                            acc[n][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, __builtin_bit_cast(bf16x8, fh[u][b]), acc[n][b], 0, 0, 0);
                            acc[n][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, __builtin_bit_cast(bf16x8, fl[u][b]), acc[n][b], 0, 0, 0);
                        }
                    }
                }
        }
    }
    if constexpr (WK == 4) {
#pragma unroll
        for (int n = 0; n < NT; ++n)
#pragma unroll
            for (int b = 0; b < MT; ++b) part[((wave * NT + n) * MT + b) * 64 + lane] = acc[n][b];
        __syncthreads();
    }
    auto whole = [&](int n, int b) {  // the finished sum
        f32x4 v = acc[n][b];
        if constexpr (WK == 4) {
            v = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const f32x4 t = part[((q * NT + n) * MT + b) * 64 + lane];
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] += t[r];
            }
        }
        return v;
    };
    if constexpr (GLU) {
        static_assert(!GLU || NT == 2, "a gate tile and its up tile");
        const int f = (nt0 >> 1) * 16 + grp * 4;
#pragma unroll
        for (int b = 0; b < MT; ++b) {
            if (WK == 4 && b % 4 != wave) continue;
            const f32x4 gate = whole(0, b), up = whole(1, b);
            const int p = p0 + b * 16 + l15;
            const float post = a.post ? a.post[p] : 1.f;
            f32x4 v;
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = (EXACT ? gate[r] / (1.0f + expf(-gate[r])) * up[r] : silu_mul(gate[r], up[r])) * post;
            if (a.out) *reinterpret_cast<float4*>(a.out + (size_t)p * a.ldo + f) = make_float4(v[0], v[1], v[2], v[3]);
            if (a.oh) put_planes4(a.oh, a.ol, p, f, 4, a.ldo, 1, v);
        }
        return;
    }
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        if (nt0 + n >= ntiles) continue;
        const int f = (nt0 + n) * 16 + grp * 4;
#pragma unroll
        for (int b = 0; b < MT; ++b) {
            if (WK == 4 && (n * MT + b) % 4 != wave) continue;
            f32x4 v = whole(n, b);
            const int p = p0 + b * 16 + l15;
            if (!a.tile_group && p >= a.x_rows) continue;
            const float pre = a.pre ? a.pre[p] : 1.f, post = a.post ? a.post[p] : 1.f;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                v[r] *= pre;
                if (a.relu2) v[r] = relu2(v[r]);
                v[r] *= post;
            }
            if (a.out) *reinterpret_cast<float4*>(a.out + (size_t)p * a.ldo + f) = make_float4(v[0], v[1], v[2], v[3]);
            if (a.oh) put_planes4(a.oh, a.ol, p, f, 4, a.ldo, 1, v);
        }
    }
}

hipError_t launch_group_gemm(const GroupGemmArgs& a, hipStream_t s) {
    const bool exact = a.xf != nullptr;
    const int nmax = a.last >= 0 ? std::max(a.N, a.Ns) : a.N, kmax = a.last >= 0 ? std::max(a.K, a.Ks) : a.K;
    if (a.N % 16 || a.K % 32 || (a.last >= 0 && (a.Ns % 16 || a.Ks % 32 || !a.ws)) || a.ldx % 32 || a.ldx < kmax || (!exact && (!a.xh || !a.xl)) ||
        (!a.out && !a.oh) || a.ldo < (a.glu ? nmax / 2 : nmax) || (a.glu && (a.N % 32 || a.last >= 0 || a.relu2 || a.pre || !a.tile_group)) || a.ldo % (a.oh ? 32 : 4) || a.x_rows < 1 || (a.align != 16 && a.align != 64))
        return hipErrorInvalidValue;
    const int tiles = a.tile_group ? a.tiles : (a.x_rows + a.align - 1) / a.align;
    if (tiles <= 0) return hipSuccess;
    const int nt = nmax / 16;
#define NVLLM_GG(MT_, NT_, WK_, EX_, GLU_) group_gemm_kernel<MT_, NT_, WK_, EX_, GLU_><<<dim3((nt + NT_ * (WK_ == 4 ? 1 : 4) - 1) / (NT_ * (WK_ == 4 ? 1 : 4)), tiles), 256, 0, s>>>(a)
    if (a.align == 64) {
        if (a.glu && exact) NVLLM_GG(4, 2, 1, true, true);
        else if (a.glu) NVLLM_GG(4, 2, 1, false, true);
        else if (exact) NVLLM_GG(4, 1, 1, true, false);
        else NVLLM_GG(4, 2, 1, false, false);
    } else {
        if (a.glu && exact) NVLLM_GG(1, 2, 4, true, true);
        else if (a.glu) NVLLM_GG(1, 2, 4, false, true);
        else if (exact) NVLLM_GG(1, 1, 4, true, false);
        else NVLLM_GG(1, 2, 4, false, false);
    }
#undef NVLLM_GG
    return hipGetLastError();
}

}  // namespace nvllm
