// gfx950 scans with carried state (f32): S <- g S; u = beta (v - S^T k) or u = v; S <- S + k u^T; o = S^T q per token and head.
//
// Columns of S are independent, channels of a column meet in two sums per token.  A wave owns eight columns of one head: lane
// (p = lane % 16, c = lane / 16) holds the channels 64 r + 4 p + i of columns 2 c and 2 c + 1 in registers, so both sums are four
// DPP steps inside a row of 16 lanes, and k, q, g of a token are read as conflict-free float4 rows.  Both sums are taken from the
// decayed state at once: with d = S^T k and e = S^T q before the write, o = e + (k . q) u, which is S^T q after it.
#include <algorithm>

#include "device_common.h"
#include "hybrid.h"

namespace nvllm {

// one token on the wave's registers
enum { DECAY_CONST, DECAY_CHANNEL, DECAY_HEAD };  // constant decays; delta rule with a decay per key channel, per head
template <int R4, int KIND>
__device__ __forceinline__ float2 recur_token(float (&S)[R4][2][4], const float4 (&k)[R4], const float4 (&q)[R4], const float4 (&g)[R4], float decay,
                                              float2 v, float beta) {
    constexpr bool DELTA = KIND != DECAY_CONST;
    float dk[2] = {0.f, 0.f}, dq[2] = {0.f, 0.f}, kq = 0.f;
#pragma unroll
    for (int r = 0; r < R4; ++r) {
        const float kv[4] = {k[r].x, k[r].y, k[r].z, k[r].w}, qv[4] = {q[r].x, q[r].y, q[r].z, q[r].w};
        const float gv[4] = {g[r].x, g[r].y, g[r].z, g[r].w};
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            kq += kv[i] * qv[i];
#pragma unroll
            for (int c = 0; c < 2; ++c) {
                S[r][c][i] *= KIND == DECAY_CHANNEL ? gv[i] : decay;
                if (DELTA) dk[c] += S[r][c][i] * kv[i];
                dq[c] += S[r][c][i] * qv[i];
            }
        }
    }
    kq = row16_sum(kq);
    float u[2], o[2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        u[c] = DELTA ? beta * ((c ? v.y : v.x) - row16_sum(dk[c])) : (c ? v.y : v.x);
        o[c] = row16_sum(dq[c]) + u[c] * kq;
    }
#pragma unroll
    for (int r = 0; r < R4; ++r) {
        const float kv[4] = {k[r].x, k[r].y, k[r].z, k[r].w};
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int c = 0; c < 2; ++c) S[r][c][i] += kv[i] * u[c];
    }
    return make_float2(o[0], o[1]);
}

template <int R4>
__device__ __forceinline__ void state_io(float (&S)[R4][2][4], float* st, int lane, bool store) {
#pragma unroll
    for (int r = 0; r < R4; ++r)
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            float4* p = reinterpret_cast<float4*>(st) + (r * 2 + c) * 64 + lane;
            if (store) *p = make_float4(S[r][c][0], S[r][c][1], S[r][c][2], S[r][c][3]);
            else {
                const float4 t = *p;
                S[r][c][0] = t.x; S[r][c][1] = t.y; S[r][c][2] = t.z; S[r][c][3] = t.w;
            }
        }
}

// one workgroup = 32 columns of one head of one segment, tokens in pieces of TT staged through LDS (two buffers)
template <int R4, int KIND>
__global__ void __launch_bounds__(256) recurrence_kernel(RecurArgs a) {
    constexpr bool DELTA = KIND != DECAY_CONST, CHANNEL = KIND == DECAY_CHANNEL;
    constexpr int DP = R4 * 64, TT = R4 <= 2 ? 16 : 8, NV = CHANNEL ? 3 : 2;
    constexpr int W4 = NV * DP / 4 + 9;             // float4 per token: k, q, (g), 32 values, beta and decay
    constexpr int NL = (TT * W4 + 255) / 256;
    __shared__ __attribute__((aligned(16))) float4 buf[2][TT * W4];
    __shared__ float obuf[TT][32];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, p = lane & 15, cg = lane >> 4;
    const int blocks = a.vdim_p / 32, head = blockIdx.x / blocks, cb = blockIdx.x % blocks, sg = blockIdx.y;
    const int row0 = a.seg.single ? sg : a.seg.row0[sg], n = a.seg.single ? 1 : a.seg.n[sg], slot = a.seg.slot[sg];
    const int qh = head / (a.heads / a.q_heads);
    float* st = a.state + ((size_t)slot * a.heads + head) * DP * a.vdim_p + (size_t)(cb * 4 + wave) * 8 * DP;
    float S[R4][2][4];
    if (a.pos[row0] > 0) {
        state_io<R4>(S, st, lane, false);
    } else {
#pragma unroll
        for (int r = 0; r < R4; ++r)
#pragma unroll
            for (int c = 0; c < 2; ++c)
#pragma unroll
                for (int i = 0; i < 4; ++i) S[r][c][i] = 0.f;
    }
    const float decay = DELTA ? 1.f : a.decay[head];  // of every token
    // slot w of token t
    auto fetch = [&](int t, int w) -> float4 {
        const size_t row = row0 + min(t, n - 1);
        if (w < DP / 4) return reinterpret_cast<const float4*>(a.k + (row * a.q_heads + qh) * DP)[w];
        if (w < 2 * (DP / 4)) return reinterpret_cast<const float4*>(a.q + (row * a.q_heads + qh) * DP)[w - DP / 4];
        if (CHANNEL && w < 3 * (DP / 4)) return reinterpret_cast<const float4*>(a.g + row * a.g_row + (size_t)head * DP)[w - 2 * (DP / 4)];
        const int x = w - NV * (DP / 4);
        if (x < 8) return reinterpret_cast<const float4*>(a.v + (row * a.heads + head) * a.vdim_p + cb * 32)[x];
        return make_float4(DELTA ? a.beta[row * a.heads + head] : 0.f, KIND == DECAY_HEAD ? a.gh[row * a.heads + head] : 0.f, 0.f, 0.f);
    };
    float4 pre[NL];
    auto load = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NL; ++i) {
            const int x = min((int)threadIdx.x + i * 256, TT * W4 - 1);
            pre[i] = fetch(t0 + x / W4, x % W4);
        }
    };
    auto park = [&](float4* b) {
#pragma unroll
        for (int i = 0; i < NL; ++i)
            if ((int)threadIdx.x + i * 256 < TT * W4) b[threadIdx.x + i * 256] = pre[i];
    };
    load(0);
    park(buf[0]);
    __syncthreads();
    int cur = 0;
    for (int t0 = 0; t0 < n; t0 += TT, cur ^= 1) {
        const int m = min(TT, n - t0);
        if (t0 + TT < n) load(t0 + TT);
        for (int t = 0; t < m; ++t) {
            const float4* b = buf[cur] + t * W4;
            float4 k[R4], q[R4], g[R4];
#pragma unroll
            for (int r = 0; r < R4; ++r) {
                k[r] = b[r * 16 + p];
                q[r] = b[DP / 4 + r * 16 + p];
                if (CHANNEL) g[r] = b[2 * (DP / 4) + r * 16 + p];
                else g[r] = make_float4(0.f, 0.f, 0.f, 0.f);
            }
            const float* bv = reinterpret_cast<const float*>(b + NV * (DP / 4));
            const float2 v = *reinterpret_cast<const float2*>(bv + wave * 8 + cg * 2);
            const float2 o = recur_token<R4, KIND>(S, k, q, g, KIND == DECAY_HEAD ? bv[33] : decay, v, bv[32]);
            if (p == 0) *reinterpret_cast<float2*>(&obuf[t][wave * 8 + cg * 2]) = o;
        }
        if (t0 + TT < n) park(buf[cur ^ 1]);
        __syncthreads();
        for (int i = threadIdx.x; i < m * 8; i += 256)
            reinterpret_cast<float4*>(a.o + ((size_t)(row0 + t0 + (i >> 3)) * a.heads + head) * a.vdim_p + cb * 32)[i & 7] =
                *reinterpret_cast<const float4*>(&obuf[i >> 3][(i & 7) * 4]);
        __syncthreads();
    }
    state_io<R4>(S, st, lane, true);
}

// ---------------------------------------------------------------------------------------------------
// decode: one workgroup = one (row, head); a wave takes every fourth block of eight columns, four blocks' state in flight.  With
// NORM (per-head norms) the gated output norm follows in the same launch.
// ---------------------------------------------------------------------------------------------------
template <int R4, int KIND, bool NORM>
__global__ void __launch_bounds__(256) recurrence_decode_kernel(RecurArgs a, GatedNormArgs n) {
    constexpr bool DELTA = KIND != DECAY_CONST, CHANNEL = KIND == DECAY_CHANNEL;
    constexpr int DP = R4 * 64, NB = R4 <= 2 ? 4 : 1;
    extern __shared__ float o_lds[];  // [vdim_p], NORM
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, p = lane & 15, cg = lane >> 4;
    const int head = blockIdx.x, row = blockIdx.y, slot = a.seg.slot[row], qh = head / (a.heads / a.q_heads), blocks = a.vdim_p / 8;
    const bool fresh = a.pos[row] == 0;
    float* st = a.state + ((size_t)slot * a.heads + head) * DP * a.vdim_p;
    float4 k[R4], q[R4], g[R4];
    const float4* kp = reinterpret_cast<const float4*>(a.k + ((size_t)row * a.q_heads + qh) * DP) + p;
    const float4* qp = reinterpret_cast<const float4*>(a.q + ((size_t)row * a.q_heads + qh) * DP) + p;
    const float4* gp = reinterpret_cast<const float4*>(CHANNEL ? a.g + (size_t)row * a.g_row + (size_t)head * DP : a.k) + p;
    const float* vp = a.v + ((size_t)row * a.heads + head) * a.vdim_p + cg * 2;
#pragma unroll
    for (int r = 0; r < R4; ++r) {
        k[r] = kp[r * 16];
        q[r] = qp[r * 16];
        g[r] = CHANNEL ? gp[r * 16] : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    const float decay = KIND == DECAY_HEAD ? a.gh[(size_t)row * a.heads + head] : DELTA ? 1.f : a.decay[head], beta = DELTA ? a.beta[(size_t)row * a.heads + head] : 0.f;
    for (int b0 = wave; b0 < blocks; b0 += 4 * NB) {
        float S[NB][R4][2][4];
        float2 v[NB];
#pragma unroll
        for (int u = 0; u < NB; ++u) {
            const int b = min(b0 + u * 4, blocks - 1);
            state_io<R4>(S[u], st + (size_t)b * 8 * DP, lane, false);
            v[u] = *reinterpret_cast<const float2*>(vp + b * 8);
        }
#pragma unroll
        for (int u = 0; u < NB; ++u) {
            const int b = b0 + u * 4;
            if (b >= blocks) continue;
            if (fresh) {
#pragma unroll
                for (int r = 0; r < R4; ++r)
#pragma unroll
                    for (int c = 0; c < 2; ++c)
#pragma unroll
                        for (int i = 0; i < 4; ++i) S[u][r][c][i] = 0.f;
            }
            const float2 o = recur_token<R4, KIND>(S[u], k, q, g, decay, v[u], beta);
            state_io<R4>(S[u], st + (size_t)b * 8 * DP, lane, true);
            if (p == 0) {
                if (NORM) *reinterpret_cast<float2*>(o_lds + b * 8 + cg * 2) = o;
                else *reinterpret_cast<float2*>(a.o + ((size_t)row * a.heads + head) * a.vdim_p + b * 8 + cg * 2) = o;
            }
        }
    }
    if constexpr (NORM) {
        __syncthreads();
        float ss = 0.f;
        for (int e = threadIdx.x; e < n.vdim; e += 256) ss += o_lds[e] * o_lds[e];
        const float rinv = 1.0f / sqrtf(block_sum(ss, red, 4) / (float)n.vdim + n.eps);
        const float* gate = n.gate + (size_t)row * n.gate_row + (size_t)head * n.gate_head;
        for (int e = threadIdx.x; e < n.vdim; e += 256) {
            float f = gate[e];
            if (n.gate_slabs) {
                f = slab_elem(gate + e, n.gate_slabs, n.gate_stride);
                f = f / (1.0f + expf(-f));
            }
            const float x = (o_lds[e] * rinv) * n.weight[e] * f;
            const int col = head * n.vdim + e;
            if (n.of) n.of[(size_t)row * n.ld + col] = x;
            if (n.oh) {
                const size_t at = n.packed ? xpack_off(row, col, n.ld >> 5) : (size_t)row * n.ld + col;
                split_bf16(x, n.oh[at], n.ol[at]);
            }
        }
    }
}

bool recur_ok(int dim, int vdim) { return dim >= 1 && dim <= 512 && vdim >= 1 && vdim <= 8192; }

template <int R4, int KIND>
static void recurrence_t(const RecurArgs& a, const GatedNormArgs* norm, hipStream_t s) {
    if (!a.seg.single) recurrence_kernel<R4, KIND><<<dim3(a.heads * (a.vdim_p / 32), a.seg.count), 256, 0, s>>>(a);
    else if (norm) recurrence_decode_kernel<R4, KIND, true><<<dim3(a.heads, a.seg.count), 256, (size_t)a.vdim_p * 4, s>>>(a, *norm);
    else recurrence_decode_kernel<R4, KIND, false><<<dim3(a.heads, a.seg.count), 256, 0, s>>>(a, GatedNormArgs());
}
template <int KIND>
static hipError_t recurrence_launch(const RecurArgs& a, const GatedNormArgs* norm, hipStream_t s) {
    switch (a.dim_p / 64) {
#define NVLLM_RC(R_) case R_: recurrence_t<R_, KIND>(a, norm, s); break;
        NVLLM_RC(1) NVLLM_RC(2) NVLLM_RC(3) NVLLM_RC(4) NVLLM_RC(5) NVLLM_RC(6) NVLLM_RC(7) NVLLM_RC(8)
#undef NVLLM_RC
        default: return hipErrorNotSupported;
    }
    return hipGetLastError();
}
hipError_t launch_recurrence(const RecurArgs& a, const GatedNormArgs* norm, hipStream_t s) {
    if (a.dim_p % 64 || a.vdim_p % 32 || a.q_heads < 1 || a.heads % a.q_heads || ((a.g || a.gh) && !a.beta) || (a.g && a.gh) || (!a.g && !a.gh && !a.decay) || (a.g_row & 3)) return hipErrorInvalidValue;
    if (norm && (!a.seg.single || norm->whole || norm->heads != a.heads || norm->vdim_p != a.vdim_p || norm->heads * norm->vdim > norm->ld)) return hipErrorInvalidValue;
    if (a.seg.count <= 0) return hipSuccess;
    if (a.gh) return recurrence_launch<DECAY_HEAD>(a, norm, s);
    return a.g ? recurrence_launch<DECAY_CHANNEL>(a, norm, s) : recurrence_launch<DECAY_CONST>(a, norm, s);
}

}  // namespace nvllm
