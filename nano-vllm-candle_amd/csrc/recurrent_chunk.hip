// gfx950 recurrences over prompt chunks in pieces of 16 tokens, everything in f32 (16x16x4 f32 MFMA).
//
// With G_i the decays multiplied up to token i of a piece, S_0 the state before it and t_j(i) = k_j * decays of tokens j+1..i:
//   delta rule:  u_i = beta_i (v_i - S_0^T (G_i k_i) - sum_{j<i} (k_i . t_j(i)) u_j)
//                o_i = S_0^T (G_i q_i) + sum_{j<=i} (q_i . t_j(i)) u_j,     S' = G_16 S_0 + sum_j t_j(16) u_j^T
// Everything but S_0 and u is known per piece: the triangular system is solved once for the columns of v and of G k,
//   (I + diag(beta) A) [V' W] = diag(beta) [V  G K],   then   u = V' - W S_0.
// delta_pieces_kernel does that for every piece in parallel (decays only ever multiply, nothing is divided or exponentiated, so decays that
// underflow are harmless); piece_scan_kernel walks the pieces of a sequence with three products per piece on the state in registers.
// Constant decays need no W and no triangular system; their powers scale rows of the accumulators.
//
// Order of a piece's tokens in the operands: accumulator register r of lane group g holds token 4 r + g, so u leaves its product in the
// B-operand order of the next ones, and the state's accumulators (channel 16 t + 4 g + r) are themselves the B operand of W S and Q S.
#include <algorithm>

#include "device_common.h"
#include "hybrid.h"

namespace nvllm {

__device__ __forceinline__ int token_slot(int j) { return ((j & 3) << 2) | (j >> 2); }  // place of token j among a row's 16: lane group, register

// ---------------------------------------------------------------------------------------------------
// one wave per (piece, head)
// ---------------------------------------------------------------------------------------------------
// HEAD: one decay per head and token, so the pair products are two plain products on the matrix cores with factors on their results
template <int R4, bool HEAD>
__global__ void __launch_bounds__(64) delta_pieces_kernel(RecurArgs a, PieceArgs c) {
    constexpr int DP = R4 * 64;
    __shared__ __attribute__((aligned(16))) float A[16 * 16];
    const int lane = threadIdx.x, dg = lane & 15, jg = lane >> 4;
    const int head = blockIdx.x, piece = blockIdx.y, row0 = c.row0[piece], n = c.n[piece], qh = head / (a.heads / a.q_heads);
    const size_t ph = (size_t)piece * a.heads + head;
    // rows past the piece's last one hold something finite that is masked
    const float* kb = a.k + ((size_t)row0 * a.q_heads + qh) * DP;
    const float* qb = a.q + ((size_t)row0 * a.q_heads + qh) * DP;
    const float* gb = HEAD ? a.gh + (size_t)row0 * a.heads + head : a.g + (size_t)row0 * a.g_row + (size_t)head * DP;
    const int ks = a.q_heads * DP, gs = HEAD ? a.heads : (int)a.g_row;
    [[maybe_unused]] float gh[16];
    if constexpr (HEAD) {
#pragma unroll
        for (int i = 0; i < 16; ++i) gh[i] = i < n ? gb[i * gs] : 1.f;
        // products of decays from token j + 1 on, j = dg: to tokens i = 4 jg + r and to the piece's end
        float f = 1.f, upto[4] = {0.f, 0.f, 0.f, 0.f}, all = 1.f;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            if (i > dg) f *= gh[i];
            all *= gh[i];
            if ((i >> 2) == jg && i >= dg) upto[i & 3] = f;
        }
        const float end = dg < n ? f : 0.f;
        const float* q = qb + min(dg, n - 1) * ks + jg * 4;
        const float* k = kb + min(dg, n - 1) * ks + jg * 4;
        float* kt = c.kt + ph * (16 * DP) + token_slot(dg);
        f32x4 kk[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}}, qk[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int t = 0; t < R4 * 4; ++t) {
            const float4 x = *reinterpret_cast<const float4*>(q + t * 16), y = *reinterpret_cast<const float4*>(k + t * 16);
            const float xv[4] = {x.x, x.y, x.z, x.w}, yv[4] = {y.x, y.y, y.z, y.w};
            float* o = kt + (t * 16 + jg * 4) * 16;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                kk[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(yv[e], yv[e], kk[t & 1], 0, 0, 0);
                qk[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(xv[e], yv[e], qk[t & 1], 0, 0, 0);
                o[e * 16] = yv[e] * end;
            }
        }
        float* pair = c.pair + ph * 256;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = jg * 4 + r, at = i * 16 + token_slot(dg);
            const float p = i < n ? upto[r] : 0.f;  // 0 for i < j too
            A[at] = (kk[0][r] + kk[1][r]) * p;
            pair[at] = (qk[0][r] + qk[1][r]) * p;
        }
        for (int d = lane; d < DP; d += 64) c.decay[ph * DP + d] = all;
    } else {
        // A and B: lane (jg, dg) carries t_j of tokens j = 4 s + jg for the channels 64 r + 4 dg + e
        float t[4][R4 * 4], all[R4 * 4];
#pragma unroll
        for (int x = 0; x < R4 * 4; ++x) {
            all[x] = 1.f;
#pragma unroll
            for (int s = 0; s < 4; ++s) t[s][x] = 0.f;
        }
        float4 kn[R4], qn[R4], gn[R4];
        auto load = [&](int i) {
#pragma unroll
            for (int r = 0; r < R4; ++r) {
                kn[r] = *reinterpret_cast<const float4*>(kb + i * ks + (r * 64 + dg * 4));
                qn[r] = *reinterpret_cast<const float4*>(qb + i * ks + (r * 64 + dg * 4));
                gn[r] = *reinterpret_cast<const float4*>(gb + i * gs + (r * 64 + dg * 4));
            }
        };
        load(0);
#pragma unroll
        for (int sh = 0; sh < 4; ++sh) {
            for (int il = 0; il < 4; ++il) {
                const int i = sh * 4 + il;
                const bool in = i < n;
                float k[R4 * 4], q[R4 * 4], g[R4 * 4];
#pragma unroll
                for (int r = 0; r < R4; ++r) {
                    const float kv[4] = {kn[r].x, kn[r].y, kn[r].z, kn[r].w}, qv[4] = {qn[r].x, qn[r].y, qn[r].z, qn[r].w};
                    const float gv[4] = {gn[r].x, gn[r].y, gn[r].z, gn[r].w};
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        k[r * 4 + e] = in ? kv[e] : 0.f;
                        q[r * 4 + e] = in ? qv[e] : 0.f;
                        g[r * 4 + e] = in ? gv[e] : 1.f;
                    }
                }
                if (i < 15) load(i + 1);
                float av[4] = {0.f, 0.f, 0.f, 0.f}, bv[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int x = 0; x < R4 * 4; ++x) {
                    all[x] *= g[x];
#pragma unroll
                    for (int s = 0; s <= sh; ++s) {
                        t[s][x] *= g[x];
                        if (s == sh && jg == il) t[s][x] = k[x];
                        av[s] += k[x] * t[s][x];
                        bv[s] += q[x] * t[s][x];
                    }
                }
#pragma unroll
                for (int s = 0; s <= sh; ++s) {
                    av[s] = row16_sum(av[s]);
                    bv[s] = row16_sum(bv[s]);
                }
                if (dg == 0) {
                    *reinterpret_cast<float4*>(&A[i * 16 + jg * 4]) = make_float4(av[0], av[1], av[2], av[3]);
                    reinterpret_cast<float4*>(c.pair + ph * 256)[i * 4 + jg] = make_float4(bv[0], bv[1], bv[2], bv[3]);
                }
            }
        }
#pragma unroll
        for (int r = 0; r < R4; ++r) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = r * 64 + dg * 4 + e, x = r * 4 + e;
                reinterpret_cast<float4*>(c.kt + ph * (16 * DP))[d * 4 + jg] = make_float4(t[0][x], t[1][x], t[2][x], t[3][x]);
            }
            if (jg == 0) reinterpret_cast<float4*>(c.decay + ph * DP)[r * 16 + dg] = make_float4(all[r * 4], all[r * 4 + 1], all[r * 4 + 2], all[r * 4 + 3]);
        }
    }
    __syncthreads();
    // forward substitution, one column per lane: W for the channels, V' for the values
    float beta[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) beta[i] = i < n ? a.beta[(size_t)(row0 + i) * a.heads + head] : 0.f;
    auto solve = [&](float (&y)[16]) {
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float s = y[i];
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                if (x > 0 && x >= i) continue;
                const float4 v = *reinterpret_cast<const float4*>(&A[i * 16 + x * 4]);  // tokens x, 4 + x, 8 + x, 12 + x
                if (x < i) s -= v.x * y[x];
                if (4 + x < i) s -= v.y * y[4 + x];
                if (8 + x < i) s -= v.z * y[8 + x];
                if (12 + x < i) s -= v.w * y[12 + x];
            }
            y[i] = beta[i] * s;
        }
    };
#pragma unroll 1
    for (int d = lane; d < DP; d += 64) {
        float y[16], f = 1.f;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const float g = HEAD ? gh[i] : gb[i * gs + d], k = kb[i * ks + d], q = qb[i * ks + d];
            f *= i < n ? g : 1.f;
            y[i] = i < n ? k * f : 0.f;
            c.qt[(ph * 16 + i) * DP + d] = i < n ? q * f : 0.f;
        }
        solve(y);
#pragma unroll
        for (int i = 0; i < 16; ++i) c.wt[(ph * 16 + i) * DP + d] = y[i];
    }
    float* v = const_cast<float*>(a.v) + ((size_t)row0 * a.heads + head) * a.vdim_p;
    const int vs = a.heads * a.vdim_p;
#pragma unroll 1
    for (int e = lane; e < a.vdim_p; e += 64) {
        float y[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const float x = v[i * vs + e];
            y[i] = i < n ? x : 0.f;
        }
        solve(y);
#pragma unroll
        for (int i = 0; i < 16; ++i)
            if (i < n) v[i * vs + e] = y[i];
    }
}

// constant decays: decay^(i - j) q_i . k_j (j <= i) and the keys decayed to the piece's end; one wave per (piece, head)
template <int R4>
__global__ void __launch_bounds__(64) linear_pieces_kernel(RecurArgs a, PieceArgs c) {
    constexpr int DP = R4 * 64;
    const int lane = threadIdx.x, l15 = lane & 15, grp = lane >> 4;
    const int head = blockIdx.x, piece = blockIdx.y, row0 = c.row0[piece], n = c.n[piece], qh = head / (a.heads / a.q_heads);
    const float* q = a.q + ((size_t)(row0 + min(l15, n - 1)) * a.q_heads + qh) * DP + grp * 4;
    const float* k = a.k + ((size_t)(row0 + min(l15, n - 1)) * a.q_heads + qh) * DP + grp * 4;
    const size_t ph = (size_t)piece * a.heads + head;
    const float decay = a.decay[head];
    float p[16];
    p[0] = 1.f;
#pragma unroll
    for (int i = 1; i < 16; ++i) p[i] = p[i - 1] * decay;
    auto power = [&](int e) {
        float f = 0.f;
#pragma unroll
        for (int x = 0; x < 16; ++x) f = e == x ? p[x] : f;
        return f;
    };
    const float end = l15 < n ? power(n - 1 - l15) : 0.f;
    float* kt = c.kt + ph * (16 * DP) + token_slot(l15);
    f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int t = 0; t < R4 * 4; ++t) {
        const float4 x = *reinterpret_cast<const float4*>(q + t * 16), y = *reinterpret_cast<const float4*>(k + t * 16);
        acc[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, acc[t & 1], 0, 0, 0);
        acc[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, acc[t & 1], 0, 0, 0);
        acc[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, acc[t & 1], 0, 0, 0);
        acc[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, acc[t & 1], 0, 0, 0);
        float* o = kt + (t * 16 + grp * 4) * 16;
        o[0] = y.x * end;
        o[16] = y.y * end;
        o[32] = y.z * end;
        o[48] = y.w * end;
    }
    float* o = c.pair + ph * 256;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int i = grp * 4 + r, j = l15;
        o[i * 16 + token_slot(j)] = i < n && j <= i ? (acc[0][r] + acc[1][r]) * power(i - j) : 0.f;
    }
}

// ---------------------------------------------------------------------------------------------------
// the pieces of one sequence in order: one workgroup = NW waves x 16 columns of one head
// ---------------------------------------------------------------------------------------------------
template <int R4, bool DELTA, int NW>
__global__ void __launch_bounds__(64 * NW) piece_scan_kernel(RecurArgs a, PieceArgs c) {
    constexpr int DP = R4 * 64, T = DP / 16, ROW = DP / 4;  // float4 per row of a [16][DP] operand
    // float4 slots of a stage: Q, K (transposed and decayed), pair, then W and the decays of the delta rule
    constexpr int oQ = 0, oK = 16 * ROW, oP = 32 * ROW, oW = oP + 64, oG = oW + 16 * ROW, N4 = DELTA ? oG + ROW : oW;
    constexpr int NI = (N4 + 64 * NW - 1) / (64 * NW);
    constexpr int SLOTS = NI * 64 * NW;
    __shared__ __attribute__((aligned(16))) float4 buf[2][SLOTS];
    const int lane = threadIdx.x & 63, l15 = lane & 15, grp = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int blocks = (a.vdim_p + 16 * NW - 1) / (16 * NW), head = blockIdx.x / blocks, col0 = ((blockIdx.x % blocks) * NW + wave) * 16;
    const int sg = blockIdx.y, slot = a.seg.slot[sg], p0 = c.seg_piece0[sg];
    const int qh = head / (a.heads / a.q_heads);
    const bool live = col0 < a.vdim_p;
    const int col = min(col0, a.vdim_p - 16) + l15;
    // Rows of Q and W are stored with their float4 units permuted by the token: reads of one unit of 16 tokens fall on different banks.
    // Every copy of a stage has a uniform base that moves on by a
    // constant per piece and a lane offset that stays; a last piece of fewer rows reads on into rows that meet zero weights.
    const int first = a.seg.row0[sg], rows = a.seg.n[sg];
    const size_t ph = (size_t)p0 * a.heads + head, lin = ((size_t)first * a.q_heads + qh) * ROW;
    const float4* src[NI];
    int move[NI];
    uint32_t off[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int x0 = (i * NW + wave) * 64, x = x0 + lane;
        const float4* base = reinterpret_cast<const float4*>(c.pair) + ph * 64;
        int mv = a.heads * 64, o = min(x - oP, 63);
        if (x0 < oP) {
            const bool isq = x0 < oK;
            const int y = isq ? x : x - oK, tok = y / ROW, unit = (y % ROW) ^ token_slot(tok);
            if (!DELTA && isq) {
                base = reinterpret_cast<const float4*>(a.q) + lin;
                mv = 16 * a.q_heads * ROW;
                o = tok * a.q_heads * ROW + unit;
            } else {
                base = reinterpret_cast<const float4*>(isq ? c.qt : c.kt) + ph * (16 * ROW);
                mv = a.heads * 16 * ROW;
                o = isq ? tok * ROW + unit : y;
            }
        } else if (DELTA && x0 >= oG) {
            base = reinterpret_cast<const float4*>(c.decay) + ph * ROW;
            mv = a.heads * ROW;
            o = min(x - oG, ROW - 1);
        } else if (DELTA && x0 >= oW) {
            const int y = x - oW, tok = y / ROW;
            base = reinterpret_cast<const float4*>(c.wt) + ph * (16 * ROW);
            mv = a.heads * 16 * ROW;
            o = tok * ROW + ((y % ROW) ^ token_slot(tok));
        }
        src[i] = base;
        move[i] = mv;
        off[i] = (uint32_t)o * 16u;
    }
    auto stage = [&](float4* b) {  // the next piece
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            __builtin_amdgcn_global_load_lds((gptr_t)(reinterpret_cast<const char*>(src[i]) + off[i]), (lptr_t)(b + (i * NW + wave) * 64), 16, 0, 0);
            src[i] += move[i];
        }
    };
    stage(buf[0]);
    f32x4 S[T];
    float* st = a.state + ((size_t)slot * a.heads + head) * DP * a.vdim_p;
    auto state_at = [&](int t) {  // channels 16 t + 4 grp .. + 3 of column col
        return reinterpret_cast<f32x4*>(st) + ((size_t)((col >> 3) * R4 + (t >> 2)) * 2 + (col & 1)) * 64 + ((col & 7) >> 1) * 16 + (t & 3) * 4 + grp;
    };
    const bool fresh = a.pos[first] == 0;
#pragma unroll
    for (int t = 0; t < T; ++t) S[t] = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : *state_at(t);
    const float decay = DELTA ? 1.f : a.decay[head];
    float pw_lo = 1.f, d4 = 1.f;  // decay^grp, decay^4
    if (!DELTA) {
        d4 = (decay * decay) * (decay * decay);
        for (int i = 0; i < grp; ++i) pw_lo *= decay;
    }
    const float rest16 = (d4 * d4) * (d4 * d4);
    float v[4];
    const int hv = a.heads * a.vdim_p;
    const float* vp = a.v + (size_t)(first + grp) * hv + (size_t)head * a.vdim_p + col;
    float* op = a.o + (size_t)(first + grp) * hv + (size_t)head * a.vdim_p + col;
    auto load_v = [&]() {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = vp[(size_t)(4 * r) * hv];
        vp += (size_t)16 * hv;
    };
    load_v();
    const int tok = token_slot(l15);  // token of this lane's operand rows
    uint32_t qa[T];  // LDS addresses in the first buffer
#pragma unroll
    for (int t = 0; t < T; ++t) qa[t] = lds_address(buf[0]) + (uint32_t)(tok * ROW + ((4 * t + grp) ^ l15)) * 16u;  // token_slot(tok) == l15
    const uint32_t ka = lds_address(buf[0]) + (uint32_t)(l15 * 4 + grp) * 16u, ga = lds_address(buf[0]) + (uint32_t)grp * 16u;
    const uint32_t pa = lds_address(buf[0]) + (uint32_t)(tok * 4 + grp) * 16u;
    dma_publish_barrier();
    for (int row = 0, cur = 0; row < rows; row += 16, cur ^= 1) {
        const uint32_t b = (uint32_t)cur * (SLOTS * 16u);
        const int n = min(16, rows - row);
        const bool more = row + 16 < rows;
        f32x4 u;
#pragma unroll
        for (int r = 0; r < 4; ++r) u[r] = 4 * r + grp < n ? v[r] : 0.f;
        if (more) {
            stage(buf[cur ^ 1]);
            load_v();
        }
        // W S and Q S: two state tiles' operands in flight ahead of the ones in use
        f32x4 qs[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}}, ws[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
        f32x4 xq[4], xw[4], xk[4], xg[4], pr;
        auto read_qw = [&](int t) {
            NVLLM_LDS_READ128(xq[t & 3], qa[t] + b, oQ * 16);
            if constexpr (DELTA) NVLLM_LDS_READ128(xw[t & 3], qa[t] + b, oW * 16);
        };
        auto read_kg = [&](int t) {
            NVLLM_LDS_READ128(xk[t & 3], ka + b + t * 1024, oK * 16);
            if constexpr (DELTA) NVLLM_LDS_READ128(xg[t & 3], ga + b + t * 64, oG * 16);
        };
        constexpr int PER = DELTA ? 2 : 1;  // reads per tile
        read_qw(0); read_qw(1);
#pragma unroll
        for (int t = 0; t < T; t += 2) {
            if (t + 2 < T) { read_qw(t + 2); read_qw(t + 3); }
            else { NVLLM_LDS_READ128(pr, pa + b, oP * 16); read_kg(0); read_kg(1); }
            if (t + 2 < T) NVLLM_LDS_WAIT(2 * PER);
            else NVLLM_LDS_WAIT(2 * PER + 1);
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int x = 0; x < 2; ++x) {
                    if constexpr (DELTA) ws[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(xw[(t + x) & 3][i], S[t + x][i], ws[x], 0, 0, 0);
                    qs[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(xq[(t + x) & 3][i], S[t + x][i], qs[x], 0, 0, 0);
                }
            __builtin_amdgcn_sched_barrier(0);
        }
        f32x4 o;
        float rest = rest16;
        if constexpr (DELTA) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                u[r] -= ws[0][r] + ws[1][r];
                o[r] = qs[0][r] + qs[1][r];
            }
        } else {
            float pw = pw_lo * decay;  // decay^(i + 1) of token i = grp
#pragma unroll
            for (int r = 0; r < 4; ++r, pw *= d4) o[r] = (qs[0][r] + qs[1][r]) * pw;
            if (n < 16) {
                rest = 1.f;
                for (int i = 0; i < n; ++i) rest *= decay;
            }
        }
#pragma unroll
        for (int t = 0; t < T; t += 2) {
            if (t + 2 < T) { read_kg(t + 2); read_kg(t + 3); NVLLM_LDS_WAIT(2 * PER); }
            else NVLLM_LDS_WAIT(0);
#pragma unroll
            for (int x = 0; x < 2; ++x)
#pragma unroll
                for (int r = 0; r < 4; ++r) S[t + x][r] *= DELTA ? xg[(t + x) & 3][r] : rest;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                if (t == 0) o = __builtin_amdgcn_mfma_f32_16x16x4f32(pr[r], u[r], o, 0, 0, 0);
#pragma unroll
                for (int x = 0; x < 2; ++x) S[t + x] = __builtin_amdgcn_mfma_f32_16x16x4f32(xk[(t + x) & 3][r], u[r], S[t + x], 0, 0, 0);
            }
            __builtin_amdgcn_sched_barrier(0);
        }
        if (more && live) {
#pragma unroll
            for (int r = 0; r < 4; ++r) op[(size_t)(4 * r) * hv] = o[r];
            op += (size_t)16 * hv;
            // the next piece has landed everywhere; the four stores may still be on their way
            asm volatile("s_waitcnt vmcnt(4)\n\ts_barrier" ::: "memory");
        } else {
            if (live) {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (4 * r + grp < n) op[(size_t)(4 * r) * hv] = o[r];
            }
            asm volatile("s_waitcnt vmcnt(0)\n\ts_barrier" ::: "memory");
        }
    }
    if (live) {
#pragma unroll
        for (int t = 0; t < T; ++t) *state_at(t) = S[t];
    }
}

bool piece_scan_ok(int dim_p) { return dim_p % 64 == 0 && dim_p <= 256; }

template <int R4, bool DELTA>
static void piece_scan_t(const RecurArgs& a, const PieceArgs& c, hipStream_t s) {
    if (DELTA && a.gh) delta_pieces_kernel<R4, true><<<dim3(a.heads, c.count), 64, 0, s>>>(a, c);
    else if (DELTA) delta_pieces_kernel<R4, false><<<dim3(a.heads, c.count), 64, 0, s>>>(a, c);
    else linear_pieces_kernel<R4><<<dim3(a.heads, c.count), 64, 0, s>>>(a, c);
    // four waves share a stage when that still fills the chip
    const int tiles = a.vdim_p / 16, base = a.heads * a.seg.count;
    const int nw = base * ((tiles + 3) / 4) >= 256 ? 4 : base * ((tiles + 1) / 2) >= 256 ? 2 : 1;
    const dim3 grid(a.heads * ((tiles + nw - 1) / nw), a.seg.count);
    if (nw == 4) piece_scan_kernel<R4, DELTA, 4><<<grid, 256, 0, s>>>(a, c);
    else if (nw == 2) piece_scan_kernel<R4, DELTA, 2><<<grid, 128, 0, s>>>(a, c);
    else piece_scan_kernel<R4, DELTA, 1><<<grid, 64, 0, s>>>(a, c);
}
hipError_t launch_piece_scan(const RecurArgs& a, const PieceArgs& c, hipStream_t s) {
    if (!piece_scan_ok(a.dim_p) || a.vdim_p % 16 || a.seg.single || !c.pair || !c.kt || ((a.g || a.gh) && (!c.qt || !c.wt || !c.decay || !a.beta)) || (a.g && a.gh) || (!a.g && !a.gh && !a.decay)) return hipErrorInvalidValue;
    if (c.count > 65535) return hipErrorNotSupported;
    if (a.seg.count <= 0 || c.count <= 0) return hipSuccess;
    switch (a.dim_p / 64) {
#define NVLLM_PS(R_) case R_: if (a.g || a.gh) piece_scan_t<R_, true>(a, c, s); else piece_scan_t<R_, false>(a, c, s); break;
        NVLLM_PS(1) NVLLM_PS(2) NVLLM_PS(3) NVLLM_PS(4)
#undef NVLLM_PS
    }
    return hipGetLastError();
}

}  // namespace nvllm
