// Host half of the selective-scan mixer: see scan_mixer.h.
#include "scan_mixer.h"

#include <algorithm>
#include <cmath>

int ScanMixer::create(nvllm_ctx* ctx, int inner_, int state_, int taps_, int rank_, int Kw, bool f32) {
    inner = inner_; state = state_; taps = taps_; rank = rank_;
    n = inner / ctx->tp_size; S = scan_states(state); n_p = up(n, scan_channels(S)); rank_p = up(rank, 32); Kc = up(n, 128);
    // wide projections: a whole number of the prompt product's 192- or 256-feature tiles
    Nin = 2 * n >= 1536 && !f32 ? up_tile(2 * n) : up(2 * n, 16);
    Nx = n >= 1536 && !f32 ? up_tile(rank_p + 2 * S) : up(rank_p + 2 * S, 16);
    int rc = alloc_packed(ctx, in, Nin, Kw);
    if (!rc) rc = alloc_packed(ctx, x, Nx, Kc);
    if (!rc) rc = alloc_packed(ctx, dt, n_p, rank_p);
    if (!rc) rc = alloc_vec(ctx, &conv, (size_t)taps * n);
    if (!rc) rc = alloc_vec(ctx, &conv_b, n);
    if (!rc) rc = alloc_vec(ctx, &dt_b, n_p);
    if (!rc) rc = alloc_vec(ctx, &A, (size_t)n_p * S);
    if (!rc) rc = alloc_vec(ctx, &D, n_p);
    return rc;
}
void ScanMixer::destroy() {
    for (PackedW* p : {&in, &x, &dt}) (void)hipFree(p->data);
    for (float* p : {conv, conv_b, dt_b, A, D}) (void)hipFree(p);
}

int ScanMixer::load(nvllm_model* m, const char* name, const char* s, const HostMat& h, int64_t rows, int64_t cols, int W) {
    nvllm_ctx* ctx = m->ctx;
    const int64_t c0 = (int64_t)ctx->tp_rank * n;
    auto want = [&](int64_t r, int64_t c) -> int {
        if (rows == r && cols == c) return NVLLM_OK;
        return fail(ctx, NVLLM_EINVAL, "tensor '%s': shape mismatch (got %lld x %lld, want %lld x %lld)", name, (long long)rows, (long long)cols, (long long)r, (long long)c);
    };
    auto put = [&](float* dst, const std::vector<float>& t) -> int {
        HIPCHK(ctx, hipMemcpy(dst, t.data(), t.size() * 4, hipMemcpyHostToDevice));
        return NVLLM_OK;
    };
    auto vec = [&](float* dst) -> int {
        int rc = want(1, inner);
        if (rc) return rc;
        std::vector<float> t(n);
        for (int i = 0; i < n; ++i) t[i] = h.f32(c0 + i);
        return put(dst, t);
    };
    int rc = NVLLM_OK;
    if (!strcmp(s, "in")) {
        if ((rc = want(2 * (int64_t)inner, W))) return rc;
        return put_rows(ctx, in, 0, 2 * n, W, -1, [&](int r, int c) { return h.at(r < n ? c0 + r : inner + c0 + r - n, c); });
    }
    if (!strcmp(s, "conv")) {  // [channels, taps] -> [taps][channels]
        if ((rc = want(inner, taps))) return rc;
        std::vector<float> t((size_t)taps * n);
        for (int i = 0; i < taps; ++i)
            for (int c = 0; c < n; ++c) t[(size_t)i * n + c] = h.f32((c0 + c) * taps + i);
        return put(conv, t);
    }
    if (!strcmp(s, "conv.b")) return vec(conv_b);
    if (!strcmp(s, "D")) return vec(D);
    if (!strcmp(s, "dt.b")) return vec(dt_b);
    if (!strcmp(s, "x")) {
        if ((rc = want(rank + 2 * (int64_t)state, inner))) return rc;
        const int src0[3] = {0, rank, rank + state}, dst0[3] = {0, rank_p, rank_p + S}, cnt[3] = {rank, state, state};
        for (int k = 0; k < 3 && !rc; ++k) rc = put_rows(ctx, x, dst0[k], cnt[k], n, -1, [&](int r, int c) { return h.at(src0[k] + r, c0 + c); });
        return rc;
    }
    if (!strcmp(s, "dt")) {
        if ((rc = want(inner, rank))) return rc;
        return put_rows(ctx, dt, 0, n, rank, -1, [&](int r, int c) { return h.at(c0 + r, c); });
    }
    if (!strcmp(s, "A_log")) {
        if ((rc = want(inner, state))) return rc;
        std::vector<float> t((size_t)n_p * S, 0.f);
        for (int c = 0; c < n; ++c)
            for (int k = 0; k < state; ++k) t[(size_t)c * S + k] = (float)(-std::exp((double)h.f32((c0 + c) * state + k)) * 1.4426950408889634);
        return put(A, t);
    }
    return 1;
}

int ScanMixer::kv_alloc(nvllm_model* m) {
    nvllm_ctx* ctx = m->ctx;
    int rc = alloc_vec(ctx, &st, (size_t)m->max_seqs * n_p * S);
    if (!rc && taps > 1) rc = alloc_vec(ctx, &history, (size_t)2 * m->max_seqs * (taps - 1) * n);
    return rc;
}
void ScanMixer::free_kv() {
    for (float** p : {&st, &history}) {
        if (*p) (void)hipFree(*p);
        *p = nullptr;
    }
}

constexpr int kShortestPiece = 64, kScanWaves = 1024;  // rows of a piece at least; waves the pieces of a chunk aim at

void ScanScratch::reserve(const ScanMixer& w, size_t R) {
    n_x = std::max(n_x, R * w.Kc);
    n_dt = std::max(n_dt, R * w.n_p);
    n_dbc = std::max(n_dbc, R * w.Nx);
    n_carry = std::max<size_t>(n_carry, (size_t)w.n_p * w.S);
    n_carry_dt = std::max<size_t>(n_carry_dt, w.n_p);
    const int v = std::max(1, w.n_p * std::min(w.S / 4, 64) / 64);
    waves = waves ? std::min(waves, v) : v;
}
int ScanScratch::alloc(nvllm_model* m, bool f32) {
    if (!n_x) return NVLLM_OK;
    nvllm_ctx* ctx = m->ctx;
    seg_cap = m->max_seqs;
    piece_cap = m->max_rows / kShortestPiece + seg_cap;
    int rc = alloc_vec(ctx, &x, n_x);  // padding columns stay zero
    if (!rc) rc = dmalloc(ctx, &dt, n_dt);
    if (!rc) rc = dmalloc(ctx, &dbc, n_dbc);
    if (!rc) rc = dmalloc(ctx, &carry, n_carry * piece_cap);
    if (!rc) rc = dmalloc(ctx, &carry_dt, n_carry_dt * piece_cap);
    if (!f32)
        for (bf16_bits** p : {&xh, &xl})
            if (!rc) rc = alloc_vec(ctx, reinterpret_cast<float**>(p), n_x / 2 + 16 * (n_x / std::max(1, m->max_rows)) / 2);  // read in whole 16-row blocks
    const size_t ints = (size_t)3 * seg_cap + 5 * piece_cap;
    if (!rc) rc = dmalloc(ctx, &d_plan, ints);
    if (!rc) HIPCHK(ctx, hipHostMalloc((void**)&h_plan, ints * sizeof(int), hipHostMallocDefault));
    return rc;
}
void ScanScratch::release() {
    for (void* p : {(void*)x, (void*)dt, (void*)dbc, (void*)carry, (void*)carry_dt, (void*)xh, (void*)xl, (void*)d_plan})
        if (p) (void)hipFree(p);
    if (h_plan) (void)hipHostFree(h_plan);
    *this = ScanScratch();
}

int ScanScratch::plan(nvllm_model* m, const int* slot, const int* seq, int R) {
    nvllm_ctx* ctx = m->ctx;
    n_seg = n_piece = several = 0;
    if (!d_plan) return NVLLM_OK;
    // as many pieces as fill the chip beside the channels, of equal length
    const int want = std::max(1, kScanWaves / waves), longest = std::max(kShortestPiece, up((R + want - 1) / want, 16));
    int *row0 = h_plan, *cnt = row0 + seg_cap, *sl = cnt + seg_cap;
    int *p_row0 = sl + seg_cap, *p_n = p_row0 + piece_cap, *p_slot = p_n + piece_cap, *p_at = p_slot + piece_cap, *p_of = p_at + piece_cap;
    for (int r = 0; r < R; ++n_seg) {
        int e = r;
        while (e < R && seq[e] == seq[r]) ++e;
        row0[n_seg] = r; cnt[n_seg] = e - r; sl[n_seg] = slot[r];
        const int of = (e - r + longest - 1) / longest;
        several |= of > 1;
        for (int k = 0; k < of; ++k, ++n_piece) {
            p_row0[n_piece] = r + k * longest; p_n[n_piece] = std::min(longest, e - r - k * longest);
            p_slot[n_piece] = slot[r]; p_at[n_piece] = k; p_of[n_piece] = of;
        }
        r = e;
    }
    // the staging buffer is free: the tile upload before this call waited for the stream
    HIPCHK(ctx, hipMemcpyAsync(d_plan, h_plan, ((size_t)3 * seg_cap + 5 * piece_cap) * sizeof(int), hipMemcpyHostToDevice, ctx->stream));
    return NVLLM_OK;
}

int run_scan(nvllm_model* m, ScanMixer& w, ScanScratch& x, const float* in, int n_slabs, float* other_slabs, int R, int qt, float* ctx_f, int ctx_packed) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    const bool f32 = ctx_f != nullptr;
    ProductPlan px;
    if (!f32) px = plan_product(m, R, w.x);
    ConvRowsArgs ca;
    ca.in = in; ca.n_slabs = n_slabs; ca.ld = w.Nin; ca.slab_stride = (int64_t)R * w.Nin;
    ca.channels = w.n; ca.taps = w.taps; ca.conv = w.conv; ca.bias = w.conv_b; ca.history = w.history; ca.slots = m->max_seqs;
    ca.seg.single = qt == 1;
    ca.seg.count = ca.seg.single ? R : x.n_seg;
    ca.seg.row0 = x.d_plan; ca.seg.n = x.d_plan + x.seg_cap; ca.seg.slot = ca.seg.single ? m->d_slot : x.d_plan + 2 * x.seg_cap;
    ca.pos = m->d_pos; ca.slot = m->d_slot;
    ca.x = x.x; ca.ldx = w.Kc; ca.packed = px.packed;
    if (!f32) { ca.xh = x.xh; ca.xl = x.xl; }
    PROF(m, PROF_QK, launch_conv_rows(ca, R, s));
    if (!ca.seg.single) PROF(m, PROF_QK, launch_conv_history(ca, s));
    int nx = 1, rc = f32 ? exact_product(m, x.x, w.x, other_slabs, R) : run_product(m, px, x.xh, x.xl, w.x, other_slabs, R, &nx);
    if (rc) return rc;
    const float* dbc = other_slabs;
    if (nx > 1 || ctx->tp_size > 1) {
        HIPCHK(ctx, launch_slab_sum(other_slabs, nx, (int64_t)R * w.Nx, nullptr, R, w.Nx, x.dbc, s));
        dbc = x.dbc;
        rc = comm_allreduce_sum(ctx, x.dbc, (size_t)R * w.Nx);
        if (rc) return rc;
    }
    HeadGemmArgs ga;
    ga.x = dbc; ga.x_row = w.Nx; ga.w = w.dt.data; ga.N = ga.n_valid = w.n_p; ga.K = w.rank_p; ga.M = R; ga.exact = f32;
    ga.y = x.dt; ga.y_row = w.n_p; ga.decay_bias = w.dt_b;
    PROF(m, PROF_GEMM, launch_delta_gates(ga, s));
    ScanArgs sa;
    sa.x = x.x; sa.ldx = w.Kc; sa.dt = x.dt; sa.bc = dbc; sa.ldbc = w.Nx; sa.b0 = w.rank_p; sa.c0 = w.rank_p + w.S;
    sa.z = in + w.n; sa.z_slabs = n_slabs; sa.ldz = w.Nin; sa.z_stride = ca.slab_stride;
    sa.A = w.A; sa.D = w.D; sa.channels = w.n; sa.channels_p = w.n_p; sa.states = w.S; sa.state = w.st; sa.pos = m->d_pos; sa.slot = m->d_slot;
    const int* p = x.d_plan + 3 * x.seg_cap;
    sa.piece_row0 = p; sa.piece_n = p + x.piece_cap; sa.piece_slot = p + 2 * x.piece_cap; sa.piece_at = p + 3 * x.piece_cap; sa.piece_of = p + 4 * x.piece_cap;
    sa.pieces = x.n_piece; sa.several = x.several; sa.carry = x.carry; sa.carry_dt = x.carry_dt;
    sa.ld = w.Kc; sa.packed = ctx_packed;
    if (f32) sa.of = ctx_f;
    else { sa.oh = m->ctxh; sa.ol = m->ctxl; }
    if (qt == 1) PROF(m, PROF_RECUR, launch_scan_decode(sa, R, s));
    else PROF(m, PROF_RECUR, launch_scan_prompt(sa, s));
    return NVLLM_OK;
}
