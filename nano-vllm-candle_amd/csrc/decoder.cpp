// Shared host half of the decoders built from layer descriptions: see decoder.h.
#include "decoder.h"
#include "hybrid.h"

#include <algorithm>

// y = x.W^T left as f32 slabs
ProductPlan plan_product(const nvllm_model* m, int R, const PackedW& w) {
    ProductPlan p;
    const size_t one = (size_t)R * w.N;
    p.max_split = (int)std::max<size_t>(1, std::min<size_t>(8, m->slab_floats / one));
    const int tmin = m->opt_tile_min_wgs;
    if (tmin > 0 && R > kFusedMaxRows) {
        const int ks = gemm_tile_splits(R, w.N, w.K, tmin, std::min(p.max_split, R <= 512 ? 8 : 4));
        if (ks > 0) { p.kind = P_TILE; p.packed = 1; p.max_split = std::min(p.max_split, R <= 512 ? 8 : 4); return p; }
    }
    const int ss = gemm_stream_splits(R, w.N, w.K);
    if (ss > 0 && (size_t)ss * one <= m->slab_floats) { p.kind = P_STREAM; p.packed = 1; return p; }
    if (R <= kFusedMaxRows && gemm_rowpar_ok(w.N, w.K, 2, R) && (size_t)gemm_rowpar_splits(w.N, w.K, 2, R) * one <= m->slab_floats) {
        p.kind = P_ROW;
        p.packed = R >= 16 && gemm_rowdir_ok(w.N, w.K, 2, R);
    }
    return p;
}
int run_product(nvllm_model* m, const ProductPlan& p, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, float* out, int R, int* n_slabs) {
    hipStream_t s = m->ctx->stream;
    if (p.kind == P_TILE) {
        PROF(m, PROF_GEMM, launch_gemm_tile(xh, xl, w, R, 0, out, nullptr, nullptr, 0, m->opt_tile_min_wgs, p.max_split, n_slabs, s));
        ++m->tile_launches;
    } else if (p.kind == P_STREAM) {
        PROF(m, PROF_GEMM, launch_gemm_stream(xh, xl, w.K, w, out, R, p.packed, s));
        *n_slabs = gemm_stream_splits(R, w.N, w.K);
    } else if (p.kind == P_ROW) {
        RowParArgs a;
        a.xh = xh; a.xl = xl; a.ldx = w.K; a.out = out; a.M = R; a.x_packed = p.packed;
        PROF(m, PROF_GEMM, launch_gemm_rowpar(a, w, 2, s));
        *n_slabs = gemm_rowpar_splits(w.N, w.K, 2, R);
    } else {
        GemmPlan g = plan_gemm(R, w.N, w.K, p.max_split);
        PROF(m, PROF_GEMM, launch_gemm(g, xh, xl, w.K, w, out, R, s));
        *n_slabs = g.n_split;
    }
    return NVLLM_OK;
}

GluPlan plan_glu(const nvllm_model* m, int R, const PackedW& w, bool want_packed_out) {
    GluPlan g;
    const int tmin = m->opt_tile_min_wgs;
    if (tmin > 0 && R > kFusedMaxRows && gemm_tile_ok(R, w.N, w.K, 2, tmin)) { g.kind = P_TILE; g.packed = 1; g.out_packed_ok = 1; return g; }
    if (R <= kFusedMaxRows && gemm_rowpar_ok(w.N, w.K, 1, R)) {
        g.kind = P_ROW;
        const bool dir = gemm_rowdir_ok(w.N, w.K, 1, R);
        g.packed = R >= 16 && dir;
        g.out_packed_ok = dir;
        return g;
    }
    if (gemm_stream_splits(R, w.N, w.K) > 0 || want_packed_out) {
        g.kind = P_STREAM;
        g.slabs = plan_product(m, R, w);
        g.packed = g.slabs.packed;
        g.out_packed_ok = 1;
    }
    return g;
}
int run_glu(nvllm_model* m, const GluPlan& g, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, int R, const GluSpec& spec,
                   bf16_bits* oh, bf16_bits* ol, int out_packed) {
    hipStream_t s = m->ctx->stream;
    if (g.kind == P_TILE) {
        PROF(m, PROF_GEMM, launch_gemm_tile(xh, xl, w, R, 2, nullptr, oh, ol, out_packed, m->opt_tile_min_wgs, 1, nullptr, s, spec));
        ++m->tile_launches;
    } else if (g.kind == P_ROW) {
        RowParArgs a;
        a.xh = xh; a.xl = xl; a.ldx = w.K; a.oh = oh; a.ol = ol; a.M = R; a.x_packed = g.packed; a.o_packed = out_packed; a.glu = spec;
        PROF(m, PROF_GEMM, launch_gemm_rowpar(a, w, 1, s));
    } else if (g.kind == P_STREAM) {
        int ns = 1;
        int rc = run_product(m, g.slabs, xh, xl, w, m->slabs, R, &ns);
        if (rc) return rc;
        PROF(m, PROF_SILU, launch_silu_mul_interleaved(m->slabs, ns, (int64_t)R * w.N, R, w.N / 2, oh, ol, out_packed, s, spec));
    } else {
        GemmPlan p = plan_gemm_swiglu(R, w.N, w.K);
        PROF(m, PROF_GEMM, launch_gemm_swiglu(p, xh, xl, w.K, w, R, oh, ol, nullptr, s, spec));
    }
    return NVLLM_OK;
}

int run_act(nvllm_model* m, const ProductPlan& p, nvllm::Act act, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, int R, bf16_bits* oh, bf16_bits* ol, int out_packed) {
    hipStream_t s = m->ctx->stream;
    if (p.kind == P_TILE && gemm_tile_ok(R, w.N, w.K, 4 + act, m->opt_tile_min_wgs)) {
        PROF(m, PROF_GEMM, launch_gemm_tile(xh, xl, w, R, 4 + act, nullptr, oh, ol, out_packed, m->opt_tile_min_wgs, 1, nullptr, s));
        ++m->tile_launches;
    } else if (p.kind == P_ROW && gemm_rowdir_ok(w.N, w.K, 3 + act, R)) {
        RowParArgs a;
        a.xh = xh; a.xl = xl; a.ldx = w.K; a.oh = oh; a.ol = ol; a.M = R; a.x_packed = p.packed; a.o_packed = out_packed;
        PROF(m, PROF_GEMM, launch_gemm_rowpar(a, w, 3 + act, s));
    } else {
        int ns = 1, rc = run_product(m, p, xh, xl, w, m->slabs, R, &ns);
        if (rc) return rc;
        PROF(m, PROF_SILU, launch_act(act, m->slabs, ns, (int64_t)R * w.N, R, w.N, oh, ol, out_packed, nullptr, s));
    }
    return NVLLM_OK;
}

// 32-bit product of row-major f32 rows
int exact_product(nvllm_model* m, const float* x, const PackedW& w, float* out, int R) {
    HeadGemmArgs a;
    a.x = x; a.x_row = w.K; a.w = w.data; a.N = a.n_valid = w.N; a.K = w.K; a.M = R; a.exact = 1; a.y = out; a.y_row = w.N;
    PROF(m, PROF_GEMM, launch_head_gemm(a, m->ctx->stream));
    return NVLLM_OK;
}

int output_head(nvllm_model* m, const PackedW& head, int Kw, int Vp, const float* y, float cap, int n_last, int logits_row0) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    const int tps = ctx->tp_size;
    uint32_t* ids_dst = tps == 1 ? m->d_next + logits_row0 : m->d_next + m->cur_n + (size_t)ctx->tp_rank * m->cur_n + logits_row0;
    float* val_dst = tps == 1 ? nullptr : m->d_maxval + (size_t)ctx->tp_rank * m->cur_n + logits_row0;
    float* lg = m->logits + (size_t)logits_row0 * m->V_l;
    if (!y && m->V_l % 16 == 0) {
        RowNorm rn;
        rn.softcap = cap;
        GemmPlan pl = plan_lmhead(n_last, m->V_l, Kw);
        PROF(m, PROF_LMHEAD, launch_gemm_argmax(pl, m->xh, m->xl, Kw, head, m->want_logits ? lg : nullptr, n_last, m->part_val, m->part_idx, &rn, s));
        const int parts = gemm_argmax_parts(pl, m->V_l);
        if (pl.lm_nt > 0) HIPCHK(ctx, launch_argmax_rows(m->part_val, m->part_idx, parts, n_last, ids_dst, val_dst, s));
        else HIPCHK(ctx, launch_argmax_parts(m->part_val, m->part_idx, parts, n_last, m->argmax_scratch, ids_dst, val_dst, s));
        return NVLLM_OK;
    }
    int ns = 1, rc = NVLLM_OK;
    if (y) rc = exact_product(m, y, head, m->slabs, n_last);
    else {
        ProductPlan ph;  // row-major planes, one slab
        rc = run_product(m, ph, m->xh, m->xl, head, m->slabs, n_last, &ns);
    }
    if (rc) return rc;
    HIPCHK(ctx, launch_logits_finish(m->slabs, ns, (int64_t)n_last * Vp, Vp, n_last, m->V_l, cap, lg, m->V_l, s));
    HIPCHK(ctx, launch_argmax(lg, n_last, m->V_l, m->V_l, ids_dst, val_dst, s));
    return NVLLM_OK;
}
