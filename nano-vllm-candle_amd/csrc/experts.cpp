// Host half of routed feed-forwards: see experts.h.
#include "experts.h"

#include <algorithm>

int ExpertsBlock::create(nvllm_ctx* ctx, int experts_, int top_, int ff_, int shared_, int W_, int Kw_, int ldr_, bool f32) {
    const int tp = ctx->tp_size;
    experts = experts_; top = top_; ff_all = ff_; shared_all = shared_; W = W_; Kw = Kw_; ldr = ldr_;
    ff = ff_all / tp; sh = shared_all / tp; ff_p = ff >= 512 && !f32 ? up_tile(ff) : up(ff, 128); sh_p = !sh ? 0 : sh >= 512 && !f32 ? up_tile(sh) : up(sh, 128);
    Nr = up(experts + (sh ? 1 : 0), 16);
    int rc = alloc_packed(ctx, router, Nr, Kw);
    if (!rc) rc = alloc_packed(ctx, wup, experts * up_rows(), Kw);
    if (!rc) rc = alloc_packed(ctx, down, experts * ldr, ff_p);
    if (!rc && sh) rc = alloc_packed(ctx, sup, sh_p, Kw);
    if (!rc && sh) rc = alloc_packed(ctx, sdown, ldr, sh_p);
    return rc;
}
void ExpertsBlock::destroy() {
    for (PackedW* p : {&router, &wup, &down, &sup, &sdown}) (void)hipFree(p->data);
}

int ExpertsBlock::load(nvllm_model* m, const char* name, const char* s, const HostMat& h, int64_t rows, int64_t cols) {
    nvllm_ctx* ctx = m->ctx;
    const int64_t f0 = (int64_t)ctx->tp_rank * ff, s0 = (int64_t)ctx->tp_rank * sh;
    auto want = [&](int64_t r, int64_t c) -> int {
        if (rows == r && cols == c) return NVLLM_OK;
        return fail(ctx, NVLLM_EINVAL, "tensor '%s': shape mismatch (got %lld x %lld, want %lld x %lld)", name, (long long)rows, (long long)cols, (long long)r, (long long)c);
    };
    auto put_up = [&](const PackedW& w, int row0, int64_t all, int n, int64_t r0, int ileave = -1) -> int {
        int rc = want(all, W);
        return rc ? rc : put_rows(ctx, w, row0, n, W, ileave, [&](int r, int c) { return h.at(r0 + r, c); });
    };
    auto put_down = [&](const PackedW& w, int row0, int64_t all, int n, int64_t c0) -> int {
        int rc = want(W, all);
        return rc ? rc : put_rows(ctx, w, row0, W, n, -1, [&](int r, int c) { return h.at(r, c0 + c); });
    };
    if (!strcmp(s, "router")) return put_up(router, 0, experts, experts, 0);
    if (sh && !strcmp(s, "shared.sg")) return put_up(router, experts, 1, 1, 0);
    if (sh && !strcmp(s, "shared.up")) return put_up(sup, 0, shared_all, sh, s0);
    if (sh && !strcmp(s, "shared.down")) return put_down(sdown, 0, shared_all, sh, s0);
    int e = -1, off = 0;
    if (sscanf(s, "e%d.%n", &e, &off) == 1 && off && e >= 0 && e < experts) {
        if (gated && !strcmp(s + off, "gate")) return put_up(wup, e * up_rows(), ff_all, ff, f0, 0);
        if (!strcmp(s + off, "up")) return put_up(wup, e * up_rows(), ff_all, ff, f0, gated ? 1 : -1);
        if (!strcmp(s + off, "down")) return put_down(down, e * ldr, ff_all, ff, f0);
    }
    return 1;
}
std::vector<std::string> ExpertsBlock::tensors() const {
    std::vector<std::string> t = {"router"};
    for (int e = 0; e < experts; ++e)
        for (const char* s : {".gate", ".up", ".down"})
            if (gated || s[1] != 'g') t.push_back("e" + std::to_string(e) + s);
    if (sh) for (const char* s : {"shared.up", "shared.down", "shared.sg"}) t.push_back(s);
    return t;
}
size_t ExpertsBlock::step_bytes() const { return router.bytes() + (wup.bytes() + down.bytes()) / std::max(1, experts) * top + sup.bytes() + sdown.bytes(); }

constexpr int kTileAlign = 256;  // rows of the widest tile a group starts at

void ExpertsScratch::reserve(const ExpertsBlock& e, size_t R) {
    const size_t per = e.top + 1;
    cap = (int)std::max<size_t>(cap, (R * per + (size_t)(e.experts + 1) * kTileAlign + kTileAlign - 1) / kTileAlign * kTileAlign);
    lda = std::max({lda, e.ff_p, e.sh_p});
    n_rows = R;
    n_z = std::max(n_z, R * e.Nr);
    n_top = std::max(n_top, R * e.top);
    n_place = std::max(n_place, R * per);
    n_out = std::max<size_t>(n_out, e.ldr);
    n_sh = std::max<size_t>(n_sh, (R + 15) / 16 * 16 * e.sh_p);
}
int ExpertsScratch::alloc(nvllm_ctx* ctx, bool f32) {
    if (!cap) return NVLLM_OK;
    int rc = dmalloc(ctx, &z, n_z);
    if (!rc) rc = dmalloc(ctx, &score, n_top);
    if (!rc) rc = dmalloc(ctx, &chosen, n_top);
    if (!rc) rc = dmalloc(ctx, &gate, n_rows);
    if (!rc) rc = dmalloc(ctx, &place, n_place);
    for (float** p : {&pre, &post}) if (!rc) rc = dmalloc(ctx, p, cap);
    if (!rc) rc = dmalloc(ctx, &src, cap);
    if (!rc) rc = dmalloc(ctx, &cursor, kMaxExperts + 1);
    if (!rc) rc = dmalloc(ctx, &tile_group, cap / 16);
    if (!rc) rc = dmalloc(ctx, &out, (size_t)cap * n_out);
    if (f32) {
        if (!rc) rc = dmalloc(ctx, &act_f, (size_t)cap * lda);
    } else {
        for (bf16_bits** p : {&ah, &al}) if (!rc) rc = dmalloc(ctx, p, (size_t)cap * lda);
        if (n_sh) for (bf16_bits** p : {&sh, &sl}) if (!rc) rc = dmalloc(ctx, p, n_sh);
    }
    return rc;
}
void ExpertsScratch::release() {
    for (void* p : {(void*)z, (void*)score, (void*)gate, (void*)pre, (void*)post, (void*)out, (void*)act_f, (void*)chosen, (void*)place, (void*)src, (void*)tile_group, (void*)cursor, (void*)ah,
                    (void*)al, (void*)sh, (void*)sl})
        if (p) (void)hipFree(p);
    *this = ExpertsScratch();
}

// prompt chunks with enough rows per expert: groups of whole blocks of the prompt product
static int tile_align(const nvllm_model* m, const ExpertsBlock& e, int R) {
    const int rows = R * e.top / e.experts;  // of an expert, on average
    if (m->opt_tile_min_wgs <= 0 || R <= kFusedMaxRows || rows < (m->opt_tile_min_wgs == 1 ? 1 : 48)) return 0;
    for (int align : {rows >= 320 ? 256 : 128, 256})
        if (gemm_tile_group_ok(e.up_rows(), e.Kw, align) && gemm_tile_group_ok(e.ldr, e.ff_p, align)) return align;
    return 0;
}
bool experts_gather(const nvllm_model* m, const ExpertsBlock& e, int R) { return tile_align(m, e, R) > 0; }

int run_experts(nvllm_model* m, ExpertsBlock& e, ExpertsScratch& x, const bf16_bits* xh, const bf16_bits* xl, int packed, const bf16_bits* rh, const bf16_bits* rl,
                const float* y, int R, float* slabs2, BranchSum* out) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    const bool f32 = y != nullptr;
    GroupGemmArgs in;  // of rows
    in.xh = xh; in.xl = xl; in.xf = y; in.ldx = e.Kw; in.x_packed = packed; in.x_rows = R;
    GroupGemmArgs rg = in;
    rg.w = e.router.data; rg.N = e.Nr; rg.K = e.Kw; rg.align = R > 64 && e.Nr > 128 ? 64 : 16; rg.out = x.z; rg.ldo = e.Nr;
    PROF(m, PROF_GEMM, launch_group_gemm(rg, s));
    RouteArgs ra;
    ra.z = x.z; ra.ld = e.Nr; ra.rows = R; ra.experts = e.experts; ra.top = e.top; ra.weight_in = e.weight_in;
    ra.softmax = e.softmax; ra.groups = e.groups; ra.keep = e.keep;
    ra.gate_col = e.sh ? e.experts : -1;
    const int tile = f32 ? 0 : tile_align(m, e, R);
    ra.shared_group = e.sh > 0 && !tile;
    ra.align = tile ? tile : R * e.top >= 32 * e.experts ? 64 : 16;
    ra.cap = x.cap;
    ra.chosen = x.chosen; ra.score = x.score; ra.gate = x.gate; ra.place = x.place; ra.src = x.src; ra.pre = x.pre; ra.post = x.post; ra.tile_group = x.tile_group; ra.cursor = x.cursor;
    PROF(m, PROF_QK, launch_route(ra, s));
    const int64_t longest = (int64_t)R * e.top + (int64_t)std::min(e.experts, R * e.top) * (ra.align - 1) + (ra.shared_group ? R + ra.align - 1 : 0);
    out->gather = x.out; out->gather_row = x.place; out->n_gather = e.top + ra.shared_group;
    if (tile) {
        const int n = (int)(longest / tile) * tile;
        TileGroups tg;
        tg.tile_group = x.tile_group; tg.align = tile; tg.w_group = (int64_t)e.up_rows() * e.Kw / 8; tg.src = x.src; tg.x_rows = R; tg.pre = x.pre; tg.post = x.post; tg.gated = e.gated;
        PackedW w = e.wup;
        w.N = e.up_rows();
        PROF(m, PROF_GEMM, launch_gemm_tile_group(rh, rl, w, n, tg, nullptr, x.ah, x.al, s));
        w = e.down;
        w.N = e.ldr;
        tg.w_group = (int64_t)e.ldr * e.ff_p / 8;
        PROF(m, PROF_GEMM, launch_gemm_tile_group(x.ah, x.al, w, n, tg, x.out, nullptr, nullptr, s));
        m->tile_launches += 2;
        if (e.sh) {
            ProductPlan pu = plan_product(m, R, e.sup), pd = plan_product(m, R, e.sdown);
            const bool ours = pu.packed == packed;  // else the row-major planes and a kernel that takes them
            if (!ours && pu.packed) pu = ProductPlan{P_GENERIC, 0, pu.max_split};
            int rc = run_act(m, pu, ACT_RELU2, ours ? xh : rh, ours ? xl : rl, e.sup, R, x.sh, x.sl, pd.packed);
            if (!rc) rc = run_product(m, pd, x.sh, x.sl, e.sdown, slabs2, R, &out->n_slabs);
            if (rc) return rc;
            out->in = slabs2; out->slab_stride = (int64_t)R * e.ldr; out->scale = x.gate;
        }
        return NVLLM_OK;
    }
    GroupGemmArgs ga = in;
    ga.src = x.src; ga.w = e.wup.data; ga.w_group = (int64_t)e.up_rows() * e.Kw / 8; ga.N = e.up_rows(); ga.K = e.Kw;
    if (ra.shared_group) { ga.ws = e.sup.data; ga.last = e.experts; ga.Ns = e.sh_p; ga.Ks = e.Kw; }
    ga.tile_group = x.tile_group; ga.align = ra.align; ga.tiles = (int)(longest / ra.align); ga.post = x.post;
    if (e.gated) ga.glu = 1;
    else { ga.pre = x.pre; ga.relu2 = 1; }
    ga.ldo = x.lda;
    if (f32) ga.out = x.act_f;
    else { ga.oh = x.ah; ga.ol = x.al; }
    PROF(m, PROF_GEMM, launch_group_gemm(ga, s));
    GroupGemmArgs gd;
    gd.xh = x.ah; gd.xl = x.al; gd.xf = f32 ? x.act_f : nullptr; gd.ldx = x.lda; gd.x_packed = 1; gd.x_rows = x.cap;
    gd.w = e.down.data; gd.w_group = (int64_t)e.ldr * e.ff_p / 8; gd.N = e.ldr; gd.K = e.ff_p;
    if (ra.shared_group) { gd.ws = e.sdown.data; gd.last = e.experts; gd.Ns = e.ldr; gd.Ks = e.sh_p; }
    gd.tile_group = x.tile_group; gd.align = ra.align; gd.tiles = ga.tiles; gd.out = x.out; gd.ldo = e.ldr;
    PROF(m, PROF_GEMM, launch_group_gemm(gd, s));
    return NVLLM_OK;
}
