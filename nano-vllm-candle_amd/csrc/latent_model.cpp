// Latent-attention decoders behind the C ABI: weights in MFMA tile layout, latent cache and step buffers, the forward of one
// chunk of rows.  Sequences, blocks, slots, scheduling of chunks, sampling and decode pipelining are the shared code of api.cpp.
//
// A layer adds two branches of the same x:  x <- x + W_o mixer(norm1 x) + ff(norm2 x), norm2 possibly being norm1.  The mixer is latent
// attention or a selective scan (scan_mixer.h), the feed-forward gated or routed to experts (experts.h).
// Mixed precision (the serving mode): products run on bf16 hi + lo planes (16 bits of the activation) with f32 accumulation,
// the cache is f16; residual, norms, rotation, scores and softmax are f32.  32-bit mode: every product and the cache in f32.
#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstring>
#include <map>

#include "decoder.h"
#include "experts.h"
#include "rope.h"
#include "scan_mixer.h"

struct LatentLayer {
    nvllm_latent_layer c{};
    int heads = 0, ff = 0;                       // this rank's share
    int dim_p = 0, rank_p = 0, rot_p = 0, vdim_p = 0, ff_p = 0;
    int Nq = 0, Kc = 0;                          // q (+ latent) projection rows (padded), context width (padded)
    int Nd = 0, Kq = 0;                          // query latents: rows of the first projection (padded), width of the second (padded)
    PackedW dq;                                  // query latents: the first projection, then the latent projection unless kv_from
    PackedW qkv, ukt, uv, o, gu, down;           // per head: ukt [rank_p x dim_p], uv [vdim_p x rank_p]
    bool expands = false;                        // prompt chunks may run the expanded form
    PackedW ukx, uvx;                            // its weights, f16 times 1 / scale: [dim_p x rank_p], [vdim_p x rank_p] per head
    float ukx_scale = 1.f, uvx_scale = 1.f;
    float *norm1 = nullptr, *norm2 = nullptr, *dkv_norm = nullptr, *dq_norm = nullptr;
    float* sink = nullptr;                       // times log2(e)
    ExpertsBlock experts;
    ScanMixer scan;
    bool own_kv() const { return c.kv_from < 0; }
    const PackedW& first() const { return scan.on() ? scan.in : c.q_rank ? dq : qkv; }  // the product the normed input meets
    int rope = 0;                                // index of the rotation table
    LatentCache cache_shape() const {
        LatentCache k;
        k.rank = c.kv_rank; k.rank_p = rank_p; k.rot = c.rot_dim; k.rot_p = rot_p;
        return k;
    }
};

struct LatentModel : DecoderImpl {
    nvllm_latent_config cfg{};
    std::vector<LatentLayer> layers;
    std::vector<int> order;            // layer of every run (a looped layer runs several times, each with its own cache)
    int ldr = 0, Kw = 0, Vp = 0;       // residual stride, width padded for the products, padded vocabulary rows of the head
    bf16_bits* embed = nullptr;        // [vocab][ldr]
    PackedW head;
    float* final_norm = nullptr;
    std::vector<RopeTable> ropes;
    // pool and step buffers
    std::vector<void*> cache;          // per run
    float *slabs2 = nullptr, *q = nullptr, *qlat = nullptr, *olat = nullptr, *part_o = nullptr, *part_ml = nullptr, *tap = nullptr;
    bf16_bits *x2h = nullptr, *x2l = nullptr;                                                 // second norm's planes
    // expanded prompt attention: scratch keys / values, the chunk's cache tiles (device) and segments
    f16_bits *kx = nullptr, *vx = nullptr;
    int exp_cap = 0, exp_n = 0;        // entries allocated; entries of this chunk (0: the absorbed form)
    int *d_exp = nullptr, *d_tile_exp = nullptr, *h_exp = nullptr;
    struct Segment { int pos0, n; };
    std::vector<Segment> segments;
    float *y1 = nullptr, *y2 = nullptr, *ctx_f = nullptr, *act_f = nullptr, *cq_f = nullptr;  // 32-bit mode
    bf16_bits *cqh = nullptr, *cql = nullptr;                                                 // normed query latents
    ExpertsScratch experts;
    ScanScratch scan;
    bool has_state = false;

    ~LatentModel() override;
    int load_tensor(nvllm_model* m, const char* name, const void* data, int dtype, const int64_t* shape, int ndim) override;
    int finalize(nvllm_model* m) override;
    int kv_alloc(nvllm_model* m) override;
    void free_kv() override;
    int64_t weight_bytes() const override;
    int64_t kv_bytes_per_token() const override;
    int64_t kv_read_bytes(int len) const override;
    int tile_rows(int qt) const override { return qt == 1 ? 1 : kLatentTileRows; }
    bool recurrent() const override { return has_state; }
    int plan_chunk(nvllm_model* m, const int* pos, const int* slot, const int* seq, int R, const int* tile_row0, int n_tiles, int qt) override;
    int forward_chunk(nvllm_model* m, int R, int n_tiles, int qt, int n_last, int logits_row0) override;
};
static LatentModel& latent(const nvllm_model* m) { return *static_cast<LatentModel*>(m->dec.get()); }

extern "C" int nvllm_model_create_latent(nvllm_ctx* ctx, const nvllm_latent_config* cfg, const nvllm_latent_layer* layers, nvllm_model** out) {
    if (!ctx || !cfg || !layers || !out) return fail(ctx, NVLLM_EINVAL, "NULL argument");
    const nvllm_latent_config& c = *cfg;
    const int tp = ctx->tp_size;
    if (c.vocab_size < 1 || c.width < 1 || c.num_layers < 1) return fail(ctx, NVLLM_EINVAL, "config has non-positive sizes");
    if (c.width > 8192) return fail(ctx, NVLLM_EINVAL, "width %d unsupported (at most 8192)", c.width);
    if (c.vocab_size % tp) return fail(ctx, NVLLM_EINVAL, "vocabulary of %d not divisible by tp_size %d", c.vocab_size, tp);
    const bool loop = c.loop_times > 1;
    if (loop && (c.loop_start < 0 || c.loop_start > c.loop_stop || c.loop_stop > c.num_layers))
        return fail(ctx, NVLLM_EINVAL, "loop [%d, %d) outside the %d layers", c.loop_start, c.loop_stop, c.num_layers);
    for (int l = 0; l < c.num_layers; ++l) {
        const nvllm_latent_layer& k = layers[l];
        if (k.ff < 0 || k.experts < 0 || (k.ff && k.experts)) return fail(ctx, NVLLM_EINVAL, "layer %d: feed-forward sizes", l);
        if (k.ff % tp || (k.experts && (k.expert_ff % tp || k.shared_ff % tp)))
            return fail(ctx, NVLLM_EINVAL, "layer %d: feed-forward width not divisible by tp_size %d", l, tp);
        if (k.ff && k.glu != NVLLM_GLU_CLAMPED && k.glu != NVLLM_GLU_GELU) return fail(ctx, NVLLM_EINVAL, "layer %d: feed-forward activation %d unknown", l, k.glu);
        if (k.ff && k.glu == NVLLM_GLU_CLAMPED && k.glu_limit <= 0) return fail(ctx, NVLLM_EINVAL, "layer %d: the feed-forward's limit must be positive", l);
        if (k.experts && (k.experts > kMaxExperts || k.top < 1 || k.top > std::min(k.experts, kMaxTop) || k.expert_ff < 1 || k.shared_ff < 0))
            return fail(ctx, NVLLM_EINVAL, "layer %d: %d of %d experts of width %d unsupported (at most %d of %d)", l, k.top, k.experts, k.expert_ff, kMaxTop, kMaxExperts);
        if (k.mixer == NVLLM_SELECTIVE_SCAN) {
            if (k.inner < 1 || k.state < 1 || k.state > kMaxScanStates || k.conv_taps < 1 || k.conv_taps > 16 || k.dt_rank < 1)
                return fail(ctx, NVLLM_EINVAL, "layer %d: scan of %d channels, %d states (at most %d), %d taps (at most 16), rank %d unsupported", l, k.inner, k.state, kMaxScanStates, k.conv_taps, k.dt_rank);
            if (k.inner % tp) return fail(ctx, NVLLM_EINVAL, "layer %d: %d channels not divisible by tp_size %d", l, k.inner, tp);
            continue;
        }
        if (k.mixer != NVLLM_LATENT_ATTENTION) return fail(ctx, NVLLM_EINVAL, "layer %d: mixer %d unknown", l, k.mixer);
        if (k.heads < 1 || k.dim < 1 || k.rot_dim < 0 || k.vdim < 1 || k.kv_rank < 1 || k.q_rank < 0 || k.q_rank > 16384) return fail(ctx, NVLLM_EINVAL, "layer %d has non-positive sizes", l);
        if (k.rot_dim % 2) return fail(ctx, NVLLM_EINVAL, "layer %d: rot_dim %d is odd", l, k.rot_dim);
        if (k.heads % tp) return fail(ctx, NVLLM_EINVAL, "layer %d: heads %d not divisible by tp_size %d", l, k.heads, tp);
        if (up(k.kv_rank, 32) + up(k.rot_dim, 32) > 2560) return fail(ctx, NVLLM_EINVAL, "layer %d: latent of %d + %d elements unsupported (at most 2560)", l, k.kv_rank, k.rot_dim);
        if (k.kv_from >= 0) {
            if (k.kv_from >= l || layers[k.kv_from].mixer != NVLLM_LATENT_ATTENTION || layers[k.kv_from].kv_from >= 0)
                return fail(ctx, NVLLM_EINVAL, "layer %d: layer %d has no latent cache of its own before it", l, k.kv_from);
            const nvllm_latent_layer& j = layers[k.kv_from];
            if (j.kv_rank != k.kv_rank || j.rot_dim != k.rot_dim) return fail(ctx, NVLLM_EINVAL, "layer %d reads the cache of layer %d, whose sizes differ", l, k.kv_from);
            if (loop) return fail(ctx, NVLLM_EINVAL, "layer %d: shared caches beside looped layers are unsupported", l);
        }
    }
    HIPCHK(ctx, hipSetDevice(ctx->device));
    nvllm_model* m = new nvllm_model();
    m->ctx = ctx;
    m->dec = std::make_unique<LatentModel>();
    LatentModel& L = latent(m);
    L.cfg = c;
    m->H = c.width; m->V_l = c.vocab_size / tp; m->kv_l = 1;
    m->cfg.vocab_size = c.vocab_size; m->cfg.hidden_size = c.width; m->cfg.max_position_embeddings = 1 << 30;
    L.ldr = up(c.width, 16); L.Kw = up(c.width, 128); L.Vp = up(m->V_l, 16);
    for (int l = 0; l < c.num_layers; ++l) {
        const int times = loop && l == c.loop_start ? c.loop_times : 1;
        if (times > 1) {
            for (int t = 0; t < times; ++t) for (int i = c.loop_start; i < c.loop_stop; ++i) L.order.push_back(i);
            if (c.loop_stop > c.loop_start) { l = c.loop_stop - 1; continue; }
        }
        L.order.push_back(l);
    }
    m->L = (int)L.order.size();
    for (int l = 0; l < c.num_layers; ++l) {
        if (layers[l].mixer == NVLLM_LATENT_ATTENTION && layers[l].window <= 0) { m->widest_window = 0; break; }
        m->widest_window = std::max(m->widest_window, (int)layers[l].window);
    }
    auto alloc_w = [&](PackedW& w, int N, int K) { return alloc_packed(ctx, w, N, K); };
    auto alloc_v = [&](float** p, size_t n) { return alloc_vec(ctx, p, n); };
    // wide projections: a whole number of the prompt product's 192- or 256-feature tiles
    auto wide = [&](int n) { return n >= 1536 && !c.f32 ? up_tile(n) : up(n, 16); };
    int rc = dmalloc(ctx, &L.embed, (size_t)c.vocab_size * L.ldr);
    if (!rc) HIPCHK(ctx, hipMemsetAsync(L.embed, 0, (size_t)c.vocab_size * L.ldr * 2, ctx->stream));
    if (!rc) rc = alloc_w(L.head, L.Vp, L.Kw);
    if (!rc) rc = alloc_v(&L.final_norm, L.Kw);
    L.layers.resize(c.num_layers);
    for (int l = 0; l < c.num_layers && !rc; ++l) {
        LatentLayer& w = L.layers[l];
        w.c = layers[l];
        w.ff = w.c.ff / tp; w.ff_p = up(w.ff, 128);
        rc = alloc_v(&w.norm1, L.Kw);
        if (w.ff) {
            if (!rc) rc = alloc_w(w.gu, 2 * w.ff_p, L.Kw);
            if (!rc) rc = alloc_w(w.down, L.ldr, w.ff_p);
        }
        if (!rc && !c.one_norm && (w.ff || w.c.experts)) rc = alloc_v(&w.norm2, L.Kw);
        w.experts.weight_in = w.c.expert_weight_in;
        if (!rc && w.c.experts) rc = w.experts.create(ctx, w.c.experts, w.c.top, w.c.expert_ff, w.c.shared_ff, c.width, L.Kw, L.ldr, c.f32);
        if (w.c.mixer == NVLLM_SELECTIVE_SCAN) {
            L.has_state = true;
            if (!rc) rc = w.scan.create(ctx, w.c.inner, w.c.state, w.c.conv_taps, w.c.dt_rank, L.Kw, c.f32);
            w.Kc = w.scan.Kc;
            if (!rc) rc = alloc_w(w.o, L.ldr, w.Kc);
            continue;
        }
        w.heads = w.c.heads / tp;
        // the expanded form has instances for the padded sizes below; layers without one keep the plain padding
        w.expands = !c.f32 && latent_prefill_dim(w.c.dim) && latent_prefill_vdim(w.c.vdim) && w.c.kv_rank <= 512 && w.c.rot_dim > 0 && w.c.rot_dim <= 64;
        w.dim_p = w.expands ? latent_prefill_dim(w.c.dim) : up(w.c.dim, 32); w.rank_p = c.f32 ? up(w.c.kv_rank, 32) : latent_rank_padded(w.c.kv_rank); w.rot_p = up(w.c.rot_dim, 32);
        w.vdim_p = w.expands ? latent_prefill_vdim(w.c.vdim) : up(w.c.vdim, 16);
        const int latent_rows = w.own_kv() ? w.c.kv_rank + w.c.rot_dim : 0;
        w.Nq = wide(w.heads * (w.c.dim + w.c.rot_dim) + (w.c.q_rank ? 0 : latent_rows));
        w.Kc = up(w.heads * w.c.vdim, 128);
        if (w.c.q_rank) {
            const int rows = w.c.q_rank + latent_rows;
            w.Nd = rows >= 512 && rows < 1536 && !c.f32 ? up(rows, 256) : wide(rows); w.Kq = up(w.c.q_rank, 128);
            if (!rc) rc = alloc_w(w.dq, w.Nd, L.Kw);
            if (!rc) rc = alloc_v(&w.dq_norm, w.Kq);
        }
        if (!rc && w.c.sink) rc = alloc_v(&w.sink, w.heads);
        if (!rc) rc = alloc_w(w.qkv, w.Nq, w.c.q_rank ? w.Kq : L.Kw);
        if (!rc) rc = alloc_w(w.ukt, w.heads * w.rank_p, w.dim_p);
        if (!rc && w.expands) rc = alloc_w(w.ukx, w.heads * w.dim_p, w.rank_p);
        if (!rc && w.expands) rc = alloc_w(w.uvx, w.heads * w.vdim_p, w.rank_p);
        if (!rc) rc = alloc_w(w.uv, w.heads * w.vdim_p, w.rank_p);
        if (!rc) rc = alloc_w(w.o, L.ldr, w.Kc);
        if (!rc) rc = alloc_v(&w.dkv_norm, w.rank_p);
        w.rope = rope_index(L.ropes, RopeTable{w.c.rot_base, w.c.yarn_factor, w.c.yarn_original, w.c.yarn_fast, w.c.yarn_slow, w.c.rot_dim});
    }
    if (!rc && hipStreamSynchronize(ctx->stream) != hipSuccess) rc = fail(ctx, NVLLM_EHIP, "weight allocation failed");
    if (rc) { nvllm_model_destroy(m); return rc; }
    *out = m;
    return NVLLM_OK;
}

void LatentModel::free_kv() {
    LatentModel& L = *this;
    for (size_t i = 0; i < L.cache.size(); ++i)
        if (L.cache[i] && L.layers[L.order[i]].own_kv()) (void)hipFree(L.cache[i]);
    L.cache.clear();
    L.experts.release();
    L.scan.release();
    for (LatentLayer& w : L.layers) w.scan.free_kv();
    void* ptrs[] = {L.cq_f, L.cqh, L.cql, L.slabs2, L.q, L.qlat, L.olat, L.part_o, L.part_ml, L.tap, L.kx, L.vx, L.d_exp, L.d_tile_exp, L.x2h, L.x2l, L.y1, L.y2, L.ctx_f, L.act_f};
    for (void* p : ptrs) if (p) (void)hipFree(p);
    L.slabs2 = L.q = L.qlat = L.olat = L.part_o = L.part_ml = L.tap = nullptr;
    L.x2h = L.x2l = nullptr;
    L.kx = L.vx = nullptr;
    L.d_exp = L.d_tile_exp = nullptr;
    if (L.h_exp) (void)hipHostFree(L.h_exp);
    L.h_exp = nullptr;
    L.exp_cap = L.exp_n = 0;
    L.y1 = L.y2 = L.ctx_f = L.act_f = L.cq_f = nullptr;
    L.cqh = L.cql = nullptr;
    for (RopeTable& r : L.ropes) r.release();
}

LatentModel::~LatentModel() {
    LatentModel& L = *this;
    free_kv();
    (void)hipFree(L.embed); (void)hipFree(L.head.data); (void)hipFree(L.final_norm);
    for (LatentLayer& w : L.layers) {
        w.experts.destroy();
        w.scan.destroy();
        (void)hipFree(w.dq_norm); (void)hipFree(w.sink);
        for (PackedW* p : {&w.dq, &w.qkv, &w.ukt, &w.ukx, &w.uv, &w.uvx, &w.o, &w.gu, &w.down}) (void)hipFree(p->data);
        (void)hipFree(w.norm1); (void)hipFree(w.norm2); (void)hipFree(w.dkv_norm);
    }
}

// ---------------------------------------------------------------------------------------------------
// weights
// ---------------------------------------------------------------------------------------------------
// weights of the expanded form: `size` rows per head as f16, scaled by the power of two that brings the largest entry of the
// (bf16-valued) matrix to [2^14, 2^15); *unscale undoes it
static int put_expand(nvllm_ctx* ctx, const PackedW& w, float* unscale, const HostMat& h, int64_t head0, int heads, int size, int size_p, int kr) {
    auto val = [&](int64_t i) {
        const uint32_t u = (uint32_t)h.at(i / kr, i % kr) << 16;
        float f;
        memcpy(&f, &u, 4);
        return f;
    };
    float big = 0.f;
    const int64_t i0 = head0 * size * kr, n = (int64_t)heads * size * kr;
    for (int64_t i = 0; i < n; ++i) big = std::max(big, std::fabs(val(i0 + i)));
    const int e = big > 0.f && std::isfinite(big) ? 14 - std::ilogb(big) : 0;
    *unscale = std::ldexp(1.0f, -e);
    return put_rows(ctx, w, 0, heads * size_p, kr, -1, [&](int r, int c) -> uint16_t {
        const int k = r / size_p, i = r % size_p;
        if (i >= size) return 0;
        const _Float16 v = (_Float16)std::ldexp(val(i0 + ((int64_t)k * size + i) * kr + c), e);
        uint16_t b;
        memcpy(&b, &v, 2);
        return b;
    });
}

// the checkpoint's tensors of a layer
static std::vector<std::string> layer_tensors(const LatentLayer& w, bool one_norm) {
    std::vector<std::string> t = {"norm1", "mix.o"};
    auto add = [&](std::initializer_list<const char*> names) { t.insert(t.end(), names.begin(), names.end()); };
    if (w.scan.on()) {
        for (const std::string& s : ScanMixer::tensors()) t.push_back("mix." + s);
    } else {
        add({"mix.uk", "mix.uv"});
        if (w.c.q_rank) add({"mix.dq", "mix.dq.norm", "mix.uq"});
        else add({"mix.q"});
        if (w.own_kv()) add({"mix.dkv", "mix.dkv.norm"});
        if (w.c.sink) add({"mix.sink"});
    }
    if (!one_norm && (w.ff || w.experts.on())) add({"norm2"});
    if (w.ff) add({"mlp.gate", "mlp.up", "mlp.down"});
    if (w.experts.on())
        for (const std::string& s : w.experts.tensors()) t.push_back("mlp." + s);
    return t;
}

int LatentModel::load_tensor(nvllm_model* m, const char* name, const void* data, int dtype, const int64_t* shape, int ndim) {
    nvllm_ctx* ctx = m->ctx;
    LatentModel& L = latent(m);
    const int rank = ctx->tp_rank;
    if (ndim != 1 && ndim != 2) return fail(ctx, NVLLM_EINVAL, "tensor '%s' has %d dimensions", name, ndim);
    const int64_t rows = ndim == 2 ? shape[0] : 1, cols = shape[ndim - 1];
    const HostMat h{data, dtype, cols};
    HIPCHK(ctx, hipSetDevice(ctx->device));
    auto want = [&](int64_t r, int64_t c) -> int {
        if (rows == r && cols == c && (ndim == 2 || r == 1)) return NVLLM_OK;
        return fail(ctx, NVLLM_EINVAL, "tensor '%s': shape mismatch (got %lld x %lld, want %lld x %lld)", name, (long long)rows, (long long)cols, (long long)r, (long long)c);
    };
    auto vec = [&](float* dst, int n) -> int {
        int rc = want(1, n);
        if (rc) return rc;
        std::vector<float> t(n);
        for (int i = 0; i < n; ++i) t[i] = h.f32(i);
        HIPCHK(ctx, hipMemcpy(dst, t.data(), (size_t)n * 4, hipMemcpyHostToDevice));
        return NVLLM_OK;
    };
    const int W = L.cfg.width, V = L.cfg.vocab_size;
    int rc = NVLLM_OK, l = -1, off = 0;
    if (!strcmp(name, "embed")) {
        if ((rc = want(V, W))) return rc;
        std::vector<uint16_t> t((size_t)V * L.ldr, 0);
        for (int r = 0; r < V; ++r) for (int c = 0; c < W; ++c) t[(size_t)r * L.ldr + c] = h.at(r, c);
        HIPCHK(ctx, hipMemcpy(L.embed, t.data(), t.size() * 2, hipMemcpyHostToDevice));
    } else if (!strcmp(name, "head")) {
        if ((rc = want(V, W))) return rc;
        const int64_t r0 = (int64_t)rank * m->V_l;
        if ((rc = put_rows(ctx, L.head, 0, m->V_l, W, -1, [&](int r, int c) { return h.at(r0 + r, c); }))) return rc;
    } else if (!strcmp(name, "final.norm")) {
        if ((rc = vec(L.final_norm, W))) return rc;
    } else {
        if (sscanf(name, "l%d.%n", &l, &off) != 1 || off == 0 || l < 0 || l >= L.cfg.num_layers) return fail(ctx, NVLLM_EINVAL, "unknown tensor name '%s'", name);
        const char* s = name + off;
        LatentLayer& w = L.layers[l];
        const int dim = w.c.dim, rot = w.c.rot_dim, vdim = w.c.vdim, kr = w.c.kv_rank, Hl = w.heads, H = w.c.heads, ff = w.c.ff;
        const int64_t h0 = (int64_t)rank * Hl, f0 = (int64_t)rank * w.ff;
        // rotated pairs of neighbours: the rows are put in the order that pairs i with i + rot / 2 (queries and keys alike: scores do not change)
        auto turned = [&](int i) { return !w.c.rot_pairs ? i : i < rot / 2 ? 2 * i : 2 * (i - rot / 2) + 1; };
        auto q_row = [&](int r) { const int n = r / (dim + rot), i = r % (dim + rot); return (h0 + n) * (dim + rot) + (i < dim ? i : dim + turned(i - dim)); };
        auto kv_row = [&](int r) { return r < kr ? r : kr + turned(r - kr); };
        auto put_o = [&](int64_t all, int n, int64_t c0) -> int {
            int e = want(W, all);
            return e ? e : put_rows(ctx, w.o, 0, W, n, -1, [&](int r, int c) { return h.at(r, c0 + c); });
        };
        const bool latents = !w.scan.on(), own = latents && w.own_kv(), narrow = latents && w.c.q_rank > 0;
        const int qr = w.c.q_rank, Q = H * (dim + rot);
        const std::vector<std::string> names = layer_tensors(w, L.cfg.one_norm);
        if (std::find(names.begin(), names.end(), s) == names.end()) return fail(ctx, NVLLM_EINVAL, "unknown tensor name '%s'", name);
        if (!strcmp(s, "norm1")) rc = vec(w.norm1, W);
        else if (w.scan.on() && !strcmp(s, "mix.o")) rc = put_o(w.c.inner, w.scan.n, (int64_t)rank * w.scan.n);
        else if (w.scan.on() && !strncmp(s, "mix.", 4)) rc = w.scan.load(m, name, s + 4, h, rows, cols, W);
        else if (w.experts.on() && !strncmp(s, "mlp.", 4)) rc = w.experts.load(m, name, s + 4, h, rows, cols);
        else if (!strcmp(s, "mix.q") || !strcmp(s, "mix.uq")) {
            const int K = narrow ? qr : W;
            if (!(rc = want(Q, K))) rc = put_rows(ctx, w.qkv, 0, Hl * (dim + rot), K, -1, [&](int r, int c) { return h.at(q_row(r), c); });
        } else if (!strcmp(s, "mix.dq")) {
            if (!(rc = want(qr, W))) rc = put_rows(ctx, w.dq, 0, qr, W, -1, [&](int r, int c) { return h.at(r, c); });
        } else if (!strcmp(s, "mix.dq.norm")) rc = vec(w.dq_norm, qr);
        else if (!strcmp(s, "mix.sink")) {
            if (!(rc = want(1, H))) {
                std::vector<float> t(Hl);
                for (int i = 0; i < Hl; ++i) t[i] = (float)(h.f32(h0 + i) * 1.4426950408889634);
                HIPCHK(ctx, hipMemcpy(w.sink, t.data(), t.size() * 4, hipMemcpyHostToDevice));
            }
        } else if (own && !strcmp(s, "mix.dkv")) {
            if (!(rc = want(kr + rot, W)))
                rc = put_rows(ctx, narrow ? w.dq : w.qkv, narrow ? qr : Hl * (dim + rot), kr + rot, W, -1, [&](int r, int c) { return h.at(kv_row(r), c); });
        } else if (!strcmp(s, "mix.dkv.norm")) rc = vec(w.dkv_norm, kr);
        else if (!strcmp(s, "mix.uk")) {  // transposed per head: the query is carried into latent space
            if (!(rc = want((int64_t)H * dim, kr)))
                rc = put_rows(ctx, w.ukt, 0, Hl * w.rank_p, dim, -1, [&](int r, int c) -> uint16_t {
                    const int n = r / w.rank_p, k = r % w.rank_p;
                    return k < kr ? h.at((h0 + n) * dim + c, k) : (uint16_t)0;
                });
            if (!rc && w.expands) rc = put_expand(ctx, w.ukx, &w.ukx_scale, h, h0, Hl, dim, w.dim_p, kr);
        } else if (!strcmp(s, "mix.uv")) {
            if (!(rc = want((int64_t)H * vdim, kr)))
                rc = put_rows(ctx, w.uv, 0, Hl * w.vdim_p, kr, -1, [&](int r, int c) -> uint16_t {
                    const int n = r / w.vdim_p, i = r % w.vdim_p;
                    return i < vdim ? h.at((h0 + n) * vdim + i, c) : (uint16_t)0;
                });
            if (!rc && w.expands) rc = put_expand(ctx, w.uvx, &w.uvx_scale, h, h0, Hl, vdim, w.vdim_p, kr);
        } else if (!strcmp(s, "mix.o")) {
            rc = put_o((int64_t)H * vdim, Hl * vdim, h0 * vdim);
        } else if (!strcmp(s, "norm2")) rc = vec(w.norm2, W);
        else if (ff && (!strcmp(s, "mlp.gate") || !strcmp(s, "mlp.up"))) {
            if (!(rc = want(ff, W))) rc = put_rows(ctx, w.gu, 0, w.ff, W, s[4] == 'g' ? 0 : 1, [&](int r, int c) { return h.at(f0 + r, c); });
        } else if (ff && !strcmp(s, "mlp.down")) {
            if (!(rc = want(W, ff))) rc = put_rows(ctx, w.down, 0, W, w.ff, -1, [&](int r, int c) { return h.at(r, f0 + c); });
        } else return fail(ctx, NVLLM_EINVAL, "unknown tensor name '%s'", name);
        if (rc) return rc;
    }
    m->loaded[name] = true;
    return NVLLM_OK;
}

int LatentModel::finalize(nvllm_model* m) {
    nvllm_ctx* ctx = m->ctx;
    for (const char* s : {"embed", "head", "final.norm"})
        if (!m->loaded.count(s)) return fail(ctx, NVLLM_ESTATE, "missing tensor %s", s);
    char name[96];
    for (int l = 0; l < latent(m).cfg.num_layers; ++l)
        for (const std::string& s : layer_tensors(latent(m).layers[l], latent(m).cfg.one_norm)) {
            snprintf(name, sizeof name, "l%d.%s", l, s.c_str());
            if (!m->loaded.count(name)) return fail(ctx, NVLLM_ESTATE, "missing tensor %s", name);
        }
    m->finalized = true;
    return NVLLM_OK;
}

int64_t LatentModel::weight_bytes() const {
    const LatentModel& L = *this;
    int64_t b = (int64_t)L.head.bytes() + (int64_t)L.cfg.width * 4;
    for (int l : L.order) {
        const LatentLayer& w = L.layers[l];
        b += (int64_t)(w.dq.bytes() + w.experts.step_bytes() + w.scan.bytes());
        b += (int64_t)(w.qkv.bytes() + w.ukt.bytes() + w.uv.bytes() + w.o.bytes() + w.gu.bytes() + w.down.bytes());
        b += (int64_t)((w.norm2 ? 2 : 1) * L.cfg.width + w.c.kv_rank) * 4;
    }
    return b;
}
int64_t LatentModel::kv_bytes_per_token() const {
    const LatentModel& L = *this;
    int64_t b = 0;
    for (int l : L.order)
        if (L.layers[l].own_kv()) b += (int64_t)(L.layers[l].rank_p + L.layers[l].rot_p) * (L.cfg.f32 ? 4 : 2);
    return b;
}
int64_t LatentModel::kv_read_bytes(int len) const {
    const LatentModel& L = *this;
    int64_t b = 0;
    for (int l : L.order) {
        const LatentLayer& w = L.layers[l];
        if (w.scan.on()) b += (int64_t)w.scan.state_bytes() * 2;  // read and written
        b += (int64_t)(w.rank_p + w.rot_p) * (L.cfg.f32 ? 4 : 2) * (w.c.window > 0 ? std::min(len, w.c.window) : len);
    }
    return b;
}

// ---------------------------------------------------------------------------------------------------
// cache and step buffers (pool sizes are set, the shared buffers exist)
// ---------------------------------------------------------------------------------------------------
int LatentModel::kv_alloc(nvllm_model* m) {
    nvllm_ctx* ctx = m->ctx;
    LatentModel& L = latent(m);
    hipStream_t s = ctx->stream;
    const bool f32 = L.cfg.f32 != 0;
    const size_t R = m->max_rows, R16 = (R + 15) / 16 * 16;
    L.cache.assign(L.order.size(), nullptr);
    for (size_t i = 0; i < L.order.size(); ++i) {
        LatentLayer& w = L.layers[L.order[i]];
        if (w.scan.on()) {  // no cache; its state once, however often the layer runs
            if (!w.scan.st) {
                int e = w.scan.kv_alloc(m);
                if (e) return e;
            }
            continue;
        }
        if (!w.own_kv()) { L.cache[i] = L.cache[w.c.kv_from]; continue; }  // no loop: run = layer
        const size_t bytes = (size_t)m->num_blocks * kBlockTokens * (w.rank_p + w.rot_p) * (f32 ? 4 : 2);
        HIPCHK(ctx, hipMalloc(&L.cache[i], bytes));
        HIPCHK(ctx, hipMemsetAsync(L.cache[i], 0, bytes, s));  // padding stays zero, unwritten tokens finite
    }
    size_t nmax = L.ldr, q_row = 0, lat_row = 0, kc = 0, ffp = 0, kq = 0;
    for (const LatentLayer& w : L.layers) {
        nmax = std::max<size_t>({nmax, (size_t)w.Nq, (size_t)w.Nd, (size_t)2 * w.ff_p, (size_t)w.scan.Nin, (size_t)w.scan.Nx, (size_t)w.experts.sh_p});
        kq = std::max<size_t>(kq, w.Kq);
        if (w.scan.on()) L.scan.reserve(w.scan, R);
        if (w.experts.on()) L.experts.reserve(w.experts, R);
        q_row = std::max<size_t>(q_row, (size_t)w.heads * (w.dim_p + w.rot_p));
        lat_row = std::max<size_t>(lat_row, (size_t)w.heads * w.rank_p);
        kc = std::max<size_t>(kc, w.Kc);
        ffp = std::max<size_t>(ffp, w.ff_p);
    }
    m->slab_floats = std::max<size_t>(R * nmax, (size_t)32 * std::min<size_t>(R, 128) * nmax);
    if (f32 || m->V_l % 16) m->slab_floats = std::max<size_t>(m->slab_floats, (size_t)m->max_seqs * L.Vp);
    auto zalloc = [&](void** p, size_t bytes) -> int {
        HIPCHK(ctx, hipMalloc(p, std::max<size_t>(bytes, 16)));
        HIPCHK(ctx, hipMemsetAsync(*p, 0, std::max<size_t>(bytes, 16), s));
        return NVLLM_OK;
    };
    int rc = zalloc((void**)&m->resid, R * L.ldr * 4);
    if (!rc) rc = dmalloc(ctx, &m->slabs, m->slab_floats);
    if (!rc) rc = dmalloc(ctx, &L.slabs2, m->slab_floats);
    if (!rc) rc = dmalloc(ctx, &m->red, R * L.ldr);
    if (!rc) rc = dmalloc(ctx, &L.tap, R * L.ldr);
    if (!rc) rc = L.experts.alloc(ctx, f32);
    if (!rc) rc = L.scan.alloc(m, f32);
    if (!rc) rc = zalloc((void**)&L.q, R * q_row * 4);
    if (!rc) rc = zalloc((void**)&L.qlat, R * lat_row * 4);
    if (!rc) rc = zalloc((void**)&L.olat, R * lat_row * 4);
    if (!f32) {
        const size_t part_rows = std::min<size_t>(m->max_seqs, 512);  // more sequences never split
        size_t hmax = 0;
        for (const LatentLayer& w : L.layers) hmax = std::max<size_t>(hmax, w.heads);
        if (!rc) rc = dmalloc(ctx, &L.part_o, part_rows * lat_row * kLatentMaxParts);
        if (!rc) rc = dmalloc(ctx, &L.part_ml, part_rows * hmax * kLatentMaxParts * 2);
    }
    if (f32) {
        if (!rc) rc = zalloc((void**)&L.y1, R * L.Kw * 4);
        if (!rc) rc = zalloc((void**)&L.y2, R * L.Kw * 4);
        if (!rc) rc = zalloc((void**)&L.ctx_f, R * kc * 4);
        if (!rc && ffp) rc = zalloc((void**)&L.act_f, R * ffp * 4);
        if (!rc && kq) rc = zalloc((void**)&L.cq_f, R * kq * 4);
    } else {
        if (kq) for (bf16_bits** p : {&L.cqh, &L.cql}) if (!rc) rc = zalloc((void**)p, R16 * kq * 2);
        // activation planes are read in whole 16-row blocks; columns past a layer's own width meet zero weights
        for (bf16_bits** p : {&m->xh, &m->xl, &L.x2h, &L.x2l}) if (!rc) rc = zalloc((void**)p, R16 * L.Kw * 2);
        for (bf16_bits** p : {&m->ctxh, &m->ctxl}) if (!rc) rc = zalloc((void**)p, R16 * kc * 2);
        if (ffp) for (bf16_bits** p : {&m->xh2, &m->xl2}) if (!rc) rc = zalloc((void**)p, R16 * ffp * 2);
    }
    size_t kx_row = 0, vx_row = 0;  // scratch elements per token
    for (const LatentLayer& w : L.layers)
        if (w.expands) {
            kx_row = std::max<size_t>(kx_row, (size_t)w.heads * w.dim_p);
            vx_row = std::max<size_t>(vx_row, (size_t)w.heads * w.vdim_p);
        }
    if (kx_row) {
        // a chunk's own rows, as much context again, and a partly filled tile or two per segment
        L.exp_cap = (int)(2 * R / 32) + 2 * std::min(m->max_seqs, 64) + 2;
        if (!rc) rc = dmalloc(ctx, &L.kx, (size_t)L.exp_cap * 32 * kx_row);
        if (!rc) rc = dmalloc(ctx, &L.vx, (size_t)L.exp_cap * 32 * vx_row);
        if (!rc) rc = dmalloc(ctx, &L.d_exp, (size_t)3 * L.exp_cap);
        if (!rc) rc = dmalloc(ctx, &L.d_tile_exp, R);
        if (!rc) HIPCHK(ctx, hipHostMalloc((void**)&L.h_exp, ((size_t)3 * L.exp_cap + R) * sizeof(int), hipHostMallocDefault));
    }
    if (rc) return rc;
    // rotation tables, one per rotation: angle p * f_i
    m->rope_len = (int)std::min<int64_t>((int64_t)m->max_blocks * kBlockTokens, 1 << 20);
    for (RopeTable& t : L.ropes) {
        rc = t.upload(ctx, m->rope_len);
        if (rc) return rc;
    }
    return NVLLM_OK;
}

// ---------------------------------------------------------------------------------------------------
// forward over one chunk of rows
// ---------------------------------------------------------------------------------------------------
int LatentModel::plan_chunk(nvllm_model* m, const int* pos, const int* slot, const int* seq, int R, const int* tile_row0, int n_tiles, int qt) {
    nvllm_ctx* ctx = m->ctx;
    LatentModel& L = latent(m);
    L.exp_n = 0;
    L.segments.clear();
    if (qt != 1 && L.has_state) {
        int rc = L.scan.plan(m, slot, seq, R);
        if (rc) return rc;
    }
    if (qt == 1 || !L.exp_cap || m->opt_latent_plain || m->opt_latent_absorb == 1) return NVLLM_OK;
    int widest = 0;  // <= 0: some layer sees everything
    bool all = false;
    for (const LatentLayer& w : L.layers)
        if (!w.scan.on()) { all |= w.c.window <= 0; widest = std::max(widest, w.c.window); }
    int n = 0;
    int *h_slot = L.h_exp, *h_tile = L.h_exp + L.exp_cap, *h_pos0 = L.h_exp + 2 * L.exp_cap, *h_te = L.h_exp + 3 * L.exp_cap;
    int k = 0;  // q-tile
    for (int r = 0; r < R;) {
        int e = r;
        while (e < R && seq[e] == seq[r]) ++e;
        const int lo = all ? 0 : std::max(0, pos[r] - widest + 1) >> 5, hi = (pos[e - 1] >> 5) + 1;
        if (n + hi - lo > L.exp_cap) return NVLLM_OK;  // much context for few rows: absorbed
        for (; k < n_tiles && tile_row0[k] < e; ++k) h_te[k] = n - lo;
        for (int t = lo; t < hi; ++t, ++n) { h_slot[n] = slot[r]; h_tile[n] = t; h_pos0[n] = pos[r]; }
        L.segments.push_back({pos[r], e - r});
        r = e;
    }
    // the staging buffer is free: the tile upload before this call waited for the stream
    HIPCHK(ctx, hipMemcpyAsync(L.d_exp, L.h_exp, (size_t)3 * L.exp_cap * sizeof(int), hipMemcpyHostToDevice, ctx->stream));
    HIPCHK(ctx, hipMemcpyAsync(L.d_tile_exp, h_te, (size_t)n_tiles * sizeof(int), hipMemcpyHostToDevice, ctx->stream));
    L.exp_n = n;
    return NVLLM_OK;
}

// products per head: expansion + expanded attention against absorbing + absorbed attention + carrying values back
static bool latent_expanded_pays(const nvllm_model* m, const LatentLayer& w, int R) {
    const LatentModel& L = latent(m);
    if (!w.expands || !L.exp_n) return false;
    if (m->opt_latent_absorb == -1) return true;
    double pairs = 0, tokens = 0;
    for (const auto& s : L.segments) {
        const double seen = w.c.window > 0 ? std::min<double>(w.c.window, s.pos0 + s.n / 2.0 + 1) : s.pos0 + s.n / 2.0 + 1;
        pairs += s.n * seen;
        tokens += s.n + (w.c.window > 0 ? std::min(s.pos0, w.c.window) : s.pos0);
    }
    const double expanded = tokens * w.rank_p * (w.dim_p + w.vdim_p) + pairs * (w.dim_p + w.rot_p + w.vdim_p);
    const double absorbed = (double)R * w.rank_p * (w.dim_p + w.vdim_p) + pairs * (3.0 * w.rank_p + w.rot_p);  // keys, transposes, values
    return expanded < absorbed;
}

// first: slabs of the product the normed input met; with query latents the second product overwrites them
static int latent_attention(nvllm_model* m, const LatentLayer& w, void* cache_data, float* first, int n_slabs, int R, int n_tiles, int qt, int ctx_packed) {
    nvllm_ctx* ctx = m->ctx;
    LatentModel& L = latent(m);
    hipStream_t s = ctx->stream;
    const bool f32 = L.cfg.f32 != 0;
    const int dq = w.dim_p + w.rot_p;
    const float* qkv = first;
    LatentRowsArgs ra;
    ra.ldq = w.Nq; ra.slab_stride = (int64_t)R * w.Nq;
    ra.heads = w.heads; ra.dim = w.c.dim; ra.dim_p = w.dim_p;
    ra.scale = (float)(w.c.scale * 1.4426950408889634);
    ra.norm_w = w.dkv_norm; ra.eps = (float)L.cfg.norm_eps;
    ra.cos = L.ropes[w.rope].cos; ra.sin = L.ropes[w.rope].sin;
    ra.pos = m->d_pos; ra.slot = m->d_slot; ra.block_tables = m->d_block_tables; ra.max_blocks = m->max_blocks;
    ra.q = L.q;
    ra.cache = w.cache_shape();
    ra.cache.data = cache_data; ra.cache.f32 = f32;
    ra.kv_slabs = n_slabs; ra.ldkv = w.c.q_rank ? w.Nd : w.Nq; ra.kv_stride = (int64_t)R * ra.ldkv;
    if (w.own_kv()) ra.kv = first + (w.c.q_rank ? w.c.q_rank : w.heads * (w.c.dim + w.c.rot_dim));
    if (w.c.q_rank) {
        ProductPlan pq;
        if (!f32) pq = plan_product(m, R, w.qkv);
        QueryLatentArgs qa;
        qa.in = first; qa.n_slabs = n_slabs; qa.ld = w.Nd; qa.slab_stride = ra.kv_stride; qa.rank = w.c.q_rank; qa.ldx = w.Kq; qa.norm_w = w.dq_norm; qa.eps = ra.eps;
        qa.xh = L.cqh; qa.xl = L.cql; qa.y = L.cq_f; qa.packed = pq.packed;
        PROF(m, PROF_QK, launch_query_latent(qa, ra, R, s));
        ra.kv = nullptr;  // written
        int rc = f32 ? exact_product(m, L.cq_f, w.qkv, first, R) : run_product(m, pq, L.cqh, L.cql, w.qkv, first, R, &n_slabs);
        if (rc) return rc;
        if (f32) n_slabs = 1;
    }
    ra.qkv = qkv; ra.n_slabs = n_slabs;
    const bool matrix_core = latent_attn_ok(ra.cache) && !m->opt_latent_plain;
    const bool fused = matrix_core && qt == 1 && !m->opt_no_fused && w.dim_p <= 1024;  // decode: the kernels around the attention in two launches
    const bool expanded = qt == 2 && latent_expanded_pays(m, w, R);
    if (expanded) { if (ra.kv) PROF(m, PROF_QK, launch_latent_cache(ra, R, s)); }
    else if (!fused) PROF(m, PROF_QK, launch_latent_rows(ra, R, s));
    if (expanded) {
        LatentExpandArgs ea;
        ea.cache = ra.cache; ea.block_tables = m->d_block_tables; ea.max_blocks = m->max_blocks;
        ea.exp_slot = L.d_exp; ea.exp_tile = L.d_exp + L.exp_cap; ea.exp_pos0 = L.d_exp + 2 * L.exp_cap;
        ea.n_tiles = L.exp_n; ea.cap = L.exp_cap; ea.window = w.c.window;
        ea.uk = w.ukx.data; ea.uv = w.uvx.data; ea.uk_scale = w.ukx_scale; ea.uv_scale = w.uvx_scale; ea.dim_p = w.dim_p; ea.vdim_p = w.vdim_p; ea.kx = L.kx; ea.vx = L.vx;
        PROF(m, PROF_GEMM, launch_latent_expand(ea, w.heads, s));
        LatentPrefillArgs pa;
        pa.qkv = qkv; pa.n_slabs = n_slabs; pa.ldq = w.Nq; pa.slab_stride = ra.slab_stride; pa.dim = w.c.dim; pa.scale = ra.scale;
        pa.cos = ra.cos; pa.sin = ra.sin; pa.cache = ra.cache; pa.block_tables = m->d_block_tables; pa.max_blocks = m->max_blocks;
        pa.kx = L.kx; pa.vx = L.vx; pa.cap = L.exp_cap;
        pa.tile_row0 = m->d_tile_row0; pa.tile_nrows = m->d_tile_nrows; pa.tile_slot = m->d_tile_slot; pa.tile_exp = L.d_tile_exp;
        pa.tile_order = m->d_tile_order; pa.pos = m->d_pos; pa.n_tiles = n_tiles; pa.heads = w.heads; pa.window = w.c.window; pa.sink = w.sink;
        pa.dim_p = w.dim_p; pa.vdim = w.c.vdim; pa.vdim_p = w.vdim_p; pa.oh = m->ctxh; pa.ol = m->ctxl; pa.ld = w.Kc; pa.packed = ctx_packed;
        PROF(m, PROF_ATTN, launch_latent_prefill(pa, s));
        ++m->latent_expanded;
        return NVLLM_OK;
    }
    // unrotated query into latent space
    if (fused) {
        PROF(m, PROF_QK, launch_latent_query(ra, w.ukt.data, L.qlat, R, s));
    } else {
        HeadGemmArgs ga;
        ga.x = L.q; ga.x_row = (int64_t)w.heads * dq; ga.x_head = dq;
        ga.w = w.ukt.data; ga.w_head = (int64_t)w.rank_p * w.dim_p / 8;
        ga.N = ga.n_valid = w.rank_p; ga.K = w.dim_p; ga.heads = w.heads; ga.M = R; ga.exact = f32;
        ga.y = L.qlat; ga.y_row = (int64_t)w.heads * w.rank_p; ga.y_head = w.rank_p;
        PROF(m, PROF_GEMM, launch_head_gemm(ga, s));
    }
    LatentAttnArgs aa;
    aa.qlat = L.qlat; aa.qrot = L.q + w.dim_p; aa.qrot_row = (int64_t)w.heads * dq; aa.qrot_head = dq;
    aa.cache = ra.cache; aa.block_tables = m->d_block_tables; aa.max_blocks = m->max_blocks;
    aa.tile_row0 = m->d_tile_row0; aa.tile_nrows = m->d_tile_nrows; aa.tile_slot = m->d_tile_slot; aa.pos = m->d_pos; aa.slot = m->d_slot;
    aa.single = qt == 1 && n_tiles == R;
    aa.heads = w.heads; aa.window = w.c.window; aa.sink = w.sink; aa.out = L.olat;
    int parts = 1;
    if (matrix_core) {
        if (fused && R <= m->max_seqs) {
            // split the visible context when (sequences x 16-head groups) alone leave CUs idle; a wave takes a 32-token tile at a time.
            // About two workgroups per CU where two fit (latents up to 256), else one.
            const int len = m->cur_max_len, seen = w.c.window > 0 ? std::min(len, w.c.window) : len;
            const int tiles = (seen + 31) / 32 + 1, base = R * ((w.heads + 15) / 16);
            const int wgs = m->opt_latent_wgs > 0 ? m->opt_latent_wgs : w.rank_p <= 256 ? 512 : 256;
            const int want = std::max(1, std::min(kLatentMaxParts, wgs / base));
            aa.part_tiles = 4 * ((tiles + 4 * want - 1) / (4 * want));
            parts = (tiles + aa.part_tiles - 1) / aa.part_tiles;
            aa.max_parts = kLatentMaxParts; aa.part_o = L.part_o; aa.part_ml = L.part_ml;
        }
        PROF(m, PROF_ATTN, launch_latent_attn(aa, n_tiles, qt == 1 ? 1 : kLatentTileRows, parts, s));
    } else {
        PROF(m, PROF_ATTN, launch_latent_attn_plain(aa, R, s));
    }
    // weighted latents to values
    if (fused) {
        PROF(m, PROF_GEMM, launch_latent_values(aa, parts, w.uv.data, w.c.vdim, w.vdim_p, m->ctxh, m->ctxl, w.Kc, ctx_packed, R, s));
        return NVLLM_OK;
    }
    HeadGemmArgs gv;
    gv.x = L.olat; gv.x_row = (int64_t)w.heads * w.rank_p; gv.x_head = w.rank_p;
    gv.w = w.uv.data; gv.w_head = (int64_t)w.vdim_p * w.rank_p / 8;
    gv.N = w.vdim_p; gv.n_valid = w.c.vdim; gv.K = w.rank_p; gv.heads = w.heads; gv.M = R; gv.exact = f32;
    if (f32) { gv.y = L.ctx_f; gv.y_row = w.Kc; gv.y_head = w.c.vdim; }
    else { gv.yh = m->ctxh; gv.yl = m->ctxl; gv.ld = w.Kc; gv.packed = ctx_packed; }
    PROF(m, PROF_GEMM, launch_head_gemm(gv, s));
    return NVLLM_OK;
}

int LatentModel::forward_chunk(nvllm_model* m, int R, int n_tiles, int qt, int n_last, int logits_row0) {
    nvllm_ctx* ctx = m->ctx;
    LatentModel& L = latent(m);
    hipStream_t s = ctx->stream;
    const bool f32 = L.cfg.f32 != 0, tp = ctx->tp_size > 1;
    m->tap_rows = R;
    AddNormArgs base;  // the sum pending on the residual stream
    base.center = L.cfg.norm == NVLLM_NORM_LAYER;
    base.W = L.cfg.width; base.ldr = L.ldr; base.ldx = L.Kw; base.eps = (float)L.cfg.norm_eps;
    base.ids = m->d_ids; base.embed = L.embed; base.embed_scale = (float)L.cfg.embed_scale;
    for (size_t run = 0; run < L.order.size(); ++run) {
        LatentLayer& w = L.layers[L.order[run]];
        const bool gelu = w.c.glu == NVLLM_GLU_GELU;
        const GluSpec spec{gelu ? 0.f : (float)w.c.glu_limit, (float)w.c.glu_alpha, (float)w.c.glu_shift, gelu};
        ProductPlan pq, po, pd;
        GluPlan pg;
        if (!f32) {
            pq = plan_product(m, R, w.first());
            po = plan_product(m, R, w.o);
            if (w.ff) {
                pd = plan_product(m, R, w.down);
                pg = plan_glu(m, R, w.gu, pd.kind == P_TILE);
                if (pd.packed && !pg.out_packed_ok) {
                    if (pd.kind == P_TILE) pd = ProductPlan{P_GENERIC, 0, pd.max_split};
                    else pd.packed = 0;
                }
            }
        }
        AddNormArgs na = base;
        na.residual_out = m->resid;
        // the feed-forward's input: its own norm's output, or the mixer's where they share the norm (twice when the products want other orders)
        const bool mlp = w.ff || w.experts.on(), gathers = w.experts.on() && !f32 && experts_gather(m, w.experts, R);
        if (w.experts.on()) pg.packed = gathers ? 0 : pq.packed;
        const bool same = L.cfg.one_norm && (f32 || pg.packed == pq.packed);
        na.w[0] = w.norm1; na.w[1] = !mlp || same ? nullptr : L.cfg.one_norm ? w.norm1 : w.norm2;
        const float* y_ff = same ? L.y1 : L.y2;
        const bf16_bits *ffh = same ? m->xh : L.x2h, *ffl = same ? m->xl : L.x2l;
        if (f32) { na.y[0] = L.y1; na.y[1] = L.y2; }
        else {
            na.xh[0] = m->xh; na.xl[0] = m->xl; na.packed[0] = pq.packed;
            na.xh[1] = L.x2h; na.xl[1] = L.x2l; na.packed[1] = pg.packed;
        }
        PROF(m, PROF_NORM, launch_add_norm(na, R, s));
        int ns = 1, rc = f32 ? exact_product(m, L.y1, w.first(), m->slabs, R) : run_product(m, pq, m->xh, m->xl, w.first(), m->slabs, R, &ns);
        if (!rc && w.scan.on()) rc = run_scan(m, w.scan, L.scan, m->slabs, ns, L.slabs2, R, qt, f32 ? L.ctx_f : nullptr, po.packed);
        else if (!rc) rc = latent_attention(m, w, L.cache[run], m->slabs, ns, R, n_tiles, qt, po.packed);
        if (rc) return rc;
        int no = 1, nd = 1;
        BranchSum ff;
        if (w.experts.on()) {
            const bool two = gathers && L.cfg.one_norm && !same;  // the mixer's planes serve the shared expert and the router
            rc = run_experts(m, w.experts, L.experts, two ? m->xh : ffh, two ? m->xl : ffl, two ? pq.packed : pg.packed, ffh, ffl, f32 ? y_ff : nullptr, R, L.slabs2, &ff);
            if (rc) return rc;
        }
        if (w.ff) {
            if (f32) {
                rc = exact_product(m, y_ff, w.gu, m->slabs, R);
                if (rc) return rc;
                PROF(m, PROF_SILU, launch_silu_mul_interleaved(m->slabs, 1, 0, R, w.ff_p, nullptr, nullptr, 0, s, spec, L.act_f));
                rc = exact_product(m, L.act_f, w.down, L.slabs2, R);
            } else {
                rc = run_glu(m, pg, ffh, ffl, w.gu, R, spec, m->xh2, m->xl2, pd.packed);
                if (!rc) rc = run_product(m, pd, m->xh2, m->xl2, w.down, L.slabs2, R, &nd);
            }
            if (rc) return rc;
            ff.in = L.slabs2; ff.n_slabs = nd; ff.slab_stride = (int64_t)R * L.ldr;
        }
        rc = f32 ? exact_product(m, L.ctx_f, w.o, m->slabs, R) : run_product(m, po, m->ctxh, m->ctxl, w.o, m->slabs, R, &no);
        if (rc) return rc;
        base.ids = nullptr;
        base.in = m->slabs; base.n_slabs = no; base.slab_stride = (int64_t)R * L.ldr;
        base.in2 = ff.in; base.n_slabs2 = ff.n_slabs; base.slab_stride2 = ff.slab_stride; base.in2_scale = ff.scale;
        base.gather = ff.gather; base.gather_row = ff.gather_row; base.n_gather = ff.n_gather;
        base.residual_in = m->resid;
        if (tp) {  // both branches of the layer in one all-reduce
            AddNormArgs sum = base;
            sum.residual_in = nullptr; sum.residual_out = m->red;
            HIPCHK(ctx, launch_add_norm(sum, R, s));
            rc = comm_allreduce_sum(ctx, m->red, (size_t)R * L.ldr);
            if (rc) return rc;
            base.in = m->red; base.n_slabs = 1; base.in2 = nullptr; base.n_gather = 0;
        }
        if (m->taps) {  // residual stream after this run
            AddNormArgs t = base;
            t.residual_out = L.tap;
            HIPCHK(ctx, launch_add_norm(t, R, s));
            HIPCHK(ctx, hipMemcpy2DAsync(m->tap_res + run * (size_t)m->max_rows * m->H, (size_t)m->H * 4, L.tap, (size_t)L.ldr * 4, (size_t)m->H * 4, R,
                                         hipMemcpyDeviceToDevice, s));
        }
    }
    if (n_last <= 0) return NVLLM_OK;
    AddNormArgs nf = base;
    nf.row_idx = m->d_last_rows;
    nf.w[0] = L.final_norm;
    if (f32) nf.y[0] = L.y1; else { nf.xh[0] = m->xh; nf.xl[0] = m->xl; }
    PROF(m, PROF_NORM, launch_add_norm(nf, n_last, s));
    return output_head(m, L.head, L.Kw, L.Vp, f32 ? L.y1 : nullptr, (float)L.cfg.logit_softcap, n_last, logits_row0);
}
