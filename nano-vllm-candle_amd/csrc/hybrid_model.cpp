// Hybrid decoders behind the C ABI: every layer has one of three token mixers -- grouped-query attention with a distance bias, a
// recurrence with constant decays, or a gated delta rule -- and optionally a feed-forward; the sublayers read the residual stream
// itself and are normed on their output:  x <- x + m norm1(mixer(x)),  x <- x + m norm2(ff(x)).
// Keys and values live in the paged cache, recurrent state and convolution history in the sequence's slot (f32).
// Mixed precision (the serving mode): products run on bf16 hi + lo planes with f32 accumulation, the cache is f16; residual, norms,
// scores, gates and recurrences are f32.  32-bit mode: every product and the cache in f32.
#include <algorithm>
#include <cmath>
#include <cstdio>

#include "decoder.h"
#include "hybrid.h"

struct HybridLayer {
    nvllm_hybrid_layer c{};
    int heads = 0, kv = 0, ff = 0;               // this rank's share
    int dim_p = 0, vdim_p = 0, ff_p = 0, rank_p = 0;
    int N = 0, Kc = 0, Ng = 0;                   // rows of the input projection (padded), context width (padded), rows of one gate matrix
    bool matrix_core = false;                    // attention: sizes have an instance
    bool last_v = false;                         // attention with value mixing: not the first such layer
    PackedW in, o, up, down, gates;              // gates: decay, then output gate, [Ng x rank_p] each
    float *norm1 = nullptr, *norm2 = nullptr;    // stored weight + norm_offset
    float *bias = nullptr, *qn = nullptr, *kn = nullptr, *table = nullptr, *vmix = nullptr;           // attention
    float *decay = nullptr, *onorm = nullptr;                                                         // recurrences
    float *conv = nullptr, *rate = nullptr, *dt = nullptr;                                            // delta rule
    int n_bias = 0;
    std::vector<int> bucket;                     // bias table row of every distance below n_bias
    void *kc = nullptr, *vc = nullptr;           // cache
    float *state = nullptr, *history = nullptr;  // per slot
    int channels() const { return 2 * kv * c.dim + heads * c.vdim; }
    bool attention() const { return c.mixer == NVLLM_MIXER_ATTENTION; }
    bool delta() const { return c.mixer == NVLLM_MIXER_DELTA; }
};

struct HybridModel : DecoderImpl {
    nvllm_hybrid_config cfg{};
    std::vector<HybridLayer> layers;
    int ldr = 0, Kw = 0, Vp = 0;       // residual stride, width padded for the products, padded vocabulary rows of the head
    bool has_state = false;
    bf16_bits* embed = nullptr;        // [vocab][ldr]
    PackedW head;
    float* final_norm = nullptr;
    // step buffers
    float *q = nullptr, *k = nullptr, *v = nullptr, *g = nullptr, *beta = nullptr, *gate_in = nullptr, *out = nullptr, *v_first = nullptr, *ssq = nullptr;
    float *part_o = nullptr, *part_ml = nullptr;
    float *y = nullptr, *ctx_f = nullptr, *act_f = nullptr;  // 32-bit mode
    int *d_seg = nullptr, *h_seg = nullptr, n_seg = 0;       // first row, rows, slot, first piece of every segment of the chunk
    int *d_piece = nullptr, n_piece = 0, piece_cap = 0;      // first row, rows of every 16-token piece (staged behind h_seg)
    float *pc_pair = nullptr, *pc_q = nullptr, *pc_w = nullptr, *pc_k = nullptr, *pc_decay = nullptr;
    int opt_scan = 0;                                        // recurrences: token by token in prompt chunks too
    int opt_plain = 0;                                       // attention: the plain kernel instead of the matrix-core ones

    ~HybridModel() override;
    int load_tensor(nvllm_model* m, const char* name, const void* data, int dtype, const int64_t* shape, int ndim) override;
    int finalize(nvllm_model* m) override;
    int kv_alloc(nvllm_model* m) override;
    void free_kv() override;
    int64_t weight_bytes() const override;
    int64_t kv_bytes_per_token() const override;
    int64_t kv_read_bytes(int len) const override;
    int tile_rows(int qt) const override { return qt == 1 ? 1 : kBiasTileRows; }
    bool recurrent() const override { return has_state; }
    int plan_chunk(nvllm_model* m, const int* pos, const int* slot, const int* seq, int R, const int* tile_row0, int n_tiles, int qt) override;
    int forward_chunk(nvllm_model* m, int R, int n_tiles, int qt, int n_last, int logits_row0) override;
    int option(const char* name, int value) override {
        if (!strcmp(name, "bias_attn_plain")) opt_plain = value;
        else if (!strcmp(name, "recur_scan")) opt_scan = value;
        else return 1;
        return 0;
    }
    int product(nvllm_model* m, const ProductPlan& p, const float* f, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, int R, int* ns) {
        *ns = 1;
        return cfg.f32 ? exact_product(m, f, w, m->slabs, R) : run_product(m, p, xh, xl, w, m->slabs, R, ns);
    }
    int attention(nvllm_model* m, HybridLayer& w, int ns, int R, int n_tiles, int qt, int ctx_packed);
    int recurrence(nvllm_model* m, HybridLayer& w, int ns, int R, int qt, int ctx_packed);
};

constexpr int kDecodeWgs = 512;  // workgroups the split of a decode step's context aims at

// row of the distance table
static int distance_bucket(int n, int rows, double far) {
    const int half = rows / 2;
    if (n < half) return n;
    if (half < 1 || far <= half) return rows - 1;
    // the exact quotient may be a whole number that the logarithms miss by a rounding
    const double f = std::log((double)n / half) / std::log(far / half) * (rows - half);
    return std::min(rows - 1, half + (int)std::floor(f + 1e-9));
}

extern "C" int nvllm_model_create_hybrid(nvllm_ctx* ctx, const nvllm_hybrid_config* cfg, const nvllm_hybrid_layer* layers, nvllm_model** out) {
    if (!ctx || !cfg || !layers || !out) return fail(ctx, NVLLM_EINVAL, "NULL argument");
    const nvllm_hybrid_config& c = *cfg;
    const int tp = ctx->tp_size;
    if (c.vocab_size < 1 || c.width < 1 || c.num_layers < 1) return fail(ctx, NVLLM_EINVAL, "config has non-positive sizes");
    if (c.width > 8192) return fail(ctx, NVLLM_EINVAL, "width %d unsupported (at most 8192)", c.width);
    if (c.vocab_size % tp) return fail(ctx, NVLLM_EINVAL, "vocabulary of %d not divisible by tp_size %d", c.vocab_size, tp);
    const nvllm_hybrid_layer* first_mix = nullptr;
    for (int l = 0; l < c.num_layers; ++l) {
        const nvllm_hybrid_layer& k = layers[l];
        if (k.heads < 1 || k.kv_heads < 1 || k.dim < 1 || k.vdim < 1 || k.ff < 0) return fail(ctx, NVLLM_EINVAL, "layer %d has non-positive sizes", l);
        if (k.heads % k.kv_heads) return fail(ctx, NVLLM_EINVAL, "layer %d: %d heads over %d key/value heads", l, k.heads, k.kv_heads);
        if (k.heads % tp || k.kv_heads % tp || k.ff % tp) return fail(ctx, NVLLM_EINVAL, "layer %d: heads %d / %d or feed-forward width %d not divisible by tp_size %d", l, k.heads, k.kv_heads, k.ff, tp);
        if (k.mixer == NVLLM_MIXER_ATTENTION) {
            if (k.dim > 4096 || k.vdim > 1024) return fail(ctx, NVLLM_EINVAL, "layer %d: head sizes %d / %d unsupported (at most 4096 / 1024)", l, k.dim, k.vdim);
            if ((k.heads / tp) * k.dim + (k.kv_heads / tp) * (k.dim + k.vdim) > 16000) return fail(ctx, NVLLM_EINVAL, "layer %d: more than 16000 query, key and value columns per rank", l);
            if (k.bias_rows < 0 || k.bias_rows > 1 << 20) return fail(ctx, NVLLM_EINVAL, "layer %d: %d rows of distance bias", l, k.bias_rows);
            if (k.v_mix && !first_mix) first_mix = &k;
            else if (k.v_mix && k.kv_heads * k.vdim != first_mix->kv_heads * first_mix->vdim)
                return fail(ctx, NVLLM_EINVAL, "layer %d mixes values of %d columns with the first mixing layer's %d", l, k.kv_heads * k.vdim, first_mix->kv_heads * first_mix->vdim);
        } else if (k.mixer == NVLLM_MIXER_LINEAR || k.mixer == NVLLM_MIXER_DELTA) {
            if (!recur_ok(k.dim, k.vdim)) return fail(ctx, NVLLM_EINVAL, "layer %d: head sizes %d / %d unsupported (key size at most 512)", l, k.dim, k.vdim);
            if (k.mixer == NVLLM_MIXER_LINEAR && (!k.decay || k.kv_heads != k.heads)) return fail(ctx, NVLLM_EINVAL, "layer %d: needs one decay and one key head per head", l);
            if (k.mixer == NVLLM_MIXER_DELTA && (k.conv_taps < 1 || k.conv_taps > 16 || k.decay_rank < 1 || k.gate_rank < 1))
                return fail(ctx, NVLLM_EINVAL, "layer %d: convolution of %d taps (1 to 16) or gate ranks %d / %d unsupported", l, k.conv_taps, k.decay_rank, k.gate_rank);
        } else {
            return fail(ctx, NVLLM_EINVAL, "layer %d: mixer %d unknown", l, k.mixer);
        }
    }
    HIPCHK(ctx, hipSetDevice(ctx->device));
    nvllm_model* m = new nvllm_model();
    m->ctx = ctx;
    auto owned = std::make_unique<HybridModel>();
    HybridModel& L = *owned;
    m->dec = std::move(owned);
    L.cfg = c;
    m->H = c.width; m->V_l = c.vocab_size / tp; m->kv_l = 1; m->L = c.num_layers;
    m->cfg.vocab_size = c.vocab_size; m->cfg.hidden_size = c.width; m->cfg.max_position_embeddings = 1 << 30;
    L.ldr = up(c.width, 16); L.Kw = up(c.width, 128); L.Vp = up(m->V_l, 16);
    auto alloc_w = [&](PackedW& w, int N, int K) -> int {
        w.N = N; w.K = K;
        HIPCHK(ctx, hipMalloc((void**)&w.data, w.bytes()));
        HIPCHK(ctx, hipMemsetAsync(w.data, 0, w.bytes(), ctx->stream));  // padding rows and columns stay zero
        return NVLLM_OK;
    };
    auto alloc_v = [&](float** p, int n) -> int {
        int rc = dmalloc(ctx, p, n);
        if (!rc) HIPCHK(ctx, hipMemsetAsync(*p, 0, (size_t)n * 4, ctx->stream));
        return rc;
    };
    int rc = dmalloc(ctx, &L.embed, (size_t)c.vocab_size * L.ldr);
    if (!rc) HIPCHK(ctx, hipMemsetAsync(L.embed, 0, (size_t)c.vocab_size * L.ldr * 2, ctx->stream));
    if (!rc) rc = alloc_w(L.head, L.Vp, L.Kw);
    if (!rc) rc = alloc_v(&L.final_norm, L.Kw);
    L.layers.resize(c.num_layers);
    bool mixes = false;
    for (int l = 0; l < c.num_layers && !rc; ++l) {
        HybridLayer& w = L.layers[l];
        w.c = layers[l];
        w.c.decay = nullptr;  // the caller's array is not kept
        const int D = w.c.dim, E = w.c.vdim;
        w.heads = w.c.heads / tp; w.kv = w.c.kv_heads / tp; w.ff = w.c.ff / tp; w.ff_p = up(w.ff, 128);
        w.Kc = up(w.heads * E, 128);
        int n = 0;
        if (w.attention()) {
            w.matrix_core = !c.f32 && bias_attn_dim(D) && bias_attn_vdim(E);
            w.dim_p = w.matrix_core ? bias_attn_dim(D) : up(D, 32);
            w.vdim_p = w.matrix_core ? bias_attn_vdim(E) : up(E, 16);
            w.last_v = w.c.v_mix && mixes;
            mixes |= w.c.v_mix != 0;
            n = w.heads * D + w.kv * (D + E);
            const int B = w.c.bias_rows;
            if (B) {
                do w.bucket.push_back(distance_bucket((int)w.bucket.size(), B, w.c.bias_max)); while (w.bucket.back() < B - 1 && w.bucket.size() < (1u << 24));
                w.n_bias = (int)w.bucket.size();
            }
        } else {
            L.has_state = true;
            w.dim_p = recur_dim(D);
            w.vdim_p = recur_vdim(E);
            if (w.delta()) {
                w.rank_p = std::max(up(w.c.decay_rank, 32), up(w.c.gate_rank, 32));
                w.Ng = w.heads * std::max(w.dim_p, w.vdim_p);
                n = w.channels() + w.heads + 2 * w.rank_p;
            } else {
                n = 2 * w.heads * (D + E);
            }
        }
        // wide projections: a whole number of the prompt product's 192- or 256-feature tiles
        w.N = n >= 1536 && !c.f32 ? std::min(up(n, 192), up(n, 256)) : up(n, 16);
        rc = alloc_w(w.in, w.N, L.Kw);
        if (!rc) rc = alloc_w(w.o, L.ldr, w.Kc);
        if (!rc) rc = alloc_v(&w.norm1, L.Kw);
        if (w.ff) {
            if (!rc) rc = alloc_w(w.up, w.ff_p, L.Kw);
            if (!rc) rc = alloc_w(w.down, L.ldr, w.ff_p);
            if (!rc) rc = alloc_v(&w.norm2, L.Kw);
        }
        if (w.attention()) {
            if (!rc) rc = alloc_v(&w.bias, w.N);
            if (!rc) rc = alloc_v(&w.qn, w.heads * D);
            if (!rc) rc = alloc_v(&w.kn, w.kv * D);
            if (!rc) rc = alloc_v(&w.vmix, 1);
            if (!rc) rc = alloc_v(&w.table, std::max(1, w.heads * w.n_bias));
        } else {
            if (!rc) rc = alloc_v(&w.onorm, w.delta() ? E : w.heads * E);
            if (w.delta()) {
                if (!rc) rc = alloc_w(w.gates, 2 * w.Ng, w.rank_p);
                if (!rc) rc = alloc_v(&w.conv, w.c.conv_taps * w.channels());
                if (!rc) rc = alloc_v(&w.rate, w.Ng);
                if (!rc) rc = alloc_v(&w.dt, w.Ng);
            } else {
                std::vector<float> d(w.heads);
                for (int h = 0; h < w.heads; ++h) d[h] = (float)layers[l].decay[ctx->tp_rank * w.heads + h];
                if (!rc) rc = alloc_v(&w.decay, w.heads);
                if (!rc && hipMemcpyAsync(w.decay, d.data(), d.size() * 4, hipMemcpyHostToDevice, ctx->stream) != hipSuccess) rc = fail(ctx, NVLLM_EHIP, "decay upload failed");
                if (!rc && hipStreamSynchronize(ctx->stream) != hipSuccess) rc = fail(ctx, NVLLM_EHIP, "decay upload failed");
            }
        }
    }
    if (!rc && hipStreamSynchronize(ctx->stream) != hipSuccess) rc = fail(ctx, NVLLM_EHIP, "weight allocation failed");
    if (rc) { nvllm_model_destroy(m); return rc; }
    *out = m;
    return NVLLM_OK;
}

void HybridModel::free_kv() {
    for (HybridLayer& w : layers) {
        for (void* p : {w.kc, w.vc, (void*)w.state, (void*)w.history}) if (p) (void)hipFree(p);
        w.kc = w.vc = nullptr;
        w.state = w.history = nullptr;
    }
    for (float** p : {&q, &k, &v, &g, &beta, &gate_in, &out, &v_first, &ssq, &part_o, &part_ml, &y, &ctx_f, &act_f, &pc_pair, &pc_q, &pc_w, &pc_k, &pc_decay}) {
        if (*p) (void)hipFree(*p);
        *p = nullptr;
    }
    if (d_seg) (void)hipFree(d_seg);
    if (h_seg) (void)hipHostFree(h_seg);
    if (d_piece) (void)hipFree(d_piece);
    d_seg = h_seg = d_piece = nullptr;
    n_seg = n_piece = 0;
}

HybridModel::~HybridModel() {
    free_kv();
    (void)hipFree(embed); (void)hipFree(head.data); (void)hipFree(final_norm);
    for (HybridLayer& w : layers) {
        for (PackedW* p : {&w.in, &w.o, &w.up, &w.down, &w.gates}) (void)hipFree(p->data);
        for (float* p : {w.norm1, w.norm2, w.bias, w.qn, w.kn, w.table, w.vmix, w.decay, w.onorm, w.conv, w.rate, w.dt}) (void)hipFree(p);
    }
}

// ---------------------------------------------------------------------------------------------------
// weights
// ---------------------------------------------------------------------------------------------------
static const char* const kAttnTensors[] = {"q", "q.b", "k", "k.b", "v", "v.b", "q.norm", "k.norm", "o"};
static const char* const kLinearTensors[] = {"q", "k", "v", "g", "norm", "o"};
static const char* const kDeltaTensors[] = {"q", "q.conv", "k", "k.conv", "v", "v.conv", "b", "A_log", "a1", "a2", "dt_bias", "g1", "g2", "norm", "o"};

int HybridModel::load_tensor(nvllm_model* m, const char* name, const void* data, int dtype, const int64_t* shape, int ndim) {
    nvllm_ctx* ctx = m->ctx;
    const int rank = ctx->tp_rank;
    if (ndim < 0 || ndim > 2) return fail(ctx, NVLLM_EINVAL, "tensor '%s' has %d dimensions", name, ndim);
    const int64_t rows = ndim == 2 ? shape[0] : 1, cols = ndim ? shape[ndim - 1] : 1;
    const HostMat h{data, dtype, cols};
    HIPCHK(ctx, hipSetDevice(ctx->device));
    auto want = [&](int64_t r, int64_t c, int nd) -> int {
        if (rows == r && cols == c && (ndim == nd || (nd == 0 && ndim == 1))) return NVLLM_OK;
        return fail(ctx, NVLLM_EINVAL, "tensor '%s': shape mismatch (got %lld x %lld, want %lld x %lld)", name, (long long)rows, (long long)cols, (long long)r, (long long)c);
    };
    auto put = [&](float* dst, const std::vector<float>& t) -> int {
        HIPCHK(ctx, hipMemcpy(dst, t.data(), t.size() * 4, hipMemcpyHostToDevice));
        return NVLLM_OK;
    };
    // n elements of a vector of `all`, from `first` on, plus an offset
    auto vec = [&](float* dst, int64_t all, int64_t first, int n, float offset) -> int {
        int rc = want(1, all, 1);
        if (rc) return rc;
        std::vector<float> t(n);
        for (int i = 0; i < n; ++i) t[i] = h.f32(first + i) + offset;
        return put(dst, t);
    };
    const int W = cfg.width, V = cfg.vocab_size;
    const float off1 = (float)cfg.norm_offset;
    int rc = NVLLM_OK, l = -1, off = 0;
    if (!strcmp(name, "embed")) {
        if ((rc = want(V, W, 2))) return rc;
        std::vector<uint16_t> t((size_t)V * ldr, 0);
        for (int r = 0; r < V; ++r) for (int c = 0; c < W; ++c) t[(size_t)r * ldr + c] = h.at(r, c);
        HIPCHK(ctx, hipMemcpy(embed, t.data(), t.size() * 2, hipMemcpyHostToDevice));
    } else if (!strcmp(name, "head")) {
        if ((rc = want(V, W, 2))) return rc;
        const int64_t r0 = (int64_t)rank * m->V_l;
        if ((rc = put_rows(ctx, head, 0, m->V_l, W, -1, [&](int r, int c) { return h.at(r0 + r, c); }))) return rc;
    } else if (!strcmp(name, "final.norm")) {
        if ((rc = vec(final_norm, W, 0, W, off1))) return rc;
    } else {
        if (sscanf(name, "l%d.%n", &l, &off) != 1 || off == 0 || l < 0 || l >= cfg.num_layers) return fail(ctx, NVLLM_EINVAL, "unknown tensor name '%s'", name);
        const char* s = name + off;
        HybridLayer& w = layers[l];
        const int D = w.c.dim, E = w.c.vdim, Hl = w.heads, Gl = w.kv, H = w.c.heads, G = w.c.kv_heads, ff = w.c.ff;
        const int64_t h0 = (int64_t)rank * Hl, g0 = (int64_t)rank * Gl, f0 = (int64_t)rank * w.ff;
        const std::string unknown = std::string("unknown tensor name '") + name + "'";
        // `n` rows per rank of the input projection from its row `at` on, out of `all`
        auto proj = [&](int at, int64_t all, int n) -> int {
            const int64_t r0 = all == n ? 0 : (int64_t)rank * n;
            int e = want(all, W, 2);
            return e ? e : put_rows(ctx, w.in, at, n, W, -1, [&](int r, int c) { return h.at(r0 + r, c); });
        };
        if (!strcmp(s, "norm1")) rc = vec(w.norm1, W, 0, W, off1);
        else if (ff && !strcmp(s, "norm2")) rc = vec(w.norm2, W, 0, W, off1);
        else if (ff && !strcmp(s, "mlp.up")) {
            if (!(rc = want(ff, W, 2))) rc = put_rows(ctx, w.up, 0, w.ff, W, -1, [&](int r, int c) { return h.at(f0 + r, c); });
        } else if (ff && !strcmp(s, "mlp.down")) {
            if (!(rc = want(W, ff, 2))) rc = put_rows(ctx, w.down, 0, W, w.ff, -1, [&](int r, int c) { return h.at(r, f0 + c); });
        } else if (strncmp(s, "mix.", 4)) return fail(ctx, NVLLM_EINVAL, "%s", unknown.c_str());
        else if (s += 4, !strcmp(s, "o")) {
            if (!(rc = want(W, (int64_t)H * E, 2))) rc = put_rows(ctx, w.o, 0, W, Hl * E, -1, [&](int r, int c) { return h.at(r, h0 * E + c); });
        } else if (w.attention()) {
            const int q0 = 0, k0 = Hl * D, v0 = k0 + Gl * D;
            if (!strcmp(s, "q")) rc = proj(q0, (int64_t)H * D, Hl * D);
            else if (!strcmp(s, "k")) rc = proj(k0, (int64_t)G * D, Gl * D);
            else if (!strcmp(s, "v")) rc = proj(v0, (int64_t)G * E, Gl * E);
            else if (!strcmp(s, "q.b")) rc = vec(w.bias + q0, (int64_t)H * D, h0 * D, Hl * D, 0.f);
            else if (!strcmp(s, "k.b")) rc = vec(w.bias + k0, (int64_t)G * D, g0 * D, Gl * D, 0.f);
            else if (!strcmp(s, "v.b")) rc = vec(w.bias + v0, (int64_t)G * E, g0 * E, Gl * E, 0.f);
            else if (!strcmp(s, "q.norm")) rc = vec(w.qn, (int64_t)H * D, h0 * D, Hl * D, 0.f);
            else if (!strcmp(s, "k.norm")) rc = vec(w.kn, (int64_t)G * D, g0 * D, Gl * D, 0.f);
            else if (w.c.bias_rows && !strcmp(s, "rel")) {
                if (!(rc = want(w.c.bias_rows, H, 2))) {
                    std::vector<float> t((size_t)Hl * w.n_bias);
                    for (int n = 0; n < Hl; ++n)
                        for (int d = 0; d < w.n_bias; ++d) t[(size_t)n * w.n_bias + d] = (float)(h.f32((int64_t)w.bucket[d] * H + h0 + n) * 1.4426950408889634);
                    rc = put(w.table, t);
                }
            } else if (!strcmp(s, "vmix")) {  // unused where nothing is mixed
                if (!(rc = want(1, 1, 0))) rc = put(w.vmix, {h.f32(0)});
            } else return fail(ctx, NVLLM_EINVAL, "%s", unknown.c_str());
        } else if (!w.delta()) {
            const int HD = Hl * D, HE = Hl * E;
            if (!strcmp(s, "q")) rc = proj(0, (int64_t)H * D, HD);
            else if (!strcmp(s, "k")) rc = proj(HD, (int64_t)H * D, HD);
            else if (!strcmp(s, "v")) rc = proj(2 * HD, (int64_t)H * E, HE);
            else if (!strcmp(s, "g")) rc = proj(2 * HD + HE, (int64_t)H * E, HE);
            else if (!strcmp(s, "norm")) rc = vec(w.onorm, (int64_t)H * E, h0 * E, HE, 0.f);
            else return fail(ctx, NVLLM_EINVAL, "%s", unknown.c_str());
        } else {
            const int GD = Gl * D, HE = Hl * E, C = w.channels(), ra = w.c.decay_rank, rg = w.c.gate_rank;
            auto conv = [&](int at, int64_t all, int n) -> int {  // [channels, taps] -> [taps][channels]
                int e = want(all, w.c.conv_taps, 2);
                if (e) return e;
                std::vector<float> t(n);
                for (int i = 0; i < w.c.conv_taps && !e; ++i) {
                    for (int r = 0; r < n; ++r) t[r] = h.f32(((int64_t)rank * n + r) * cols + i);
                    e = put(w.conv + (size_t)i * C + at, t);
                }
                return e;
            };
            auto gate = [&](int at, int size, int size_p, int r) -> int {  // rows head * size + i -> head * size_p + i
                int e = want((int64_t)H * size, r, 2);
                return e ? e : put_rows(ctx, w.gates, at, Hl * size_p, r, -1, [&](int row, int c) -> uint16_t {
                    const int n = row / size_p, i = row % size_p;
                    return i < size ? h.at((h0 + n) * size + i, c) : (uint16_t)0;
                });
            };
            if (!strcmp(s, "q")) rc = proj(0, (int64_t)G * D, GD);
            else if (!strcmp(s, "k")) rc = proj(GD, (int64_t)G * D, GD);
            else if (!strcmp(s, "v")) rc = proj(2 * GD, (int64_t)H * E, HE);
            else if (!strcmp(s, "b")) rc = proj(C, H, Hl);
            else if (!strcmp(s, "a1")) rc = proj(C + Hl, ra, ra);
            else if (!strcmp(s, "g1")) rc = proj(C + Hl + w.rank_p, rg, rg);
            else if (!strcmp(s, "q.conv")) rc = conv(0, (int64_t)G * D, GD);
            else if (!strcmp(s, "k.conv")) rc = conv(GD, (int64_t)G * D, GD);
            else if (!strcmp(s, "v.conv")) rc = conv(2 * GD, (int64_t)H * E, HE);
            else if (!strcmp(s, "a2")) rc = gate(0, D, w.dim_p, ra);
            else if (!strcmp(s, "g2")) rc = gate(w.Ng, E, w.vdim_p, rg);
            else if (!strcmp(s, "norm")) rc = vec(w.onorm, E, 0, E, 0.f);
            else if (!strcmp(s, "A_log")) {
                if (!(rc = want(1, H, 1))) {
                    std::vector<float> t(w.Ng, 0.f);
                    for (int i = 0; i < Hl * w.dim_p; ++i) t[i] = std::exp(h.f32(h0 + i / w.dim_p));
                    rc = put(w.rate, t);
                }
            } else if (!strcmp(s, "dt_bias")) {
                if (!(rc = want(1, (int64_t)H * D, 1))) {
                    std::vector<float> t(w.Ng, 0.f);
                    for (int i = 0; i < Hl * w.dim_p; ++i) if (i % w.dim_p < D) t[i] = h.f32((h0 + i / w.dim_p) * D + i % w.dim_p);
                    rc = put(w.dt, t);
                }
            } else return fail(ctx, NVLLM_EINVAL, "%s", unknown.c_str());
        }
        if (rc) return rc;
    }
    m->loaded[name] = true;
    return NVLLM_OK;
}

int HybridModel::finalize(nvllm_model* m) {
    nvllm_ctx* ctx = m->ctx;
    auto need = [&](const std::string& s) { return m->loaded.count(s) ? NVLLM_OK : fail(ctx, NVLLM_ESTATE, "missing tensor %s", s.c_str()); };
    int rc = NVLLM_OK;
    for (const char* s : {"embed", "head", "final.norm"}) if (!rc) rc = need(s);
    for (int l = 0; l < cfg.num_layers && !rc; ++l) {
        const HybridLayer& w = layers[l];
        const std::string p = "l" + std::to_string(l) + ".";
        rc = need(p + "norm1");
        if (w.attention()) {
            for (const char* s : kAttnTensors) if (!rc) rc = need(p + "mix." + s);
            if (!rc && w.c.bias_rows) rc = need(p + "mix.rel");
            if (!rc && w.last_v) rc = need(p + "mix.vmix");
        } else if (w.delta()) {
            for (const char* s : kDeltaTensors) if (!rc) rc = need(p + "mix." + s);
        } else {
            for (const char* s : kLinearTensors) if (!rc) rc = need(p + "mix." + s);
        }
        if (w.ff) for (const char* s : {"norm2", "mlp.up", "mlp.down"}) if (!rc) rc = need(p + s);
    }
    if (!rc) m->finalized = true;
    return rc;
}

int64_t HybridModel::weight_bytes() const {
    int64_t b = (int64_t)head.bytes() + (int64_t)cfg.width * 4;
    for (const HybridLayer& w : layers)
        b += (int64_t)(w.in.bytes() + w.o.bytes() + w.up.bytes() + w.down.bytes() + w.gates.bytes()) + (int64_t)(w.ff ? 2 : 1) * cfg.width * 4;
    return b;
}
int64_t HybridModel::kv_bytes_per_token() const {
    int64_t b = 0;
    for (const HybridLayer& w : layers)
        if (w.attention()) b += (int64_t)w.kv * (w.dim_p + w.vdim_p) * (cfg.f32 ? 4 : 2);
    return b;
}
int64_t HybridModel::kv_read_bytes(int len) const {
    int64_t b = kv_bytes_per_token() * len;
    for (const HybridLayer& w : layers)
        if (!w.attention()) {
            b += (int64_t)recur_state_floats(w.heads, w.dim_p, w.vdim_p) * 8;  // read and written
            if (w.delta()) b += (int64_t)(w.c.conv_taps - 1) * w.channels() * 8;
        }
    return b;
}

// ---------------------------------------------------------------------------------------------------
// cache, state and step buffers (pool sizes are set, the shared buffers exist)
// ---------------------------------------------------------------------------------------------------
int HybridModel::kv_alloc(nvllm_model* m) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    const bool f32 = cfg.f32 != 0;
    const size_t R = m->max_rows, R16 = (R + 15) / 16 * 16;
    auto zalloc = [&](void** p, size_t bytes) -> int {
        HIPCHK(ctx, hipMalloc(p, std::max<size_t>(bytes, 16)));
        HIPCHK(ctx, hipMemsetAsync(*p, 0, std::max<size_t>(bytes, 16), s));
        return NVLLM_OK;
    };
    int rc = NVLLM_OK;
    size_t nmax = ldr, kc = 0, ffp = 0, nq = 0, nk = 0, nv = 0, ng = 0, nb = 0, nin = 0, no = 0, nvf = 0, po = 0, pm = 0;
    for (HybridLayer& w : layers) {
        nmax = std::max<size_t>({nmax, (size_t)w.N, (size_t)w.ff_p});
        kc = std::max<size_t>(kc, w.Kc);
        ffp = std::max<size_t>(ffp, w.ff_p);
        nq = std::max<size_t>(nq, (size_t)w.heads * w.dim_p);
        if (w.attention()) {
            // padding stays zero, unwritten tokens finite
            const size_t toks = (size_t)m->num_blocks * kBlockTokens * w.kv * (f32 ? 4 : 2);
            if (!rc) rc = zalloc(&w.kc, toks * w.dim_p);
            if (!rc) rc = zalloc(&w.vc, toks * w.vdim_p);
            if (w.c.v_mix) nvf = std::max<size_t>(nvf, (size_t)w.kv * w.c.vdim);
            po = std::max<size_t>(po, (size_t)kDecodeWgs * 16 * w.vdim_p);
            pm = (size_t)kDecodeWgs * 16 * 2;
        } else {
            nk = std::max<size_t>(nk, (size_t)w.heads * w.dim_p);
            nv = std::max<size_t>(nv, (size_t)w.heads * w.vdim_p);
            ng = std::max<size_t>(ng, w.delta() ? (size_t)2 * w.Ng : (size_t)w.heads * w.vdim_p);
            nb = std::max<size_t>(nb, w.heads);
            nin = std::max<size_t>(nin, (size_t)2 * w.rank_p);
            no = std::max<size_t>(no, (size_t)w.heads * w.vdim_p);
            if (!rc) rc = zalloc((void**)&w.state, (size_t)m->max_seqs * recur_state_floats(w.heads, w.dim_p, w.vdim_p) * 4);
            if (!rc && w.delta() && w.c.conv_taps > 1) rc = zalloc((void**)&w.history, (size_t)2 * m->max_seqs * (w.c.conv_taps - 1) * w.channels() * 4);
        }
    }
    m->slab_floats = std::max<size_t>(R * nmax, (size_t)32 * std::min<size_t>(R, 128) * nmax);
    if (f32 || m->V_l % 16) m->slab_floats = std::max<size_t>(m->slab_floats, (size_t)m->max_seqs * Vp);
    if (!rc) rc = zalloc((void**)&m->resid, R * ldr * 4);
    if (!rc) rc = dmalloc(ctx, &m->slabs, m->slab_floats);
    if (!rc) rc = dmalloc(ctx, &m->red, R * ldr);
    struct { float** p; size_t n; } bufs[] = {{&q, nq}, {&k, nk}, {&v, nv}, {&g, ng}, {&beta, nb}, {&gate_in, nin}, {&out, no}, {&v_first, nvf}};
    for (auto& b : bufs) if (!rc && b.n) rc = zalloc((void**)b.p, (R + kPiece) * b.n * 4);  // pieces read past the last row
    if (!rc) rc = dmalloc(ctx, &ssq, R * 2);
    if (!rc && po && !f32) rc = dmalloc(ctx, &part_o, po);
    if (!rc && pm && !f32) rc = dmalloc(ctx, &part_ml, pm);
    if (f32) {
        if (!rc) rc = zalloc((void**)&y, R * Kw * 4);
        if (!rc) rc = zalloc((void**)&ctx_f, R * kc * 4);
        if (!rc && ffp) rc = zalloc((void**)&act_f, R * ffp * 4);
    } else {
        // activation planes are read in whole 16-row blocks; columns past a layer's own width meet zero weights
        for (bf16_bits** p : {&m->xh, &m->xl}) if (!rc) rc = zalloc((void**)p, R16 * Kw * 2);
        for (bf16_bits** p : {&m->ctxh, &m->ctxl}) if (!rc) rc = zalloc((void**)p, R16 * kc * 2);
        if (ffp) for (bf16_bits** p : {&m->xh2, &m->xl2}) if (!rc) rc = zalloc((void**)p, R16 * ffp * 2);
    }
    piece_cap = (int)(R / kPiece) + m->max_seqs;
    size_t ph = 0, pd = 0, pdd = 0;  // heads, channels of the layers that run in pieces, channels of the delta rule's alone
    for (const HybridLayer& w : layers)
        if (!w.attention() && piece_scan_ok(w.dim_p)) {
            ph = std::max<size_t>(ph, w.heads);
            pd = std::max<size_t>(pd, (size_t)w.heads * w.dim_p);
            if (w.delta()) pdd = std::max<size_t>(pdd, (size_t)w.heads * w.dim_p);
        }
    struct { float** p; size_t n; } pieces[] = {{&pc_pair, ph * kPiece * kPiece}, {&pc_k, pd * kPiece}, {&pc_q, pdd * kPiece}, {&pc_w, pdd * kPiece}, {&pc_decay, pdd}};
    for (auto& b : pieces) if (!rc && b.n) rc = dmalloc(ctx, b.p, (size_t)piece_cap * b.n);
    if (!rc) rc = dmalloc(ctx, &d_seg, (size_t)4 * m->max_seqs);
    if (!rc) rc = dmalloc(ctx, &d_piece, (size_t)2 * piece_cap);
    if (!rc) HIPCHK(ctx, hipHostMalloc((void**)&h_seg, ((size_t)4 * m->max_seqs + 2 * piece_cap) * sizeof(int), hipHostMallocDefault));
    m->rope_len = (int)std::min<int64_t>((int64_t)m->max_blocks * kBlockTokens, 1 << 20);  // positions a block table covers
    return rc;
}

// ---------------------------------------------------------------------------------------------------
// forward over one chunk of rows
// ---------------------------------------------------------------------------------------------------
int HybridModel::plan_chunk(nvllm_model* m, const int*, const int* slot, const int* seq, int R, const int*, int, int qt) {
    nvllm_ctx* ctx = m->ctx;
    n_seg = n_piece = 0;
    if (qt == 1) return NVLLM_OK;
    const int cap = m->max_seqs;
    int *h_piece0 = h_seg + 3 * cap, *h_row0 = h_seg + 4 * cap, *h_n = h_row0 + piece_cap;
    for (int r = 0; r < R; ++n_seg) {
        int e = r;
        while (e < R && seq[e] == seq[r]) ++e;
        h_seg[n_seg] = r; h_seg[cap + n_seg] = e - r; h_seg[2 * cap + n_seg] = slot[r];
        h_piece0[n_seg] = n_piece;
        for (; r < e; r += kPiece, ++n_piece) { h_row0[n_piece] = r; h_n[n_piece] = std::min(kPiece, e - r); }
        r = e;
    }
    // the staging buffer is free: the tile upload before this call waited for the stream
    HIPCHK(ctx, hipMemcpyAsync(d_seg, h_seg, (size_t)4 * cap * sizeof(int), hipMemcpyHostToDevice, ctx->stream));
    HIPCHK(ctx, hipMemcpyAsync(d_piece, h_row0, (size_t)2 * piece_cap * sizeof(int), hipMemcpyHostToDevice, ctx->stream));
    return NVLLM_OK;
}

int HybridModel::attention(nvllm_model* m, HybridLayer& w, int ns, int R, int n_tiles, int qt, int ctx_packed) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    AttnRowsArgs ra;
    ra.in = m->slabs; ra.n_slabs = ns; ra.ld = w.N; ra.slab_stride = (int64_t)R * w.N; ra.bias = w.bias;
    ra.heads = w.heads; ra.qn = w.qn; ra.kn = w.kn; ra.eps = (float)cfg.norm_eps; ra.q_scale = (float)(w.c.scale * 1.4426950408889634);
    ra.q_all = w.c.heads * w.c.dim; ra.k_all = w.c.kv_heads * w.c.dim;
    ra.mix = w.c.v_mix ? (w.last_v ? 2 : 1) : 0; ra.lambda = w.vmix; ra.v_first = v_first;
    ra.pos = m->d_pos; ra.slot = m->d_slot; ra.block_tables = m->d_block_tables; ra.max_blocks = m->max_blocks; ra.q = q;
    ra.kv.k = w.kc; ra.kv.v = w.vc; ra.kv.f32 = cfg.f32; ra.kv.kv = w.kv;
    ra.kv.dim = w.c.dim; ra.kv.dim_p = w.dim_p; ra.kv.vdim = w.c.vdim; ra.kv.vdim_p = w.vdim_p;
    if (ctx->tp_size > 1) {  // the norms run over every rank's columns
        const int c0[2] = {0, w.heads * w.c.dim}, n[2] = {w.heads * w.c.dim, w.kv * w.c.dim};
        HIPCHK(ctx, launch_rows_ssq(m->slabs, ns, ra.slab_stride, w.N, w.bias, c0, n, R, ssq, s));
        int rc = comm_allreduce_sum(ctx, ssq, (size_t)R * 2);
        if (rc) return rc;
        ra.ssq = ssq;
    }
    PROF(m, PROF_QK, launch_attn_rows(ra, R, s));
    BiasAttnArgs aa;
    aa.q = q; aa.kv = ra.kv; aa.heads = w.heads; aa.bias = w.table; aa.n_bias = w.n_bias; aa.sink = w.c.sink;
    aa.block_tables = m->d_block_tables; aa.max_blocks = m->max_blocks;
    aa.tile_row0 = m->d_tile_row0; aa.tile_nrows = m->d_tile_nrows; aa.tile_slot = m->d_tile_slot; aa.tile_order = m->d_tile_order;
    aa.pos = m->d_pos; aa.slot = m->d_slot; aa.ld = w.Kc; aa.packed = ctx_packed;
    if (cfg.f32) aa.of = ctx_f;
    else { aa.oh = m->ctxh; aa.ol = m->ctxl; }
    if (!w.matrix_core || opt_plain) {
        PROF(m, PROF_ATTN, launch_bias_attn_plain(aa, R, s));
    } else if (qt == 1) {
        // split the context when (sequences x groups of heads) alone leave CUs idle
        const int gqa = w.heads / w.kv, base = R * w.kv * ((gqa + 15) / 16), tiles = (m->cur_max_len + 31) / 32;
        const int want = std::max(1, std::min(kBiasMaxParts, kDecodeWgs / base));
        aa.part_tiles = 4 * ((tiles + 4 * want - 1) / (4 * want));
        const int parts = (tiles + aa.part_tiles - 1) / aa.part_tiles;
        aa.max_parts = parts; aa.part_o = part_o; aa.part_ml = part_ml;
        PROF(m, PROF_ATTN, launch_bias_decode(aa, R, parts, s));
    } else {
        PROF(m, PROF_ATTN, launch_bias_prefill(aa, n_tiles, s));
    }
    return NVLLM_OK;
}

int HybridModel::recurrence(nvllm_model* m, HybridLayer& w, int ns, int R, int qt, int ctx_packed) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    Segments seg;
    seg.single = qt == 1;
    seg.count = seg.single ? R : n_seg;
    seg.row0 = d_seg; seg.n = d_seg + m->max_seqs; seg.slot = seg.single ? m->d_slot : d_seg + 2 * m->max_seqs;
    RecurArgs rc;
    rc.q = q; rc.k = k; rc.v = v; rc.heads = w.heads; rc.q_heads = w.kv; rc.dim_p = w.dim_p; rc.vdim = w.c.vdim; rc.vdim_p = w.vdim_p;
    rc.state = w.state; rc.seg = seg; rc.pos = m->d_pos; rc.o = out;
    GatedNormArgs gn;
    gn.o = out; gn.heads = w.heads; gn.vdim = w.c.vdim; gn.vdim_p = w.vdim_p; gn.gate_head = w.vdim_p;
    gn.weight = w.onorm; gn.eps = (float)cfg.norm_eps; gn.ld = w.Kc; gn.packed = ctx_packed;
    if (cfg.f32) gn.of = ctx_f;
    else { gn.oh = m->ctxh; gn.ol = m->ctxl; }
    if (w.delta()) {
        DeltaRowsArgs da;
        da.in = m->slabs; da.n_slabs = ns; da.ld = w.N; da.slab_stride = (int64_t)R * w.N;
        da.heads = w.heads; da.kv = w.kv; da.dim = w.c.dim; da.dim_p = w.dim_p; da.vdim = w.c.vdim; da.vdim_p = w.vdim_p; da.rank_p = w.rank_p; da.taps = w.c.conv_taps;
        da.conv = w.conv; da.q_scale = 1.0f / std::sqrt((float)w.c.dim);
        da.history = w.history; da.slots = m->max_seqs; da.seg = seg; da.pos = m->d_pos; da.slot = m->d_slot;
        da.q = q; da.k = k; da.v = v; da.beta = beta; da.gate_in = gate_in;
        PROF(m, PROF_QK, launch_delta_rows(da, R, s));
        if (!seg.single) PROF(m, PROF_QK, launch_delta_history(da, s));
        HeadGemmArgs ga;
        ga.x = gate_in; ga.x_row = 2 * w.rank_p; ga.x_head = w.rank_p;
        ga.w = w.gates.data; ga.w_head = (int64_t)w.Ng * w.rank_p / 8; ga.N = ga.n_valid = w.Ng; ga.K = w.rank_p; ga.heads = 2; ga.M = R; ga.exact = cfg.f32;
        ga.y = g; ga.y_row = 2 * w.Ng; ga.y_head = w.Ng; ga.decay_rate = w.rate; ga.decay_bias = w.dt;
        PROF(m, PROF_GEMM, launch_delta_gates(ga, s));
        rc.g = g; rc.g_row = 2 * w.Ng; rc.beta = beta;
        gn.gate = g + w.Ng; gn.gate_row = 2 * w.Ng;
    } else {
        LinearRowsArgs la;
        la.in = m->slabs; la.n_slabs = ns; la.ld = w.N; la.slab_stride = (int64_t)R * w.N;
        la.heads = w.heads; la.dim = w.c.dim; la.dim_p = w.dim_p; la.vdim = w.c.vdim; la.vdim_p = w.vdim_p;
        la.q = q; la.k = k; la.v = v; la.gate = g;
        PROF(m, PROF_QK, launch_linear_rows(la, R, s));
        rc.decay = w.decay;
        gn.gate = g; gn.gate_row = (int64_t)w.heads * w.vdim_p;
        gn.whole = 1; gn.all = w.c.heads * w.c.vdim;
    }
    if (seg.single && !gn.whole) {
        PROF(m, PROF_RECUR, launch_recurrence(rc, &gn, s));
        return NVLLM_OK;
    }
    // in pieces of 16 tokens unless most of them would be padding
    if (!seg.single && !opt_scan && piece_scan_ok(w.dim_p) && R >= 4 * n_seg && n_piece <= 65535) {
        PieceArgs pc;
        pc.row0 = d_piece; pc.n = d_piece + piece_cap; pc.seg_piece0 = d_seg + 3 * m->max_seqs; pc.count = n_piece;
        pc.pair = pc_pair; pc.qt = pc_q; pc.wt = pc_w; pc.kt = pc_k; pc.decay = pc_decay;
        PROF(m, PROF_RECUR, launch_piece_scan(rc, pc, s));
    } else {
        PROF(m, PROF_RECUR, launch_recurrence(rc, nullptr, s));
    }
    if (gn.whole && ctx->tp_size > 1) {  // the norm runs over every rank's heads (padding columns are zero)
        const int n = w.heads * w.vdim_p, c0[2] = {0, 0}, nn[2] = {n, 0};
        HIPCHK(ctx, launch_rows_ssq(out, 1, 0, n, nullptr, c0, nn, R, ssq, s));
        int e = comm_allreduce_sum(ctx, ssq, (size_t)R * 2);
        if (e) return e;
        gn.ssq = ssq;
    }
    PROF(m, PROF_NORM, launch_gated_norm(gn, R, s));
    return NVLLM_OK;
}

int HybridModel::forward_chunk(nvllm_model* m, int R, int n_tiles, int qt, int n_last, int logits_row0) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    const bool f32 = cfg.f32 != 0;
    m->tap_rows = R;
    AddNormArgs base;
    base.W = cfg.width; base.ldr = ldr; base.ldx = Kw; base.eps = (float)cfg.norm_eps;
    auto plan = [&](const PackedW& w) { return f32 ? ProductPlan() : plan_product(m, R, w); };
    auto outputs = [&](AddNormArgs& a, int packed) {
        if (f32) a.y[0] = y;
        else { a.xh[0] = m->xh; a.xl[0] = m->xl; a.packed[0] = packed; }
    };
    ProductPlan pin = plan(layers[0].in);
    AddNormArgs first = base;
    first.ids = m->d_ids; first.embed = embed; first.embed_scale = (float)cfg.embed_scale;
    first.residual_out = m->resid; first.raw = 1;
    outputs(first, pin.packed);
    PROF(m, PROF_NORM, launch_add_norm(first, R, s));
    // x <- x + mult norm(slabs); the planes of x for the product `next`, or the normed rows of the head after the last sublayer
    float* const tap = ctx->tp_size > 1 ? m->slabs : m->red;  // not the last sum's input
    auto add = [&](int ns, const float* weight, const ProductPlan* next) -> int {
        AddNormArgs a = base;
        a.in = m->slabs; a.n_slabs = ns; a.slab_stride = (int64_t)R * ldr;
        if (ctx->tp_size > 1) {
            AddNormArgs sum = a;
            sum.residual_out = m->red;
            HIPCHK(ctx, launch_add_norm(sum, R, s));
            int rc = comm_allreduce_sum(ctx, m->red, (size_t)R * ldr);
            if (rc) return rc;
            a.in = m->red; a.n_slabs = 1;
        }
        a.post_w = weight; a.post_mult = (float)cfg.residual_mult; a.residual_in = m->resid;
        if (next) {
            a.residual_out = m->resid; a.raw = 1;
            outputs(a, next->packed);
            PROF(m, PROF_NORM, launch_add_norm(a, R, s));
            return NVLLM_OK;
        }
        if (m->taps) {
            AddNormArgs t = a;
            t.residual_out = tap;
            HIPCHK(ctx, launch_add_norm(t, R, s));
        }
        if (n_last <= 0) return NVLLM_OK;
        a.row_idx = m->d_last_rows;
        a.w[0] = final_norm;
        outputs(a, 0);
        PROF(m, PROF_NORM, launch_add_norm(a, n_last, s));
        return NVLLM_OK;
    };
    for (size_t l = 0; l < layers.size(); ++l) {
        HybridLayer& w = layers[l];
        const bool last = l + 1 == layers.size();
        const ProductPlan po = plan(w.o), pnext = last ? ProductPlan() : plan(layers[l + 1].in);
        ProductPlan pu, pd;
        if (w.ff) { pu = plan(w.up); pd = plan(w.down); }
        int ns = 1, rc = product(m, pin, y, m->xh, m->xl, w.in, R, &ns);
        if (!rc) rc = w.attention() ? attention(m, w, ns, R, n_tiles, qt, po.packed) : recurrence(m, w, ns, R, qt, po.packed);
        if (!rc) rc = product(m, po, ctx_f, m->ctxh, m->ctxl, w.o, R, &ns);
        if (!rc) rc = add(ns, w.norm1, w.ff ? &pu : last ? nullptr : &pnext);
        if (!rc && w.ff) {
            if (f32) {
                rc = exact_product(m, y, w.up, m->slabs, R);
                if (rc) return rc;
                PROF(m, PROF_SILU, launch_relu2(m->slabs, 1, 0, R, w.ff_p, nullptr, nullptr, 0, act_f, s));
            } else {
                rc = run_relu2(m, pu, m->xh, m->xl, w.up, R, m->xh2, m->xl2, pd.packed);
                if (rc) return rc;
            }
            rc = product(m, pd, act_f, m->xh2, m->xl2, w.down, R, &ns);
            if (!rc) rc = add(ns, w.norm2, last ? nullptr : &pnext);
        }
        if (rc) return rc;
        pin = pnext;
        if (m->taps)
            HIPCHK(ctx, hipMemcpy2DAsync(m->tap_res + l * (size_t)m->max_rows * m->H, (size_t)m->H * 4, last ? tap : m->resid, (size_t)ldr * 4, (size_t)m->H * 4, R,
                                         hipMemcpyDeviceToDevice, s));
    }
    if (n_last <= 0) return NVLLM_OK;
    return output_head(m, head, Kw, Vp, f32 ? y : nullptr, 0.f, n_last, logits_row0);
}
