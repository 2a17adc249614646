// Hybrid decoders behind the C ABI: every layer mixes tokens by grouped-query attention, a recurrence with constant decays or a gated delta
// rule, or by two of them side by side, and optionally has a feed-forward (plain or routed to experts).  Sublayers are normed on their output,
//   x <- x + m norm(mixer(x)),  x <- x + m norm(ff(x)),   with pre_norm on their input too,
// and a range of layers may be passed through several times, every pass with a cache and state of its own.
// Keys and values live in the paged cache, recurrent state and convolution history in the sequence's slot (f32).
// Mixed precision (the serving mode): products run on bf16 hi + lo planes with f32 accumulation, the cache is f16; residual, norms,
// scores, gates and recurrences are f32.  32-bit mode: every product and the cache in f32.
#include <algorithm>
#include <cmath>
#include <cstdio>

#include "decoder.h"
#include "experts.h"
#include "hybrid.h"
#include "rope.h"

struct HybridMixer {
    nvllm_hybrid_mixer c{};
    std::string prefix;                          // of its tensor names behind the layer's
    int heads = 0, kv = 0;                       // this rank's share
    int dim_p = 0, vdim_p = 0, rank_p = 0;
    int col0 = 0, cols = 0, gate0 = 0;           // columns of the layer's input projection; first one of a gate of one step
    int Kc = 0, Ng = 0;                          // context width (padded), rows of one gate matrix
    bool matrix_core = false;                    // attention: sizes have an instance
    bool last_v = false;                         // attention with value mixing: not the first such layer
    PackedW o, gates;                            // gates: decay, then output gate, [Ng x rank_p] each
    float *bias = nullptr, *qn = nullptr, *kn = nullptr, *table = nullptr, *vmix = nullptr, *sink = nullptr, *ob = nullptr;  // attention
    float *decay = nullptr, *onorm = nullptr;                                                                             // recurrences
    float *conv = nullptr, *rate = nullptr, *dt = nullptr;                                                                // convolutions, delta rule
    float* out_norm = nullptr;                   // of two mixers side by side
    int n_bias = 0, rope = -1;
    std::vector<int> bucket;                     // bias table row of every distance below n_bias
    bool attention() const { return c.mixer == NVLLM_MIXER_ATTENTION; }
    bool delta() const { return c.mixer == NVLLM_MIXER_DELTA; }
    bool head_decay() const { return delta() && !c.decay_rank; }
    bool per_head_norm() const { return attention() && c.qk_norm == NVLLM_QK_NORM_HEAD; }
    int channels() const { return attention() ? heads * c.dim + kv * (c.dim + c.vdim) : 2 * kv * c.dim + heads * c.vdim; }  // convolved
};

struct HybridLayer {
    nvllm_hybrid_layer c{};
    int ff = 0, ff_p = 0;                        // this rank's share
    int N = 0;                                   // rows of the input projection (padded)
    int branches = 1;
    HybridMixer mix[2];
    PackedW in, up, down;
    ExpertsBlock experts;
    float *norm1 = nullptr, *norm2 = nullptr;    // of the sublayers' outputs: stored weight + norm_offset
    float *pre1 = nullptr, *pre2 = nullptr;      // of their inputs
    Act act() const { return c.act == NVLLM_ACT_GELU ? ACT_GELU : ACT_RELU2; }
};

// what one mixer of one run carries
struct MixerState {
    void *kc = nullptr, *vc = nullptr;
    float *state = nullptr, *history = nullptr;  // per slot
};
struct HybridRun {
    int layer = 0;
    bool again = false;                          // first layer of a pass but the first
    MixerState st[2];
};

struct HybridModel : DecoderImpl {
    nvllm_hybrid_config cfg{};
    std::vector<HybridLayer> layers;
    std::vector<HybridRun> runs;
    std::vector<RopeTable> ropes;
    int ldr = 0, Kw = 0, Vp = 0;       // residual stride, width padded for the products, padded vocabulary rows of the head
    bool has_state = false, two = false;
    bf16_bits* embed = nullptr;        // [vocab][ldr]
    PackedW head;
    float* final_norm = nullptr;
    // step buffers
    float *q = nullptr, *k = nullptr, *v = nullptr, *g = nullptr, *beta = nullptr, *gate_in = nullptr, *out = nullptr, *v_first = nullptr, *ssq = nullptr;
    float *part_o = nullptr, *part_ml = nullptr, *slabs2 = nullptr;
    float *y = nullptr, *ctx_f[2] = {nullptr, nullptr}, *act_f = nullptr;  // 32-bit mode
    bf16_bits *ctx2h = nullptr, *ctx2l = nullptr;                          // the second mixer's context
    ExpertsScratch experts;
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
    int product(nvllm_model* m, const ProductPlan& p, const float* f, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, float* out, int R, int* ns) {
        *ns = 1;
        return cfg.f32 ? exact_product(m, f, w, out, R) : run_product(m, p, xh, xl, w, out, R, ns);
    }
    Segments segments(const nvllm_model* m, int R, int qt) const {
        Segments s;
        s.single = qt == 1;
        s.count = s.single ? R : n_seg;
        s.row0 = d_seg; s.n = d_seg + m->max_seqs; s.slot = s.single ? m->d_slot : d_seg + 2 * m->max_seqs;
        return s;
    }
    int create_mixer(nvllm_ctx* ctx, HybridMixer& w, const nvllm_hybrid_mixer& c, bool* mixes);
    int load_mixer(nvllm_model* m, HybridLayer& l, HybridMixer& w, const char* name, const char* s, const HostMat& h, int64_t rows, int64_t cols, int ndim);
    // mixer of R rows from the slabs of the input projection (rows of ld columns) up to the context of branch b
    int attention(nvllm_model* m, HybridMixer& w, MixerState& st, int b, int ns, int ld, int R, int n_tiles, int qt, int ctx_packed);
    int recurrence(nvllm_model* m, HybridMixer& w, MixerState& st, int b, int ns, int ld, int R, int qt, int ctx_packed);
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

static int check_mixer(nvllm_ctx* ctx, const nvllm_hybrid_mixer& k, int l) {
    const int tp = ctx->tp_size;
    if (k.heads < 1 || k.kv_heads < 1 || k.dim < 1 || k.vdim < 1) return fail(ctx, NVLLM_EINVAL, "layer %d has non-positive sizes", l);
    if (k.heads % k.kv_heads) return fail(ctx, NVLLM_EINVAL, "layer %d: %d heads over %d key/value heads", l, k.heads, k.kv_heads);
    if (k.heads % tp || k.kv_heads % tp) return fail(ctx, NVLLM_EINVAL, "layer %d: heads %d / %d not divisible by tp_size %d", l, k.heads, k.kv_heads, tp);
    if (k.mixer == NVLLM_MIXER_ATTENTION) {
        if (k.qk_norm == NVLLM_QK_NORM_HEAD) {
            if (k.dim > kConvAttnDim || k.vdim > kConvAttnDim) return fail(ctx, NVLLM_EINVAL, "layer %d: head sizes %d / %d unsupported (at most %d)", l, k.dim, k.vdim, kConvAttnDim);
            if (k.conv_taps < 1 || k.conv_taps > 16) return fail(ctx, NVLLM_EINVAL, "layer %d: convolution of %d taps (1 to 16) unsupported", l, k.conv_taps);
            if (k.rot_dim < 0 || k.rot_dim % 2 || k.rot_dim > k.dim) return fail(ctx, NVLLM_EINVAL, "layer %d: %d rotated dimensions of %d", l, k.rot_dim, k.dim);
            if (k.v_mix) return fail(ctx, NVLLM_EINVAL, "layer %d: value mixing beside norms per head unsupported", l);
        } else {
            if (k.dim > 4096 || k.vdim > 1024) return fail(ctx, NVLLM_EINVAL, "layer %d: head sizes %d / %d unsupported (at most 4096 / 1024)", l, k.dim, k.vdim);
            if ((k.heads / tp) * k.dim + (k.kv_heads / tp) * (k.dim + k.vdim) > 16000) return fail(ctx, NVLLM_EINVAL, "layer %d: more than 16000 query, key and value columns per rank", l);
            if (k.conv_taps || k.rot_dim) return fail(ctx, NVLLM_EINVAL, "layer %d: convolutions and rotation go with norms per head", l);
        }
        if (k.bias_rows < 0 || k.bias_rows > 1 << 20) return fail(ctx, NVLLM_EINVAL, "layer %d: %d rows of distance bias", l, k.bias_rows);
        if (k.sink < NVLLM_SINK_NONE || k.sink > NVLLM_SINK_HEAD) return fail(ctx, NVLLM_EINVAL, "layer %d: sink %d unknown", l, k.sink);
    } else if (k.mixer == NVLLM_MIXER_LINEAR || k.mixer == NVLLM_MIXER_DELTA) {
        if (!recur_ok(k.dim, k.vdim)) return fail(ctx, NVLLM_EINVAL, "layer %d: head sizes %d / %d unsupported (key size at most 512)", l, k.dim, k.vdim);
        if (k.mixer == NVLLM_MIXER_LINEAR && (!k.decay || k.kv_heads != k.heads)) return fail(ctx, NVLLM_EINVAL, "layer %d: needs one decay and one key head per head", l);
        if (k.mixer == NVLLM_MIXER_DELTA && (k.conv_taps < 1 || k.conv_taps > 16 || k.decay_rank < 0 || k.gate_rank < 0 || !k.decay_rank != !k.gate_rank))
            return fail(ctx, NVLLM_EINVAL, "layer %d: convolution of %d taps (1 to 16) or gate ranks %d / %d unsupported", l, k.conv_taps, k.decay_rank, k.gate_rank);
    } else {
        return fail(ctx, NVLLM_EINVAL, "layer %d: mixer %d unknown", l, k.mixer);
    }
    return NVLLM_OK;
}

extern "C" int nvllm_model_create_hybrid(nvllm_ctx* ctx, const nvllm_hybrid_config* cfg, const nvllm_hybrid_layer* layers, nvllm_model** out) {
    if (!ctx || !cfg || !layers || !out) return fail(ctx, NVLLM_EINVAL, "NULL argument");
    const nvllm_hybrid_config& c = *cfg;
    const int tp = ctx->tp_size;
    if (c.vocab_size < 1 || c.width < 1 || c.num_layers < 1) return fail(ctx, NVLLM_EINVAL, "config has non-positive sizes");
    if (c.width > 8192) return fail(ctx, NVLLM_EINVAL, "width %d unsupported (at most 8192)", c.width);
    if (c.vocab_size % tp) return fail(ctx, NVLLM_EINVAL, "vocabulary of %d not divisible by tp_size %d", c.vocab_size, tp);
    const bool loop = c.loop_times > 1;
    if (loop && (c.loop_start < 0 || c.loop_start >= c.loop_stop || c.loop_stop > c.num_layers))
        return fail(ctx, NVLLM_EINVAL, "loop [%d, %d) outside the %d layers", c.loop_start, c.loop_stop, c.num_layers);
    const nvllm_hybrid_mixer* first_mix = nullptr;
    for (int l = 0; l < c.num_layers; ++l) {
        const nvllm_hybrid_layer& k = layers[l];
        for (int b = 0; b < (k.branches == 2 ? 2 : 1); ++b) {
            const nvllm_hybrid_mixer& x = b ? k.side : k.mix;
            int rc = check_mixer(ctx, x, l);
            if (rc) return rc;
            if (x.mixer == NVLLM_MIXER_ATTENTION && x.v_mix) {
                if (loop) return fail(ctx, NVLLM_EINVAL, "layer %d: value mixing beside looped layers is unsupported", l);
                if (!first_mix) first_mix = &x;
                else if (x.kv_heads * x.vdim != first_mix->kv_heads * first_mix->vdim)
                    return fail(ctx, NVLLM_EINVAL, "layer %d mixes values of %d columns with the first mixing layer's %d", l, x.kv_heads * x.vdim, first_mix->kv_heads * first_mix->vdim);
            }
            if (b && x.mixer == NVLLM_MIXER_ATTENTION && x.out_bias) return fail(ctx, NVLLM_EINVAL, "layer %d: output bias on the second mixer unsupported", l);
        }
        if (k.ff < 0 || k.experts < 0 || (k.ff && k.experts)) return fail(ctx, NVLLM_EINVAL, "layer %d: feed-forward sizes", l);
        if (k.ff % tp || (k.experts && k.expert_ff % tp)) return fail(ctx, NVLLM_EINVAL, "layer %d: feed-forward width not divisible by tp_size %d", l, tp);
        if (k.ff && k.act != NVLLM_ACT_RELU2 && k.act != NVLLM_ACT_GELU) return fail(ctx, NVLLM_EINVAL, "layer %d: feed-forward activation %d unknown", l, k.act);
        if (k.experts && (k.experts > kMaxExperts || k.top < 1 || k.top > std::min(k.experts, kMaxTop) || k.expert_ff < 1))
            return fail(ctx, NVLLM_EINVAL, "layer %d: %d of %d experts of width %d unsupported (at most %d of %d)", l, k.top, k.experts, k.expert_ff, kMaxTop, kMaxExperts);
        if (k.experts && (k.groups < 1 || k.experts % k.groups || k.groups_kept < 1 || k.groups_kept > k.groups || k.top > k.groups_kept * (k.experts / k.groups)))
            return fail(ctx, NVLLM_EINVAL, "layer %d: %d of %d groups of %d experts, %d chosen", l, k.groups_kept, k.groups, k.experts, k.top);
    }
    HIPCHK(ctx, hipSetDevice(ctx->device));
    nvllm_model* m = new nvllm_model();
    m->ctx = ctx;
    auto owned = std::make_unique<HybridModel>();
    HybridModel& L = *owned;
    m->dec = std::move(owned);
    L.cfg = c;
    m->H = c.width; m->V_l = c.vocab_size / tp; m->kv_l = 1;
    m->cfg.vocab_size = c.vocab_size; m->cfg.hidden_size = c.width; m->cfg.max_position_embeddings = 1 << 30;
    L.ldr = up(c.width, 16); L.Kw = up(c.width, 128); L.Vp = up(m->V_l, 16);
    for (int l = 0; l < c.num_layers; ++l) {
        if (loop && l == c.loop_start) {
            for (int t = 0; t < c.loop_times; ++t)
                for (int i = c.loop_start; i < c.loop_stop; ++i) { L.runs.emplace_back(); L.runs.back().layer = i; L.runs.back().again = t && i == c.loop_start; }
            l = c.loop_stop - 1;
            continue;
        }
        L.runs.emplace_back();
        L.runs.back().layer = l;
    }
    m->L = (int)L.runs.size();
    int rc = dmalloc(ctx, &L.embed, (size_t)c.vocab_size * L.ldr);
    if (!rc) HIPCHK(ctx, hipMemsetAsync(L.embed, 0, (size_t)c.vocab_size * L.ldr * 2, ctx->stream));
    if (!rc) rc = alloc_packed(ctx, L.head, L.Vp, L.Kw);
    if (!rc) rc = alloc_vec(ctx, &L.final_norm, L.Kw);
    L.layers.resize(c.num_layers);
    bool mixes = false, unbounded = false;
    for (int l = 0; l < c.num_layers && !rc; ++l) {
        HybridLayer& w = L.layers[l];
        w.c = layers[l];
        w.branches = w.c.branches == 2 ? 2 : 1;
        L.two |= w.branches == 2;
        w.ff = w.c.ff / tp; w.ff_p = up(w.ff, 128);
        int n = 0;
        for (int b = 0; b < w.branches && !rc; ++b) {
            HybridMixer& x = w.mix[b];
            x.prefix = w.branches == 2 ? (b ? "mix.right." : "mix.left.") : "mix.";
            x.col0 = n;
            rc = L.create_mixer(ctx, x, b ? layers[l].side : layers[l].mix, &mixes);
            if (!rc && w.branches == 2) rc = alloc_vec(ctx, &x.out_norm, L.Kw);
            if (x.attention()) {
                unbounded |= x.c.window <= 0;
                m->widest_window = std::max(m->widest_window, (int)x.c.window);
            }
            n = b + 1 < w.branches ? up(n + x.cols, 16) : n + x.cols;
        }
        // wide projections: a whole number of the prompt product's 192- or 256-feature tiles
        w.N = n >= 1536 && !c.f32 ? std::min(up(n, 192), up(n, 256)) : up(n, 16);
        if (!rc) rc = alloc_packed(ctx, w.in, w.N, L.Kw);
        if (!rc) rc = alloc_vec(ctx, &w.norm1, L.Kw);
        if (!rc && c.pre_norm) rc = alloc_vec(ctx, &w.pre1, L.Kw);
        if (w.ff) {
            if (!rc) rc = alloc_packed(ctx, w.up, w.ff_p, L.Kw);
            if (!rc) rc = alloc_packed(ctx, w.down, L.ldr, w.ff_p);
        }
        if (w.c.experts) {
            w.experts.weight_in = 0; w.experts.gated = 1; w.experts.softmax = 1; w.experts.groups = w.c.groups; w.experts.keep = w.c.groups_kept;
            if (!rc) rc = w.experts.create(ctx, w.c.experts, w.c.top, w.c.expert_ff, 0, c.width, L.Kw, L.ldr, c.f32);
        }
        if (w.ff || w.c.experts) {
            if (!rc) rc = alloc_vec(ctx, &w.norm2, L.Kw);
            if (!rc && c.pre_norm) rc = alloc_vec(ctx, &w.pre2, L.Kw);
        }
    }
    if (unbounded) m->widest_window = 0;
    if (!rc && hipStreamSynchronize(ctx->stream) != hipSuccess) rc = fail(ctx, NVLLM_EHIP, "weight allocation failed");
    if (rc) { nvllm_model_destroy(m); return rc; }
    *out = m;
    return NVLLM_OK;
}

// sizes and everything but the input projection
int HybridModel::create_mixer(nvllm_ctx* ctx, HybridMixer& w, const nvllm_hybrid_mixer& c, bool* mixes) {
    const int tp = ctx->tp_size, D = c.dim, E = c.vdim;
    w.c = c;
    w.c.decay = nullptr;  // the caller's array is not kept
    w.heads = c.heads / tp; w.kv = c.kv_heads / tp;
    w.Kc = up(w.heads * E, 128);
    if (w.attention()) {
        w.matrix_core = !cfg.f32 && bias_attn_dim(D) && bias_attn_vdim(E);
        w.dim_p = w.matrix_core ? bias_attn_dim(D) : up(D, 32);
        w.vdim_p = w.matrix_core ? bias_attn_vdim(E) : up(E, 16);
        w.last_v = c.v_mix && *mixes;
        *mixes |= c.v_mix != 0;
        w.cols = w.channels();
        if (c.bias_rows) {
            do w.bucket.push_back(distance_bucket((int)w.bucket.size(), c.bias_rows, c.bias_max)); while (w.bucket.back() < c.bias_rows - 1 && w.bucket.size() < (1u << 24));
            w.n_bias = (int)w.bucket.size();
        }
        if (c.conv_taps > 1) has_state = true;
        if (c.rot_dim) w.rope = rope_index(ropes, RopeTable{c.rot_base, c.yarn_factor, c.yarn_original, c.yarn_fast, c.yarn_slow, c.rot_dim});
    } else {
        has_state = true;
        w.dim_p = recur_dim(D);
        w.vdim_p = recur_vdim(E);
        if (w.head_decay()) {
            w.gate0 = up(w.channels() + 2 * w.heads, 4);
            w.cols = w.gate0 + w.heads * E;
        } else if (w.delta()) {
            w.rank_p = std::max(up(c.decay_rank, 32), up(c.gate_rank, 32));
            w.Ng = w.heads * std::max(w.dim_p, w.vdim_p);
            w.cols = w.channels() + w.heads + 2 * w.rank_p;
        } else {
            w.cols = 2 * w.heads * (D + E);
        }
    }
    auto vec = [&](float** p, size_t n) { return alloc_vec(ctx, p, n); };
    int rc = alloc_packed(ctx, w.o, ldr, w.Kc);
    if (w.attention()) {
        if (!rc) rc = vec(&w.bias, up(w.cols, 16));
        if (!rc && !w.per_head_norm()) rc = vec(&w.qn, w.heads * D);
        if (!rc && !w.per_head_norm()) rc = vec(&w.kn, w.kv * D);
        if (!rc) rc = vec(&w.vmix, 1);
        if (!rc) rc = vec(&w.table, std::max(1, w.heads * w.n_bias));
        if (!rc && c.sink) rc = vec(&w.sink, w.heads);  // NVLLM_SINK_ONE: stays zero
        if (!rc && c.out_bias) rc = vec(&w.ob, Kw);
        if (!rc && c.conv_taps) rc = vec(&w.conv, c.conv_taps * w.channels());
        return rc;
    }
    if (!rc) rc = vec(&w.onorm, w.delta() ? E : w.heads * E);
    if (w.delta()) {
        if (!rc && w.Ng) rc = alloc_packed(ctx, w.gates, 2 * w.Ng, w.rank_p);
        if (!rc) rc = vec(&w.conv, c.conv_taps * w.channels());
        if (!rc) rc = vec(&w.rate, w.head_decay() ? w.heads : w.Ng);
        if (!rc) rc = vec(&w.dt, w.head_decay() ? w.heads : w.Ng);
        return rc;
    }
    std::vector<float> d(w.heads);
    for (int h = 0; h < w.heads; ++h) d[h] = (float)c.decay[ctx->tp_rank * w.heads + h];
    if (!rc) rc = vec(&w.decay, w.heads);
    if (!rc && hipMemcpyAsync(w.decay, d.data(), d.size() * 4, hipMemcpyHostToDevice, ctx->stream) != hipSuccess) rc = fail(ctx, NVLLM_EHIP, "decay upload failed");
    if (!rc && hipStreamSynchronize(ctx->stream) != hipSuccess) rc = fail(ctx, NVLLM_EHIP, "decay upload failed");
    return rc;
}

void HybridModel::free_kv() {
    for (HybridRun& r : runs)
        for (MixerState& s : r.st) {
            for (void* p : {s.kc, s.vc, (void*)s.state, (void*)s.history}) if (p) (void)hipFree(p);
            s = MixerState();
        }
    for (RopeTable& r : ropes) r.release();
    experts.release();
    for (float** p : {&q, &k, &v, &g, &beta, &gate_in, &out, &v_first, &ssq, &part_o, &part_ml, &slabs2, &y, &ctx_f[0], &ctx_f[1], &act_f, &pc_pair, &pc_q, &pc_w, &pc_k, &pc_decay}) {
        if (*p) (void)hipFree(*p);
        *p = nullptr;
    }
    for (bf16_bits** p : {&ctx2h, &ctx2l}) {
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
    for (HybridLayer& l : layers) {
        l.experts.destroy();
        for (PackedW* p : {&l.in, &l.up, &l.down}) (void)hipFree(p->data);
        for (float* p : {l.norm1, l.norm2, l.pre1, l.pre2}) (void)hipFree(p);
        for (HybridMixer& w : l.mix) {
            for (PackedW* p : {&w.o, &w.gates}) (void)hipFree(p->data);
            for (float* p : {w.bias, w.qn, w.kn, w.table, w.vmix, w.sink, w.ob, w.decay, w.onorm, w.conv, w.rate, w.dt, w.out_norm}) (void)hipFree(p);
        }
    }
}

// ---------------------------------------------------------------------------------------------------
// weights
// ---------------------------------------------------------------------------------------------------
// the tensors a mixer cannot do without
static std::vector<std::string> mixer_tensors(const HybridMixer& w) {
    std::vector<std::string> t = {"q", "k", "v", "o"};
    auto add = [&](std::initializer_list<const char*> names) { t.insert(t.end(), names.begin(), names.end()); };
    if (w.attention()) {
        add({"q.b", "k.b", "v.b"});
        if (!w.per_head_norm()) add({"q.norm", "k.norm"});
        if (w.c.bias_rows) add({"rel"});
        if (w.last_v) add({"vmix"});
        if (w.c.sink == NVLLM_SINK_HEAD) add({"sink"});
        if (w.c.out_bias) add({"o.b"});
    } else {
        add({"norm"});
        if (w.delta()) add({"b", "A_log", "dt_bias"});
        if (w.delta() && !w.head_decay()) add({"a1", "a2", "g1", "g2"});
        if (w.head_decay()) add({"a"});
        if (!w.delta() || w.head_decay()) add({"g"});
    }
    if (w.c.conv_taps && (w.attention() || w.delta())) add({"q.conv", "k.conv", "v.conv"});
    if (w.out_norm) add({"out"});
    return t;
}

static int want_shape(nvllm_ctx* ctx, const char* name, int64_t rows, int64_t cols, int ndim, int64_t r, int64_t c, int nd) {
    if (rows == r && cols == c && (ndim == nd || (nd == 0 && ndim == 1))) return NVLLM_OK;
    return fail(ctx, NVLLM_EINVAL, "tensor '%s': shape mismatch (got %lld x %lld, want %lld x %lld)", name, (long long)rows, (long long)cols, (long long)r, (long long)c);
}

int HybridModel::load_mixer(nvllm_model* m, HybridLayer& l, HybridMixer& w, const char* name, const char* s, const HostMat& h, int64_t rows, int64_t cols, int ndim) {
    nvllm_ctx* ctx = m->ctx;
    const int rank = ctx->tp_rank, W = cfg.width;
    const int D = w.c.dim, E = w.c.vdim, Hl = w.heads, Gl = w.kv, H = w.c.heads, G = w.c.kv_heads;
    const int64_t h0 = (int64_t)rank * Hl, g0 = (int64_t)rank * Gl;
    auto want = [&](int64_t r, int64_t c, int nd) { return want_shape(ctx, name, rows, cols, ndim, r, c, nd); };
    auto is = [&](const char* t) { return !strcmp(s, t); };
    auto put = [&](float* dst, const std::vector<float>& t) -> int {
        HIPCHK(ctx, hipMemcpy(dst, t.data(), t.size() * 4, hipMemcpyHostToDevice));
        return NVLLM_OK;
    };
    // n elements of a vector of `all`, from `first` on, through f
    auto vec_f = [&](float* dst, int64_t all, int64_t first, int n, auto f) -> int {
        int rc = want(1, all, 1);
        if (rc) return rc;
        std::vector<float> t(n);
        for (int i = 0; i < n; ++i) t[i] = f(h.f32(first + i));
        return put(dst, t);
    };
    auto vec = [&](float* dst, int64_t all, int64_t first, int n) { return vec_f(dst, all, first, n, [](float x) { return x; }); };
    // `n` rows per rank of the input projection from the mixer's row `at` on, out of `all`
    auto proj = [&](int at, int64_t all, int n) -> int {
        const int64_t r0 = all == n ? 0 : (int64_t)rank * n;
        int e = want(all, W, 2);
        return e ? e : put_rows(ctx, l.in, w.col0 + at, n, W, -1, [&](int r, int c) { return h.at(r0 + r, c); });
    };
    auto conv = [&](int at, int64_t all, int n) -> int {  // [channels, taps] -> [taps][channels]
        int e = want(all, w.c.conv_taps, 2);
        if (e) return e;
        std::vector<float> t(n);
        for (int i = 0; i < w.c.conv_taps && !e; ++i) {
            for (int r = 0; r < n; ++r) t[r] = h.f32(((int64_t)rank * n + r) * cols + i);
            e = put(w.conv + (size_t)i * w.channels() + at, t);
        }
        return e;
    };
    if (is("o")) {
        int rc = want(W, (int64_t)H * E, 2);
        return rc ? rc : put_rows(ctx, w.o, 0, W, Hl * E, -1, [&](int r, int c) { return h.at(r, h0 * E + c); });
    }
    if (w.out_norm && is("out")) return vec(w.out_norm, W, 0, W);
    const bool convs = w.c.conv_taps && (w.attention() || w.delta());
    if (w.attention()) {
        const int k0 = Hl * D, v0 = k0 + Gl * D;
        if (is("q")) return proj(0, (int64_t)H * D, Hl * D);
        if (is("k")) return proj(k0, (int64_t)G * D, Gl * D);
        if (is("v")) return proj(v0, (int64_t)G * E, Gl * E);
        if (is("q.b")) return vec(w.bias, (int64_t)H * D, h0 * D, Hl * D);
        if (is("k.b")) return vec(w.bias + k0, (int64_t)G * D, g0 * D, Gl * D);
        if (is("v.b")) return vec(w.bias + v0, (int64_t)G * E, g0 * E, Gl * E);
        if (w.qn && is("q.norm")) return vec(w.qn, (int64_t)H * D, h0 * D, Hl * D);
        if (w.kn && is("k.norm")) return vec(w.kn, (int64_t)G * D, g0 * D, Gl * D);
        if (convs && is("q.conv")) return conv(0, (int64_t)H * D, Hl * D);
        if (convs && is("k.conv")) return conv(k0, (int64_t)G * D, Gl * D);
        if (convs && is("v.conv")) return conv(v0, (int64_t)G * E, Gl * E);
        if (w.ob && is("o.b")) return vec(w.ob, W, 0, W);
        if (w.c.sink == NVLLM_SINK_HEAD && is("sink")) return vec_f(w.sink, H, h0, Hl, [](float x) { return (float)(x * 1.4426950408889634); });
        if (w.c.bias_rows && is("rel")) {
            int rc = want(w.c.bias_rows, H, 2);
            if (rc) return rc;
            std::vector<float> t((size_t)Hl * w.n_bias);
            for (int n = 0; n < Hl; ++n)
                for (int d = 0; d < w.n_bias; ++d) t[(size_t)n * w.n_bias + d] = (float)(h.f32((int64_t)w.bucket[d] * H + h0 + n) * 1.4426950408889634);
            return put(w.table, t);
        }
        if (w.qn && is("vmix")) {  // unused where nothing is mixed
            int rc = want(1, 1, 0);
            return rc ? rc : put(w.vmix, {h.f32(0)});
        }
    } else if (!w.delta()) {
        const int HD = Hl * D, HE = Hl * E;
        if (is("q")) return proj(0, (int64_t)H * D, HD);
        if (is("k")) return proj(HD, (int64_t)H * D, HD);
        if (is("v")) return proj(2 * HD, (int64_t)H * E, HE);
        if (is("g")) return proj(2 * HD + HE, (int64_t)H * E, HE);
        if (is("norm")) return vec(w.onorm, (int64_t)H * E, h0 * E, HE);
    } else {
        const int GD = Gl * D, HE = Hl * E, C = w.channels(), ra = w.c.decay_rank, rg = w.c.gate_rank;
        auto gate = [&](int at, int size, int size_p, int r) -> int {  // rows head * size + i -> head * size_p + i
            int e = want((int64_t)H * size, r, 2);
            return e ? e : put_rows(ctx, w.gates, at, Hl * size_p, r, -1, [&](int row, int c) -> uint16_t {
                const int n = row / size_p, i = row % size_p;
                return i < size ? h.at((h0 + n) * size + i, c) : (uint16_t)0;
            });
        };
        if (is("q")) return proj(0, (int64_t)G * D, GD);
        if (is("k")) return proj(GD, (int64_t)G * D, GD);
        if (is("v")) return proj(2 * GD, (int64_t)H * E, HE);
        if (is("b")) return proj(C, H, Hl);
        if (is("q.conv")) return conv(0, (int64_t)G * D, GD);
        if (is("k.conv")) return conv(GD, (int64_t)G * D, GD);
        if (is("v.conv")) return conv(2 * GD, (int64_t)H * E, HE);
        if (is("norm")) return vec(w.onorm, E, 0, E);
        if (w.head_decay()) {
            if (is("a")) return proj(C + Hl, H, Hl);
            if (is("g")) return proj(w.gate0, (int64_t)H * E, HE);
            if (is("A_log")) return vec_f(w.rate, H, h0, Hl, [](float x) { return std::exp(x); });
            if (is("dt_bias")) return vec(w.dt, H, h0, Hl);
        } else {
            if (is("a1")) return proj(C + Hl, ra, ra);
            if (is("g1")) return proj(C + Hl + w.rank_p, rg, rg);
            if (is("a2")) return gate(0, D, w.dim_p, ra);
            if (is("g2")) return gate(w.Ng, E, w.vdim_p, rg);
            if (is("A_log")) {
                int rc = want(1, H, 1);
                if (rc) return rc;
                std::vector<float> t(w.Ng, 0.f);
                for (int i = 0; i < Hl * w.dim_p; ++i) t[i] = std::exp(h.f32(h0 + i / w.dim_p));
                return put(w.rate, t);
            }
            if (is("dt_bias")) {
                int rc = want(1, (int64_t)H * D, 1);
                if (rc) return rc;
                std::vector<float> t(w.Ng, 0.f);
                for (int i = 0; i < Hl * w.dim_p; ++i) if (i % w.dim_p < D) t[i] = h.f32((h0 + i / w.dim_p) * D + i % w.dim_p);
                return put(w.dt, t);
            }
        }
    }
    return fail(ctx, NVLLM_EINVAL, "unknown tensor name '%s'", name);
}

int HybridModel::load_tensor(nvllm_model* m, const char* name, const void* data, int dtype, const int64_t* shape, int ndim) {
    nvllm_ctx* ctx = m->ctx;
    const int rank = ctx->tp_rank;
    if (ndim < 0 || ndim > 2) return fail(ctx, NVLLM_EINVAL, "tensor '%s' has %d dimensions", name, ndim);
    const int64_t rows = ndim == 2 ? shape[0] : 1, cols = ndim ? shape[ndim - 1] : 1;
    const HostMat h{data, dtype, cols};
    HIPCHK(ctx, hipSetDevice(ctx->device));
    auto want = [&](int64_t r, int64_t c, int nd) { return want_shape(ctx, name, rows, cols, ndim, r, c, nd); };
    const int W = cfg.width, V = cfg.vocab_size;
    auto norm = [&](float* dst) -> int {
        int rc = want(1, W, 1);
        if (rc) return rc;
        std::vector<float> t(W);
        for (int i = 0; i < W; ++i) t[i] = h.f32(i) + (float)cfg.norm_offset;
        HIPCHK(ctx, hipMemcpy(dst, t.data(), t.size() * 4, hipMemcpyHostToDevice));
        return NVLLM_OK;
    };
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
        if ((rc = norm(final_norm))) return rc;
    } else {
        if (sscanf(name, "l%d.%n", &l, &off) != 1 || off == 0 || l < 0 || l >= cfg.num_layers) return fail(ctx, NVLLM_EINVAL, "unknown tensor name '%s'", name);
        const char* s = name + off;
        HybridLayer& w = layers[l];
        const int64_t f0 = (int64_t)rank * w.ff;
        HybridMixer* mixer = nullptr;
        for (int b = 0; b < w.branches; ++b)
            if (!strncmp(s, w.mix[b].prefix.c_str(), w.mix[b].prefix.size())) mixer = &w.mix[b];
        if (!strcmp(s, "norm1")) rc = norm(cfg.pre_norm ? w.pre1 : w.norm1);
        else if (w.norm2 && !strcmp(s, "norm2")) rc = norm(cfg.pre_norm ? w.pre2 : w.norm2);
        else if (cfg.pre_norm && !strcmp(s, "norm1b")) rc = norm(w.norm1);
        else if (cfg.pre_norm && w.norm2 && !strcmp(s, "norm2b")) rc = norm(w.norm2);
        else if (w.ff && !strcmp(s, "mlp.up")) {
            if (!(rc = want(w.c.ff, W, 2))) rc = put_rows(ctx, w.up, 0, w.ff, W, -1, [&](int r, int c) { return h.at(f0 + r, c); });
        } else if (w.ff && !strcmp(s, "mlp.down")) {
            if (!(rc = want(W, w.c.ff, 2))) rc = put_rows(ctx, w.down, 0, W, w.ff, -1, [&](int r, int c) { return h.at(r, f0 + c); });
        } else if (mixer) rc = load_mixer(m, w, *mixer, name, s + mixer->prefix.size(), h, rows, cols, ndim);
        else {
            rc = w.experts.on() && !strncmp(s, "mlp.", 4) ? w.experts.load(m, name, s + 4, h, rows, cols) : 1;
            if (rc == 1) rc = fail(ctx, NVLLM_EINVAL, "unknown tensor name '%s'", name);
        }
        if (rc) return rc;
    }
    m->loaded[name] = true;
    return NVLLM_OK;
}

int HybridModel::finalize(nvllm_model* m) {
    nvllm_ctx* ctx = m->ctx;
    std::vector<std::string> names = {"embed", "head", "final.norm"};
    for (int l = 0; l < cfg.num_layers; ++l) {
        const HybridLayer& w = layers[l];
        const std::string p = "l" + std::to_string(l) + ".";
        names.push_back(p + "norm1");
        if (cfg.pre_norm) names.push_back(p + "norm1b");
        for (int b = 0; b < w.branches; ++b)
            for (const std::string& s : mixer_tensors(w.mix[b])) names.push_back(p + w.mix[b].prefix + s);
        if (w.norm2) names.push_back(p + "norm2");
        if (w.norm2 && cfg.pre_norm) names.push_back(p + "norm2b");
        if (w.ff) for (const char* s : {"mlp.up", "mlp.down"}) names.push_back(p + s);
        if (w.experts.on()) for (const std::string& s : w.experts.tensors()) names.push_back(p + "mlp." + s);
    }
    for (const std::string& s : names)
        if (!m->loaded.count(s)) return fail(ctx, NVLLM_ESTATE, "missing tensor %s", s.c_str());
    m->finalized = true;
    return NVLLM_OK;
}

int64_t HybridModel::weight_bytes() const {
    int64_t b = (int64_t)head.bytes() + (int64_t)cfg.width * 4;
    for (const HybridRun& r : runs) {
        const HybridLayer& w = layers[r.layer];
        b += (int64_t)(w.in.bytes() + w.up.bytes() + w.down.bytes() + w.experts.step_bytes());
        for (const HybridMixer& x : w.mix) b += (int64_t)(x.o.bytes() + x.gates.bytes() + (x.out_norm ? cfg.width * 4 : 0));
        for (const float* p : {w.norm1, w.norm2, w.pre1, w.pre2}) b += p ? (int64_t)cfg.width * 4 : 0;
    }
    return b;
}
int64_t HybridModel::kv_bytes_per_token() const {
    int64_t b = 0;
    for (const HybridRun& r : runs)
        for (const HybridMixer& w : layers[r.layer].mix)
            if (w.heads && w.attention()) b += (int64_t)w.kv * (w.dim_p + w.vdim_p) * (cfg.f32 ? 4 : 2);
    return b;
}
int64_t HybridModel::kv_read_bytes(int len) const {
    int64_t b = 0;
    for (const HybridRun& r : runs)
        for (const HybridMixer& w : layers[r.layer].mix) {
            if (!w.heads) continue;
            if (w.attention()) b += (int64_t)w.kv * (w.dim_p + w.vdim_p) * (cfg.f32 ? 4 : 2) * (w.c.window > 0 ? std::min(len, w.c.window) : len);
            else b += (int64_t)recur_state_floats(w.heads, w.dim_p, w.vdim_p) * 8;  // read and written
            if (w.conv) b += (int64_t)(w.c.conv_taps - 1) * w.channels() * 8;
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
    for (HybridRun& r : runs)
        for (int b = 0; b < layers[r.layer].branches; ++b) {
            const HybridMixer& w = layers[r.layer].mix[b];
            MixerState& st = r.st[b];
            if (w.attention()) {
                // padding stays zero, unwritten tokens finite
                const size_t toks = (size_t)m->num_blocks * kBlockTokens * w.kv * (f32 ? 4 : 2);
                if (!rc) rc = zalloc(&st.kc, toks * w.dim_p);
                if (!rc) rc = zalloc(&st.vc, toks * w.vdim_p);
            } else if (!rc) {
                rc = zalloc((void**)&st.state, (size_t)m->max_seqs * recur_state_floats(w.heads, w.dim_p, w.vdim_p) * 4);
            }
            if (!rc && w.conv && w.c.conv_taps > 1) rc = zalloc((void**)&st.history, (size_t)2 * m->max_seqs * (w.c.conv_taps - 1) * w.channels() * 4);
        }
    size_t nmax = ldr, kc = 0, ffp = 0, nq = 0, nk = 0, nv = 0, ng = 0, nb = 0, nin = 0, no = 0, nvf = 0, po = 0, pm = 0;
    size_t ph = 0, pd = 0, pdd = 0;  // heads, channels of the layers that run in pieces, channels of the delta rule's alone
    for (HybridLayer& l : layers) {
        nmax = std::max<size_t>({nmax, (size_t)l.N, (size_t)l.ff_p});
        ffp = std::max<size_t>(ffp, l.ff_p);
        if (l.experts.on()) experts.reserve(l.experts, R);
        for (int b = 0; b < l.branches; ++b) {
            const HybridMixer& w = l.mix[b];
            kc = std::max<size_t>(kc, w.Kc);
            nq = std::max<size_t>(nq, (size_t)w.heads * w.dim_p);
            if (w.attention()) {
                if (w.c.v_mix) nvf = std::max<size_t>(nvf, (size_t)w.kv * w.c.vdim);
                po = std::max<size_t>(po, (size_t)kDecodeWgs * 16 * w.vdim_p);
                pm = (size_t)kDecodeWgs * 16 * 2;
                continue;
            }
            nk = std::max<size_t>(nk, (size_t)w.heads * w.dim_p);
            nv = std::max<size_t>(nv, (size_t)w.heads * w.vdim_p);
            ng = std::max<size_t>(ng, w.head_decay() ? (size_t)w.heads : w.delta() ? (size_t)2 * w.Ng : (size_t)w.heads * w.vdim_p);
            nb = std::max<size_t>(nb, w.heads);
            nin = std::max<size_t>(nin, (size_t)2 * w.rank_p);
            no = std::max<size_t>(no, (size_t)w.heads * w.vdim_p);
            if (piece_scan_ok(w.dim_p)) {
                ph = std::max<size_t>(ph, w.heads);
                pd = std::max<size_t>(pd, (size_t)w.heads * w.dim_p);
                if (w.delta()) pdd = std::max<size_t>(pdd, (size_t)w.heads * w.dim_p);
            }
        }
    }
    m->slab_floats = std::max<size_t>(R * nmax, (size_t)32 * std::min<size_t>(R, 128) * nmax);
    if (f32 || m->V_l % 16) m->slab_floats = std::max<size_t>(m->slab_floats, (size_t)m->max_seqs * Vp);
    if (!rc) rc = zalloc((void**)&m->resid, R * ldr * 4);
    if (!rc) rc = dmalloc(ctx, &m->slabs, m->slab_floats);
    if (!rc && two) rc = dmalloc(ctx, &slabs2, m->slab_floats);
    if (!rc) rc = dmalloc(ctx, &m->red, R * ldr * (two ? 2 : 1));
    struct { float** p; size_t n; } bufs[] = {{&q, nq}, {&k, nk}, {&v, nv}, {&g, ng}, {&beta, nb}, {&gate_in, nin}, {&out, no}, {&v_first, nvf}};
    for (auto& b : bufs) if (!rc && b.n) rc = zalloc((void**)b.p, (R + kPiece) * b.n * 4);  // pieces read past the last row
    if (!rc) rc = dmalloc(ctx, &ssq, R * 2);
    if (!rc && po && !f32) rc = dmalloc(ctx, &part_o, po);
    if (!rc && pm && !f32) rc = dmalloc(ctx, &part_ml, pm);
    if (!rc) rc = experts.alloc(ctx, f32);
    if (f32) {
        if (!rc) rc = zalloc((void**)&y, R * Kw * 4);
        for (int b = 0; b < (two ? 2 : 1); ++b) if (!rc) rc = zalloc((void**)&ctx_f[b], R * kc * 4);
        if (!rc && ffp) rc = zalloc((void**)&act_f, R * ffp * 4);
    } else {
        // activation planes are read in whole 16-row blocks; columns past a layer's own width meet zero weights
        for (bf16_bits** p : {&m->xh, &m->xl}) if (!rc) rc = zalloc((void**)p, R16 * Kw * 2);
        for (bf16_bits** p : {&m->ctxh, &m->ctxl}) if (!rc) rc = zalloc((void**)p, R16 * kc * 2);
        if (two) for (bf16_bits** p : {&ctx2h, &ctx2l}) if (!rc) rc = zalloc((void**)p, R16 * kc * 2);
        if (ffp) for (bf16_bits** p : {&m->xh2, &m->xl2}) if (!rc) rc = zalloc((void**)p, R16 * ffp * 2);
    }
    piece_cap = (int)(R / kPiece) + m->max_seqs;
    struct { float** p; size_t n; } pieces[] = {{&pc_pair, ph * kPiece * kPiece}, {&pc_k, pd * kPiece}, {&pc_q, pdd * kPiece}, {&pc_w, pdd * kPiece}, {&pc_decay, pdd}};
    for (auto& b : pieces) if (!rc && b.n) rc = dmalloc(ctx, b.p, (size_t)piece_cap * b.n);
    if (!rc) rc = dmalloc(ctx, &d_seg, (size_t)4 * m->max_seqs);
    if (!rc) rc = dmalloc(ctx, &d_piece, (size_t)2 * piece_cap);
    if (!rc) HIPCHK(ctx, hipHostMalloc((void**)&h_seg, ((size_t)4 * m->max_seqs + 2 * piece_cap) * sizeof(int), hipHostMallocDefault));
    m->rope_len = (int)std::min<int64_t>((int64_t)m->max_blocks * kBlockTokens, 1 << 20);  // positions a block table covers
    for (RopeTable& r : ropes) if (!rc) rc = r.upload(ctx, m->rope_len);
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

int HybridModel::attention(nvllm_model* m, HybridMixer& w, MixerState& st, int b, int ns, int ld, int R, int n_tiles, int qt, int ctx_packed) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    PagedKV kv;
    kv.k = st.kc; kv.v = st.vc; kv.f32 = cfg.f32; kv.kv = w.kv;
    kv.dim = w.c.dim; kv.dim_p = w.dim_p; kv.vdim = w.c.vdim; kv.vdim_p = w.vdim_p;
    const float* in = m->slabs + w.col0;
    const int64_t stride = (int64_t)R * ld;
    const float q_scale = (float)(w.c.scale * 1.4426950408889634);
    if (w.per_head_norm()) {
        ConvAttnRowsArgs ra;
        ra.in = in; ra.n_slabs = ns; ra.ld = ld; ra.slab_stride = stride; ra.in_bias = w.bias;
        ra.heads = w.heads; ra.taps = w.c.conv_taps; ra.conv = w.conv; ra.eps = (float)cfg.norm_eps; ra.q_scale = q_scale;
        if (w.rope >= 0) { ra.rot = w.c.rot_dim; ra.cos = ropes[w.rope].cos; ra.sin = ropes[w.rope].sin; }
        ra.history = st.history; ra.slots = m->max_seqs; ra.seg = segments(m, R, qt); ra.pos = m->d_pos; ra.slot = m->d_slot;
        ra.block_tables = m->d_block_tables; ra.max_blocks = m->max_blocks; ra.q = q; ra.kv = kv;
        PROF(m, PROF_QK, launch_conv_attn_rows(ra, R, s));
        if (!ra.seg.single) PROF(m, PROF_QK, launch_conv_attn_history(ra, s));
    } else {
        AttnRowsArgs ra;
        ra.in = in; ra.n_slabs = ns; ra.ld = ld; ra.slab_stride = stride; ra.bias = w.bias;
        ra.heads = w.heads; ra.qn = w.qn; ra.kn = w.kn; ra.eps = (float)cfg.norm_eps; ra.q_scale = q_scale;
        ra.q_all = w.c.heads * w.c.dim; ra.k_all = w.c.kv_heads * w.c.dim;
        ra.mix = w.c.v_mix ? (w.last_v ? 2 : 1) : 0; ra.lambda = w.vmix; ra.v_first = v_first;
        ra.pos = m->d_pos; ra.slot = m->d_slot; ra.block_tables = m->d_block_tables; ra.max_blocks = m->max_blocks; ra.q = q;
        ra.kv = kv;
        if (ctx->tp_size > 1) {  // the norms run over every rank's columns
            const int c0[2] = {0, w.heads * w.c.dim}, n[2] = {w.heads * w.c.dim, w.kv * w.c.dim};
            HIPCHK(ctx, launch_rows_ssq(in, ns, stride, ld, w.bias, c0, n, R, ssq, s));
            int rc = comm_allreduce_sum(ctx, ssq, (size_t)R * 2);
            if (rc) return rc;
            ra.ssq = ssq;
        }
        PROF(m, PROF_QK, launch_attn_rows(ra, R, s));
    }
    BiasAttnArgs aa;
    aa.q = q; aa.kv = kv; aa.heads = w.heads; aa.bias = w.table; aa.n_bias = w.n_bias; aa.window = w.c.window; aa.sink = w.sink;
    aa.block_tables = m->d_block_tables; aa.max_blocks = m->max_blocks;
    aa.tile_row0 = m->d_tile_row0; aa.tile_nrows = m->d_tile_nrows; aa.tile_slot = m->d_tile_slot; aa.tile_order = m->d_tile_order;
    aa.pos = m->d_pos; aa.slot = m->d_slot; aa.ld = w.Kc; aa.packed = ctx_packed;
    if (cfg.f32) aa.of = ctx_f[b];
    else { aa.oh = b ? ctx2h : m->ctxh; aa.ol = b ? ctx2l : m->ctxl; }
    if (!w.matrix_core || opt_plain) {
        PROF(m, PROF_ATTN, launch_bias_attn_plain(aa, R, s));
    } else if (qt == 1) {
        // split the visible context when (sequences x groups of heads) alone leave CUs idle; a window may begin inside a tile
        const int gqa = w.heads / w.kv, base = R * w.kv * ((gqa + 15) / 16), len = m->cur_max_len;
        const int tiles = w.c.window > 0 && w.c.window < len ? (w.c.window + 31) / 32 + 1 : (len + 31) / 32;
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

int HybridModel::recurrence(nvllm_model* m, HybridMixer& w, MixerState& st, int b, int ns, int ld, int R, int qt, int ctx_packed) {
    nvllm_ctx* ctx = m->ctx;
    hipStream_t s = ctx->stream;
    const Segments seg = segments(m, R, qt);
    const float* in = m->slabs + w.col0;
    const int64_t stride = (int64_t)R * ld;
    RecurArgs rc;
    rc.q = q; rc.k = k; rc.v = v; rc.heads = w.heads; rc.q_heads = w.kv; rc.dim_p = w.dim_p; rc.vdim = w.c.vdim; rc.vdim_p = w.vdim_p;
    rc.state = st.state; rc.seg = seg; rc.pos = m->d_pos; rc.o = out;
    GatedNormArgs gn;
    gn.o = out; gn.heads = w.heads; gn.vdim = w.c.vdim; gn.vdim_p = w.vdim_p; gn.gate_head = w.vdim_p;
    gn.weight = w.onorm; gn.eps = (float)cfg.norm_eps; gn.ld = w.Kc; gn.packed = ctx_packed;
    if (cfg.f32) gn.of = ctx_f[b];
    else { gn.oh = b ? ctx2h : m->ctxh; gn.ol = b ? ctx2l : m->ctxl; }
    if (w.delta()) {
        DeltaRowsArgs da;
        da.in = in; da.n_slabs = ns; da.ld = ld; da.slab_stride = stride;
        da.heads = w.heads; da.kv = w.kv; da.dim = w.c.dim; da.dim_p = w.dim_p; da.vdim = w.c.vdim; da.vdim_p = w.vdim_p; da.rank_p = w.rank_p; da.taps = w.c.conv_taps;
        da.conv = w.conv; da.q_scale = 1.0f / std::sqrt((float)w.c.dim);
        da.history = st.history; da.slots = m->max_seqs; da.seg = seg; da.pos = m->d_pos; da.slot = m->d_slot;
        da.q = q; da.k = k; da.v = v; da.beta = beta; da.gate_in = gate_in;
        if (w.head_decay()) { da.rate = w.rate; da.dt = w.dt; da.decay = g; }
        PROF(m, PROF_QK, launch_delta_rows(da, R, s));
        if (!seg.single) PROF(m, PROF_QK, launch_delta_history(da, s));
        rc.beta = beta;
        if (w.head_decay()) {
            rc.gh = g;
            gn.gate = in + w.gate0; gn.gate_row = ld; gn.gate_head = w.c.vdim; gn.gate_slabs = ns; gn.gate_stride = stride;
        } else {
            HeadGemmArgs ga;
            ga.x = gate_in; ga.x_row = 2 * w.rank_p; ga.x_head = w.rank_p;
            ga.w = w.gates.data; ga.w_head = (int64_t)w.Ng * w.rank_p / 8; ga.N = ga.n_valid = w.Ng; ga.K = w.rank_p; ga.heads = 2; ga.M = R; ga.exact = cfg.f32;
            ga.y = g; ga.y_row = 2 * w.Ng; ga.y_head = w.Ng; ga.decay_rate = w.rate; ga.decay_bias = w.dt;
            PROF(m, PROF_GEMM, launch_delta_gates(ga, s));
            rc.g = g; rc.g_row = 2 * w.Ng;
            gn.gate = g + w.Ng; gn.gate_row = 2 * w.Ng;
        }
    } else {
        LinearRowsArgs la;
        la.in = in; la.n_slabs = ns; la.ld = ld; la.slab_stride = stride;
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
    const bool f32 = cfg.f32 != 0, tp = ctx->tp_size > 1;
    m->tap_rows = R;
    AddNormArgs base;
    base.W = cfg.width; base.ldr = ldr; base.ldx = Kw; base.eps = (float)cfg.norm_eps;
    base.ids = m->d_ids; base.embed = embed; base.embed_scale = (float)cfg.embed_scale;
    auto plan = [&](const PackedW& w) { return f32 ? ProductPlan() : plan_product(m, R, w); };
    // the next sublayer's input: the stream or its norm `pre`, as planes in the order its product wants
    auto outputs = [&](AddNormArgs& a, const float* pre, int packed) {
        a.w[0] = pre;
        a.raw = !pre;
        if (f32) a.y[0] = y;
        else { a.xh[0] = m->xh; a.xl[0] = m->xl; a.packed[0] = packed; }
    };
    ProductPlan pin = plan(layers[runs[0].layer].in);
    AddNormArgs first = base;
    first.residual_out = m->resid;
    outputs(first, layers[runs[0].layer].pre1, pin.packed);
    PROF(m, PROF_NORM, launch_add_norm(first, R, s));
    // a sublayer's output, pending on the stream: x <- x + mult norm(sum)
    AddNormArgs sum = base;
    float* const tap = tp ? m->slabs : m->red;  // not the last sum's input
    bool reduced = false;
    auto reduce = [&]() -> int {
        if (!tp || reduced) return NVLLM_OK;
        reduced = true;
        AddNormArgs a = base;
        a.ids = nullptr;
        a.in = sum.in; a.n_slabs = sum.n_slabs; a.slab_stride = sum.slab_stride;
        a.gather = sum.gather; a.gather_row = sum.gather_row; a.n_gather = sum.n_gather;
        a.residual_out = m->red;
        HIPCHK(ctx, launch_add_norm(a, R, s));
        if (sum.in2) {
            a.in = sum.in2; a.n_slabs = sum.n_slabs2; a.slab_stride = sum.slab_stride2; a.residual_out = m->red + (size_t)R * ldr;
            HIPCHK(ctx, launch_add_norm(a, R, s));
        }
        int rc = comm_allreduce_sum(ctx, m->red, (size_t)R * ldr * (sum.in2 ? 2 : 1));
        if (rc) return rc;
        sum.in = m->red; sum.n_slabs = 1; sum.n_gather = 0;
        if (sum.in2) { sum.in2 = m->red + (size_t)R * ldr; sum.n_slabs2 = 1; }
        return NVLLM_OK;
    };
    auto add = [&](const float* weight, const float* pre, int packed, bool again) -> int {
        int rc = reduce();
        if (rc) return rc;
        AddNormArgs a = sum;
        a.post_w = weight; a.post_mult = (float)cfg.residual_mult; a.residual_in = m->resid;
        a.residual_out = m->resid; a.again = again;
        outputs(a, pre, packed);
        PROF(m, PROF_NORM, launch_add_norm(a, R, s));
        return NVLLM_OK;
    };
    auto add_tap = [&](const float* weight) -> int {  // the stream after this sublayer, left beside the stream itself
        int rc = reduce();
        if (rc) return rc;
        AddNormArgs t = sum;
        t.post_w = weight; t.post_mult = (float)cfg.residual_mult; t.residual_in = m->resid; t.residual_out = tap;
        HIPCHK(ctx, launch_add_norm(t, R, s));
        return NVLLM_OK;
    };
    for (size_t run = 0; run < runs.size(); ++run) {
        HybridLayer& w = layers[runs[run].layer];
        const bool last = run + 1 == runs.size(), mlp = w.ff || w.experts.on();
        const HybridLayer* next = last ? nullptr : &layers[runs[run + 1].layer];
        const bool again = !last && runs[run + 1].again;
        const ProductPlan pnext = last ? ProductPlan() : plan(next->in);
        ProductPlan po[2], pu, pd;
        for (int b = 0; b < w.branches; ++b) po[b] = plan(w.mix[b].o);
        if (w.ff) { pu = plan(w.up); pd = plan(w.down); }
        int ns = 1, rc = product(m, pin, y, m->xh, m->xl, w.in, m->slabs, R, &ns);
        for (int b = 0; b < w.branches && !rc; ++b)
            rc = w.mix[b].attention() ? attention(m, w.mix[b], runs[run].st[b], b, ns, w.N, R, n_tiles, qt, po[b].packed)
                                      : recurrence(m, w.mix[b], runs[run].st[b], b, ns, w.N, R, qt, po[b].packed);
        sum = base;
        reduced = false;
        sum.in = m->slabs; sum.slab_stride = (int64_t)R * ldr; sum.in_bias = w.mix[0].ob;
        if (!rc) rc = product(m, po[0], ctx_f[0], m->ctxh, m->ctxl, w.mix[0].o, m->slabs, R, &sum.n_slabs);
        if (!rc && w.branches == 2) {
            sum.in2 = slabs2; sum.slab_stride2 = (int64_t)R * ldr;
            sum.branch_w[0] = w.mix[0].out_norm; sum.branch_w[1] = w.mix[1].out_norm;
            rc = product(m, po[1], ctx_f[1], ctx2h, ctx2l, w.mix[1].o, slabs2, R, &sum.n_slabs2);
        }
        if (rc) return rc;
        const float* weight = w.norm1;
        if (mlp) {
            const int packed = w.ff ? pu.packed : f32 || experts_gather(m, w.experts, R) ? 0 : 1;
            rc = add(w.norm1, w.pre2, packed, false);
            if (rc) return rc;
            sum = base;
            reduced = false;
            if (w.ff && f32) {
                rc = exact_product(m, y, w.up, m->slabs, R);
                if (rc) return rc;
                PROF(m, PROF_SILU, launch_act(w.act(), m->slabs, 1, 0, R, w.ff_p, nullptr, nullptr, 0, act_f, s));
            } else if (w.ff) {
                rc = run_act(m, pu, w.act(), m->xh, m->xl, w.up, R, m->xh2, m->xl2, pd.packed);
            }
            if (!rc && w.ff) {
                sum.in = m->slabs; sum.slab_stride = (int64_t)R * ldr;
                rc = product(m, pd, act_f, m->xh2, m->xl2, w.down, m->slabs, R, &sum.n_slabs);
            } else if (!rc) {
                BranchSum ff;
                rc = run_experts(m, w.experts, experts, m->xh, m->xl, packed, m->xh, m->xl, f32 ? y : nullptr, R, nullptr, &ff);
                sum.gather = ff.gather; sum.gather_row = ff.gather_row; sum.n_gather = ff.n_gather;
            }
            if (rc) return rc;
            weight = w.norm2;
        }
        if (m->taps && (last || again)) rc = add_tap(weight);
        if (!rc && !last) rc = add(weight, next->pre1, pnext.packed, again);
        if (rc) return rc;
        pin = pnext;
        if (m->taps)
            HIPCHK(ctx, hipMemcpy2DAsync(m->tap_res + run * (size_t)m->max_rows * m->H, (size_t)m->H * 4, last || again ? tap : m->resid, (size_t)ldr * 4, (size_t)m->H * 4, R,
                                         hipMemcpyDeviceToDevice, s));
        if (last && n_last > 0) {
            rc = reduce();
            if (rc) return rc;
            AddNormArgs a = sum;
            a.post_w = weight; a.post_mult = (float)cfg.residual_mult; a.residual_in = m->resid;
            a.row_idx = m->d_last_rows;
            outputs(a, final_norm, 0);
            PROF(m, PROF_NORM, launch_add_norm(a, n_last, s));
        }
    }
    if (n_last <= 0) return NVLLM_OK;
    return output_head(m, head, Kw, Vp, f32 ? y : nullptr, 0.f, n_last, logits_row0);
}
