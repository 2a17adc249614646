// Host half of a routed feed-forward (moe.h) for the decoders built from layer descriptions: weights, scratch shared by the layers, forward.
#pragma once
#include "decoder.h"
#include "moe.h"

// a feed-forward's summands of the residual, as AddNormArgs takes them
struct BranchSum {
    const float* in = nullptr;
    int n_slabs = 1;
    int64_t slab_stride = 0;
    const float* scale = nullptr;
    const float* gather = nullptr;
    const int* gather_row = nullptr;
    int n_gather = 0;
};

struct ExpertsBlock {
    int experts = 0, top = 0, ff_all = 0, shared_all = 0;  // widths of the whole model (shared_all 0: no shared expert)
    int ff = 0, ff_p = 0, sh = 0, sh_p = 0;                // this rank's share, padded
    int weight_in = 1;
    int gated = 0, softmax = 0, groups = 1, keep = 1;      // set before create: experts silu(gate) up (else squared ReLU; no shared one beside), scores and groups as in RouteArgs
    int up_rows() const { return gated ? 2 * ff_p : ff_p; }
    int W = 0, Kw = 0, ldr = 0, Nr = 0;
    PackedW router;                                        // a row per expert, then the shared gate's
    PackedW wup, down, sup, sdown;                         // wup [experts * up_rows x Kw], down [experts * ldr x ff_p]
    bool on() const { return experts > 0; }
    int create(nvllm_ctx* ctx, int experts, int top, int ff, int shared, int W, int Kw, int ldr, bool f32);
    void destroy();
    // `s`: the name behind "mlp."; 1: not a tensor of this block
    int load(nvllm_model* m, const char* name, const char* s, const HostMat& h, int64_t rows, int64_t cols);
    std::vector<std::string> tensors() const;
    size_t bytes() const { return router.bytes() + wup.bytes() + down.bytes() + sup.bytes() + sdown.bytes(); }
    size_t step_bytes() const;                             // weights one token reads
};

struct ExpertsScratch {
    int cap = 0, lda = 0;
    float *z = nullptr, *score = nullptr, *gate = nullptr, *pre = nullptr, *post = nullptr, *out = nullptr, *act_f = nullptr;
    int *chosen = nullptr, *place = nullptr, *src = nullptr, *tile_group = nullptr, *cursor = nullptr;
    bf16_bits *ah = nullptr, *al = nullptr, *sh = nullptr, *sl = nullptr;
    void reserve(const ExpertsBlock& e, size_t rows);       // sizes first, for every block, ...
    int alloc(nvllm_ctx* ctx, bool f32);                    // ... then the buffers
    void release();
private:
    size_t n_z = 0, n_top = 0, n_place = 0, n_rows = 0, n_out = 0, n_sh = 0;
    friend struct ExpertsBlock;
};

// long prompt chunks gather the experts' rows from row-major planes, beside those of the shared expert (an ordinary product) and the router
bool experts_gather(const nvllm_model* m, const ExpertsBlock& e, int R);
// the branch of R normed rows: planes xh / xl (ld Kw), and rh / rl row-major where experts_gather says so, or f32 rows y (32-bit mode); slabs2:
// scratch of slab_floats
int run_experts(nvllm_model* m, ExpertsBlock& e, ExpertsScratch& x, const bf16_bits* xh, const bf16_bits* xl, int packed, const bf16_bits* rh, const bf16_bits* rl,
                const float* y, int R, float* slabs2, BranchSum* out);
