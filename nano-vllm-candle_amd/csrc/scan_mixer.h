// Host half of the selective-scan mixer (scan.h) for the decoders built from layer descriptions: weights, state, plan of a chunk, forward.
#pragma once
#include "decoder.h"
#include "scan.h"

struct ScanMixer {
    int inner = 0, state = 0, taps = 0, rank = 0;      // of the whole model (inner 0: the layer has another mixer)
    int n = 0, n_p = 0, S = 0, rank_p = 0, Kc = 0;     // this rank's channels, padded; padded states; width of the context planes
    int Nin = 0, Nx = 0;
    PackedW in, x, dt;                                 // [x | z], [dt | B | C] (parts at 0, rank_p, rank_p + S), step sizes
    float *conv = nullptr, *conv_b = nullptr, *dt_b = nullptr, *A = nullptr, *D = nullptr;
    float *st = nullptr, *history = nullptr;           // per slot
    bool on() const { return inner > 0; }
    int create(nvllm_ctx* ctx, int inner, int state, int taps, int rank, int Kw, bool f32);
    void destroy();
    int load(nvllm_model* m, const char* name, const char* s, const HostMat& h, int64_t rows, int64_t cols, int W);  // `s`: behind "mix."; 1: not a tensor of the mixer
    static std::vector<std::string> tensors() { return {"in", "conv", "conv.b", "x", "dt", "dt.b", "A_log", "D"}; }
    int kv_alloc(nvllm_model* m);
    void free_kv();
    size_t bytes() const { return in.bytes() + x.bytes() + dt.bytes() + (size_t)(n_p * S + n * (taps + 3)) * 4; }
    size_t state_bytes() const { return (size_t)(n_p * S + (taps - 1) * n) * 4; }
};

struct ScanScratch {
    float *x = nullptr, *dt = nullptr, *dbc = nullptr, *carry = nullptr, *carry_dt = nullptr;
    bf16_bits *xh = nullptr, *xl = nullptr;
    int *d_plan = nullptr, *h_plan = nullptr, piece_cap = 0, seg_cap = 0;
    int n_seg = 0, n_piece = 0, several = 0;
    void reserve(const ScanMixer& w, size_t rows);
    int alloc(nvllm_model* m, bool f32);
    void release();
    int plan(nvllm_model* m, const int* slot, const int* seq, int R);  // segments and pieces of a prompt chunk
private:
    size_t n_x = 0, n_dt = 0, n_dbc = 0, n_carry = 0, n_carry_dt = 0;
    int waves = 0;  // of one piece in the narrowest layer
};

// mixer of R rows up to the context planes m->ctxh / ctxl (or ctx_f), read from the input projection's slabs `in`; other_slabs: scratch of slab_floats
int run_scan(nvllm_model* m, ScanMixer& w, ScanScratch& x, const float* in, int n_slabs, float* other_slabs, int R, int qt, float* ctx_f, int ctx_packed);
