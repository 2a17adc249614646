// What the decoders built from layer descriptions share on the host side: the interface api.cpp drives them through, reading of host
// tensors into packed weights, matrix products with the kernel that fits the row count, the output head.
#pragma once
#include <algorithm>
#include <cstring>
#include <string>

#include "model.h"

// A decoder behind nvllm_model's shared half (sequences, blocks, slots, chunks of rows, sampling, decode pipelining: api.cpp).
struct DecoderImpl {
    virtual ~DecoderImpl() = default;
    virtual int load_tensor(nvllm_model* m, const char* name, const void* data, int dtype, const int64_t* shape, int ndim) = 0;
    virtual int finalize(nvllm_model* m) = 0;
    virtual int kv_alloc(nvllm_model* m) = 0;   // pool sizes are set, the shared buffers exist
    virtual void free_kv() = 0;
    virtual int64_t weight_bytes() const = 0;
    virtual int64_t kv_bytes_per_token() const = 0;
    virtual int64_t kv_read_bytes(int len) const = 0;  // cache (and state) bytes a decode step moves for a sequence of len tokens
    virtual int tile_rows(int qt) const = 0;           // rows of a q-tile (qt = 1: decode)
    virtual bool recurrent() const { return false; }   // carries state that cannot step back: such a step starts the sequence again
    // metadata of the chunk about to run beyond the q-tiles (R rows; tiles already uploaded); decode continued on the device needs none
    virtual int plan_chunk(nvllm_model* m, const int* pos, const int* slot, const int* seq, int R, const int* tile_row0, int n_tiles, int qt) = 0;
    virtual int forward_chunk(nvllm_model* m, int R, int n_tiles, int qt, int n_last, int logits_row0) = 0;
    virtual int option(const char* name, int value) { (void)name; (void)value; return 1; }        // 0: taken
    virtual int counter(const char* name, int64_t* value) const { (void)name; (void)value; return 1; }
};

static inline int up(int v, int q) { return (v + q - 1) / q * q; }
// features of a wide matrix: a whole number of the prompt product's 192- or 256-feature tiles
static inline int up_tile(int v) { return v <= 256 ? 256 : std::min(up(v, 192), up(v, 256)); }

// ---- host tensors ---------------------------------------------------------------------------------------------------------
// bf16 view of a host tensor
struct HostMat {
    const void* p;
    int dtype;
    int64_t cols;
    uint16_t at(int64_t r, int64_t c) const {
        const int64_t i = r * cols + c;
        return dtype == NVLLM_DTYPE_F32 ? host_f32_to_bf16(((const float*)p)[i]) : ((const uint16_t*)p)[i];
    }
    float f32(int64_t i) const {
        if (dtype == NVLLM_DTYPE_F32) return ((const float*)p)[i];
        const uint32_t u = (uint32_t)((const uint16_t*)p)[i] << 16;
        float f;
        memcpy(&f, &u, 4);
        return f;
    }
};

// rows [row0, row0 + rows) of w <- elem(r, c), c < cols (columns beyond are zero)
template <typename F>
static int put_rows(nvllm_ctx* ctx, const PackedW& w, int row0, int rows, int cols, int ileave, F elem) {
    std::vector<uint16_t> tmp((size_t)rows * w.K, 0);
    for (int r = 0; r < rows; ++r)
        for (int c = 0; c < cols; ++c) tmp[(size_t)r * w.K + c] = elem(r, c);
    bf16_bits* d = nullptr;
    HIPCHK(ctx, hipMalloc((void**)&d, tmp.size() * 2));
    hipError_t e = hipMemcpyAsync(d, tmp.data(), tmp.size() * 2, hipMemcpyHostToDevice, ctx->stream);
    if (e == hipSuccess) e = launch_pack_rows(w, row0, rows, d, w.K, ileave, ctx->stream);
    if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
    (void)hipFree(d);
    HIPCHK(ctx, e);
    return NVLLM_OK;
}

// weights and vectors on the device, zero until loaded (padding stays zero)
static inline int alloc_packed(nvllm_ctx* ctx, PackedW& w, int N, int K) {
    w.N = N; w.K = K;
    HIPCHK(ctx, hipMalloc((void**)&w.data, w.bytes()));
    HIPCHK(ctx, hipMemsetAsync(w.data, 0, w.bytes(), ctx->stream));
    return NVLLM_OK;
}
static inline int alloc_vec(nvllm_ctx* ctx, float** p, size_t n) {
    int rc = dmalloc(ctx, p, n);
    if (!rc) HIPCHK(ctx, hipMemsetAsync(*p, 0, std::max<size_t>(n * 4, 16), ctx->stream));
    return rc;
}

// ---- products ---------------------------------------------------------------------------------------------------------------
enum { P_GENERIC = 0, P_ROW, P_STREAM, P_TILE };
struct ProductPlan {
    int kind = P_GENERIC;
    int packed = 0;     // input planes in fragment order
    int max_split = 1;  // K slabs that fit the slab buffer
};

// gate/up + activation as hi/lo planes: fused into the product where a kernel has the epilogue, else slabs + one row kernel
struct GluPlan {
    int kind = P_GENERIC;  // P_STREAM: slabs + activation kernel on a product plan
    int packed = 0, out_packed_ok = 0;
    ProductPlan slabs;
};
// y = x.W^T left as f32 slabs
ProductPlan plan_product(const nvllm_model* m, int R, const PackedW& w);
int run_product(nvllm_model* m, const ProductPlan& p, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, float* out, int R, int* n_slabs);
GluPlan plan_glu(const nvllm_model* m, int R, const PackedW& w, bool want_packed_out);
int run_glu(nvllm_model* m, const GluPlan& g, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, int R, const GluSpec& spec,
            bf16_bits* oh, bf16_bits* ol, int out_packed);
// activation of x.W^T as hi/lo planes oh / ol on the plan of the product, through m->slabs where no epilogue fits
int run_act(nvllm_model* m, const ProductPlan& p, nvllm::Act act, const bf16_bits* xh, const bf16_bits* xl, const PackedW& w, int R, bf16_bits* oh, bf16_bits* ol, int out_packed);
// 32-bit product of row-major f32 rows
int exact_product(nvllm_model* m, const float* x, const PackedW& w, float* out, int R);

// logits (soft-capped when cap > 0) and arg-max of n_last normed rows: f32 rows y, or the planes m->xh / m->xl (row-major) when y is null
int output_head(nvllm_model* m, const PackedW& head, int Kw, int Vp, const float* y, float cap, int n_last, int logits_row0);
