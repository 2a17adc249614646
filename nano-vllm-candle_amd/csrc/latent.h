// Latent-attention decoders (compressed K/V: every token caches one latent vector and one rotated key part shared by all
// heads): launchers of latent_ops.hip / latent_attn.hip / latent_prefill.hip.
#pragma once
#include "kernels.h"

namespace nvllm {

constexpr int kLatentTileRows = 128;  // rows of one q-tile of a prompt chunk (a decode tile is one row)
constexpr int kLatentMaxParts = 64;   // split-KV partitions per row

// ---- residual add + up to two norms of the same row ---------------------------------------------------------------------
// s = sum of the partial sums in / in2 (or embed[id] * embed_scale) (+ residual); residual_out = s; post_w: s = residual + post_mult * norm(sum) instead;
// output k = s / sqrt(mean(s^2) + eps) * w[k], as bf16 hi/lo planes and/or f32.  Rows are W wide, stored with stride ldr
// (multiple of 16, zeros beyond W); planes / y have stride ldx (zeros beyond W).
struct AddNormArgs {
    const float* in = nullptr;
    int n_slabs = 1;
    int64_t slab_stride = 0;
    const float* in2 = nullptr;        // a second product's partial sums (the other branch of a parallel layer)
    int n_slabs2 = 1;
    int64_t slab_stride2 = 0;
    const float* in2_scale = nullptr;  // [rows] factor of in2
    const float* gather = nullptr;     // more summands: rows gather_row[r][0 .. n_gather) of a [*][ldr] array
    const int* gather_row = nullptr;
    int n_gather = 0;
    const uint32_t* ids = nullptr;
    const bf16_bits* embed = nullptr;  // [vocab][ldr]
    float embed_scale = 1.f;
    const float* residual_in = nullptr;
    float* residual_out = nullptr;
    const int* row_idx = nullptr;      // input row of output row r (outputs are compact)
    int W = 0, ldr = 0, ldx = 0;
    int ld_in = 0;                     // row stride of `in` where it is not ldr (16-row form only)
    float eps = 0.f;
    const float* in_bias = nullptr;    // [ldr] added to the sum of `in`
    const float* post_w = nullptr;
    float post_mult = 1.f;
    const float* branch_w[2] = {nullptr, nullptr};  // both set, with post_w: half the sum of `in` and `in2`, each RMS-normed with its weight first
    int again = 0;                     // with post_w: the new residual takes embed[id] * embed_scale on top (`in` is read beside ids)
    const float* w[2] = {nullptr, nullptr};  // nullptr: output k absent
    int center = 0;                    // layer norm: the mean is taken off before the root mean square and the weight
    int raw = 0;                       // output 0 is s itself (w[0] unused)
    bf16_bits* xh[2] = {nullptr, nullptr};
    bf16_bits* xl[2] = {nullptr, nullptr};
    float* y[2] = {nullptr, nullptr};
    int packed[2] = {0, 0};            // planes in xpack_off order (ldx % 32 == 0)
};
hipError_t launch_add_norm(const AddNormArgs& a, int rows, hipStream_t s);

// ---- latent cache ------------------------------------------------------------------------------------------------------
// One cached token = D = rank_p + rot_p elements (rank and rot padded to multiples of 32, zeros): the normed latent, then the
// rotated shared key part.  Blocks of kBlockTokens tokens in QK^T fragment order (k_packed_offset with hd = D), f16 or f32.
struct LatentCache {
    void* data = nullptr;  // [num_blocks][kBlockTokens * D]
    int f32 = 0;
    int rank = 0, rank_p = 0, rot = 0, rot_p = 0;
    __host__ __device__ int D() const { return rank_p + rot_p; }
};

// ---- rows after the q / latent projection: split, norm, rotate, cache write ---------------------------------------------
// qkv row: [heads][dim + rot] query; kv row: rank + rot of the latent projection (kv nullptr: the rows write no cache).  Writes q [rows][heads][dim_p + rot_p] f32
// (scaled; unrotated part, then rotated part; zero padded) and the token's latent and key part into the cache.
struct LatentRowsArgs {
    const float* qkv = nullptr;
    int n_slabs = 1, ldq = 0;
    int64_t slab_stride = 0;
    const float* kv = nullptr;
    int kv_slabs = 1, ldkv = 0;
    int64_t kv_stride = 0;
    int heads = 0, dim = 0, dim_p = 0;
    float scale = 1.f;             // score scale * log2(e)
    const float* norm_w = nullptr; // [rank]
    float eps = 0.f;
    const float* cos = nullptr;    // [positions][rot / 2]
    const float* sin = nullptr;
    const int* pos = nullptr;
    const int* slot = nullptr;
    const int* block_tables = nullptr;
    int max_blocks = 0;
    float* q = nullptr;
    LatentCache cache;
};
hipError_t launch_latent_rows(const LatentRowsArgs& a, int rows, hipStream_t s);
// the cache half of it alone (the expanded prompt kernel splits and rotates the query itself)
hipError_t launch_latent_cache(const LatentRowsArgs& a, int rows, hipStream_t s);

// query latents: RMS norm of the first `rank` columns of the input projection, as planes / f32 rows [rows][ldx]; kv (kv.kv set): the rows'
// latents and key parts into the cache
struct QueryLatentArgs {
    const float* in = nullptr;
    int n_slabs = 1, ld = 0;
    int64_t slab_stride = 0;
    int rank = 0, ldx = 0;
    const float* norm_w = nullptr;
    float eps = 0.f;
    bf16_bits* xh = nullptr;
    bf16_bits* xl = nullptr;
    float* y = nullptr;
    int packed = 0;
};
hipError_t launch_query_latent(const QueryLatentArgs& a, const LatentRowsArgs& kv, int rows, hipStream_t s);

// ---- per-head products and 32-bit products -------------------------------------------------------------------------------
// y[r][h][n] = sum_k x[r][h][k] W[h][n][k]: x f32 (element strides), W packed per head (N % 16 == 0, K % 32 == 0).
// exact = 0: x as bf16 hi + lo, 16x16x32 bf16 MFMA; exact = 1: everything in f32 (16x16x4 f32 MFMA, weights widened).
// decay_bias set (f32 output): softplus(y + decay_bias[n]); decay_rate too: head 0 leaves exp(-decay_rate[n] softplus(y + decay_bias[n])),
// every other head sigmoid(y).
// Output: f32 with strides, or bf16 hi/lo planes [rows][ld] at column h * n_valid + n (n < n_valid).
struct HeadGemmArgs {
    const float* x = nullptr;
    int64_t x_row = 0, x_head = 0;
    const uint4* w = nullptr;
    int64_t w_head = 0;            // uint4 per head
    int N = 0, K = 0, heads = 1, M = 0, n_valid = 0;
    int exact = 0;
    const float* decay_rate = nullptr;
    const float* decay_bias = nullptr;
    float* y = nullptr;            // columns >= n_valid are not written
    int64_t y_row = 0, y_head = 0;
    bf16_bits* yh = nullptr;
    bf16_bits* yl = nullptr;
    int ld = 0, packed = 0;
};
hipError_t launch_head_gemm(const HeadGemmArgs& a, hipStream_t s);

// ---- attention over the latent cache (absorbed form) ----------------------------------------------------------------------
// score = qlat . c + qrot . k_rot (scale folded into q); weights over positions [pos - window + 1, pos]; output the weighted
// latent [rows][heads][rank_p] f32.
struct LatentAttnArgs {
    const float* qlat = nullptr;   // [rows][heads][rank_p]
    const float* qrot = nullptr;   // rotated part of q: element strides below
    int64_t qrot_row = 0, qrot_head = 0;
    LatentCache cache;
    const int* block_tables = nullptr;
    int max_blocks = 0;
    const int* tile_row0 = nullptr;
    const int* tile_nrows = nullptr;
    const int* tile_slot = nullptr;
    const int* pos = nullptr;
    const int* slot = nullptr;     // per row
    int single = 0;                // every q-tile is one row, tile i = row i
    int heads = 0, window = 0;     // window <= 0: causal without a window
    const float* sink = nullptr;   // [heads] one more term 2^sink of every denominator; nullptr: none
    float* out = nullptr;          // [rows][heads][rank_p]
    // split-KV: workgroup z covers part_tiles 32-token tiles counted from the first visible tile of its q-tile
    int part_tiles = 0, max_parts = 1;
    float* part_o = nullptr;       // [rows][heads][max_parts][rank_p]
    float* part_ml = nullptr;      // [rows][heads][max_parts][2]
};
// any size, f16 or f32 cache: one workgroup per (row, head)
hipError_t launch_latent_attn_plain(const LatentAttnArgs& a, int rows, hipStream_t s);
// matrix-core form (latent_attn.hip): f16 cache, rank_p <= 512, 32 <= rot_p <= 64; tile_rows: rows of the longest q-tile;
// n_parts_max > 1 (decode tiles only): split-KV, partials left for launch_latent_values
int latent_rank_padded(int rank);  // rank_p the kernel is instantiated for
bool latent_attn_ok(const LatentCache& c);
hipError_t launch_latent_attn(const LatentAttnArgs& a, int n_tiles, int tile_rows, int n_parts_max, hipStream_t s);

// ---- decode: the steps around the attention kernel, fused --------------------------------------------------------------------
// launch_latent_rows + the product that carries the unrotated query into latent space: y [rows][heads][rank_p] f32; of q only the
// rotated part is written.  w: per head [rank_p x dim_p] packed.
hipError_t launch_latent_query(const LatentRowsArgs& a, const uint4* w, float* y, int rows, hipStream_t s);
// split-KV combine + the product that carries the weighted latents to values: planes [rows][ld], column head * vdim (n < vdim).
// a: the attention launch's arguments (n_parts_max of that launch).  w: per head [vdim_p x rank_p] packed.
hipError_t launch_latent_values(const LatentAttnArgs& a, int n_parts_max, const uint4* w, int vdim, int vdim_p, bf16_bits* oh, bf16_bits* ol,
                                int ld, int packed, int rows, hipStream_t s);

// ---- expanded form for prompt chunks (latent_prefill.hip) --------------------------------------------------------------------
// The 32-token cache tiles some row of the chunk sees, listed once per chunk for the widest window: entry e = (slot, tile, first
// position of its segment).  kx / vx: per (head, entry) a K fragment set [2 halves][dim_p / 32][64][8] and a V set [vdim_p / 16][64][8].
struct LatentExpandArgs {
    LatentCache cache;
    const int* block_tables = nullptr;
    int max_blocks = 0;
    const int* exp_slot = nullptr;
    const int* exp_tile = nullptr;
    const int* exp_pos0 = nullptr;
    int n_tiles = 0, cap = 0;      // entries, entries per head allocated
    int window = 0;
    const uint4* uk = nullptr;     // [heads][dim_p x rank_p] packed, f16 times 1 / uk_scale
    const uint4* uv = nullptr;     // [heads][vdim_p x rank_p] packed, f16 times 1 / uv_scale
    float uk_scale = 1.f, uv_scale = 1.f;
    int dim_p = 0, vdim_p = 0;
    f16_bits* kx = nullptr;
    f16_bits* vx = nullptr;
};
hipError_t launch_latent_expand(const LatentExpandArgs& a, int heads, hipStream_t s);
struct LatentPrefillArgs {
    const float* qkv = nullptr;    // query part of the q / latent projection, as in LatentRowsArgs
    int n_slabs = 1, ldq = 0;
    int64_t slab_stride = 0;
    int dim = 0;
    float scale = 1.f;
    const float* cos = nullptr;
    const float* sin = nullptr;
    LatentCache cache;             // rotated key part
    const int* block_tables = nullptr;
    int max_blocks = 0;
    const f16_bits* kx = nullptr;
    const f16_bits* vx = nullptr;
    int cap = 0;
    const int* tile_row0 = nullptr;
    const int* tile_nrows = nullptr;
    const int* tile_slot = nullptr;
    const int* tile_exp = nullptr;   // per q-tile: entry of cache tile t = tile_exp + t
    const int* tile_order = nullptr; // longest context first
    const int* pos = nullptr;
    int n_tiles = 0, heads = 0, window = 0;
    const float* sink = nullptr;   // as in LatentAttnArgs
    int dim_p = 0, vdim = 0, vdim_p = 0;
    bf16_bits* oh = nullptr;       // context planes [rows][ld], column head * vdim
    bf16_bits* ol = nullptr;
    int ld = 0, packed = 0;
};
int latent_prefill_dim(int dim);    // padded sizes of the instances; 0: no instance
int latent_prefill_vdim(int vdim);
hipError_t launch_latent_prefill(const LatentPrefillArgs& a, hipStream_t s);

// ---- output head -----------------------------------------------------------------------------------------------------------
// logits[r][n] = cap(sum of slabs), n < V; accurate tanh; softcap <= 0: none
hipError_t launch_logits_finish(const float* in, int n_slabs, int64_t slab_stride, int ld_in, int rows, int V, float softcap,
                                float* logits, int64_t ld_out, hipStream_t s);

}  // namespace nvllm
