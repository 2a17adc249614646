// Decoders whose layers mix tokens by recurrence, by grouped-query attention or by two mixers side by side (hybrid_model.cpp): launchers of
// hybrid_ops.hip and conv_attn.hip (row kernels), recurrent.hip and recurrent_chunk.hip (carried-state scans) and bias_attn.hip (attention).
#pragma once
#include "latent.h"

namespace nvllm {

// ---- rows of one sequence inside a chunk ---------------------------------------------------------------------------------------
struct Segments {
    const int* row0 = nullptr;  // first row, number of rows, slot of segment i
    const int* n = nullptr;
    const int* slot = nullptr;
    int count = 0;
    int single = 0;             // decode: segment i is row i, its slot is slot[i] (row0, n unused)
};

// ---- feed-forward activation of the summed slabs, as bf16 hi/lo planes [rows][F] or f32 -------------------------------------------
hipError_t launch_act(Act act, const float* in, int n_slabs, int64_t slab_stride, int rows, int F, bf16_bits* hi, bf16_bits* lo, int packed, float* y,
                      hipStream_t s);

// ---- grouped-query attention ------------------------------------------------------------------------------------------------
// K in QK^T fragment order with dim_p, V in PV fragment order with vdim_p (device_common.h), blocks of kBlockTokens tokens per kv head:
// [block][kv][kBlockTokens * dim_p] / [block][kv][kBlockTokens * vdim_p]; f16 or f32; padding zero.
struct PagedKV {
    void* k = nullptr;
    void* v = nullptr;
    int f32 = 0, kv = 0, dim = 0, dim_p = 0, vdim = 0, vdim_p = 0;
};
// rows after the fused q / k / v projection: biases, RMS norm over all of q and all of k, value mixing, cache write
struct AttnRowsArgs {
    const float* in = nullptr;       // slabs [n_slabs][rows][ld]: H * dim query, kv * dim key, kv * vdim value columns
    int n_slabs = 1, ld = 0;
    int64_t slab_stride = 0;
    const float* bias = nullptr;     // [ld], nullptr: none
    int heads = 0;
    const float* qn = nullptr;       // [heads * dim]
    const float* kn = nullptr;       // [kv * dim]
    float eps = 0.f, q_scale = 1.f;  // q_scale: score scale * log2(e)
    const float* ssq = nullptr;      // [rows][2] sums of squares over every rank's share (q, k); nullptr: this rank holds everything
    int q_all = 0, k_all = 0;        // elements those sums run over
    int mix = 0;                     // 0 plain values, 1 plain and kept in v_first, 2 mixed: (1 - lambda) v + lambda v_first
    const float* lambda = nullptr;   // one float (device)
    float* v_first = nullptr;        // [rows][kv * vdim]
    const int* pos = nullptr;
    const int* slot = nullptr;
    const int* block_tables = nullptr;
    int max_blocks = 0;
    float* q = nullptr;              // [rows][heads][dim_p], scaled, padding zero
    PagedKV kv;
};
hipError_t launch_attn_rows(const AttnRowsArgs& a, int rows, hipStream_t s);
// sums of squares of column ranges of biased slab rows: out[row][k] over columns [c0[k], c0[k] + n[k])
hipError_t launch_rows_ssq(const float* in, int n_slabs, int64_t slab_stride, int ld, const float* bias, const int c0[2], const int n[2], int rows,
                           float* out, hipStream_t s);

constexpr int kBiasTileRows = 128;  // tokens of one q-tile of a prompt chunk (a decode tile is one token)
constexpr int kBiasMaxParts = 64;
struct BiasAttnArgs {
    const float* q = nullptr;        // [rows][heads][dim_p]
    PagedKV kv;
    int heads = 0;
    const float* bias = nullptr;     // [heads][n_bias] by distance, times log2(e); distances from n_bias - 1 on share the last entry
    int n_bias = 0;                  // 0: no bias
    int window = 0;                  // > 0: a token sees itself and the window - 1 before it
    const float* sink = nullptr;     // [heads] one more term 2^sink in the denominator; nullptr: none
    const int* block_tables = nullptr;
    int max_blocks = 0;
    const int* tile_row0 = nullptr;
    const int* tile_nrows = nullptr;
    const int* tile_slot = nullptr;
    const int* tile_order = nullptr; // prompt: longest context first
    const int* pos = nullptr;
    const int* slot = nullptr;       // per row
    bf16_bits* oh = nullptr;         // context planes [rows][ld], column head * vdim
    bf16_bits* ol = nullptr;
    float* of = nullptr;             // or f32
    int ld = 0, packed = 0;
    // split over the context (decode): workgroup z takes part_tiles 32-token tiles
    int part_tiles = 0, max_parts = 1;
    float* part_o = nullptr;         // [rows][heads][max_parts][vdim_p]
    float* part_ml = nullptr;        // [rows][heads][max_parts][2]
};
// any size, f16 or f32 cache: one workgroup per (row, head)
hipError_t launch_bias_attn_plain(const BiasAttnArgs& a, int rows, hipStream_t s);
// matrix-core forms, f16 cache; sizes they have instances for (padded; 0: none)
int bias_attn_dim(int dim);
int bias_attn_vdim(int vdim);
hipError_t launch_bias_decode(const BiasAttnArgs& a, int rows, int parts, hipStream_t s);  // one row per tile; parts > 1: split + combine
hipError_t launch_bias_prefill(const BiasAttnArgs& a, int n_tiles, hipStream_t s);

// ---- recurrences: S <- g S; u = beta (v - S^T k) or u = v; S <- S + k u^T; o = S^T q --------------------------------------------------
// dim_p is a multiple of 64, vdim_p of 32; lane (part p = lane % 16, group c = lane / 16) of column block cb holds the channels
// 64 r + 4 p + i of columns 8 cb + 2 c + {0, 1}:  state [slot][head][vdim_p / 8][dim_p / 64][2][64 lanes][4] f32.
inline int recur_dim(int dim) { return (dim + 63) / 64 * 64; }
inline int recur_vdim(int vdim) { return (vdim + 31) / 32 * 32; }
bool recur_ok(int dim, int vdim);
inline size_t recur_state_floats(int heads, int dim_p, int vdim_p) { return (size_t)heads * dim_p * vdim_p; }
struct RecurArgs {
    const float* q = nullptr;        // [rows][q_heads][dim_p]
    const float* k = nullptr;
    const float* v = nullptr;        // [rows][heads][vdim_p]
    int heads = 0, q_heads = 0, dim_p = 0, vdim = 0, vdim_p = 0;
    // delta rule: decays per key channel (g) or per head (gh) and write strengths; nullptr: constant decays per head
    const float* g = nullptr;        // rows of stride g_row, head * dim_p
    int64_t g_row = 0;
    const float* gh = nullptr;       // [rows][heads] one decay per head instead
    const float* beta = nullptr;     // [rows][heads]
    const float* decay = nullptr;    // [heads]
    float* state = nullptr;
    Segments seg;
    const int* pos = nullptr;        // position 0: the state starts at zero
    float* o = nullptr;              // [rows][heads][vdim_p]
};
// RMS norm of o over one head or over all heads, times weight and gate, as context planes / f32 rows [rows][ld], column head * vdim
struct GatedNormArgs {
    const float* o = nullptr;        // [rows][heads][vdim_p]
    const float* gate = nullptr;     // the factor itself, or with gate_slabs > 0 the slabs of a projection z, the factor being silu(z)
    int64_t gate_row = 0, gate_stride = 0;  // rows, slabs
    int gate_head = 0, gate_slabs = 0;      // heads
    int heads = 0, vdim = 0, vdim_p = 0;
    int whole = 0;                   // 1: one norm over all heads, weight [heads * vdim]; 0: per head, weight [vdim]
    const float* ssq = nullptr;      // whole: [rows][2], entry 0 the sum of squares over every rank's heads
    int all = 0;                     // ... and the elements it runs over
    const float* weight = nullptr;
    float eps = 0.f;
    bf16_bits* oh = nullptr;
    bf16_bits* ol = nullptr;
    float* of = nullptr;
    int ld = 0, packed = 0;
};
hipError_t launch_gated_norm(const GatedNormArgs& a, int rows, hipStream_t s);
// norm (nullable): decode with per-head norms, the gated output norm in the same launch (o is not written)
hipError_t launch_recurrence(const RecurArgs& a, const GatedNormArgs* norm, hipStream_t s);

// prompt chunks: the same recurrences in pieces of 16 tokens (recurrent_chunk.hip); a sequence's pieces follow each other
constexpr int kPiece = 16;
struct PieceArgs {
    const int* row0 = nullptr;       // first row and number of rows of every piece
    const int* n = nullptr;
    const int* seg_piece0 = nullptr; // first piece of every segment
    int count = 0;
    float* pair = nullptr;           // scratch per (piece, head): [16][16] decayed products of queries and keys,
    float* kt = nullptr;             // [dim_p][16] keys decayed to the piece's end;
    float* qt = nullptr;             // delta rule: [16][dim_p] decayed queries,
    float* wt = nullptr;             // [16][dim_p] solved keys,
    float* decay = nullptr;          // [dim_p] decays of the whole piece
};
bool piece_scan_ok(int dim_p);
// q, k, v, g and beta hold kPiece more rows than the chunk (anything finite); v is overwritten for the delta rule
hipError_t launch_piece_scan(const RecurArgs& a, const PieceArgs& c, hipStream_t s);

// rows after the q / k / v / gate projection of the constant-decay recurrence: silu(q, k, v), sigmoid(gate)
struct LinearRowsArgs {
    const float* in = nullptr;       // columns: heads * dim query, heads * dim key, heads * vdim value, heads * vdim gate
    int n_slabs = 1, ld = 0;
    int64_t slab_stride = 0;
    int heads = 0, dim = 0, dim_p = 0, vdim = 0, vdim_p = 0;
    float* q = nullptr;
    float* k = nullptr;
    float* v = nullptr;
    float* gate = nullptr;           // [rows][heads][vdim_p]
};
hipError_t launch_linear_rows(const LinearRowsArgs& a, int rows, hipStream_t s);

// rows after the projection of the delta rule: causal convolution + silu of q, k, v (history in the sequence's slot), unit q and k,
// beta, and the inputs of the two-step gate projections
struct DeltaRowsArgs {
    // columns: kv * dim query, kv * dim key, heads * vdim value, heads beta, then rank_p decay and rank_p gate inputs (two-step gates), or
    // heads decay inputs (rate set)
    const float* in = nullptr;
    int n_slabs = 1, ld = 0;
    int64_t slab_stride = 0;
    int heads = 0, kv = 0, dim = 0, dim_p = 0, vdim = 0, vdim_p = 0, rank_p = 0, taps = 1;
    const float* in_bias = nullptr;  // unused (short_conv.h)
    const float* conv = nullptr;     // [taps][channels], channels = 2 kv dim + heads vdim in column order
    float q_scale = 1.f;
    // history: raw projections of the last taps - 1 tokens, [2][slots][taps - 1][channels]; a segment that starts at position p reads
    // half p % 2, one that ends before position p writes half p % 2
    float* history = nullptr;
    int slots = 0;
    Segments seg;
    const int* pos = nullptr;
    const int* slot = nullptr;
    float* q = nullptr;              // [rows][kv][dim_p]
    float* k = nullptr;
    float* v = nullptr;              // [rows][heads][vdim_p]
    float* beta = nullptr;           // [rows][heads]
    float* gate_in = nullptr;        // two-step gates: [rows][2][rank_p]
    // one decay per head: exp(-rate softplus(decay input + dt))
    const float* rate = nullptr;     // [heads]
    const float* dt = nullptr;       // [heads]
    float* decay = nullptr;          // [rows][heads]
    __host__ __device__ int channels() const { return 2 * kv * dim + heads * vdim; }
    __host__ __device__ int extras() const { return heads + (rate ? heads : 2 * rank_p); }  // columns behind the channels
};
constexpr float kUnitNormEps = 1e-6f;
hipError_t launch_delta_rows(const DeltaRowsArgs& a, int rows, hipStream_t s);
// rows after the q / k / v projection of attention with short convolutions: bias, causal convolution, rotation of neighbouring dimensions,
// RMS norm per head (no weight), cache write; history as in DeltaRowsArgs (biased projections)
struct ConvAttnRowsArgs {
    const float* in = nullptr;       // columns: heads * dim query, kv * dim key, kv * vdim value
    int n_slabs = 1, ld = 0;
    int64_t slab_stride = 0;
    const float* in_bias = nullptr;  // [channels], nullptr: none
    int heads = 0, taps = 1;
    const float* conv = nullptr;     // [taps][channels]
    int rot = 0;                     // rotated dimensions (even)
    const float* cos = nullptr;      // [positions][rot / 2]
    const float* sin = nullptr;
    float eps = 0.f, q_scale = 1.f;  // q_scale: score scale * log2(e)
    float* history = nullptr;
    int slots = 0;
    Segments seg;
    const int* pos = nullptr;
    const int* slot = nullptr;
    const int* block_tables = nullptr;
    int max_blocks = 0;
    float* q = nullptr;              // [rows][heads][dim_p], scaled, padding zero
    PagedKV kv;
    __host__ __device__ int channels() const { return (heads + kv.kv) * kv.dim + kv.kv * kv.vdim; }
    __host__ __device__ int units() const { return heads + 2 * kv.kv; }  // waves per row
};
constexpr int kConvAttnDim = 512;    // widest head
hipError_t launch_conv_attn_rows(const ConvAttnRowsArgs& a, int rows, hipStream_t s);
// the history half of it for chunks with longer segments (after launch_conv_attn_rows)
hipError_t launch_conv_attn_history(const ConvAttnRowsArgs& a, hipStream_t s);

// gate_in -> decays and output gates (HeadGemmArgs with decay_rate set), or step sizes alone (decay_bias without it)
hipError_t launch_delta_gates(const HeadGemmArgs& a, hipStream_t s);
// the history half of it for chunks with longer segments (after launch_delta_rows)
hipError_t launch_delta_history(const DeltaRowsArgs& a, hipStream_t s);

}  // namespace nvllm
