// Internal host-side state shared by the translation units behind the C ABI: context, sequence / block bookkeeping, model.
#pragma once
#include <hip/hip_runtime.h>
#include <rccl/rccl.h>

#include <condition_variable>
#include <memory>
#include <mutex>
#include <string>
#include <unordered_map>
#include <vector>

#include "../../include/nvllm_amd.h"
#include "../../include/nvllm_amd_debug.h"
#include "kernels.h"
#include "latent.h"

using namespace nvllm;

// In-process loopback communicator (tests only): contexts created with the same group name by different
// host threads of ONE process exchange through host memory.  It exercises every tensor-parallel code path
// (sharded load, per-rank kernels, all-reduce placement, vocab-parallel arg-max) on a single GPU; production
// uses RCCL.
struct LoopGroup {
    std::mutex mu;
    std::condition_variable cv;
    int size = 0, arrived = 0;
    uint64_t generation = 0;
    std::vector<float> acc;
    std::vector<unsigned char> gather;
    std::vector<float*> os_data;      // one-shot all-reduce buffers of the ranks (same process, same device: plain pointers)
    std::vector<uint32_t*> os_flag;
};
struct nvllm_ctx {
    std::shared_ptr<LoopGroup> loop;
    bool null_comm = false;  // projection mode: tp_size > 1 shard shapes, every collective skipped (results meaningless)
    int device = 0;
    hipStream_t stream = nullptr;
    hipEvent_t ev0 = nullptr, ev1 = nullptr;
    int tp_rank = 0, tp_size = 1;
    ncclComm_t comm = nullptr;
    std::string err;
    // one-shot all-reduce (oneshot.hip), opt-in; empty when not set up
    bool oneshot = false;
    float* os_data = nullptr;     // [2 generations][tp][os_slot] f32, uncached device memory
    uint32_t* os_flag = nullptr;  // [2][tp]
    unsigned* os_done = nullptr;  // push kernel's workgroup counter
    int* os_err = nullptr;        // set by a wait that timed out
    int* os_agree = nullptr;      // [tp] error words gathered at the end of a step: every rank takes the same decision
    size_t os_slot = 0, os_data_bytes = 0, os_flag_bytes = 0;
    uint64_t os_calls = 0;
    OneShotPeers os_peers;
    std::vector<void*> os_ipc;    // peer mappings opened with hipIpcOpenMemHandle
};

int fail(nvllm_ctx* ctx, int code, const char* fmt, ...);
int model_fail(nvllm_model* m, int code, const char* fmt, ...);

#define HIPCHK(ctx, expr)                                                                              \
    do {                                                                                               \
        hipError_t e_ = (expr);                                                                        \
        if (e_ != hipSuccess) return fail(ctx, NVLLM_EHIP, "%s -> %s", #expr, hipGetErrorString(e_)); \
    } while (0)
#define NCCLCHK(ctx, expr)                                                                               \
    do {                                                                                                 \
        ncclResult_t r_ = (expr);                                                                        \
        if (r_ != ncclSuccess) return fail(ctx, NVLLM_ERCCL, "%s -> %s", #expr, ncclGetErrorString(r_)); \
    } while (0)

// sum over the tensor-parallel group, in place (no-op for one rank)
int comm_allreduce_sum(nvllm_ctx* ctx, float* buf, size_t n);

template <typename T>
static int dmalloc(nvllm_ctx* c, T** p, size_t count) {
    HIPCHK(c, hipMalloc((void**)p, std::max<size_t>(count * sizeof(T), 16)));
    return NVLLM_OK;
}

constexpr int kFusedMaxRows = 128;  // the fused decode path (deferred norms, row-parallel epilogues) handles up to this many rows
constexpr int kMaxPending = 4;   // decode steps that may be enqueued before one is collected
constexpr int kAttnMaxParts = 64;  // split-KV partitions per sequence (partition grows with context beyond 8K)

struct LayerW {
    PackedW qkv, o, gu, down;
    float *ln1 = nullptr, *ln2 = nullptr, *qn = nullptr, *kn = nullptr;
};

struct SeqState {
    int slot = -1;
    int cached = 0;  // tokens whose K/V are in the cache
    std::vector<int> blocks;
    int released = 0;  // leading blocks given back because no window reaches them (blocks[i] = -1)
};

struct DecoderImpl;  // decoder.h

struct nvllm_model {
    nvllm_model();
    ~nvllm_model();
    nvllm_ctx* ctx = nullptr;
    std::unique_ptr<DecoderImpl> dec;  // a decoder built from layer descriptions; nullptr: Qwen3
    nvllm_qwen3_config cfg{};
    int H = 0, hd = 0, L = 0, nh_l = 0, kv_l = 0, I_l = 0, V_l = 0, gqa = 1;
    bf16_bits* embed = nullptr;  // [V][H] row-major bf16 (gather table, replicated)
    PackedW lm_head;             // [V_l][H]
    float* norm = nullptr;
    std::vector<LayerW> layers;
    std::unordered_map<std::string, bool> loaded;
    bool finalized = false;
    float *cosv = nullptr, *sinv = nullptr;
    int rope_len = 0;

    // KV pool
    int widest_window = 0;  // > 0: no layer sees further back than this
    int num_blocks = 0, max_seqs = 0, max_blocks = 0, max_rows = 0;
    std::vector<f16_bits*> kcache, vcache;
    std::vector<uint8_t*> vlocache;  // 24-bit V (opt_kv_v_bits == 24): one residual byte per V element, else empty
    std::vector<uint8_t*> klocache;  // 24-bit K (opt_kv_k_bits == 24, only with 24-bit V): the same for K
    std::vector<int> free_blocks, free_slots;
    std::unordered_map<int64_t, SeqState> seqs;
    int* d_block_tables = nullptr;
    std::vector<int> h_block_tables;

    // step buffers
    uint32_t* d_ids = nullptr;
    int *d_pos = nullptr, *d_slot = nullptr, *d_tile_row0 = nullptr, *d_tile_nrows = nullptr, *d_tile_slot = nullptr,
        *d_last_rows = nullptr, *d_tile_order = nullptr, *d_tile_last = nullptr, *d_group_order = nullptr;
    float *resid = nullptr, *slabs = nullptr, *qbuf = nullptr, *logits = nullptr, *d_maxval = nullptr, *red = nullptr;
    bf16_bits *xh = nullptr, *xl = nullptr, *xh2 = nullptr, *xl2 = nullptr, *ctxh = nullptr, *ctxl = nullptr;
    float *ssqA = nullptr, *ssqB = nullptr;  // deferred-norm partial sums of squares [groups][kFusedMaxRows]
    uint64_t* d_keys = nullptr;              // device sampling: per-row RNG keys and temperatures
    float* d_temps = nullptr;
    // The streaming GEMM's in-launch split-K combine (epilogues 1-3) is OFF by default: measured slower than slabs + a
    // consumer launch on MI355X (Qwen3-8B batch 64: 8.6 vs 6.4 ms/step; 32B TP=8 shard: 8.9 vs 6.5 ms) -- one workgroup
    // per n-group reads every slab behind an agent-scope release of all the others.  nvllm_debug_set_option turns it on.
    int opt_stream_combine = 0;
    int opt_oneshot_allreduce = 0;  // TP decode: one-shot all-reduce instead of the communicator's (set before kv_alloc; opt-in)
    int opt_kv_v_bits = 16;            // 24: V as f16 + e5m2 residual (13..14 significant bits, V bytes x1.5); read at kv_alloc
    int opt_kv_k_bits = 16;            // 24: K likewise (needs kv_v_bits = 24: K/V bytes x1.5 together); read at kv_alloc
    int opt_oneshot_skip_push = 0;     // test hook: this rank "forgets" its next N pushes (the give-up path of its peers' waits)
    int opt_oneshot_spins = 20000000;  // bound of the one-shot wait kernel's poll (~ seconds): a missing peer is an error code
    int opt_no_fused = 0, opt_no_xpack = 0, opt_no_rowpar = 0;  // A/B switches (nvllm_debug_set_option): force the generic paths
    int opt_no_attn_prologue = 0;  // A/B: decode q/k-norm + RoPE + KV write in their own row kernel, not in the attention prologue
    int opt_tile_fuse_qk = 1;    // QKV tile GEMM with the q/k-norm + RoPE + KV-write epilogue (head_dim 128, 256-wide blocks)
    int opt_latent_absorb = 0;   // prompt chunks of latent attention: 1 always absorbed, -1 expanded whenever possible, 0 by cost
    int opt_latent_wgs = 0;      // decode: workgroups the split of the visible context aims at (0: by latent size)
    int64_t latent_expanded = 0; // layer runs served by the expanded form so far
    int opt_latent_plain = 0;    // latent attention: the plain kernel instead of the matrix-core one (A/B, tests)
    int opt_tile_min_wgs = 192;  // prefill tile GEMM: smallest grid it is used for (256-row tiles need rows to fill 256 CUs)
    unsigned* tickets = nullptr;             // arrival counters of the streaming GEMM's in-launch combine (zero between launches)
    float* qkv_out = nullptr;                // complete QKV sums of the streaming GEMM (its combine reads the slabs in m->slabs)
    uint32_t* d_next = nullptr;
    float *attn_po = nullptr, *attn_pml = nullptr;  // split-KV partials [max_seqs][nh_l][kAttnMaxParts][hd] / [..][2]
    int attn_part_tiles = 4, attn_parts_max = 1;   // this step's split geometry (decode only)
    float* part_val = nullptr;  // fused LM-head arg-max partials [V_l/16][max_seqs]
    int* part_idx = nullptr;
    unsigned long long* argmax_scratch = nullptr;  // ticket + per-row keys of argmax_parts_kernel
    bool want_logits = false;   // this step stores the last-row logits
    int cur_n = 0;              // sequences of the step in flight
    int cur_max_len = 0;        // longest of them (tokens, the new ones included)
    size_t slab_floats = 0;
    void* h_stage = nullptr;  // pinned
    size_t h_stage_bytes = 0;
    float *tap_h = nullptr, *tap_res = nullptr;
    bool taps = false;
    int tap_rows = 0;

    // last step (for nvllm_decode_next / byte accounting)
    std::vector<int64_t> last_ids;
    std::vector<int> last_lens;
    int64_t last_bytes = 0;
    bool decode_resident = false;  // device metadata describes a pure-decode batch == last_ids
    // pipelined decode (nvllm_decode_enqueue / _collect)
    uint32_t* pin_ids = nullptr;
    hipEvent_t pend_ev[4] = {nullptr, nullptr, nullptr, nullptr};
    std::vector<int> pending;
    int pend_next = 0;

    // diagnostic build (-DNVLLM_STAMPS): in-kernel time stamps of every launch of the fused decode path
    unsigned long long* stamps = nullptr;
    bool stamps_on = false;
    int stamp_launch = 0;
    int64_t tile_launches = 0;  // projections run by the tile GEMM so far (tests assert the path they force was taken)

    // per-kernel-class HIP-event timing (bench roofline leg); 0 = off
    int prof_kind = 0;
    std::vector<hipEvent_t> prof_ev;
    size_t prof_used = 0;
};

#ifdef NVLLM_STAMPS
constexpr int kStampLaunches = 160;               // launches recorded per step (fused decode path: 5 per layer)
constexpr size_t kStampStride = (size_t)1024 * 16 * 8;  // u64 per launch: [<= 1024 workgroups][16 waves][8 points]
#define STAMPS(args_, m_)                                                                                        \
    do {                                                                                                         \
        if ((m_)->stamps_on && (m_)->stamp_launch < kStampLaunches) (args_).stamps = (m_)->stamps + (size_t)((m_)->stamp_launch++) * kStampStride; \
    } while (0)
#else
#define STAMPS(args_, m_) do { } while (0)
#endif

enum { PROF_ATTN = 1, PROF_GEMM = 2, PROF_NORM = 3, PROF_QK = 4, PROF_SILU = 5, PROF_LMHEAD = 6, PROF_EMPTY = 7, PROF_RECUR = 8 };

// bracket one launch with HIP events on the library stream when its class is being profiled
#define PROF(m_, kind_, expr_)                                                           \
    do {                                                                                  \
        if ((m_)->prof_kind == (kind_)) {                                                 \
            if ((m_)->prof_used + 2 > (m_)->prof_ev.size()) {                             \
                for (int i_ = 0; i_ < 256; ++i_) {                                        \
                    hipEvent_t evn_;                                                      \
                    HIPCHK((m_)->ctx, hipEventCreate(&evn_));                              \
                    (m_)->prof_ev.push_back(evn_);                                        \
                }                                                                         \
            }                                                                             \
            HIPCHK((m_)->ctx, hipEventRecord((m_)->prof_ev[(m_)->prof_used], (m_)->ctx->stream));     \
            HIPCHK((m_)->ctx, expr_);                                                     \
            HIPCHK((m_)->ctx, hipEventRecord((m_)->prof_ev[(m_)->prof_used + 1], (m_)->ctx->stream)); \
            (m_)->prof_used += 2;                                                         \
        } else {                                                                          \
            HIPCHK((m_)->ctx, expr_);                                                     \
        }                                                                                 \
    } while (0)

// y (f32 slabs) = x.W^T with the kernel that fits the row count (api.cpp)
int gemm_slabs(nvllm_model* m, const bf16_bits* xh, const bf16_bits* xl, int ldx, const PackedW& w, float* out, int R,
               int max_split, int* n_slabs, int x_packed = 0);
uint16_t host_f32_to_bf16(float f);
