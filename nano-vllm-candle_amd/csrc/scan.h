// Selective scan (state-space recurrence with input-dependent step sizes, a decay per channel and state):
//   S[c][n] <- exp(dt_c A[c][n]) S[c][n] + dt_c x_c B_n;   y_c = sum_n S[c][n] C_n + D_c x_c;   out = y silu(z)
// x: causal short convolution + silu of the input projection.  Launchers of scan.hip.
#pragma once
#include "hybrid.h"

namespace nvllm {

// convolution with bias + silu of columns [0, channels) of the input projection; history as in DeltaRowsArgs
struct ConvRowsArgs {
    const float* in = nullptr;       // slabs [n_slabs][rows][ld]
    int n_slabs = 1, ld = 0;
    int64_t slab_stride = 0;
    int channels = 0, taps = 1;
    const float* in_bias = nullptr;  // [channels] added to the input (nullable)
    const float* conv = nullptr;     // [taps][channels]
    const float* bias = nullptr;     // [channels]
    float* history = nullptr;        // [2][slots][taps - 1][channels]
    int slots = 0;
    Segments seg;
    const int* pos = nullptr;
    const int* slot = nullptr;
    float* x = nullptr;              // [rows][ldx]
    bf16_bits* xh = nullptr;         // the same as planes [rows][ldx] (nullable)
    bf16_bits* xl = nullptr;
    int ldx = 0, packed = 0;
};
hipError_t launch_conv_rows(const ConvRowsArgs& a, int rows, hipStream_t s);  // decode: leaves the next history too
hipError_t launch_conv_history(const ConvRowsArgs& a, hipStream_t s);         // prompt chunks, after launch_conv_rows

// states are padded to a power of two of at least four, channels to a multiple of scan_channels
inline int scan_states(int state) { int p = 4; while (p < state) p *= 2; return p; }
inline int scan_channels(int states) { return states >= 16 ? 64 : 1024 / states; }
constexpr int kMaxScanStates = 1024;
struct ScanArgs {
    const float* x = nullptr;        // [rows][ldx]
    int ldx = 0;
    const float* dt = nullptr;       // [rows][channels_p] step sizes
    const float* bc = nullptr;       // rows of stride ldbc: B at column b0, C at column c0 (states each)
    int ldbc = 0, b0 = 0, c0 = 0;
    const float* z = nullptr;        // gate, slabs of stride z_stride, rows of stride ldz
    int z_slabs = 1, ldz = 0;
    int64_t z_stride = 0;
    const float* A = nullptr;        // [channels_p][states], times log2(e)
    const float* D = nullptr;        // [channels_p]
    int channels = 0, channels_p = 0, states = 0;
    float* state = nullptr;          // [slot][channels_p][states]
    const int* pos = nullptr;
    const int* slot = nullptr;       // decode: per row
    // prompt chunks: pieces of consecutive rows of one sequence, those of a segment in order.  A segment of several pieces runs twice: every
    // piece but the last from a zero state (its end state and its sum of step sizes into the scratch), then all of them.
    const int* piece_row0 = nullptr;
    const int* piece_n = nullptr;
    const int* piece_slot = nullptr;
    const int* piece_at = nullptr;   // number in the segment
    const int* piece_of = nullptr;   // pieces of the segment
    int pieces = 0, several = 0;     // several: some segment has more than one piece
    float* carry = nullptr;          // [piece][channels_p][states]: state before the segment (first piece), end state of the piece before
    float* carry_dt = nullptr;       // [piece][channels_p]: sum of step sizes of the piece before
    bf16_bits* oh = nullptr;         // planes [rows][ld] (columns >= channels: not written), or f32 rows
    bf16_bits* ol = nullptr;
    float* of = nullptr;
    int ld = 0, packed = 0;
};
hipError_t launch_scan_decode(const ScanArgs& a, int rows, hipStream_t s);
hipError_t launch_scan_prompt(const ScanArgs& a, hipStream_t s);

}  // namespace nvllm
