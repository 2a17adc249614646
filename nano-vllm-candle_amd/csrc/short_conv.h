// Causal short convolutions over the rows of a chunk (device code): what a row sees of earlier tokens, and the history a segment leaves.
// A: any argument structure with in, n_slabs, slab_stride, ld (channel c of a row is column c), in_bias, taps, history, slots, seg, pos, slot as in
// DeltaRowsArgs (hybrid.h).
#pragma once
#include "device_common.h"
#include "hybrid.h"

namespace nvllm {

// what a row sees of the tokens before its chunk: rows back to its segment's start, then the slot's history
struct RowPast {
    int in_chunk = 0;  // earlier rows of the same sequence in this chunk, at most taps - 1
    int pos0 = 0;      // position of the segment's first row (valid when in_chunk < taps - 1)
    int slot = 0;
};
template <class A>
__device__ __forceinline__ RowPast row_past(const A& a, int row) {
    RowPast p;
    p.slot = a.slot[row];
    const int pos = a.pos[row];
    while (p.in_chunk < a.taps - 1 && row - p.in_chunk - 1 >= 0 && a.slot[row - p.in_chunk - 1] == p.slot) ++p.in_chunk;
    p.pos0 = pos - p.in_chunk;
    return p;
}
// input of channel c
template <class A>
__device__ __forceinline__ float conv_input(const A& a, int row, int c) {
    return slab_elem(a.in + (size_t)row * a.ld + c, a.n_slabs, a.slab_stride) + (a.in_bias ? a.in_bias[c] : 0.f);
}
// input of channel c, j tokens before the row
template <class A>
__device__ __forceinline__ float past_input(const A& a, const RowPast& p, int row, int j, int c, int channels) {
    if (j <= p.in_chunk) return conv_input(a, row - j, c);
    const int back = j - p.in_chunk;  // tokens before the segment
    if (back > p.pos0) return 0.f;
    return a.history[((((size_t)(p.pos0 & 1) * a.slots + p.slot) * (a.taps - 1)) + (a.taps - 1 - back)) * channels + c];
}
// one thread per (segment, channel): everything the segment leaves behind is read before it is written
constexpr int kMaxTaps = 16;
template <class A>
__global__ void __launch_bounds__(256) conv_history_kernel(A a, int channels) {
    const int c = blockIdx.x * 256 + threadIdx.x, sg = blockIdx.y;
    if (c >= channels) return;
    const int row = a.seg.row0[sg] + a.seg.n[sg] - 1;
    RowPast p;
    p.slot = a.seg.slot[sg];
    p.in_chunk = a.seg.n[sg] - 1;
    p.pos0 = a.pos[a.seg.row0[sg]];
    float x[kMaxTaps - 1];
#pragma unroll
    for (int i = 0; i < kMaxTaps - 1; ++i)
        if (i < a.taps - 1) x[i] = past_input(a, p, row, a.taps - 2 - i, c, channels);
    float* next = a.history + ((size_t)((a.pos[row] + 1) & 1) * a.slots + p.slot) * (a.taps - 1) * channels;
#pragma unroll
    for (int i = 0; i < kMaxTaps - 1; ++i)
        if (i < a.taps - 1) next[(size_t)i * channels + c] = x[i];
}
}  // namespace nvllm
