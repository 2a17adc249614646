// Routed feed-forwards: every row goes through `top` of `experts` small feed-forwards and, optionally, through a shared one.
// Launchers of moe.hip.  Rows are put into groups (one per expert, the shared feed-forward last), each starting at a multiple of `align`
// positions; products then run over tiles of `align` positions that belong to one group.
#pragma once
#include "latent.h"

namespace nvllm {

constexpr int kMaxExperts = 1024, kMaxTop = 64;

struct RouteArgs {
    const float* z = nullptr;    // router logits [rows][ld]: a column per expert, then the shared gate's when there is one
    int ld = 0, rows = 0, experts = 0, top = 0;
    int gate_col = -1;           // column of the shared gate (-1: none)
    int shared_group = 0;        // every row is a member of group `experts` too
    int weight_in = 1;           // the score multiplies the expert's input (else its output)
    int softmax = 0;             // scores: softmax over all experts (else the sigmoid of each logit)
    int groups = 1, keep = 1;    // equal groups of neighbours; only experts of the `keep` groups with the largest logits can be chosen
    int align = 16, cap = 0;     // cap: positions allocated (a multiple of align)
    int* chosen = nullptr;       // [rows][top]
    float* score = nullptr;      // [rows][top] scores of the chosen
    float* gate = nullptr;       // [rows] sigmoid of the shared gate's logit
    int* place = nullptr;        // [rows][top + shared_group] position of the row in each of its groups
    int* src = nullptr;          // [cap] row of a position (padding: -1)
    float* pre = nullptr;        // [cap] factor of the expert's input
    float* post = nullptr;       // [cap] factor of its output
    int* tile_group = nullptr;   // [cap / align] group of a tile, -1: unused
    int* cursor = nullptr;       // [experts + 1] scratch
};
hipError_t launch_route(const RouteArgs& a, hipStream_t s);

// y[p] = post act(pre x[src[p]] . W_g^T) for the positions p of group g's tiles
struct GroupGemmArgs {
    const bf16_bits* xh = nullptr;   // planes of rows (of positions when src is nullptr), or f32 rows (exact)
    const bf16_bits* xl = nullptr;
    const float* xf = nullptr;
    int ldx = 0, x_packed = 0, x_rows = 0;
    const int* src = nullptr;
    const uint4* w = nullptr;        // packed [N x K] per group, group g at w + g * w_group
    int64_t w_group = 0;
    int N = 0, K = 0;
    const uint4* ws = nullptr;       // weights of group `last` where they differ from the others'; its sizes
    int last = -1, Ns = 0, Ks = 0;
    const int* tile_group = nullptr; // nullptr: one group, positions 0 .. x_rows
    int align = 16, tiles = 0;       // align: 16 or 64
    const float* pre = nullptr;
    const float* post = nullptr;
    int relu2 = 0;                   // act: squared ReLU (else none)
    int glu = 0;                     // silu(gate) up of features in interleaved 16-row tiles (N, ldo: of the weights, of the result); no pre
    float* out = nullptr;            // f32 [positions][ldo], or
    bf16_bits* oh = nullptr;         // planes of positions in fragment order, ldo columns
    bf16_bits* ol = nullptr;
    int ldo = 0;
};
hipError_t launch_group_gemm(const GroupGemmArgs& a, hipStream_t s);

}  // namespace nvllm
