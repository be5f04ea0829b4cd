// moe.h -- mixture of experts: a sigmoid router, the chosen experts' rows sorted by expert, and the sum of their results.
// The chosen weight scales an expert's INPUT; its score is not renormalised.
#pragma once

#include "nvllm_internal.h"

namespace nvllm {

// The rows of a batch sorted by expert, every expert's segment padded to `pad` rows.
struct RoutePlan {
    int T, E, top, pad;
    int capacity;          // rows, a multiple of pad: no batch of T tokens needs more
    int* block_expert;     // [capacity / 16]
    int* source;           // [capacity] row -> token (padding and unused rows: token 0)
    float* weight;         // [capacity] row -> its expert's score (padding: 0)
    int* row_of;           // [T][top] row of a token's j-th choice
    int* choice;           // [T][top] expert
    float* score;          // [T][top]
};
int route_pad(int T, int E, int top);               // group size that suits a batch
size_t route_ints(int T, int E, int top, int pad);  // 4-byte words route_plan() lays out
RoutePlan route_plan(int* mem, int T, int E, int top, int pad);
// z: [T][ldz] router logits in columns 0 .. E-1; the `top` largest (the first of equals) are chosen
void launch_route(const RoutePlan& r, const float* z, int ldz);

// the rows x * gain of a batch in the plan's order, as activation tiles (x [T][ld])
void launch_expert_rows(__half* dst, const float* x, const float* gain, const RoutePlan& r, int ld);

// x += sum of the chosen experts' rows + sigmoid(z_shared) * shared;  then what the next sublayer needs of x
struct MoeCombine {
    float* x;                  // [T][ld]
    const float* rows;         // expert results [row][ld], rows by row_of (null: by token and choice, [T][top][ld])
    const int* row_of;
    int top;
    const float* shared;       // [T][ld] or null
    const float* z;            // its gate's logits: z[t * ldz + z_col]
    int ldz, z_col;
    const float* gain;         // next norm
    __half* out_b16;           // x * gain tiles, and ...
    float* ss;                 // ... sums of squares per 32 features (both null: fp32 path)
    int ld;
};
void launch_moe_combine(const MoeCombine& m, int T);
// fp32 path: out[i][n] = sum_k w[expert(i)][n][k] * scale(i) * in[row(i)][k], i = token * top + choice;
// row(i) = i, or the token when by_token (then the input is scaled by its score)
void launch_matmul_experts_f32(float* out, const float* in, const float* w, const RoutePlan& r, bool by_token, int K, int N);
void launch_relu2(float* x, long n);

}  // namespace nvllm
