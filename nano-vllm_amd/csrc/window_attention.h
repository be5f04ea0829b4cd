// window_attention.h -- grouped-query attention over a paged cache with a sliding window whose first tokens stay
// visible, an optional soft cap on the scores, and the step before it: a short causal convolution over time on the
// projected channels, half-split rotation, cache write.  Sizes, window, cap, taps and base are parameters.
#pragma once

#include "nvllm_internal.h"
#include "step_arrays.h"

namespace nvllm {

// One layer's slice of the block pool: keys, then values.
//   fp32 (elem_bytes 4): rows [position row][group][dim] and [position row][group][vdim].
//   bf16 (elem_bytes 2): per 16 positions and group a key page and a value page in matrix-core operand order; dim and
//     vdim are padded to multiples of 32 (zeros), block_size is a multiple of 16:
//       key page    (key, d) at half (d >> 5) * 512 + (key + 16 * ((d >> 3) & 3)) * 8 + (d & 7)
//       value page  (key, d) at half (d >> 4) * 256 + ((key >> 2) * 16 + (d & 15)) * 4 + (key & 3)
struct KvPages {
    void* keys;
    void* values;
    int elem_bytes, block_size;
    int G, dim, vdim;
    int dim_ld, vdim_ld;   // as stored
};
constexpr int KV_PAGE = 16;
KvPages kv_pages(void* base, int elem_bytes, int block_size, int num_blocks, int G, int dim, int vdim);
size_t kv_pages_bytes(int elem_bytes, int block_size, int num_blocks, int G, int dim, int vdim);

// Convolution, rotation and cache write of a batch's projected rows.
struct ConvRope {
    const void* raw;       // [T][raw_ld] of the pool's element type: H*dim query, G*dim key, G*vdim value channels
    int raw_ld;
    const float* taps;     // [taps][channels], the last row meets the current token; null with n_taps 1: no convolution
    int n_taps;
    void* state;           // [slot][n_taps - 1][channels] of the same type: the last projected values of each sequence
    const float2* rope;    // rot/2 {cos, sin} pairs per position (rot 0: no rotation)
    int rot;
    int H;
    void* q_out;           // [T][H][dim_ld]
};
void launch_conv_rope(const ConvRope& c, const KvPages& pool, const StepArrays& st);

struct WindowAttn {
    KvPages pool;
    const void* q;         // [T][H][dim_ld], the pool's element type
    int H;
    float scale;
    float cap;             // score <- cap * tanh(score / cap); 0: none
    int size, keep_first;  // position i sees j <= i with i - j < size or j < keep_first
    __half* out_b16;       // activation tiles of [T][H * vdim_ld] (bf16 pool) ...
    float* out_f32;        // ... or rows [T][H * vdim] (fp32 pool)
};
constexpr int WINDOW_RUN = 64;   // stage_step(attn_ct, multi_first): tokens per run at most
void launch_window_attention(const WindowAttn& a, const StepArrays& st);

}  // namespace nvllm
