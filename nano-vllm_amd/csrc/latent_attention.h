// latent_attention.h -- attention over cached latents: per position ONE row shared by all heads, [latent c |
// rotated key part], that serves as key and (its first part) as value.  Queries come with the key
// up-projection absorbed, q_row = [W_uk^T q_plain | rotated q], and the result is the attended latent, to
// which the caller applies the value up-projection.
#pragma once

#include "nvllm_internal.h"
#include "step_arrays.h"

namespace nvllm {

// One layer run's slice of the block pool.
//   fp32 (elem_bytes 4): rows [block][position][rank + rot].
//   bf16 (elem_bytes 2): "latent pages" of 16 positions, each row_ld/32 tiles of 1 KiB in the operand order of
//     v_mfma_f32_16x16x32_bf16: element (key, d) of a page sits at half
//     (d >> 5) * 512 + (key + 16 * ((d >> 3) & 3)) * 8 + (d & 7).
//     rank and rot are padded to multiples of 32 (zeros); block_size is a multiple of 16.
struct LatentPool {
    void* base;
    int elem_bytes;
    int block_size;
    int rank, rot;         // latent and rotated sizes
    int rank_ld, rot_ld;   // as stored
    int row() const { return rank_ld + rot_ld; }
};
constexpr int LATENT_PAGE = 16;
LatentPool latent_pool(void* base, int elem_bytes, int block_size, int rank, int rot);
static inline size_t latent_pool_bytes(const LatentPool& p, int num_blocks) { return (size_t)num_blocks * p.block_size * p.row() * p.elem_bytes; }

// Norm (plain weight), rotation and cache write of a batch's new rows.  raw: fp32 [T][raw_ld], the latent at 0 and
// the rotated part's input at rot_at; rope: rot/2 {cos, sin} pairs per position.
void launch_latent_kv(const LatentPool& pool, const float* raw, int raw_ld, int rot_at, const float* gain, float eps, const float2* rope,
                      const StepArrays& st);

// the same as a rider of the query projection (launch_gemm_b16)
struct LatentKvRider;
LatentKvRider latent_kv_rider(const LatentPool& pool, const float* raw, int raw_ld, int rot_at, const float* gain, float eps, const float2* rope,
                              const StepArrays& st);

struct LatentAttn {
    LatentPool pool;
    const void* q;         // [T][H][pool.row()], element type as the pool's
    const float* sink;     // [H]: the softmax denominator also holds exp(sink)
    float scale;
    int H;
    float* out_f32;        // fp32 pool: [T][H][rank]
    __half* out_b16;       // bf16 pool: activation tiles of [T, H * rank_ld]
};
constexpr int LATENT_RUN = 32;   // stage_step(attn_ct, multi_first): tokens per run at most
void launch_latent_attention(const LatentAttn& a, const StepArrays& st);

// fp32 models: q [T][H * (dim + rot)] -> rows [T][H][rank + rot] (W_uk [H * dim, rank] absorbed, rotated part turned)
void launch_latent_q_f32(float* rows, const float* q, const float* uk, const float2* rope, const int* pos, int T, int H, int dim, int rot, int rank);
// attended latents [T][H][rank] -> values [T][H * vdim] (W_uv [H * vdim, rank])
void launch_latent_v_f32(float* out, const float* lat, const float* uv, int T, int H, int vdim, int rank);

// fp32 rows -> bf16 rows padded to row_ld halves per row, in two parts (latent, rotated); and bf16 activation tiles -> fp32
// rows: the operator entry points use them around the bf16 kernels
void launch_latent_rows_b16(__half* dst, const float* src, int rows, const LatentPool& pool);
void launch_untile_b16(float* dst, const __half* tiles, int T, int H, int width, int width_ld);

}  // namespace nvllm
