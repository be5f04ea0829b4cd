// lightning.h -- linear attention with a per-head decay: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, the state
// carried from pass to pass in 32-bit floats, one slot per sequence.
#pragma once

#include "nvllm_internal.h"
#include "step_arrays.h"

namespace nvllm {

constexpr int LIGHTNING_CHUNK = 64;   // tokens per step of the chunked kernels
// stage_step(chunk_len) for a batch of T tokens: tokens a workgroup of the chunked kernels walks
int lightning_group(int T, int H, int vdim);

// One layer run over a batch.  Every sequence's portion starts from its slot's state (from zero at position 0) and
// leaves the state behind its last token there.
struct Lightning {
    int H, dim, vdim;
    const float* decay;     // [H][LIGHTNING_CHUNK + 1]: decay^0 .. decay^CHUNK
    float* state;           // [slot][H][dim][vdim]
    // bf16: rows [T][ld] of q, k (H * dim_ld each), v, gate (H * vdim_ld each), heads padded to 32 with zeros;
    // results: o * gain * sigmoid(gate) as activation tiles [T][H * vdim_ld], and sums of squares of o per 16 values
    const __half* rows = nullptr;
    int ld = 0, dim_ld = 0, vdim_ld = 0;
    const float* gain = nullptr;   // [H * vdim_ld], padded with zeros
    __half* out_b16 = nullptr;
    float* ss_out = nullptr;       // [T][H * vdim_ld / 16]
    // fp32: q, k, v [T][H * dim | dim | vdim], out [T][H * vdim]
    const float *q32 = nullptr, *k32 = nullptr, *v32 = nullptr;
    float* out_f32 = nullptr;
};
static inline size_t lightning_state_floats(int H, int dim, int vdim) { return (size_t)H * dim * vdim; }   // of one slot
void launch_lightning(const Lightning& a, const StepArrays& st);

// out = x * sigmoid(g) (fp32 path: the gate on the normed heads)
void launch_sigmoid_gate(float* out, const float* x, const float* g, long n);
void launch_silu(float* x, long n);

}  // namespace nvllm
