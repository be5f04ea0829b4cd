// hyper.hip -- hyper-connections (several residual streams per token) with the Dynamic Tanh norm, and the
// other element-wise operators of the designs that use them, as launches of their own: the fp32 path, models
// with more streams than the projection epilogue holds in registers (gemm_common.h, hyper_update_4), the
// step from the embedding into the first layer, and the operator entry points.
#include "gemm_common.h"

namespace nvllm {

// one thread per (token, feature); the old streams of the thread's element live in LDS: any number of streams
__global__ __launch_bounds__(256) void k_hyper_step(HyperStep h, int T, int Kb) {
    extern __shared__ float s_old[];   // [streams][256]
    const long i = (long)blockIdx.x * 256 + threadIdx.x;
    const int S = h.streams, ld = h.ld;
    if (i >= (long)T * ld) return;
    const int t = (int)(i / ld), n = (int)(i % ld);
    const float* mix = h.record;
    const float* out = mix + S * S;
    const float* in = out + S;
    float* xr = h.x + (size_t)t * S * ld + n;
    float u = 0.f;
    if (h.y) {
        float y = h.y[i];
        if (h.bias) y += h.bias[n];
        if (h.scale) y *= h.scale[n];
        for (int s = 0; s < S; s++) s_old[s * 256 + threadIdx.x] = xr[(size_t)s * ld];
        for (int to = 0; to < S; to++) {
            float v = out[to] * y;
            for (int s = 0; s < S; s++) v = fmaf(mix[s * S + to], s_old[s * 256 + threadIdx.x], v);
            xr[(size_t)to * ld] = v;
            u = fmaf(in[to], v, u);
        }
    } else {
        for (int s = 0; s < S; s++) u = fmaf(in[s], xr[(size_t)s * ld], u);
    }
    const float z = h.norm_w ? fmaf(tanhf(in[S] * u), h.norm_w[n], h.norm_b[n]) : u;
    if (h.out_f32) h.out_f32[i] = z;
    if (h.out_b16)
        reinterpret_cast<__bf16*>(h.out_b16)[((size_t)(t >> 4) * Kb + (n >> 5)) * TILE_HALVES + (size_t)((t & 15) + 16 * ((n >> 3) & 3)) * 8 + (n & 7)] = (__bf16)z;
}
void launch_hyper_step(const HyperStep& h, int T) {
    if (T <= 0) return;
    if (h.streams < 1 || h.streams > 64) NVLLM_FATAL("hyper-connections: %d streams (1 to 64 are supported)", h.streams);
    if (h.out_b16 && h.ld % 32) NVLLM_FATAL("hyper-connections: a row of %d is not padded to 32", h.ld);
    const long n = (long)T * h.ld;
    ProfScope ps(PC_HYPER, (double)n * 4.0 * (h.streams * (h.y ? 2 : 1) + 1), 0);
    NVLLM_LAUNCH(k_hyper_step, dim3((unsigned)((n + 255) / 256)), dim3(256), (size_t)h.streams * 256 * sizeof(float), h, T, h.ld / 32);
}

template <bool B16>
__global__ __launch_bounds__(256) void k_embed_streams(float* __restrict__ x, const void* __restrict__ table, const int* __restrict__ tokens, int S, int ld,
                                                       const int* __restrict__ tok_src, const int* __restrict__ prev) {
    const int t = blockIdx.x;
    const int tok = (tok_src && tok_src[t] >= 0) ? prev[tok_src[t]] : tokens[t];
    for (int n = threadIdx.x; n < ld; n += 256) {
        const size_t i = (size_t)tok * ld + n;
        const float v = B16 ? (float)reinterpret_cast<const __bf16*>(table)[i] : reinterpret_cast<const float*>(table)[i];
        for (int s = 0; s < S; s++) x[((size_t)t * S + s) * ld + n] = v;
    }
}
void launch_embed_streams(float* x, const void* table, bool bf16, const int* tokens, int T, int streams, int ld, const int* tok_src, const int* prev) {
    if (T <= 0) return;
    ProfScope ps(PC_EMBED, (double)T * ld * (4.0 * streams + (bf16 ? 2.0 : 4.0)), 0);
    if (bf16) NVLLM_LAUNCH((k_embed_streams<true>), dim3(T), dim3(256), 0, x, table, tokens, streams, ld, tok_src, prev);
    else NVLLM_LAUNCH((k_embed_streams<false>), dim3(T), dim3(256), 0, x, table, tokens, streams, ld, tok_src, prev);
}

// a thread per four features: eight neighbouring threads cover the 32 of a sum of squares
__global__ __launch_bounds__(256) void k_embed_norm_b16(float* __restrict__ x, __half* __restrict__ act, float* __restrict__ ss, const __bf16* __restrict__ table,
                                                        const int* __restrict__ tokens, const float* __restrict__ gain, int ld, const int* __restrict__ tok_src,
                                                        const int* __restrict__ prev) {
    const int t = blockIdx.x, Kb = ld >> 5;
    const int tok = (tok_src && tok_src[t] >= 0) ? prev[tok_src[t]] : tokens[t];
    for (int n = threadIdx.x * 4; n < ((ld + 255) & ~255); n += 1024) {
        float sq = 0.f;
        if (n < ld) {
            const b4_t r = *reinterpret_cast<const b4_t*>(table + (size_t)tok * ld + n);
            const f4_t g = *reinterpret_cast<const f4_t*>(gain + n);
            const float v[4] = {(float)r[0], (float)r[1], (float)r[2], (float)r[3]};
            const float z[4] = {v[0] * g[0], v[1] * g[1], v[2] * g[2], v[3] * g[3]};
            *reinterpret_cast<float4*>(x + (size_t)t * ld + n) = make_float4(v[0], v[1], v[2], v[3]);
            store_b16_4(act, Kb, t, n, z);
            sq = v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
        sq += __shfl_xor(sq, 1, 64);
        sq += __shfl_xor(sq, 2, 64);
        sq += __shfl_xor(sq, 4, 64);
        if ((threadIdx.x & 7) == 0 && n < ld) ss[(size_t)t * Kb + (n >> 5)] = sq;
    }
}
void launch_embed_norm_b16(float* x, __half* act, float* ss, const void* table, const int* tokens, const float* gain, int T, int ld, const int* tok_src, const int* prev) {
    if (T <= 0) return;
    if (ld % 32) NVLLM_FATAL("embedding: a row of %d is not padded to 32", ld);
    ProfScope ps(PC_EMBED, (double)T * ld * 8.0, 0);
    NVLLM_LAUNCH(k_embed_norm_b16, dim3(T), dim3(256), 0, x, act, ss, (const __bf16*)table, tokens, gain, ld, tok_src, prev);
}

__global__ __launch_bounds__(256) void k_gather_b16(__half* __restrict__ dst, const __half* __restrict__ src, const int* __restrict__ idx, int Kb) {
    const int r = blockIdx.x, t = idx[r];
    for (int c = threadIdx.x; c < Kb * 4; c += 256) {   // 8-element chunks of the row
        const size_t in_tile = (size_t)(16 * (c & 3)) * 8;
        *reinterpret_cast<u4_t*>(dst + ((size_t)(r >> 4) * Kb + (c >> 2)) * TILE_HALVES + (r & 15) * 8 + in_tile) =
            *reinterpret_cast<const u4_t*>(src + ((size_t)(t >> 4) * Kb + (c >> 2)) * TILE_HALVES + (t & 15) * 8 + in_tile);
    }
}
void launch_gather_b16(__half* dst, const __half* src, const int* idx, int B, int K) {
    if (B <= 0) return;
    ProfScope ps(PC_ELEMWISE, (double)B * K * 4.0, 0);
    NVLLM_LAUNCH(k_gather_b16, dim3(B), dim3(256), 0, dst, src, idx, K / 32);
}

__global__ __launch_bounds__(256) void k_swiglu_bias(float* out, const float* g, const float* u, const float* __restrict__ bg, const float* __restrict__ bu,
                                                     long n, int F) {
    const long i = (long)blockIdx.x * 256 + threadIdx.x;
    if (i < n) out[i] = silu_mul(g[i] + bg[i % F], u[i] + bu[i % F]);
}
void launch_swiglu_bias(float* out, const float* g, const float* u, const float* bg, const float* bu, int T, int F) {
    if (T <= 0) return;
    const long n = (long)T * F;
    ProfScope ps(PC_ELEMWISE, (double)n * 12.0, 0);
    NVLLM_LAUNCH(k_swiglu_bias, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, out, g, u, bg, bu, n, F);
}

__global__ __launch_bounds__(256) void k_softcap(float* x, float cap, long n) {
    const long i = (long)blockIdx.x * 256 + threadIdx.x;
    if (i < n) x[i] = cap * tanhf(x[i] / cap);
}
void launch_softcap(float* x, float cap, long n) {
    if (n <= 0) return;
    ProfScope ps(PC_ELEMWISE, (double)n * 8.0, 0);
    NVLLM_LAUNCH(k_softcap, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, x, cap, n);
}

}  // namespace nvllm
