// gemm_common.h -- what the projection kernels share: the launch record and the
// element-wise pieces of their epilogues (see gemm.hip for what each epilogue does).
#pragma once

#include "nvllm_internal.h"

namespace nvllm {

typedef _Float16 h8_t __attribute__((ext_vector_type(8)));
typedef float f4_t __attribute__((ext_vector_type(4)));
typedef unsigned int u4_t __attribute__((ext_vector_type(4)));

typedef __bf16 b8_t __attribute__((ext_vector_type(8)));
typedef __bf16 b4_t __attribute__((ext_vector_type(4)));

// How activations enter a projection, and the multiply that goes with it.  Fragments travel as eight 16-bit
// values per lane either way (h8_t); OpBf16 reinterprets their bits.
struct OpF16x2 {   // fp16 weights; fp32 activations as fp16 hi + lo planes
    static constexpr int PLANES = 2;
    static __device__ __forceinline__ f4_t mfma(h8_t w, h8_t a, f4_t c) { return __builtin_amdgcn_mfma_f32_16x16x32_f16(w, a, c, 0, 0, 0); }
};
struct OpBf16 {    // bf16 weights, bf16 activations
    static constexpr int PLANES = 1;
    static __device__ __forceinline__ f4_t mfma(h8_t w, h8_t a, f4_t c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(b8_t, w), __builtin_bit_cast(b8_t, a), c, 0, 0, 0);
    }
};
// epilogues that act on four consecutive features of one token at a time (epi_point below)
constexpr bool epi_is_point(int kind) { return kind >= GemmEpilogue::TILE_B16 && kind != GemmEpilogue::RESID_B16; }
// epilogues that also leave sums of squares per 32 features
constexpr bool epi_has_ss(int kind) { return kind == GemmEpilogue::RESID_A16 || kind == GemmEpilogue::LATENT_IN || kind == GemmEpilogue::RESID_B16; }

// What a launch may carry besides its tiles: the norm, rotation and cache write of the batch's latent rows (latent_kv.h)
// in extra workgroups, a wave per token.  Their input comes from the launch before and their output is for the launch
// after, so they cost no time of their own.
struct LatentKvRider {
    void* base = nullptr;   // null: nobody rides
    const float* raw;
    const float* gain;
    const float2* rope;
    const int* pos;
    const int* kv_row;
    float eps;
    int raw_ld, rot_at, T, rank, rot, rank_ld, rot_ld;
};

struct GemmArgs {
    const __half* W;
    long nb_stride;   // halves between 16-row blocks
    int NB;           // 16-row blocks
    int Kb;           // k tiles
    const __half* A;  // activation tiles [Tb][Kb][2][512]
    int Tb;
    int N, T;
    int act_Kb;       // k tiles per token block of A (Kb, or Kb * groups of a block-diagonal product)
    int group_nb;     // block-diagonal product: 16-row blocks per group, 0 = one group ...
    int group_tiles;  // ... and feature tiles per group (streaming kernel: grid columns)
    const int* block_expert;   // rows sorted by expert (ExpertRows): expert of a row block ...
    const int* source;         // ... row of A that a row reads (null: its own) ...
    long expert_stride;        // ... and halves between the experts' matrices
    int kb_per_split;
    int ksplit;
    float* slab;      // [tile][slice][round][item] float4
    unsigned* counters;
    int close_sc1;    // K split: the closing workgroup loads the partials past the vector cache instead of invalidating it
                      // (launches of at most one workgroup per CU over a hipMalloc slab)
    GemmEpilogue e;
    LatentKvRider ride;
    int ride_from;    // first workgroup (grid x) of the riders
#ifdef NVLLM_STAMPS
    unsigned long long* stamps;   // diagnostic builds only: [workgroup][8] constant-rate clock readings
#endif
};

// In-kernel timeline for diagnostic builds (tools/gemm_stamps.py): wave 0 of every workgroup
// records the 100 MHz constant-rate clock once the value `dep` exists.  Compiled out otherwise.
#ifdef NVLLM_STAMPS
#define NVLLM_STAMP(k, dep)                                                                                   \
    do {                                                                                                      \
        unsigned long long t__;                                                                               \
        asm volatile("s_memrealtime %0\n\ts_waitcnt lgkmcnt(0)" : "=s"(t__) : "v"(dep) : "memory");            \
        if (p.stamps && threadIdx.x == 0)                                                                     \
            p.stamps[(size_t)((blockIdx.z * gridDim.y + blockIdx.y) * gridDim.x + blockIdx.x) * 8 + (k)] = t__; \
    } while (0)
// the same inside gemm_tile(), whose caller says where the tile's eight readings go (`stamps_wg`)
#define NVLLM_TSTAMP(k, dep)                                                                        \
    do {                                                                                            \
        unsigned long long t__;                                                                     \
        asm volatile("s_memrealtime %0\n\ts_waitcnt lgkmcnt(0)" : "=s"(t__) : "v"(dep) : "memory");  \
        if (stamps_wg && tid == 0) stamps_wg[(k)] = t__;                                    \
    } while (0)
#else
#define NVLLM_STAMP(k, dep) do {} while (0)
#define NVLLM_TSTAMP(k, dep) do {} while (0)
#endif

__device__ __forceinline__ float silu_mul(float g, float u) {
    // reference layers.c:156-158: g / (1 + expf(-g)) * u
    return __fmul_rn(__fdiv_rn(g, __fadd_rn(1.0f, expf(-g))), u);
}

__device__ __forceinline__ void split16_4(const float* y, __half* hi, __half* lo) {
#pragma unroll
    for (int r = 0; r < 4; r++) {
        const float c = fminf(fmaxf(y[r], -65504.f), 65504.f);
        hi[r] = __float2half_rn(c);
        lo[r] = __float2half_rn(c - __half2float(hi[r]));
    }
}

// store 4 consecutive k of token t into hi/lo tiles (n % 4 == 0)
__device__ __forceinline__ void store_a16_4(__half* a16, int Kb_out, int t, int n, const float* y) {
    alignas(8) __half hi[4], lo[4];
    split16_4(y, hi, lo);
    const size_t tile = ((size_t)(t >> 4) * Kb_out + (n >> 5)) * 2;
    const size_t off = (size_t)((t & 15) + 16 * ((n >> 3) & 3)) * 8 + (n & 7);
    *reinterpret_cast<uint2*>(a16 + tile * TILE_HALVES + off) = *reinterpret_cast<uint2*>(hi);
    *reinterpret_cast<uint2*>(a16 + (tile + 1) * TILE_HALVES + off) = *reinterpret_cast<uint2*>(lo);
}

template <typename KVT>
__device__ __forceinline__ void kv_put4(KVT* dst, const float* y);
template <>
__device__ __forceinline__ void kv_put4<float>(float* dst, const float* y) {
    *reinterpret_cast<float4*>(dst) = make_float4(y[0], y[1], y[2], y[3]);
}
__device__ __forceinline__ __half kv_sat_half(float v) {   // finite fp16 only: masked keys need 0 * finite = 0
    return __float2half_rn(fminf(fmaxf(v, -65504.f), 65504.f));
}
template <>
__device__ __forceinline__ void kv_put4<__half>(__half* dst, const float* y) {
    alignas(8) __half h[4] = {kv_sat_half(y[0]), kv_sat_half(y[1]), kv_sat_half(y[2]), kv_sat_half(y[3])};
    *reinterpret_cast<uint2*>(dst) = *reinterpret_cast<uint2*>(h);
}
// four consecutive dims of one key in a V page: 4 halves apart
template <typename KVT>
__device__ __forceinline__ void kv_put4_strided(KVT* dst, const float* y);
template <>
__device__ __forceinline__ void kv_put4_strided<float>(float*, const float*) {}
template <>
__device__ __forceinline__ void kv_put4_strided<__half>(__half* dst, const float* y) {
#pragma unroll
    for (int e = 0; e < 4; e++) dst[4 * e] = kv_sat_half(y[e]);
}

__device__ __forceinline__ b4_t to_b4(const float* y) {
    const f4_t v = {y[0], y[1], y[2], y[3]};
    return __builtin_convertvector(v, b4_t);
}
// 4 consecutive k of token t into bf16 activation tiles (n % 4 == 0)
__device__ __forceinline__ void store_b16_4(__half* act, int Kb_out, int t, int n, const float* y) {
    const size_t tile = (size_t)(t >> 4) * Kb_out + (n >> 5);
    const size_t off = (size_t)((t & 15) + 16 * ((n >> 3) & 3)) * 8 + (n & 7);
    *reinterpret_cast<b4_t*>(act + tile * TILE_HALVES + off) = to_b4(y);
}

// Hyper-connection update of one token's features n .. n+3 and the next sublayer's input from it:
//   x_to <- sum_from mix[from][to] x_from + out[to] * (y + bias) * scale;   u = sum_s in[s] x_s;
//   act = tanh(alpha u) w + b
// in two halves: what does not depend on y is loaded early, so that it travels while the sums are completed.
template <int SMAX>
struct HyperIn {
    f4_t xs[SMAX], scale, bias, w, b;
};
template <int SMAX>
__device__ __forceinline__ void hyper_load_4(HyperIn<SMAX>& in, const GemmEpilogue& ep, int N, int t, int n) {
    const float* xr = ep.x + (size_t)t * ep.streams * N + n;
#pragma unroll
    for (int s = 0; s < SMAX; s++) in.xs[s] = *reinterpret_cast<const f4_t*>(xr + (size_t)min(s, ep.streams - 1) * N);
    in.scale = *reinterpret_cast<const f4_t*>(ep.hyper_scale + n);
    in.bias = ep.bias ? *reinterpret_cast<const f4_t*>(ep.bias + n) : f4_t{0.f, 0.f, 0.f, 0.f};
    in.w = *reinterpret_cast<const f4_t*>(ep.norm_w + n);
    in.b = *reinterpret_cast<const f4_t*>(ep.norm_b + n);
}
template <int SMAX>
__device__ __forceinline__ void hyper_update_4(const HyperIn<SMAX>& in, const GemmEpilogue& ep, int N, int t, int n, const float* y_in) {
    const int S = ep.streams;
    float y[4];
#pragma unroll
    for (int r = 0; r < 4; r++) y[r] = (y_in[r] + in.bias[r]) * in.scale[r];
    float* xr = ep.x + (size_t)t * S * N + n;
    const float* mix = ep.hyper;
    const float* out = mix + S * S;
    const float* weight = out + S;
    const float alpha = weight[S];
    f4_t u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int to = 0; to < SMAX; to++)
        if (to < S) {
            const float o = out[to], ii = weight[to];
            f4_t v;
#pragma unroll
            for (int r = 0; r < 4; r++) v[r] = o * y[r];
#pragma unroll
            for (int s = 0; s < SMAX; s++)
                if (s < S) {
                    const float m = mix[s * S + to];
#pragma unroll
                    for (int r = 0; r < 4; r++) v[r] = fmaf(m, in.xs[s][r], v[r]);
                }
            *reinterpret_cast<f4_t*>(xr + (size_t)to * N) = v;
#pragma unroll
            for (int r = 0; r < 4; r++) u[r] = fmaf(ii, v[r], u[r]);
        }
    float z[4];
#pragma unroll
    for (int r = 0; r < 4; r++) z[r] = fmaf(tanhf(alpha * u[r]), in.w[r], in.b[r]);
    store_b16_4(ep.a16_out, ep.Kb_out, t, n, z);
}
constexpr int hyper_streams(int kind) { return kind == GemmEpilogue::HYPER_2 ? 2 : kind == GemmEpilogue::HYPER_4 ? 4 : 0; }   // 0: another epilogue

// Residual add of one token's features n .. n+3: xr <- xo + y, x * gain -> tiles; returns their sum of squares.
__device__ __forceinline__ float resid_b16_4(const GemmEpilogue& ep, int N, int t, int n, const float4 xo, const float4 g, const float* y) {
    const float xn[4] = {xo.x + y[0], xo.y + y[1], xo.z + y[2], xo.w + y[3]};
    *reinterpret_cast<float4*>(ep.x + (size_t)t * N + n) = make_float4(xn[0], xn[1], xn[2], xn[3]);
    const float z[4] = {xn[0] * g.x, xn[1] * g.y, xn[2] * g.z, xn[3] * g.w};
    store_b16_4(ep.a16_out, ep.Kb_out, t, n, z);
    return xn[0] * xn[0] + xn[1] * xn[1] + xn[2] * xn[2] + xn[3] * xn[3];
}

// One token's features n .. n+3 through a point epilogue other than HYPER_*; returns their share of the sum of squares.
template <int EPI>
__device__ __forceinline__ float epi_point(const GemmEpilogue& ep, int N, int t, int n, const float* y) {
    if constexpr (EPI == GemmEpilogue::TILE_B16) {
        if (ep.relu2) {
            float z[4];
#pragma unroll
            for (int r = 0; r < 4; r++) z[r] = fmaxf(y[r], 0.f) * fmaxf(y[r], 0.f);
            store_b16_4(ep.a16_out, ep.Kb_out, t, n, z);
            return 0.f;
        }
        store_b16_4(ep.a16_out, ep.Kb_out, t, n, y);
    } else if constexpr (EPI == GemmEpilogue::ROWS_B16) {
        const int h = n / ep.head_ld, d = n - h * ep.head_ld;
        float z[4] = {y[0], y[1], y[2], y[3]};
        if (n < ep.silu_to)
#pragma unroll
            for (int r = 0; r < 4; r++) z[r] = silu_mul(y[r], 1.f);
        *reinterpret_cast<b4_t*>(ep.q_rows + ((size_t)t * ep.q_heads + h) * ep.q_row + d) = to_b4(z);
    } else if constexpr (EPI == GemmEpilogue::LATENT_IN) {
        if (n < ep.latent_q) {
            const f4_t g = *reinterpret_cast<const f4_t*>(ep.gain_next + n);
            const float z[4] = {y[0] * g[0], y[1] * g[1], y[2] * g[2], y[3] * g[3]};
            store_b16_4(ep.a16_out, ep.Kb_out, t, n, z);
            return y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3];
        }
        *reinterpret_cast<f4_t*>(ep.out + (size_t)t * ep.ldo + (n - ep.latent_q)) = f4_t{y[0], y[1], y[2], y[3]};
    } else if constexpr (EPI == GemmEpilogue::LATENT_Q) {
        if (n < ep.q_plain) {
            store_b16_4(ep.a16_out, ep.Kb_out, t, n, y);
        } else {
            const int m = n - ep.q_plain, h = m / ep.rot_ld, d = m - h * ep.rot_ld;
            float z[4] = {0.f, 0.f, 0.f, 0.f};
            const float2* tab = ep.rope + (size_t)ep.pos[t] * (ep.rot_dim >> 1);
#pragma unroll
            for (int e = 0; e < 4; e += 2)
                if (d + e < ep.rot_dim) {   // (features past rot_dim are padding)
                    const float2 cs = tab[(d + e) >> 1];
                    z[e] = y[e] * cs.x - y[e + 1] * cs.y;
                    z[e + 1] = y[e + 1] * cs.x + y[e] * cs.y;
                }
            *reinterpret_cast<b4_t*>(ep.q_rows + ((size_t)t * ep.q_heads + h) * ep.q_row + ep.head_ld + d) = to_b4(z);
        }
    }
    return 0.f;
}

typedef __attribute__((address_space(3))) void lds_void;
// One wave copies one 1-KiB tile global -> LDS without passing through registers: lane l's
// 16 bytes land at lds_byte_address + 16*l.  Written as an asm statement on purpose: the
// compiler then keeps no account of the copy, and the waits below are the only ones (with
// the builtin it drains every copy in flight before the next read of the LDS array).
// M0 carries the LDS address and is restored inside the statement.
__device__ __forceinline__ void copy_tile_to_lds(const __half* lane_src, unsigned lds_byte_address) {
    unsigned keep;
    asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off\n\ts_mov_b32 m0, %0"
                 : "=&s"(keep)
                 : "v"(lane_src), "s"(lds_byte_address)
                 : "memory");
}

// gemm_prefill.hip: 128 x 128 output tiles through LDS, for batches of hundreds of tokens
void launch_gemm_prefill(GemmArgs a);

}  // namespace nvllm
