// latent_kv.h -- one token's latent row for the cache: RMS norm of the latent (plain weight), rotation of the
// shared key part, both written to the token's place in the pool.  One wave per token.  Run by a launch of its own
// (latent_attention.hip) or by the extra workgroups of the query projection (LatentKvRider).
#pragma once

#include "gemm_common.h"

namespace nvllm {

// half index of element d of the bf16 row at pool row r (block * block_size + slot)
__device__ __forceinline__ size_t latent_off(long r, int d, int row) {
    return (size_t)(r >> 4) * 16 * row + (size_t)(d >> 5) * 512 + (size_t)(((int)r & 15) + 16 * ((d >> 3) & 3)) * 8 + (d & 7);
}

// v = src[0 .. rank) normed and [rot_at ..) rotated, element by element through put(d, v), d in the stored row
template <typename Put>
__device__ __forceinline__ void latent_kv_token(const LatentKvRider& a, int t, int lane, Put&& put) {
    const float* src = a.raw + (size_t)t * a.raw_ld;
    float ss = 0.f;
    for (int d = lane; d < a.rank; d += 64) ss = fmaf(src[d], src[d], ss);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float rms = sqrtf(ss / (float)a.rank + a.eps);
    for (int d = lane; d < a.rank_ld; d += 64) put(d, d < a.rank ? src[d] / rms * a.gain[d] : 0.f);
    const float2* tab = a.rope + (size_t)a.pos[t] * (a.rot >> 1);
    for (int i = lane; i < a.rot_ld >> 1; i += 64) {
        float u = 0.f, v = 0.f;
        if (2 * i < a.rot) {
            const float2 cs = tab[i];
            const float p = src[a.rot_at + 2 * i], q = src[a.rot_at + 2 * i + 1];
            u = p * cs.x - q * cs.y;
            v = q * cs.x + p * cs.y;
        }
        put(a.rank_ld + 2 * i, u);
        put(a.rank_ld + 2 * i + 1, v);
    }
}
// bf16 pages.  A lane owns chunks of eight stored elements (16 bytes of the page); when the input is laid out like the stored
// row (zeros in the padding) and two chunks per lane cover it, everything the token needs is requested before the first sum.
__device__ __forceinline__ void latent_kv_ride(const LatentKvRider& a, int t, int lane) {
    if (t >= a.T) return;
    const long row = a.kv_row[t];
    const int width = a.rank_ld + a.rot_ld, chunks = width >> 3;
    __half* base = reinterpret_cast<__half*>(a.base);
    if (a.rot_at != a.rank_ld || a.raw_ld != width || chunks > 128) {
        if (row < 0) return;
        latent_kv_token(a, t, lane, [&](int d, float v) { reinterpret_cast<__bf16*>(base)[latent_off(row, d, width)] = (__bf16)v; });
        return;
    }
    const float* src = a.raw + (size_t)t * a.raw_ld;
    const float2* tab = a.rope + (size_t)a.pos[t] * (a.rot >> 1);
    f4_t v[2][2], g[2][2];   // the chunk's values; gain, or {cos, sin} pairs
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < 2; u++) {
        const int d = 8 * (lane + 64 * u);
        if (d >= width) continue;
#pragma unroll
        for (int e = 0; e < 2; e++) v[u][e] = *reinterpret_cast<const f4_t*>(src + d + 4 * e);
        if (d < a.rank_ld) {
#pragma unroll
            for (int e = 0; e < 2; e++) g[u][e] = *reinterpret_cast<const f4_t*>(a.gain + d + 4 * e);
        } else {
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int i = ((d - a.rank_ld) >> 1) + e;
                const float2 cs = tab[min(i, (a.rot >> 1) - 1)];   // (pairs past `rot` are zeros)
                g[u][e >> 1][2 * (e & 1)] = cs.x;
                g[u][e >> 1][2 * (e & 1) + 1] = cs.y;
            }
        }
    }
#pragma unroll
    for (int u = 0; u < 2; u++)
        if (8 * (lane + 64 * u) < a.rank_ld)
#pragma unroll
            for (int e = 0; e < 8; e++) ss = fmaf(v[u][e >> 2][e & 3], v[u][e >> 2][e & 3], ss);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float rms = sqrtf(ss / (float)a.rank + a.eps);
    if (row < 0) return;
#pragma unroll
    for (int u = 0; u < 2; u++) {
        const int d = 8 * (lane + 64 * u);
        if (d >= width) continue;
        float z[8];
        if (d < a.rank_ld) {
#pragma unroll
            for (int e = 0; e < 8; e++) z[e] = v[u][e >> 2][e & 3] / rms * g[u][e >> 2][e & 3];
        } else {
#pragma unroll
            for (int e = 0; e < 8; e += 2) {
                const float p = v[u][e >> 2][e & 3], q = v[u][e >> 2][(e & 3) + 1], c = g[u][e >> 2][e & 3], s = g[u][e >> 2][(e & 3) + 1];
                z[e] = p * c - q * s;
                z[e + 1] = q * c + p * s;
            }
        }
        alignas(16) b4_t out[2] = {to_b4(z), to_b4(z + 4)};
        *reinterpret_cast<u4_t*>(base + latent_off(row, d, width)) = *reinterpret_cast<const u4_t*>(out);
    }
}

}  // namespace nvllm
