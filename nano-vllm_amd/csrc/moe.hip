// moe.hip -- routing, sorting and summing for mixtures of experts (moe.h).
#include "moe.h"

#include <algorithm>

#include "attn_tile.h"
#include "gemm_common.h"

namespace nvllm {

namespace {
constexpr int ROUTE_ONE = 256;      // up to here one workgroup routes and sorts
constexpr int MAX_EXPERTS = 4096;
}

int route_pad(int T, int E, int top) {
    const long per = (long)T * top / E;   // rows an expert gets on average
    return per >= 96 ? 128 : per >= 40 ? 64 : per > 20 ? 32 : 16;
}
static int route_capacity(int T, int E, int top, int pad) {
    const long rows = (long)T * top, groups = std::min(rows, rows / pad + E);   // full groups, and one partly filled per expert
    return (int)(groups * pad);
}
size_t route_ints(int T, int E, int top, int pad) {
    const size_t cap = (size_t)route_capacity(T, E, top, pad);
    return cap / 16 + 2 * cap + 3 * (size_t)T * top + 64;
}
RoutePlan route_plan(int* mem, int T, int E, int top, int pad) {
    RoutePlan r{};
    r.T = T; r.E = E; r.top = top; r.pad = pad;
    r.capacity = route_capacity(T, E, top, pad);
    r.block_expert = mem;
    r.source = r.block_expert + r.capacity / 16;
    r.weight = (float*)(r.source + r.capacity);
    r.row_of = (int*)(r.weight + r.capacity);
    r.choice = r.row_of + (size_t)T * top;
    r.score = (float*)(r.choice + (size_t)T * top);
    return r;
}

// Maximum over a wave, in every lane, on the vector unit alone (many waves of one CU would queue for the LDS crossbar):
// rotations within rows of 16 lanes, then the rows.
template <int N>
__device__ __forceinline__ float row_rotate(float x) {
    const int v = __builtin_bit_cast(int, x);
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(v, v, 0x120 + N, 0xf, 0xf, false));
}
__device__ __forceinline__ float wave_max(float x) {
    x = fmaxf(x, row_rotate<8>(x));
    x = fmaxf(x, row_rotate<4>(x));
    x = fmaxf(x, row_rotate<2>(x));
    x = fmaxf(x, row_rotate<1>(x));
    return rows_max(x);
}

// One wave chooses for one token: `top` times the best of what comes after the previous choice in the order
// (score descending, index ascending).
__device__ __forceinline__ void route_token(const RoutePlan& r, const float* __restrict__ z, int t, int lane) {
    float last = INFINITY;
    int last_e = -1;
    for (int j = 0; j < r.top; j++) {
        float best = -INFINITY;
        int best_e = 0x7fffffff;
        for (int e = lane; e < r.E; e += 64) {
            const float v = z[e];
            const bool open = v < last || (v == last && e > last_e);
            if (open && v > best) {
                best = v;
                best_e = e;
            }
        }
        const float top = wave_max(best);
        int first = best == top ? best_e : 0x7fffffff;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) first = min(first, __shfl_xor(first, o, 64));
        best = top;
        best_e = first;
        if (best_e >= r.E) best_e = 0;   // (no number compares: NaN logits)
        last = best;
        last_e = best_e;
        if (lane == 0) {
            r.choice[(size_t)t * r.top + j] = best_e;
            r.score[(size_t)t * r.top + j] = 1.f / (1.f + expf(-best));
        }
    }
}
__global__ __launch_bounds__(256) void k_route(RoutePlan r, const float* __restrict__ z, int ldz) {
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t < r.T) route_token(r, z + (size_t)t * ldz, t, threadIdx.x & 63);
}

// One workgroup: counts, segment starts, then every choice takes a row of its expert's segment (in any order: a row's
// result does not depend on its place).
template <bool CHOOSE>
__global__ __launch_bounds__(1024) void k_route_sort(RoutePlan r, const float* __restrict__ z, int ldz) {
    extern __shared__ int lds_r[];   // counts [E], next free row [E], segment start [E + 1], CHOOSE: choices and scores [T * top]
    int* count = lds_r;
    int* cursor = count + r.E;
    int* start = cursor + r.E;
    const int tid = threadIdx.x, lane = tid & 63, pairs = r.T * r.top;
    int *choice = CHOOSE ? start + r.E + 1 : r.choice, *out_choice = r.choice;
    float* out_score = r.score;
    float* score = CHOOSE ? reinterpret_cast<float*>(choice + pairs) : r.score;
    for (int e = tid; e < r.E; e += 1024) count[e] = 0;
    if (CHOOSE) {
        r.choice = choice;   // (route_token fills the LDS copies)
        r.score = score;
        if (r.E <= 64) {   // a logit per lane, four tokens at a time
            for (int t0 = tid >> 6; t0 < r.T; t0 += 64) {
                float v[4];
#pragma unroll
                for (int u = 0; u < 4; u++) v[u] = lane < r.E ? z[(size_t)min(t0 + 16 * u, r.T - 1) * ldz + lane] : -INFINITY;
                for (int j = 0; j < r.top; j++) {
                    float best[4];
#pragma unroll
                    for (int u = 0; u < 4; u++) best[u] = wave_max(v[u]);
#pragma unroll
                    for (int u = 0; u < 4; u++) {
                        const int t = t0 + 16 * u;
                        const unsigned long long at = __ballot(v[u] == best[u] && lane < r.E);
                        const int e = at ? __ffsll(at) - 1 : 0;   // (no number compares: NaN logits)
                        if (lane == e) v[u] = -INFINITY;
                        if (lane == 0 && t < r.T) {
                            choice[t * r.top + j] = e;
                            score[t * r.top + j] = 1.f / (1.f + expf(-best[u]));
                        }
                    }
                }
            }
        } else {
            for (int t = tid >> 6; t < r.T; t += 16) route_token(r, z + (size_t)t * ldz, t, lane);
        }
    }
    __syncthreads();
    for (int i = tid; i < pairs; i += 1024) atomicAdd(count + choice[i], 1);
    __syncthreads();
    if (tid < 64) {   // the first wave sums the padded counts
        int base = 0;
        for (int e0 = 0; e0 < r.E; e0 += 64) {
            const int e = e0 + tid, n = e < r.E ? (count[e] + r.pad - 1) / r.pad * r.pad : 0;
            int sum = n;
#pragma unroll
            for (int o = 1; o < 64; o <<= 1) {
                const int v = __shfl_up(sum, o, 64);
                if (tid >= o) sum += v;
            }
            if (e < r.E) start[e] = cursor[e] = base + sum - n;
            base += __shfl(sum, 63, 64);
        }
        if (tid == 0) start[r.E] = base;
    }
    __syncthreads();   // the last one: from here on everybody only writes results (a barrier would wait for the stores)
    const int used = start[r.E];
    for (int b = used / 16 + tid; b < r.capacity / 16; b += 1024) r.block_expert[b] = -1;
    for (int i = used + tid; i < r.capacity; i += 1024) {   // (a tile may look up rows behind its own: they name a token too)
        r.source[i] = 0;
        r.weight[i] = 0.f;
    }
    for (int e = tid >> 4; e < r.E; e += 64) {   // 16 threads per expert: its blocks, and the padding of its segment
        const int lo = start[e], hi = start[e + 1], n = count[e];
        for (int b = lo / 16 + (tid & 15); b < hi / 16; b += 16) r.block_expert[b] = e;
        for (int i = lo + n + (tid & 15); i < hi; i += 16) {
            r.source[i] = 0;
            r.weight[i] = 0.f;
        }
    }
    for (int i = tid; i < pairs; i += 1024) {
        const int row = atomicAdd(cursor + choice[i], 1);
        r.source[row] = i / r.top;
        r.weight[row] = score[i];
        r.row_of[i] = row;
        if (CHOOSE) {
            out_choice[i] = choice[i];
            out_score[i] = score[i];
        }
    }
}

void launch_route(const RoutePlan& r, const float* z, int ldz) {
    if (r.T <= 0) return;
    if (r.E < 1 || r.E > MAX_EXPERTS || r.top < 1 || r.top > r.E) NVLLM_FATAL("routing: %d of %d experts per token", r.top, r.E);
    const size_t lds = ((size_t)3 * r.E + 1) * sizeof(int);
    const double bytes = (double)r.T * (r.E * 4.0 + r.top * 20.0);
    const size_t lds_one = lds + (size_t)r.T * r.top * 8;
    if (r.T <= ROUTE_ONE && lds_one <= 64 * 1024) {
        ProfScope ps(PC_ROUTE, bytes, 0);
        NVLLM_LAUNCH((k_route_sort<true>), dim3(1), dim3(1024), lds_one, r, z, ldz);
        return;
    }
    {
        ProfScope ps(PC_ROUTE, bytes, 0);
        NVLLM_LAUNCH(k_route, dim3(cdiv(r.T, 4)), dim3(256), 0, r, z, ldz);
    }
    ProfScope ps(PC_ROUTE, (double)r.T * r.top * 28.0, 0);
    NVLLM_LAUNCH((k_route_sort<false>), dim3(1), dim3(1024), lds, r, z, ldz);
}

// A workgroup per 16 rows, a wave per tile: lane (row, k group) reads 32 bytes of its row and writes its piece of the tile.
__global__ __launch_bounds__(256) void k_expert_rows(__half* __restrict__ dst, const float* __restrict__ x, const float* __restrict__ gain, RoutePlan r, int ld) {
    const int blk = blockIdx.x, lane = threadIdx.x & 63, Kb = ld >> 5;
    if (r.block_expert[blk] < 0) return;
    const float* row = x + (size_t)r.source[blk * 16 + (lane & 15)] * ld + 8 * (lane >> 4);
    for (int kb = threadIdx.x >> 6; kb < Kb; kb += 4) {
        const f4_t a = *reinterpret_cast<const f4_t*>(row + kb * 32), b = *reinterpret_cast<const f4_t*>(row + kb * 32 + 4);
        const f4_t ga = *reinterpret_cast<const f4_t*>(gain + kb * 32 + 8 * (lane >> 4)), gb = *reinterpret_cast<const f4_t*>(gain + kb * 32 + 8 * (lane >> 4) + 4);
        b8_t v;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            v[e] = (__bf16)(a[e] * ga[e]);
            v[4 + e] = (__bf16)(b[e] * gb[e]);
        }
        *reinterpret_cast<b8_t*>(dst + ((size_t)blk * Kb + kb) * TILE_HALVES + lane * 8) = v;
    }
}
void launch_expert_rows(__half* dst, const float* x, const float* gain, const RoutePlan& r, int ld) {
    if (r.T <= 0) return;
    if (ld % 32) NVLLM_FATAL("expert rows: a row of %d is not padded to 32", ld);
    ProfScope ps(PC_EXPERT_ROWS, (double)r.T * r.top * ld * 2.0 + (double)r.T * ld * 4.0, 0);
    NVLLM_LAUNCH(k_expert_rows, dim3(r.capacity / 16), dim3(256), 0, dst, x, gain, r, ld);
}

// One workgroup per token.  VEC 4: eight neighbouring threads cover 32 features.
template <int VEC>
__global__ __launch_bounds__(256) void k_moe_combine(MoeCombine m, int top) {
    const int t = blockIdx.x, Kb = m.ld >> 5;
    struct alignas(4 * VEC) Vec { float v[VEC]; };
    const float gate = m.shared ? 1.f / (1.f + expf(-m.z[(size_t)t * m.ldz + m.z_col])) : 0.f;
    const int wide = VEC == 4 ? ((m.ld + 255) & ~255) : m.ld;   // (whole waves: the sums cross lanes)
    for (int n = threadIdx.x * VEC; n < wide; n += 256 * VEC) {
        float sq = 0.f;
        if (n < m.ld) {
            Vec y;
#pragma unroll
            for (int e = 0; e < VEC; e++) y.v[e] = 0.f;
            for (int j = 0; j < top; j++) {
                const size_t row = m.row_of ? (size_t)m.row_of[(size_t)t * top + j] : (size_t)t * top + j;
                const Vec r = *reinterpret_cast<const Vec*>(m.rows + row * m.ld + n);
#pragma unroll
                for (int e = 0; e < VEC; e++) y.v[e] += r.v[e];
            }
            if (m.shared) {
                const Vec r = *reinterpret_cast<const Vec*>(m.shared + (size_t)t * m.ld + n);
#pragma unroll
                for (int e = 0; e < VEC; e++) y.v[e] = fmaf(gate, r.v[e], y.v[e]);
            }
            Vec* xp = reinterpret_cast<Vec*>(m.x + (size_t)t * m.ld + n);
            Vec xv = *xp;
#pragma unroll
            for (int e = 0; e < VEC; e++) {
                xv.v[e] += y.v[e];
                sq += xv.v[e] * xv.v[e];
            }
            *xp = xv;
            if (VEC == 4 && m.out_b16) {
                const f4_t g = *reinterpret_cast<const f4_t*>(m.gain + n);
                const float w[4] = {xv.v[0] * g[0], xv.v[1 % VEC] * g[1], xv.v[2 % VEC] * g[2], xv.v[3 % VEC] * g[3]};
                store_b16_4(m.out_b16, Kb, t, n, w);
            }
        }
        if (VEC == 4 && m.ss) {
            sq += __shfl_xor(sq, 1, 64);
            sq += __shfl_xor(sq, 2, 64);
            sq += __shfl_xor(sq, 4, 64);
            if ((threadIdx.x & 7) == 0 && n < m.ld) m.ss[(size_t)t * Kb + (n >> 5)] = sq;
        }
    }
}
void launch_moe_combine(const MoeCombine& m, int T) {
    if (T <= 0) return;
    if (m.out_b16 && m.ld % 32) NVLLM_FATAL("sum of experts: a row of %d is not padded to 32", m.ld);
    ProfScope ps(PC_MOE_COMBINE, (double)T * m.ld * (4.0 * m.top + (m.shared ? 4.0 : 0.0) + 8.0 + (m.out_b16 ? 2.0 : 0.0)), 0);
    if (m.ld % 4 == 0) NVLLM_LAUNCH((k_moe_combine<4>), dim3(T), dim3(256), 0, m, m.top);
    else NVLLM_LAUNCH((k_moe_combine<1>), dim3(T), dim3(256), 0, m, m.top);
}

// ------------------------------------------------------------------ fp32 path
__global__ __launch_bounds__(256) void k_matmul_experts_f32(float* __restrict__ out, const float* __restrict__ in, const float* __restrict__ w,
                                                            const int* __restrict__ choice, const float* __restrict__ score, int top, int by_token, int K, int N) {
    const int i = blockIdx.x, n = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (n >= N) return;
    const float* x = in + (size_t)(by_token ? i / top : i) * K;
    const float* wr = w + ((size_t)choice[i] * N + n) * K;
    const float scale = by_token ? score[i] : 1.f;
    float acc = 0.f;
    for (int k = lane; k < K; k += 64) acc = fmaf(scale * x[k], wr[k], acc);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) acc += __shfl_xor(acc, o, 64);
    if (lane == 0) out[(size_t)i * N + n] = acc;
}
void launch_matmul_experts_f32(float* out, const float* in, const float* w, const RoutePlan& r, bool by_token, int K, int N) {
    const int pairs = r.T * r.top;
    if (pairs <= 0) return;
    ProfScope ps(PC_GEMM_OTHER, (double)std::min(r.E, pairs) * N * K * 4.0 + (double)pairs * (K + N) * 4.0, 2.0 * pairs * (double)N * K);
    NVLLM_LAUNCH(k_matmul_experts_f32, dim3(pairs, cdiv(N, 4)), dim3(256), 0, out, in, w, r.choice, r.score, r.top, by_token ? 1 : 0, K, N);
}
__global__ __launch_bounds__(256) void k_relu2(float* x, long n) {
    const long i = (long)blockIdx.x * 256 + threadIdx.x;
    if (i < n) {
        const float v = fmaxf(x[i], 0.f);
        x[i] = v * v;
    }
}
void launch_relu2(float* x, long n) {
    if (n <= 0) return;
    ProfScope ps(PC_ELEMWISE, (double)n * 8.0, 0);
    NVLLM_LAUNCH(k_relu2, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, x, n);
}

}  // namespace nvllm
