// lightning.hip -- linear attention with decay (lightning.h).
//
// Portions of several tokens (bf16) go in chunks of 64 tokens, a few neighbouring chunks (a group) to a workgroup, as many as
// still leave the chip full; three launches:
//   k_lightning_add    what a group adds to the state, chunk by chunk: U = decay^n U + sum_s k_s (decay^(n-1-s) v_s)^T
//   k_lightning_scan   the states groups start from, over a portion's groups, element by element; U gives way to S
//   k_lightning_out    o_t = decay^(t+1) S^T q_t + sum_{s <= t} decay^(t-s) (k_s . q_t) v_s chunk by chunk, S carried along
// A workgroup takes a group's head x 64 value columns, a wave 16 of them, the state in its registers.  q, k and v are bf16
// values.  The 32-bit factors -- S, the decayed products P[s, t] of queries and keys, the decayed v -- enter the matrix
// cores as three bf16 parts (truncations: 8 + 8 + 8 bits, together the exact value), so every product is that of the 32-bit
// numbers.  The state's result registers are already in the k order of S^T q, P's in that of P v.
//
// k_lightning_step (single tokens, and everything in fp32): a workgroup per (portion, head), the state streamed once per
// token as float4 columns.
#include "lightning.h"

#include "gemm_common.h"

namespace nvllm {

typedef short s4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s4_t lds_s4;
typedef unsigned int u2_t __attribute__((ext_vector_type(2)));

__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(z * -1.44269504088896340736f)); }
__device__ __forceinline__ float b16_f(unsigned short v) { return __builtin_bit_cast(float, (unsigned)v << 16); }

// x = a + b + c exactly, each with at most 8 significant bits (their upper halves are bf16 values)
__device__ __forceinline__ void split3(float x, unsigned& a, unsigned& b, unsigned& c) {
    a = __builtin_bit_cast(unsigned, x) & 0xffff0000u;
    const float r = x - __builtin_bit_cast(float, a);
    b = __builtin_bit_cast(unsigned, r) & 0xffff0000u;
    c = __builtin_bit_cast(unsigned, r - __builtin_bit_cast(float, b));
}
__device__ __forceinline__ unsigned upper_halves(unsigned lo, unsigned hi) { return __builtin_amdgcn_perm(hi, lo, 0x07060302u); }
// eight fp32 values -> three operands
__device__ __forceinline__ void split3_frag(const float (&v)[8], b8_t (&out)[3]) {
    u4_t p[3];
#pragma unroll
    for (int i = 0; i < 4; i++) {
        unsigned a0, b0, c0, a1, b1, c1;
        split3(v[2 * i], a0, b0, c0);
        split3(v[2 * i + 1], a1, b1, c1);
        p[0][i] = upper_halves(a0, a1);
        p[1][i] = upper_halves(b0, b1);
        p[2][i] = upper_halves(c0, c1);
    }
#pragma unroll
    for (int s = 0; s < 3; s++) out[s] = __builtin_bit_cast(b8_t, p[s]);
}

constexpr int CH = LIGHTNING_CHUNK;
constexpr int VROW = 64 + 8;   // LDS row of a chunk's values, halves (rows 16-byte aligned, banks shifted)
constexpr int qk_row(int DC) { return DC * 32 + 8; }
constexpr int add_lds(int DC) { return CH * qk_row(DC) * 2 + CH * VROW * 2 + (CH + 1) * 4; }
constexpr int out_lds(int DC) { return 2 * CH * qk_row(DC) * 2 + CH * VROW * 2 + 4 * 2 * 3 * 1024 + (CH + 1) * 4; }

// What the chunk kernels share: a workgroup = group of chunks x head x 64 value columns, a wave = 16 of the columns.
struct ChunkArgs {
    Lightning a;
    const int4* spans;     // (first token, count, first position, sequence)
    const int2* groups;    // (span, group of the span): `per_group` neighbouring chunks
    int n_spans, vslices, per_group;
    float* mem;            // [group][H][value tile][dim tile][64][4]: a tile as the matrix cores leave it, lane (x, g) = S[16 i + 4 g + r][16 j + x]
    int d_tiles, v_tiles;
};
struct ChunkId {
    int slot, h, vs, first, n;   // the group, its first token of the batch and its number of tokens
};
__device__ __forceinline__ ChunkId chunk_id(const ChunkArgs& c) {
    ChunkId id;
    int idx = blockIdx.x;
    id.vs = idx % c.vslices;
    idx /= c.vslices;
    id.h = idx % c.a.H;
    id.slot = idx / c.a.H;
    const int2 gr = c.groups[id.slot];
    const int4 span = c.spans[gr.x];
    id.first = span.x + gr.y * c.per_group * CH;
    id.n = min(c.per_group * CH, span.y - gr.y * c.per_group * CH);
    return id;
}
__device__ __forceinline__ f4_t* chunk_tiles(const ChunkArgs& c, int slot, int h, int vtile) {   // dim tile 0, lane 0
    return reinterpret_cast<f4_t*>(c.mem) + (((size_t)slot * c.a.H + h) * c.v_tiles + vtile) * c.d_tiles * 64;
}
// rows of a chunk, PER 16-byte pieces each by neighbouring threads, zeros behind the n-th row and the last of `pieces`
template <int PER, int U>
__device__ __forceinline__ void chunk_rows(u4_t (&r)[U], const __half* base, int ld, int n, int pieces) {
#pragma unroll
    for (int u = 0; u < U; u++) {
        const int i = (int)threadIdx.x + 256 * u, row = i / PER, piece = i - row * PER;
        r[u] = row < n && piece < pieces ? *reinterpret_cast<const u4_t*>(base + (size_t)row * ld + piece * 8) : u4_t{0, 0, 0, 0};
    }
}
template <int PER, int ROW, int U>
__device__ __forceinline__ void chunk_rows_to_lds(__half* dst, const u4_t (&r)[U]) {
#pragma unroll
    for (int u = 0; u < U; u++) {
        const int i = (int)threadIdx.x + 256 * u, row = i / PER, piece = i - row * PER;
        *reinterpret_cast<u4_t*>(dst + row * ROW + piece * 8) = r[u];
    }
}
// tokens as k of an operand: {32 pair + 4 g .., 32 pair + 16 + 4 g ..} of 16 columns, by the LDS transpose read (16 lanes bring
// 4 rows x 16 columns, lane x receives column x of the four rows)
__device__ __forceinline__ b8_t token_frag(const __half* lds, int row_halves, int col0, int pair) {
    const int x = threadIdx.x & 15, g = (threadIdx.x >> 4) & 3;
    const __half* p = lds + (size_t)(32 * pair + 4 * g + (x >> 2)) * row_halves + col0 + 4 * (x & 3);
    const u2_t lo = __builtin_bit_cast(u2_t, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)p));
    const u2_t hi = __builtin_bit_cast(u2_t, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)(p + (size_t)16 * row_halves)));
    return __builtin_bit_cast(b8_t, u4_t{lo[0], lo[1], hi[0], hi[1]});
}

// S <- decay^n S + sum_s k_s (decay^(n-1-s) v_s)^T over a chunk of n tokens
template <int DC>
__device__ __forceinline__ void chunk_update(f4_t (&S)[2 * DC], const __half* s_k, const b8_t (&vf)[2], const float* s_dec, int n) {
    const int g = (threadIdx.x >> 4) & 3;
    const float fade = s_dec[n];
#pragma unroll
    for (int i = 0; i < 2 * DC; i++) S[i] *= fade;
#pragma unroll
    for (int pair = 0; pair < 2; pair++) {
        float e[8];
#pragma unroll
        for (int i = 0; i < 8; i++) {
            const int s = 32 * pair + 16 * (i >> 2) + 4 * g + (i & 3);
            e[i] = s < n ? (float)vf[pair][i] * s_dec[max(n - 1 - s, 0)] : 0.f;
        }
        b8_t parts[3];
        split3_frag(e, parts);
#pragma unroll
        for (int i = 0; i < 2 * DC; i++) {
            const b8_t kt = token_frag(s_k, qk_row(DC), 16 * i, pair);
#pragma unroll
            for (int k = 2; k >= 0; k--) S[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kt, parts[k], S[i], 0, 0, 0);
        }
    }
}

// ---- 1. what a group of chunks adds to the state
template <int DC>
__global__ __launch_bounds__(256, 2) void k_lightning_add(ChunkArgs c) {
    constexpr int ROW = qk_row(DC);
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_l[];
    __half* s_k = reinterpret_cast<__half*>(lds_l);   // [CH][ROW]
    __half* s_v = s_k + CH * ROW;                     // [CH][VROW]
    float* s_dec = reinterpret_cast<float*>(s_v + CH * VROW);
    const Lightning& a = c.a;
    const ChunkId id = chunk_id(c);
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int v0 = id.vs * 64, my_v = v0 + wave * 16;
    const bool has_v = my_v < a.vdim_ld;
    u4_t rk[DC], rv[2];
    auto fetch = [&](int c0) {
        const __half* base = a.rows + (size_t)(id.first + c0) * a.ld;
        chunk_rows<4 * DC>(rk, base + (a.H + id.h) * a.dim_ld, a.ld, id.n - c0, a.dim_ld / 8);
        chunk_rows<8>(rv, base + 2 * a.H * a.dim_ld + id.h * a.vdim_ld + v0, a.ld, id.n - c0, (a.vdim_ld - v0) / 8);
    };
    fetch(0);
    if (tid <= CH) s_dec[tid] = a.decay[id.h * (CH + 1) + tid];
    f4_t S[2 * DC];
#pragma unroll
    for (int i = 0; i < 2 * DC; i++) S[i] = f4_t{0.f, 0.f, 0.f, 0.f};
    for (int c0 = 0; c0 < id.n; c0 += CH) {
        chunk_rows_to_lds<4 * DC, ROW>(s_k, rk);
        chunk_rows_to_lds<8, VROW>(s_v, rv);
        __syncthreads();
        if (c0 + CH < id.n) fetch(c0 + CH);
        if (has_v) {
            const b8_t vf[2] = {token_frag(s_v, VROW, wave * 16, 0), token_frag(s_v, VROW, wave * 16, 1)};
            chunk_update<DC>(S, s_k, vf, s_dec, min(CH, id.n - c0));
        }
        __syncthreads();   // the chunk's rows have been read
    }
    if (!has_v) return;
    f4_t* out = chunk_tiles(c, id.slot, id.h, my_v >> 4) + lane;
#pragma unroll
    for (int i = 0; i < 2 * DC; i++)
        if (i < c.d_tiles) out[i * 64] = S[i];
}

// ---- 2. from what groups add to the states they start from, and the sequence's state behind its portion.  A thread per four
// elements of a state; first_group: of every portion.
__global__ __launch_bounds__(256) void k_lightning_scan(ChunkArgs c, const int* __restrict__ first_group) {
    const Lightning& a = c.a;
    const int tiles = c.v_tiles * c.d_tiles, item = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y;
    if (item >= tiles * 64) return;
    const int4 span = c.spans[blockIdx.z];
    const int lane = item & 63, j = (item >> 6) / c.d_tiles, i = (item >> 6) - j * c.d_tiles;
    const int v = 16 * j + (lane & 15), d0 = 16 * i + 4 * (lane >> 4);
    float* st = a.state + ((size_t)span.w * a.H + h) * a.dim * a.vdim;
    f4_t S;
#pragma unroll
    for (int r = 0; r < 4; r++) S[r] = span.z > 0 && d0 + r < a.dim && v < a.vdim ? st[(size_t)(d0 + r) * a.vdim + v] : 0.f;
    const int len = c.per_group * CH, n_groups = (span.y + len - 1) / len;
    const size_t stride = (size_t)a.H * tiles * 64;
    f4_t* p = reinterpret_cast<f4_t*>(c.mem) + (size_t)first_group[blockIdx.z] * stride + (size_t)h * tiles * 64 + item;
    const float* dec = a.decay + h * (CH + 1);
    auto faded = [&](int tokens) {   // decay^tokens
        float f = 1.f;
        for (; tokens > CH; tokens -= CH) f *= dec[CH];
        return f * dec[tokens];
    };
    const float whole = faded(len), tail = faded(span.y - (n_groups - 1) * len);
    for (int k0 = 0; k0 < n_groups; k0 += 8) {
        f4_t u[8];
#pragma unroll
        for (int k = 0; k < 8; k++) u[k] = p[min(k0 + k, n_groups - 1) * stride];
#pragma unroll
        for (int k = 0; k < 8; k++)
            if (k0 + k < n_groups) {
                p[(k0 + k) * stride] = S;
                S = S * (k0 + k == n_groups - 1 ? tail : whole) + u[k];
            }
    }
#pragma unroll
    for (int r = 0; r < 4; r++)
        if (d0 + r < a.dim && v < a.vdim) st[(size_t)(d0 + r) * a.vdim + v] = S[r];
}

// ---- 3. the results, chunk by chunk from the state the group starts from
template <int DC>
__global__ __launch_bounds__(256, 2) void k_lightning_out(ChunkArgs c) {
    constexpr int ROW = qk_row(DC);
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_l[];
    __half* s_q = reinterpret_cast<__half*>(lds_l);   // [CH][ROW]
    __half* s_k = s_q + CH * ROW;                     // [CH][ROW]
    __half* s_v = s_k + CH * ROW;                     // [CH][VROW]
    b8_t* s_p = reinterpret_cast<b8_t*>(s_v + CH * VROW);            // [t tile][s pair][part][64]
    float* s_dec = reinterpret_cast<float*>(s_p + 4 * 2 * 3 * 64);   // [CH + 1]
    const Lightning& a = c.a;
    const ChunkId id = chunk_id(c);
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), x = lane & 15, g = lane >> 4;
    const int h = id.h, v0 = id.vs * 64, my_v = v0 + wave * 16;
    const bool has_v = my_v < a.vdim_ld;
    u4_t rq[DC], rk[DC], rv[2];
    u2_t rg[4];   // gates of this wave's columns my_v + 4 g .. + 3, tokens 16 i + x
    auto fetch = [&](int c0) {
        const __half* base = a.rows + (size_t)(id.first + c0) * a.ld;
        const int left = id.n - c0;
        chunk_rows<4 * DC>(rq, base + h * a.dim_ld, a.ld, left, a.dim_ld / 8);
        chunk_rows<4 * DC>(rk, base + (a.H + h) * a.dim_ld, a.ld, left, a.dim_ld / 8);
        chunk_rows<8>(rv, base + 2 * a.H * a.dim_ld + h * a.vdim_ld + v0, a.ld, left, (a.vdim_ld - v0) / 8);
#pragma unroll
        for (int i = 0; i < 4; i++)
            rg[i] = has_v ? *reinterpret_cast<const u2_t*>(base + (size_t)min(16 * i + x, left - 1) * a.ld + 2 * a.H * a.dim_ld + (a.H + h) * a.vdim_ld + my_v + 4 * g) : u2_t{0, 0};
    };
    fetch(0);
    f4_t S[2 * DC], gain = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 2 * DC; i++) S[i] = f4_t{0.f, 0.f, 0.f, 0.f};
    if (has_v) {
        const f4_t* in = chunk_tiles(c, id.slot, h, my_v >> 4) + lane;
#pragma unroll
        for (int i = 0; i < 2 * DC; i++)
            if (i < c.d_tiles) S[i] = in[i * 64];
        gain = *reinterpret_cast<const f4_t*>(a.gain + h * a.vdim_ld + my_v + 4 * g);
    }
    if (tid <= CH) s_dec[tid] = a.decay[h * (CH + 1) + tid];
    const int ss_ld = a.H * a.vdim_ld / 16, Kb_out = a.H * a.vdim_ld / 32, col = h * a.vdim_ld + my_v;
    for (int c0 = 0; c0 < id.n; c0 += CH) {
        const int n = min(CH, id.n - c0);
        chunk_rows_to_lds<4 * DC, ROW>(s_q, rq);
        chunk_rows_to_lds<4 * DC, ROW>(s_k, rk);
        chunk_rows_to_lds<8, VROW>(s_v, rv);
        u2_t gates[4];
#pragma unroll
        for (int i = 0; i < 4; i++) gates[i] = rg[i];
        __syncthreads();
        const bool more = c0 + CH < id.n;
        if (more) fetch(c0 + CH);
        // operands over dims in the order of the state's registers: {32 cc + 4 g .., 32 cc + 16 + 4 g ..} of row 16 i + x
        auto frag = [&](const __half* lds, int i, int cc) {
            const __half* p = lds + (16 * i + x) * ROW + 32 * cc + 4 * g;
            const u2_t lo = *reinterpret_cast<const u2_t*>(p), hi = *reinterpret_cast<const u2_t*>(p + 16);
            return __builtin_bit_cast(b8_t, u4_t{lo[0], lo[1], hi[0], hi[1]});
        };
        // ---- P of token tile `wave`: rows s (tiles 0 .. wave), columns t
        if (wave * 16 < n) {
            b8_t qf[DC];
#pragma unroll
            for (int cc = 0; cc < DC; cc++) qf[cc] = frag(s_q, wave, cc);
            const int t = wave * 16 + x;
#pragma unroll
            for (int pair = 0; pair < 2; pair++) {
                if (2 * pair > wave) break;
                float e[8];
#pragma unroll
                for (int half = 0; half < 2; half++) {
                    f4_t p = {0.f, 0.f, 0.f, 0.f};
                    const int i = 2 * pair + half;
                    if (i <= wave) {
#pragma unroll
                        for (int cc = 0; cc < DC; cc++) p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(frag(s_k, i, cc), qf[cc], p, 0, 0, 0);
                    }
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const int s = 16 * i + 4 * g + r;
                        e[4 * half + r] = s <= t ? p[r] * s_dec[max(t - s, 0)] : 0.f;
                    }
                }
                b8_t parts[3];
                split3_frag(e, parts);
#pragma unroll
                for (int k = 0; k < 3; k++) s_p[((wave * 2 + pair) * 3 + k) * 64 + lane] = parts[k];
            }
        }
        b8_t sf[DC][3];   // the state as operand, three exact parts
#pragma unroll
        for (int cc = 0; cc < DC; cc++) {
            float e[8];
#pragma unroll
            for (int i = 0; i < 8; i++) e[i] = S[2 * cc + (i >> 2)][i & 3];
            split3_frag(e, sf[cc]);
        }
        __syncthreads();
        if (has_v) {
            const b8_t vf[2] = {token_frag(s_v, VROW, wave * 16, 0), token_frag(s_v, VROW, wave * 16, 1)};
            // (the four token tiles are independent chains of products)
            f4_t o[4];
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] = f4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int cc = 0; cc < DC; cc++) {
                b8_t qf[4];
#pragma unroll
                for (int i = 0; i < 4; i++) qf[i] = frag(s_q, i, cc);
#pragma unroll
                for (int k = 2; k >= 0; k--)
#pragma unroll
                    for (int i = 0; i < 4; i++) o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sf[cc][k], qf[i], o[i], 0, 0, 0);
            }
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] *= s_dec[i * 16 + x + 1];
#pragma unroll
            for (int pair = 0; pair < 2; pair++)
#pragma unroll
                for (int k = 2; k >= 0; k--)
#pragma unroll
                    for (int i = 2 * pair; i < 4; i++)   // (P of tiles past the chunk's end is whatever LDS holds; their results are not stored)
                        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[pair], s_p[((i * 2 + pair) * 3 + k) * 64 + lane], o[i], 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                float sq = o[i][0] * o[i][0] + o[i][1] * o[i][1] + o[i][2] * o[i][2] + o[i][3] * o[i][3];
                sq += __shfl_xor(sq, 16, 64);
                sq += __shfl_xor(sq, 32, 64);
                const int tl = i * 16 + x, t = id.first + c0 + tl;
                if (tl < n) {
                    float y[4];
#pragma unroll
                    for (int r = 0; r < 4; r++) y[r] = o[i][r] * gain[r] * sigmoid_f(b16_f((unsigned short)(gates[i][r >> 1] >> (16 * (r & 1)))));
                    store_b16_4(a.out_b16, Kb_out, t, col + 4 * g, y);
                    if (g == 0) a.ss_out[(size_t)t * ss_ld + (col >> 4)] = sq;
                }
            }
            if (more) chunk_update<DC>(S, s_k, vf, s_dec, n);
        }
        __syncthreads();   // the chunk's rows and P have been read
    }
}

// A workgroup per (portion, head).  Thread = VEC neighbouring value columns x every ROWS-th dim.
template <bool B16, int VEC>
__global__ __launch_bounds__(256) void k_lightning_step(Lightning a, const int4* __restrict__ spans) {
    extern __shared__ float lds_s[];   // q [dim], k [dim], v [vdim], partial results [256 * VEC], result [vdim], reduction [4]
    float* s_q = lds_s;
    float* s_k = s_q + a.dim;
    float* s_v = s_k + a.dim;
    float* s_part = s_v + a.vdim;
    float* s_o = s_part + 256 * VEC;
    float* s_red = s_o + a.vdim;
    const int tid = threadIdx.x, h = blockIdx.x;
    const int4 span = spans[blockIdx.y];
    const float decay = a.decay[h * (CH + 1) + 1];
    float* st = a.state + ((size_t)span.w * a.H + h) * a.dim * a.vdim;
    const int cols = a.vdim / VEC, per = min(cols, 256), rows = 256 / per;   // per columns side by side, `rows` rows of threads
    const int row0 = tid / per, col0 = tid - row0 * per;
    const bool on = row0 < rows;
    const unsigned short* src = reinterpret_cast<const unsigned short*>(a.rows);
    const int ss_ld = a.H * a.vdim_ld / 16, tiles = a.vdim_ld / 16, Kb_out = a.H * a.vdim_ld / 32;
    for (int i = 0; i < span.y; i++) {
        const int t = span.x + i;
        for (int d = tid; d < a.dim; d += 256) {
            if (B16) {
                s_q[d] = b16_f(src[(size_t)t * a.ld + h * a.dim_ld + d]);
                s_k[d] = b16_f(src[(size_t)t * a.ld + (a.H + h) * a.dim_ld + d]);
            } else {
                s_q[d] = a.q32[((size_t)t * a.H + h) * a.dim + d];
                s_k[d] = a.k32[((size_t)t * a.H + h) * a.dim + d];
            }
        }
        for (int v = tid; v < a.vdim; v += 256)
            s_v[v] = B16 ? b16_f(src[(size_t)t * a.ld + 2 * a.H * a.dim_ld + h * a.vdim_ld + v]) : a.v32[((size_t)t * a.H + h) * a.vdim + v];
        __syncthreads();
        const bool fresh = span.z + i == 0;
        for (int cb = 0; cb < cols; cb += per) {   // (one round unless the values are very wide)
            const int col = cb + col0;
            float part[VEC];
#pragma unroll
            for (int e = 0; e < VEC; e++) part[e] = 0.f;
            if (on && col < cols) {
                float vv[VEC];
#pragma unroll
                for (int e = 0; e < VEC; e++) vv[e] = s_v[col * VEC + e];
                struct alignas(4 * VEC) Vec { float v[VEC]; };
                constexpr int AHEAD = 4;   // rows in flight
                for (int d0 = row0; d0 < a.dim; d0 += AHEAD * rows) {
                    Vec s[AHEAD];
#pragma unroll
                    for (int u = 0; u < AHEAD; u++)
                        s[u] = *reinterpret_cast<const Vec*>(st + (size_t)min(d0 + u * rows, a.dim - 1) * a.vdim + col * VEC);
#pragma unroll
                    for (int u = 0; u < AHEAD; u++) {
                        const int d = d0 + u * rows;
                        if (d >= a.dim) break;
                        const float kd = s_k[d], qd = s_q[d];
#pragma unroll
                        for (int e = 0; e < VEC; e++) {
                            s[u].v[e] = fmaf(kd, vv[e], fresh ? 0.f : decay * s[u].v[e]);
                            part[e] = fmaf(qd, s[u].v[e], part[e]);
                        }
                        *reinterpret_cast<Vec*>(st + (size_t)d * a.vdim + col * VEC) = s[u];
                    }
                }
            }
#pragma unroll
            for (int e = 0; e < VEC; e++) s_part[tid * VEC + e] = part[e];
            __syncthreads();
            for (int v = tid; v < per * VEC && cb * VEC + v < a.vdim; v += 256) {
                float o = 0.f;
                for (int r = 0; r < rows; r++) o += s_part[r * per * VEC + v];
                s_o[cb * VEC + v] = o;
            }
            __syncthreads();
        }
        if (!B16) {
            for (int v = tid; v < a.vdim; v += 256) a.out_f32[((size_t)t * a.H + h) * a.vdim + v] = s_o[v];
        } else {
            float sq = 0.f;
            for (int v = tid; v < a.vdim_ld; v += 256) {
                const float o = v < a.vdim ? s_o[v] : 0.f;
                sq += o * o;
                const int c = h * a.vdim_ld + v;
                const float gate = b16_f(src[(size_t)t * a.ld + 2 * a.H * a.dim_ld + a.H * a.vdim_ld + c]);
                reinterpret_cast<__bf16*>(a.out_b16)[((size_t)(t >> 4) * Kb_out + (c >> 5)) * TILE_HALVES + (size_t)((t & 15) + 16 * ((c >> 3) & 3)) * 8 + (c & 7)] =
                    (__bf16)(o * a.gain[c] * sigmoid_f(gate));
            }
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) sq += __shfl_xor(sq, o, 64);
            if ((tid & 63) == 0) s_red[tid >> 6] = sq;
            __syncthreads();
            // the head's whole sum stands in its first place
            for (int k = tid; k < tiles; k += 256)
                a.ss_out[(size_t)t * ss_ld + h * tiles + k] = k == 0 ? (s_red[0] + s_red[1]) + (s_red[2] + s_red[3]) : 0.f;
        }
        __syncthreads();   // the token's vectors are free again
    }
}

template <int DC>
static void launch_add(const ChunkArgs& c, int n_groups) {
    constexpr int shmem = add_lds(DC);
    static_assert(shmem <= 64 * 1024, "no attribute needed");
    NVLLM_LAUNCH((k_lightning_add<DC>), dim3(n_groups * c.a.H * c.vslices), dim3(256), shmem, c);
}
template <int DC>
static void launch_out(const ChunkArgs& c, int n_groups) {
    constexpr int shmem = out_lds(DC);
    static bool enabled = false;
    if (shmem > 64 * 1024 && !enabled) {
        HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_lightning_out<DC>), hipFuncAttributeMaxDynamicSharedMemorySize, shmem));
        enabled = true;
    }
    NVLLM_LAUNCH((k_lightning_out<DC>), dim3(n_groups * c.a.H * c.vslices), dim3(256), shmem, c);
}
// Portions of several tokens: the chunks' additions, the scan over them, the chunks' results.
static void launch_chunks(const Lightning& a, const StepArrays& st, double bytes, double flops) {
    ChunkArgs c{};
    c.a = a;
    c.spans = (const int4*)st.d_spans;
    c.groups = (const int2*)st.d_chunks;
    c.per_group = st.chunk_len / CH;
    c.n_spans = st.n_spans_multi;
    c.vslices = cdiv(a.vdim_ld, 64);
    c.d_tiles = a.dim_ld / 16;
    c.v_tiles = a.vdim_ld / 16;
    const size_t tiles = (size_t)a.H * c.d_tiles * c.v_tiles;   // of a state
    c.mem = (float*)ws_get(WS_STATES, st.n_chunks * tiles * 1024);
    const int DC = a.dim_ld / 32, n = st.n_chunks;
    // the algorithm's bytes and flops: those of the recurrence, split over the three launches
    {
        ProfScope ps(PC_LIGHTNING, bytes / 3, flops / 3);
        if (DC == 1) launch_add<1>(c, n);
        else if (DC == 2) launch_add<2>(c, n);
        else if (DC == 3) launch_add<3>(c, n);
        else if (DC == 4) launch_add<4>(c, n);
        else launch_add<8>(c, n);
    }
    {
        ProfScope ps(PC_LIGHTNING, bytes / 3, flops / 3);
        NVLLM_LAUNCH(k_lightning_scan, dim3(cdiv(c.d_tiles * c.v_tiles * 64, 256), a.H, c.n_spans), dim3(256), 0, c, (const int*)st.d_first_chunk);
    }
    ProfScope ps(PC_LIGHTNING, bytes / 3, flops / 3);
    if (DC == 1) launch_out<1>(c, n);
    else if (DC == 2) launch_out<2>(c, n);
    else if (DC == 3) launch_out<3>(c, n);
    else if (DC == 4) launch_out<4>(c, n);
    else launch_out<8>(c, n);
}

int lightning_group(int T, int H, int vdim) {
    const long wgs = (long)cdiv(T, CH) * H * cdiv(vdim, 64);   // with one chunk each
    int per = 1;
    while (per < 8 && wgs / (2 * per) >= 2 * rt().num_cus) per *= 2;
    return per * CH;
}

void launch_lightning(const Lightning& a, const StepArrays& st) {
    if (st.T <= 0) return;
    if (!st.d_spans) NVLLM_FATAL("linear attention: the batch was staged without its portions");
    const bool b16 = a.rows != nullptr;
    const int n_single = st.n_spans - st.n_spans_multi, multi_tokens = st.T - n_single;
    const double state_bytes = (double)lightning_state_floats(a.H, a.dim, a.vdim) * 8.0;   // read and written
    const double elem = b16 ? 2.0 : 4.0, token_bytes = (double)a.H * (2.0 * a.dim + 3.0 * a.vdim) * elem;
    const double pair = 2.0 * a.H * (double)(a.dim + a.vdim), token_flops = 4.0 * a.H * (double)a.dim * a.vdim;
    const int DC = a.dim_ld / 32;
    const bool chunked = b16 && DC <= 8;
    if (chunked && st.n_spans_multi > 0) {
        if (st.chunk_len < CH || st.chunk_len % CH) NVLLM_FATAL("linear attention: the batch was staged in chunks of %d tokens", st.chunk_len);
        launch_chunks(a, st, st.n_spans_multi * state_bytes + multi_tokens * token_bytes, multi_tokens * (token_flops + pair * 0.5 * std::min(st.max_span, CH)));
    }
    const int from = chunked ? st.n_spans_multi : 0, n = st.n_spans - from;
    if (n <= 0) return;
    const bool wide = a.vdim % 4 == 0;
    const size_t lds = ((size_t)2 * a.dim + 2 * a.vdim + 256 * (wide ? 4 : 1) + 4) * sizeof(float);
    if (lds > 64 * 1024) NVLLM_FATAL("linear attention heads of %d and %d values are too wide", a.dim, a.vdim);
    const int4* spans = (const int4*)st.d_spans + from;
    ProfScope ps(PC_LIGHTNING_TOK, n * state_bytes + (chunked ? n_single : st.T) * token_bytes, (chunked ? n_single : st.T) * token_flops);
    const dim3 grid(a.H, n);
    if (b16 && wide) NVLLM_LAUNCH((k_lightning_step<true, 4>), grid, dim3(256), lds, a, spans);
    else if (b16) NVLLM_LAUNCH((k_lightning_step<true, 1>), grid, dim3(256), lds, a, spans);
    else if (wide) NVLLM_LAUNCH((k_lightning_step<false, 4>), grid, dim3(256), lds, a, spans);
    else NVLLM_LAUNCH((k_lightning_step<false, 1>), grid, dim3(256), lds, a, spans);
}

// ------------------------------------------------------------------ element-wise steps of the fp32 path
__global__ __launch_bounds__(256) void k_sigmoid_gate(float* out, const float* x, const float* __restrict__ g, long n) {
    const long i = (long)blockIdx.x * 256 + threadIdx.x;
    if (i < n) out[i] = x[i] * sigmoid_f(g[i]);
}
void launch_sigmoid_gate(float* out, const float* x, const float* g, long n) {
    if (n <= 0) return;
    ProfScope ps(PC_ELEMWISE, (double)n * 12.0, 0);
    NVLLM_LAUNCH(k_sigmoid_gate, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, out, x, g, n);
}
__global__ __launch_bounds__(256) void k_silu(float* x, long n) {
    const long i = (long)blockIdx.x * 256 + threadIdx.x;
    if (i < n) x[i] = silu_mul(x[i], 1.f);
}
void launch_silu(float* x, long n) {
    if (n <= 0) return;
    ProfScope ps(PC_ELEMWISE, (double)n * 8.0, 0);
    NVLLM_LAUNCH(k_silu, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, x, n);
}

}  // namespace nvllm
