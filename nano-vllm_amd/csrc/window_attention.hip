// window_attention.hip -- attention with a sliding window and kept first tokens (window_attention.h).
//
// k_window_attn (bf16 pages).  Pages are stored in the operand order of the matrix cores, so a wave reads a key page
// (operand A of S^T = K Q^T) and a value page (operand A of O^T = V^T P^T) straight from memory into registers; a score
// tile's result registers are already in the k order of the second product, and a column (one query) stays on its lane
// through scores, weights, sums and results: no LDS and no barrier in the loop.  A step takes two pages (32 keys) while
// the next step's travel.
//   prompts        a wave owns C groups of 16 neighbouring tokens x up to four heads of a key/value group;
//   single tokens  the columns are the heads of a group; the waves of a workgroup (and, when there are few items,
//                  several workgroups) take every n-th pair of pages and their sums meet in LDS (and in a merge launch).
// The walk visits the pages of the kept first tokens and those the item's window touches; only pages at an edge are masked.
// A soft cap bounds every score, so with a cap of up to 32 the largest weight is known beforehand: weights are
// exp(score - cap), no running maximum and no rescaling (exp(-2 * 32) is far inside the range of fp32 and bf16).
// Scores, caps, maxima and sums are fp32.
//
// k_window_attn_any (fp32 rows, and heads too wide for the kernel above): one workgroup per (token, head).
#include "window_attention.h"

#include "attn_tile.h"
#include "gemm_common.h"
#include "model_dir.h"

namespace nvllm {

KvPages kv_pages(void* base, int elem_bytes, int block_size, int num_blocks, int G, int dim, int vdim) {
    KvPages p{base, nullptr, elem_bytes, block_size, G, dim, vdim, dim, vdim};
    if (elem_bytes == 2) {
        if (block_size % KV_PAGE) NVLLM_FATAL("bf16 key and value pages hold 16 positions: block size %d is not a multiple of 16", block_size);
        p.dim_ld = pad32(dim);
        p.vdim_ld = pad32(vdim);
    }
    if (base) p.values = (char*)base + (size_t)num_blocks * block_size * G * p.dim_ld * elem_bytes;
    return p;
}
size_t kv_pages_bytes(int elem_bytes, int block_size, int num_blocks, int G, int dim, int vdim) {
    const KvPages p = kv_pages(nullptr, elem_bytes, block_size, num_blocks, G, dim, vdim);
    return ((size_t)num_blocks * block_size * G * (p.dim_ld + p.vdim_ld) * elem_bytes + 255) & ~(size_t)255;
}

__device__ __forceinline__ float b16_f32(unsigned short v) { return __builtin_bit_cast(float, (unsigned)v << 16); }
__device__ __forceinline__ size_t key_off(long row, int g, int G, int d, int dim_ld) {
    return ((size_t)(row >> 4) * G + g) * (KV_PAGE * dim_ld) + (d >> 5) * 512 + ((row & 15) + 16 * ((d >> 3) & 3)) * 8 + (d & 7);
}
__device__ __forceinline__ size_t value_off(long row, int g, int G, int d, int vdim_ld) {
    return ((size_t)(row >> 4) * G + g) * (KV_PAGE * vdim_ld) + (d >> 4) * 256 + (((row & 15) >> 2) * 16 + (d & 15)) * 4 + (row & 3);
}

// ------------------------------------------------------------------ convolution, rotation, cache write
struct ConvKArgs {
    ConvRope c;
    KvPages pool;
    const int4* spans;
    const int* span_of;
    const int* kv_row;
    int channels, QD, KD;
    int items_q, items_k, items_v, items;   // work items of a query head, a key head, a value head; of a token
};

template <typename RT, int VEC>
struct alignas(sizeof(RT) * VEC) ConvVec {
    RT v[VEC];
};

// A thread owns VEC neighbouring channels of a token, together with their rotation partners when they turn.  The tokens
// that still see the state of earlier passes belong to the thread of the portion's first token, which then renews it.
template <typename RT, int VEC>
__global__ __launch_bounds__(256) void k_conv_rope(ConvKArgs a) {
    typedef ConvVec<RT, VEC> Vec;
    const int item = blockIdx.y * 256 + threadIdx.x;
    if (item >= a.items) return;
    const int t_mine = blockIdx.x, keep = a.c.n_taps - 1;
    const int4 span = a.spans[a.span_of[t_mine]];   // (first token, count, first position, sequence)
    const int off_mine = t_mine - span.x;
    if (off_mine > 0 && off_mine < keep) return;
    const int n_mine = off_mine == 0 ? min(span.y, max(keep, 1)) : 1;
    const RT* raw = reinterpret_cast<const RT*>(a.c.raw) + (size_t)span.x * a.c.raw_ld;
    RT* state = keep > 0 ? reinterpret_cast<RT*>(a.c.state) + (size_t)span.w * keep * a.channels : nullptr;

    // which head, which dims: part 0 query, 1 key, 2 value
    int part, head, at, i = item;
    if (i < a.c.H * a.items_q) {
        part = 0;
        head = i / a.items_q;
        at = i - head * a.items_q;
    } else if ((i -= a.c.H * a.items_q) < a.pool.G * a.items_k) {
        part = 1;
        head = i / a.items_k;
        at = i - head * a.items_k;
    } else {
        i -= a.pool.G * a.items_k;
        part = 2;
        head = i / a.items_v;
        at = i - head * a.items_v;
    }
    const int half = part == 2 ? 0 : a.c.rot >> 1, turning = half / VEC;
    const bool turns = at < turning;
    const int d0 = turns ? at * VEC : 2 * half + (at - turning) * VEC;
    const int dim = part == 2 ? a.pool.vdim : a.pool.dim;
    const bool live = d0 < dim;   // (past it: the padding of a query row)
    const int ch0 = (part == 0 ? 0 : part == 1 ? a.QD : a.QD + a.KD) + head * dim;

    // the projected value at place `off` of this portion (negative: from the state; before the sequence: zero)
    auto input = [&](int off, int ch) {
        Vec v;
        if (off >= 0) {
            v = *reinterpret_cast<const Vec*>(raw + (size_t)off * a.c.raw_ld + ch);
        } else if (span.z + off >= 0) {
            v = *reinterpret_cast<const Vec*>(state + (size_t)(keep + off) * a.channels + ch);
        } else {
#pragma unroll
            for (int e = 0; e < VEC; e++) v.v[e] = (RT)0.f;
        }
        return v;
    };
    auto conv = [&](int off, int ch, float* y) {
        if (!a.c.taps) {
            const Vec u = input(off, ch);
#pragma unroll
            for (int e = 0; e < VEC; e++) y[e] = (float)u.v[e];
            return;
        }
#pragma unroll
        for (int e = 0; e < VEC; e++) y[e] = 0.f;
        for (int j = 0; j <= keep; j++) {
            const Vec u = input(off - keep + j, ch);
            const float* w = a.c.taps + (size_t)j * a.channels + ch;
#pragma unroll
            for (int e = 0; e < VEC; e++) y[e] = fmaf(w[e], (float)u.v[e], y[e]);
        }
    };
    auto store = [&](int t, int d, const float* y) {
        if (part == 0) {
            Vec v;
#pragma unroll
            for (int e = 0; e < VEC; e++) v.v[e] = (RT)y[e];
            *reinterpret_cast<Vec*>(reinterpret_cast<RT*>(a.c.q_out) + ((size_t)t * a.c.H + head) * a.pool.dim_ld + d) = v;
            return;
        }
        const int row = a.kv_row[t];
        if (row < 0) return;
        if (sizeof(RT) == 4) {
            float* p = part == 1 ? (float*)a.pool.keys : (float*)a.pool.values;
#pragma unroll
            for (int e = 0; e < VEC; e++) p[((size_t)row * a.pool.G + head) * dim + d + e] = y[e];
        } else if (part == 1) {   // VEC 8: one 16-byte piece of the page (d is a multiple of VEC)
            Vec v;
#pragma unroll
            for (int e = 0; e < VEC; e++) v.v[e] = (RT)y[e];
            *reinterpret_cast<Vec*>(reinterpret_cast<RT*>(a.pool.keys) + key_off(row, head, a.pool.G, d, a.pool.dim_ld)) = v;
        } else {
#pragma unroll
            for (int e = 0; e < VEC; e++) reinterpret_cast<RT*>(a.pool.values)[value_off(row, head, a.pool.G, d + e, a.pool.vdim_ld)] = (RT)y[e];
        }
    };

    for (int k = 0; k < n_mine; k++) {
        const int off = off_mine + k, t = span.x + off;
        float y[VEC], z[VEC];
        if (!live) {
#pragma unroll
            for (int e = 0; e < VEC; e++) y[e] = 0.f;
            store(t, d0, y);
            continue;
        }
        conv(off, ch0 + d0, y);
        if (turns) {
            conv(off, ch0 + d0 + half, z);
            const float2* cs = a.c.rope + (size_t)(span.z + off) * half + d0;
#pragma unroll
            for (int e = 0; e < VEC; e++) {
                const float2 r = cs[e];
                const float u = y[e], v = z[e];
                y[e] = u * r.x - v * r.y;
                z[e] = v * r.x + u * r.y;
            }
            store(t, d0 + half, z);
        }
        store(t, d0, y);
    }
    if (off_mine == 0 && keep > 0 && live) {   // ascending rows: a row's source lies at or behind it
        for (int r = 0; r < keep; r++) {
            const int off = span.y - keep + r;
            RT* dst = state + (size_t)r * a.channels + ch0 + d0;
            const Vec v = input(off, ch0 + d0);
            *reinterpret_cast<Vec*>(dst) = v;
            if (turns) {
                const Vec w = input(off, ch0 + d0 + half);
                *reinterpret_cast<Vec*>(dst + half) = w;
            }
        }
    }
}

// The same for bf16 rows of 16-byte pieces and KEEP + 1 taps: a thread walks TOK neighbouring tokens with the taps and the
// last KEEP inputs in registers (what the tokens need is requested up front), and on to the end of those that see the state
// of a portion that starts among them.
struct alignas(16) Piece {
    __bf16 v[8];
};
template <int KEEP, int TOK>
__global__ __launch_bounds__(256) void k_conv_rope_walk(ConvKArgs a, int T) {
    const int item = blockIdx.y * 256 + threadIdx.x, t0 = blockIdx.x * TOK;
    if (item >= a.items) return;
    int part, head, at, i = item;
    if (i < a.c.H * a.items_q) {
        part = 0;
        head = i / a.items_q;
        at = i - head * a.items_q;
    } else if ((i -= a.c.H * a.items_q) < a.pool.G * a.items_k) {
        part = 1;
        head = i / a.items_k;
        at = i - head * a.items_k;
    } else {
        i -= a.pool.G * a.items_k;
        part = 2;
        head = i / a.items_v;
        at = i - head * a.items_v;
    }
    const int half = part == 2 ? 0 : a.c.rot >> 1, turning = half / 8;
    const bool turns = at < turning;
    const int d0 = turns ? at * 8 : 2 * half + (at - turning) * 8;
    const int dim = part == 2 ? a.pool.vdim : a.pool.dim;
    const bool live = d0 < dim;   // (past it: the padding of a query row)
    const int ch = (part == 0 ? 0 : part == 1 ? a.QD : a.QD + a.KD) + head * dim + (live ? d0 : 0), partner = turns ? half : 0;
    const __bf16* raw = reinterpret_cast<const __bf16*>(a.c.raw) + ch;
    int4 spans[TOK];   // (first token, count, first position, sequence)
    int rows[TOK];
    Piece in[TOK], inz[TOK];
#pragma unroll
    for (int u = 0; u < TOK; u++) {
        const int t = min(t0 + u, T - 1);
        spans[u] = a.spans[a.span_of[t]];
        rows[u] = a.kv_row[t];
        in[u] = *reinterpret_cast<const Piece*>(raw + (size_t)t * a.c.raw_ld);
        inz[u] = *reinterpret_cast<const Piece*>(raw + (size_t)t * a.c.raw_ld + partner);
    }
    float w[KEEP + 1][8], wz[KEEP + 1][8];
#pragma unroll
    for (int j = 0; j <= KEEP; j++)
#pragma unroll
        for (int e = 0; e < 8; e += 4) {
            const f4_t one = {1.f, 1.f, 1.f, 1.f};
            const f4_t u = a.c.taps ? *reinterpret_cast<const f4_t*>(a.c.taps + (size_t)j * a.channels + ch + e) : one;
            const f4_t v = a.c.taps ? *reinterpret_cast<const f4_t*>(a.c.taps + (size_t)j * a.channels + ch + partner + e) : one;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                w[j][e + r] = u[r];
                wz[j][e + r] = v[r];
            }
        }
    Piece win[KEEP + 1], winz[KEEP + 1];   // inputs of tokens t - KEEP .. t
    int have = -1;                         // the token they are complete for, but for its own input
    // values of four tokens that are a quarter of a page: stored together, a dim's four keys lie side by side
    bool quarter = false;
    if (TOK % 4 == 0 && part == 2) {
        const int off = t0 - spans[0].x;
        quarter = t0 + TOK <= T && spans[TOK - 1].x == spans[0].x && (spans[0].z + off) % 4 == 0 && (off == 0 || off >= KEEP) && rows[0] >= 0 && rows[TOK - 1] >= 0;
    }
    Piece values[TOK];
    auto token = [&](const int t, const int4 span, const int row, const Piece own, const Piece ownz, Piece& value) __attribute__((always_inline)) {
        const int off = t - span.x;
        __bf16* state = reinterpret_cast<__bf16*>(a.c.state) + (size_t)span.w * KEEP * a.channels + ch;
        if (have != t || off == 0) {
#pragma unroll
            for (int j = 0; j < KEEP; j++) {
                const int o = off - KEEP + j;
                const Piece zero = {};
                win[j] = winz[j] = zero;
                if (span.z + o >= 0) {
                    const __bf16* src = o >= 0 ? raw + (size_t)(span.x + o) * a.c.raw_ld : state + (size_t)(KEEP + o) * a.channels;
                    win[j] = *reinterpret_cast<const Piece*>(src);
                    winz[j] = *reinterpret_cast<const Piece*>(src + partner);
                }
            }
        }
        win[KEEP] = own;
        winz[KEEP] = ownz;
        float y[8], z[8];
#pragma unroll
        for (int e = 0; e < 8; e++) y[e] = z[e] = 0.f;
#pragma unroll
        for (int j = 0; j <= KEEP; j++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                y[e] = fmaf(w[j][e], (float)win[j].v[e], y[e]);
                z[e] = fmaf(wz[j][e], (float)winz[j].v[e], z[e]);
            }
        if (turns) {
            const float4* cs = reinterpret_cast<const float4*>(a.c.rope + (size_t)(span.z + off) * half + d0);   // {cos, sin} x 2
#pragma unroll
            for (int e = 0; e < 8; e += 2) {
                const float4 r = cs[e >> 1];
                const float u0 = y[e], v0 = z[e], u1 = y[e + 1], v1 = z[e + 1];
                y[e] = u0 * r.x - v0 * r.y;
                z[e] = v0 * r.x + u0 * r.y;
                y[e + 1] = u1 * r.z - v1 * r.w;
                z[e + 1] = v1 * r.z + u1 * r.w;
            }
        }
        Piece py, pz;
#pragma unroll
        for (int e = 0; e < 8; e++) {
            py.v[e] = (__bf16)(live ? y[e] : 0.f);
            pz.v[e] = (__bf16)z[e];
        }
        if (part == 0) {
            __bf16* q = reinterpret_cast<__bf16*>(a.c.q_out) + ((size_t)t * a.c.H + head) * a.pool.dim_ld + d0;
            *reinterpret_cast<Piece*>(q) = py;
            if (turns) *reinterpret_cast<Piece*>(q + half) = pz;
        } else if (row >= 0) {
            if (part == 1) {
                __bf16* k = reinterpret_cast<__bf16*>(a.pool.keys);
                *reinterpret_cast<Piece*>(k + key_off(row, head, a.pool.G, d0, a.pool.dim_ld)) = py;
                if (turns) *reinterpret_cast<Piece*>(k + key_off(row, head, a.pool.G, d0 + half, a.pool.dim_ld)) = pz;
            } else if (quarter) {
                value = py;
            } else {
                __bf16* v = reinterpret_cast<__bf16*>(a.pool.values) + value_off(row, head, a.pool.G, d0, a.pool.vdim_ld);
#pragma unroll
                for (int e = 0; e < 8; e++) v[4 * e] = py.v[e];   // (d0 is a multiple of 8: the dims stay in one tile)
            }
        }
#pragma unroll
        for (int j = 0; j < KEEP; j++) {
            win[j] = win[j + 1];
            winz[j] = winz[j + 1];
        }
        have = t + 1;
        if (KEEP > 0 && live && off == min(span.y, KEEP) - 1) {   // nobody needs the old state any more
#pragma unroll
            for (int j = 0; j < KEEP; j++) {
                Piece u = win[j], v = winz[j];
                if (span.y > KEEP) {
                    const __bf16* src = raw + (size_t)(span.x + span.y - KEEP + j) * a.c.raw_ld;
                    u = *reinterpret_cast<const Piece*>(src);
                    v = *reinterpret_cast<const Piece*>(src + partner);
                }
                *reinterpret_cast<Piece*>(state + (size_t)j * a.channels) = u;
                if (turns) *reinterpret_cast<Piece*>(state + (size_t)j * a.channels + half) = v;
            }
        }
    };
#pragma unroll
    for (int u = 0; u < TOK; u++) {
        const int t = t0 + u, off = t - spans[u].x;
        // (a token that sees the state of a portion that starts in front of these belongs to the thread of its first token)
        if (t < T && !(off > 0 && off < KEEP && spans[u].x < t0)) token(t, spans[u], rows[u], in[u], inz[u], values[u]);
    }
    if (quarter) {
#pragma unroll
        for (int u = 0; u + 3 < TOK; u += 4) {
            b4_t* v = reinterpret_cast<b4_t*>(reinterpret_cast<__bf16*>(a.pool.values) + value_off(rows[u], head, a.pool.G, d0, a.pool.vdim_ld));
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = b4_t{values[u].v[e], values[u + 1].v[e], values[u + 2].v[e], values[u + 3].v[e]};
        }
    }
    Piece unused;
    quarter = false;
    const int4 last = spans[TOK - 1];   // the portion the next tokens may belong to
    for (int t = t0 + TOK; t < last.x + min(last.y, KEEP) && last.x >= t0; t++)
        token(t, last, a.kv_row[t], *reinterpret_cast<const Piece*>(raw + (size_t)t * a.c.raw_ld), *reinterpret_cast<const Piece*>(raw + (size_t)t * a.c.raw_ld + partner), unused);
}

template <int KEEP>
static void launch_walk(const ConvKArgs& a, int T) {
    const dim3 threads(std::min(256, (a.items + 63) & ~63));
    const int y = cdiv(a.items, 256);
    if ((long)T * a.items >= 4L * 64 * 16 * rt().num_cus)   // (enough waves even so; fewer loads of the taps)
        NVLLM_LAUNCH((k_conv_rope_walk<KEEP, 4>), dim3(cdiv(T, 4), y), threads, 0, a, T);
    else if (T >= 256) NVLLM_LAUNCH((k_conv_rope_walk<KEEP, 2>), dim3(cdiv(T, 2), y), threads, 0, a, T);
    else NVLLM_LAUNCH((k_conv_rope_walk<KEEP, 1>), dim3(T, y), threads, 0, a, T);
}

void launch_conv_rope(const ConvRope& c, const KvPages& pool, const StepArrays& st) {
    if (st.T <= 0) return;
    if (!st.d_spans || !st.d_kv_row) NVLLM_FATAL("convolution over time: the batch was staged without its portions");
    if (c.rot % 2 || c.rot > pool.dim || c.n_taps < 1) NVLLM_FATAL("convolution over time: %d taps, %d of %d dimensions rotated", c.n_taps, c.rot, pool.dim);
    ConvKArgs a{};
    a.c = c;
    a.pool = pool;
    a.spans = (const int4*)st.d_spans;
    a.span_of = st.d_span_of;
    a.kv_row = st.d_kv_row;
    a.QD = c.H * pool.dim;
    a.KD = pool.G * pool.dim;
    a.channels = a.QD + a.KD + pool.G * pool.vdim;
    const int half = c.rot / 2;
    const bool wide = pool.elem_bytes == 2 && pool.dim % 8 == 0 && pool.vdim % 8 == 0 && half % 8 == 0 && c.raw_ld % 8 == 0;
    const int vec = wide ? 8 : 1;
    a.items_q = half / vec + (pool.dim_ld - c.rot) / vec;
    a.items_k = half / vec + (pool.dim - c.rot) / vec;
    a.items_v = pool.vdim / vec;
    a.items = c.H * a.items_q + pool.G * (a.items_k + a.items_v);
    const double elems = (double)st.T * a.channels * 2.0;
    ProfScope ps(PC_CONV_ROPE, elems * pool.elem_bytes + (double)a.channels * c.n_taps * 4.0, elems * c.n_taps);
    const dim3 grid(st.T, cdiv(a.items, 256));
    if (wide && c.n_taps <= 5 && (c.taps || c.n_taps == 1)) {
        switch (c.n_taps) {
            case 1: launch_walk<0>(a, st.T); break;
            case 2: launch_walk<1>(a, st.T); break;
            case 3: launch_walk<2>(a, st.T); break;
            case 4: launch_walk<3>(a, st.T); break;
            default: launch_walk<4>(a, st.T); break;
        }
        return;
    }
    if (pool.elem_bytes == 4) NVLLM_LAUNCH((k_conv_rope<float, 1>), grid, dim3(256), 0, a);
    else if (wide) NVLLM_LAUNCH((k_conv_rope<__bf16, 8>), grid, dim3(256), 0, a);
    else NVLLM_LAUNCH((k_conv_rope<__bf16, 1>), grid, dim3(256), 0, a);
}

// ------------------------------------------------------------------ attention, any size
template <bool B16>
__global__ __launch_bounds__(256) void k_window_attn_any(KvPages pool, const void* q, float scale, float cap, int size, int keep, const int* __restrict__ pos,
                                                         const int* __restrict__ seq, const int* __restrict__ tbl_off, const int* __restrict__ tables, int H,
                                                         float* out_f32, __half* out_b16, int Kb_out) {
    extern __shared__ float lds_any[];   // query [dim_ld], accumulators [vdim_ld], weights [256], reductions [8], rows [256]
    float* sq = lds_any;
    float* acc = sq + pool.dim_ld;
    float* sp = acc + pool.vdim_ld;
    float* red = sp + 256;
    int* srow = reinterpret_cast<int*>(red + 8);
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = h / (H / pool.G);
    for (int d = tid; d < pool.dim; d += 256) {
        const size_t i = ((size_t)t * H + h) * pool.dim_ld + d;
        sq[d] = B16 ? b16_f32(reinterpret_cast<const unsigned short*>(q)[i]) : reinterpret_cast<const float*>(q)[i];
    }
    for (int d = tid; d < pool.vdim_ld; d += 256) acc[d] = 0.f;
    const int p = pos[t], lo = max(0, p - size + 1), first = min(keep, lo), n_keys = first + p - lo + 1;
    const int* table = tables + tbl_off[seq[t]];
    float m = -INFINITY, l = 0.f;   // the same in every thread
    __syncthreads();
    for (int k0 = 0; k0 < n_keys; k0 += 256) {
        const int k = k0 + tid;
        float s = -INFINITY;
        if (k < n_keys) {
            const int key = k < first ? k : lo + k - first;
            const int row = table[key / pool.block_size] * pool.block_size + key % pool.block_size;
            srow[tid] = row;
            float dot = 0.f;
            for (int d = 0; d < pool.dim; d++) {
                const float kv = B16 ? b16_f32(reinterpret_cast<const unsigned short*>(pool.keys)[key_off(row, g, pool.G, d, pool.dim_ld)])
                                     : reinterpret_cast<const float*>(pool.keys)[((size_t)row * pool.G + g) * pool.dim + d];
                dot = fmaf(sq[d], kv, dot);
            }
            s = dot * scale;
            if (cap > 0.f) s = cap * tanhf(s / cap);
        }
        float mx = s;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
        if (lane == 0) red[wave] = mx;
        __syncthreads();
        const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float e = k < n_keys ? expf(s - mn) : 0.f;
        sp[tid] = e;
        float sum = e;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
        if (lane == 0) red[4 + wave] = sum;
        __syncthreads();
        const float alpha = m == -INFINITY ? 0.f : expf(m - mn);
        l = l * alpha + ((red[4] + red[5]) + (red[6] + red[7]));
        m = mn;
        const int n = min(256, n_keys - k0);
        for (int d = tid; d < pool.vdim; d += 256) {
            float o = acc[d] * alpha;
            for (int j = 0; j < n; j++) {
                const float vv = B16 ? b16_f32(reinterpret_cast<const unsigned short*>(pool.values)[value_off(srow[j], g, pool.G, d, pool.vdim_ld)])
                                     : reinterpret_cast<const float*>(pool.values)[((size_t)srow[j] * pool.G + g) * pool.vdim + d];
                o = fmaf(sp[j], vv, o);
            }
            acc[d] = o;
        }
        __syncthreads();   // weights, rows and reductions are free again
    }
    for (int d = tid; d < pool.vdim_ld; d += 256) {
        const float o = d < pool.vdim ? acc[d] / l : 0.f;
        if (B16) {
            const int k = h * pool.vdim_ld + d;
            reinterpret_cast<__bf16*>(out_b16)[((size_t)(t >> 4) * Kb_out + (k >> 5)) * TILE_HALVES + (size_t)((t & 15) + 16 * ((k >> 3) & 3)) * 8 + (k & 7)] = (__bf16)o;
        } else {
            out_f32[((size_t)t * H + h) * pool.vdim + d] = o;
        }
    }
}

// ------------------------------------------------------------------ attention, bf16 pages
struct WindowKArgs {
    const __half* keys;
    const __half* values;
    const __half* q;
    const int* tables;
    const int4* runs;      // (first token, count, last position, table offset)
    int n_runs, n_sub;     // items of CT tokens per run
    int HW, NHG;           // heads per item (prompts: 1, 2 or 4; single tokens: 16); head groups of a key/value group
    int G, rep, H;
    int kc, vt;            // dim_ld / 32, vdim_ld / 16
    int size, keep;
    float scale, cap;
    int nsplit;
    int page_shift;        // log2(pages per block)
    __half* out;
    int Kb_out;
    float* part_acc;       // [run][head][slice][16 * vt]
    float* part_ml;        // [run][head][slice][2], log2 domain
};
typedef const __attribute__((address_space(4))) int* const_int_p;   // read-only for the whole launch: scalar loads
typedef unsigned int u2_t __attribute__((ext_vector_type(2)));
constexpr float LOG2E = 1.44269504088896340736f;
constexpr float CAP_FIXED = 32.f;   // caps up to here: the shift of the weights is the cap itself
constexpr int window_waves(int VT, bool single) { return !single || VT > 8 ? 4 : 8; }
static size_t window_lds(int VT, int waves) { return (size_t)waves * (VT * 1024 + 16 * 8); }

// KC key chunks of 32 dims, VT value tiles of 16 dims held; C column groups of 16 per wave; CAP: 0 no cap, 1 cap with the
// shift known beforehand, 2 cap with a running maximum; EXACT: the sizes are KC and VT.
template <int KC, int VT, int C, bool SINGLE, int CAP, bool EXACT>
__global__ __launch_bounds__(64 * window_waves(VT, SINGLE), 2) void k_window_attn(WindowKArgs a) {
    constexpr int WAVES = window_waves(VT, SINGLE);
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_win[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int x = lane & 15, g4 = lane >> 4;
    const int kc = EXACT ? KC : a.kc, vt = EXACT ? VT : a.vt;

    // ---- the item: neighbouring items share keys and values and sit behind one L2 (workgroups are dealt to 8 XCDs)
    int idx;
    {
        const int n = gridDim.x, xcd = blockIdx.x & 7, slot = blockIdx.x >> 3, qd = n >> 3, r = n & 7;
        idx = (xcd < r ? xcd * (qd + 1) : r * (qd + 1) + (xcd - r) * qd) + slot;
    }
    int split = 0;
    if (SINGLE) {
        split = idx % a.nsplit;
        idx /= a.nsplit;
    } else {
        idx = idx * WAVES + wave;
    }
    const int hg = idx % a.NHG;
    idx /= a.NHG;
    const int sub = SINGLE ? 0 : idx % a.n_sub;
    if (!SINGLE) idx /= a.n_sub;
    const int run_id = idx % a.n_runs, grp = idx / a.n_runs;
    if (grp >= a.G) return;
    const int4 run = a.runs[run_id];
    const int CT = SINGLE ? 1 : 16 * C / a.HW;
    const int first = sub * CT;
    if (first >= run.y) return;
    const int ntok = __builtin_amdgcn_readfirstlane(min(CT, run.y - first));
    const int pos_lo = __builtin_amdgcn_readfirstlane(run.z - run.y + 1 + first), pos_hi = pos_lo + ntok - 1;
    const const_int_p table = (const_int_p)(uintptr_t)(a.tables + __builtin_amdgcn_readfirstlane(run.w));

    // this lane's column of group c: (token of the item, head of the group); position -1 where there is none
    auto column = [&](int c, int& tok, int& h) {
        const int hl = SINGLE ? x : c % a.HW;
        tok = SINGLE ? 0 : (c / a.HW) * 16 + x;
        h = hg * a.HW + hl;
        const bool valid = tok < ntok && h < a.rep;
        tok = valid ? tok : 0;
        h = valid ? grp * a.rep + h : -1;
    };
    int pos[C];
    b8_t qf[C][KC];
#pragma unroll
    for (int c = 0; c < C; c++) {
        int tok, h;
        column(c, tok, h);
        pos[c] = h >= 0 ? pos_lo + tok : -1;
        const b8_t* qr = reinterpret_cast<const b8_t*>(a.q + ((size_t)(run.x + first + tok) * a.H + max(h, 0)) * (kc * 32)) + g4;
#pragma unroll
        for (int k = 0; k < KC; k++) qf[c][k] = qr[(EXACT ? k : min(k, kc - 1)) * 4];
    }

    // ---- the pages: those of the kept first tokens, then those the window touches
    const int first_pg = max(0, pos_lo - a.size + 1) >> 4, last_pg = pos_hi >> 4;
    const int n_kept = min((a.keep + 15) >> 4, first_pg), n_pages = n_kept + last_pg - first_pg + 1;
    const int n_pairs = (n_pages + 1) >> 1;
    const int per = SINGLE ? (n_pairs + a.nsplit - 1) / a.nsplit : n_pairs;
    const int it0 = split * per + (SINGLE ? wave : 0), it1 = min(n_pairs, split * per + per);
    constexpr int STRIDE = SINGLE ? WAVES : 1;
    auto page_at = [&](int i) { return i < n_kept ? i : first_pg + i - n_kept; };   // position / 16

    // Pages in registers: of two steps (DEEP: a step's are requested before the step ahead of it is computed) or of one.
    constexpr bool DEEP = EXACT && 2 * (8 * KC + 4 * VT) + C * 4 * (KC + VT) <= 176;
    constexpr int SETS = DEEP ? 2 : 1;
    h8_t kf[SETS][2][KC];
    u2_t vf[SETS][2][VT];
    // The step that is requested next: entries of the block table (looked up a step earlier; used as late as possible, so that
    // nothing waits for the look-up) and the pages' places in their blocks.
    int entry[2], inside[2];
    auto look_up = [&](int it) {
#pragma unroll
        for (int p = 0; p < 2; p++) {
            const int pg = page_at(min(2 * it + p, n_pages - 1));
            entry[p] = table[pg >> a.page_shift];
            inside[p] = pg & ((1 << a.page_shift) - 1);
        }
    };
    auto page_id = [&](int p) { return (entry[p] << a.page_shift) + inside[p]; };
    auto load_keys = [&](int set) {
#pragma unroll
        for (int p = 0; p < 2; p++) {
            const h8_t* src = reinterpret_cast<const h8_t*>(a.keys + ((size_t)page_id(p) * a.G + grp) * (KV_PAGE * 32 * kc)) + lane;
#pragma unroll
            for (int k = 0; k < KC; k++)
                if (EXACT || k < kc) kf[set][p][k] = src[k * 64];
        }
    };
    auto load_values = [&](int set) {
#pragma unroll
        for (int p = 0; p < 2; p++) {
            const u2_t* src = reinterpret_cast<const u2_t*>(a.values + ((size_t)page_id(p) * a.G + grp) * (KV_PAGE * 16 * vt)) + lane;
#pragma unroll
            for (int v = 0; v < VT; v++)
                if (EXACT || v < vt) vf[set][p][v] = src[v * 64];
        }
    };

    float m[C], lsum[C];
    f4_t acc[VT][C];
#pragma unroll
    for (int c = 0; c < C; c++) {
        m[c] = -1e30f;   // (finite: no difference of infinities)
        lsum[c] = 0.f;
#pragma unroll
        for (int v = 0; v < VT; v++) acc[v][c] = f4_t{0.f, 0.f, 0.f, 0.f};
    }
    const float plain = a.scale * LOG2E;                                            // no cap: log2-domain scores
    const float grow = CAP ? 2.f * a.scale / a.cap * LOG2E : 0.f;                   // cap: tanh(s/cap) = 1 - 2 / (1 + 2^(grow s))
    const float top = a.cap * LOG2E;

    // set: where this step's pages are.  The next step's are requested whether or not there is one (the last pages again, then:
    // no memory traffic): where paths with and without requests meet, the compiler waits for every request in flight.
    auto step = [&](const int it, const int set) __attribute__((always_inline)) {
        if (DEEP && (!SINGLE || it + STRIDE < it1)) {   // (single tokens: few steps, so that the last one's would weigh)
            load_keys(set ^ 1);
            load_values(set ^ 1);
            look_up(it + 2 * STRIDE);
        }
        f4_t s[2][C];
#pragma unroll
        for (int p = 0; p < 2; p++)
#pragma unroll
            for (int c = 0; c < C; c++) s[p][c] = f4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KC; k++)
            if (EXACT || k < kc)
#pragma unroll
                for (int p = 0; p < 2; p++)
#pragma unroll
                    for (int c = 0; c < C; c++)
                        s[p][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(b8_t, kf[set][p][k]), qf[c][k], s[p][c], 0, 0, 0);
        if (!DEEP) load_keys(0);
        // ---- weights
        const int pg0 = page_at(2 * it), pg1 = 2 * it + 1 < n_pages ? page_at(2 * it + 1) : 1 << 26;   // (a page that is not there lies past every query)
        auto open = [&](int pg) { return pg * 16 + 15 <= pos_lo && (pg * 16 > pos_hi - a.size || pg * 16 + 15 < a.keep); };
        const bool masked = !(open(pg0) && open(pg1)) || (!SINGLE && ntok < CT);
        b8_t pw[C];
#pragma unroll
        for (int c = 0; c < C; c++) {
            float e[8];
#pragma unroll
            for (int i = 0; i < 8; i++) {
                const float z = s[i >> 2][c][i & 3];
                if (CAP == 0) e[i] = z * plain;
                else {
                    const float r = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(z * grow));
                    e[i] = CAP == 1 ? -2.f * top * r : fmaf(-2.f * top, r, top);
                }
            }
            if (masked) {
#pragma unroll
                for (int i = 0; i < 8; i++) {
                    const int key = (i < 4 ? pg0 : pg1) * 16 + 4 * g4 + (i & 3);
                    const bool seen = key <= pos[c] && (key > pos[c] - a.size || key < a.keep);
                    e[i] = seen ? e[i] : -INFINITY;
                }
            }
            if (CAP != 1) {
                float mx = e[0];
#pragma unroll
                for (int i = 1; i < 8; i++) mx = fmaxf(mx, e[i]);
                const float mn = fmaxf(m[c], rows_max(mx));
                if (__any(mn > m[c])) {
                    const float alpha = __builtin_amdgcn_exp2f(m[c] - mn);
                    lsum[c] *= alpha;
#pragma unroll
                    for (int v = 0; v < VT; v++)
                        if (EXACT || v < vt) acc[v][c] *= alpha;
                    m[c] = mn;
                }
#pragma unroll
                for (int i = 0; i < 8; i++) e[i] -= m[c];
            }
            float part = 0.f;
#pragma unroll
            for (int i = 0; i < 8; i++) {
                e[i] = __builtin_amdgcn_exp2f(e[i]);
                part += e[i];
            }
            const f4_t lo = {e[0], e[1], e[2], e[3]}, hi = {e[4], e[5], e[6], e[7]};
            pw[c] = __builtin_shufflevector(__builtin_convertvector(lo, b4_t), __builtin_convertvector(hi, b4_t), 0, 1, 2, 3, 4, 5, 6, 7);
            lsum[c] += part;
        }
        // ---- values
#pragma unroll
        for (int v = 0; v < VT; v++)
            if (EXACT || v < vt) {
                const u4_t both = {vf[set][0][v][0], vf[set][0][v][1], vf[set][1][v][0], vf[set][1][v][1]};
#pragma unroll
                for (int c = 0; c < C; c++)
                    acc[v][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(b8_t, both), pw[c], acc[v][c], 0, 0, 0);
            }
        if (!DEEP) {
            load_values(0);
            look_up(it + 2 * STRIDE);
        }
    };
    if (it0 < it1) {
        look_up(it0);
        load_keys(0);
        load_values(0);
        look_up(it0 + STRIDE);
        if constexpr (DEEP) {
#pragma clang loop unroll(disable)
            for (int it = it0; it < it1; it += 2 * STRIDE) {
                step(it, 0);
                if (it + STRIDE < it1) step(it + STRIDE, 1);
            }
        } else {
#pragma clang loop unroll(disable)
            for (int it = it0; it < it1; it += STRIDE) step(it, 0);
        }
    }
#pragma unroll
    for (int c = 0; c < C; c++) {   // the four lane rows of a column hold different keys
        lsum[c] += __shfl_xor(lsum[c], 16, 64);
        lsum[c] += __shfl_xor(lsum[c], 32, 64);
    }
    if (!SINGLE) {
#pragma unroll
        for (int c = 0; c < C; c++) {
            int tok, h;
            column(c, tok, h);
            if (h < 0) continue;
            const float inv = 1.f / lsum[c];
#pragma unroll
            for (int v = 0; v < VT; v++)
                if (EXACT || v < vt) {
                    const float y[4] = {acc[v][c][0] * inv, acc[v][c][1] * inv, acc[v][c][2] * inv, acc[v][c][3] * inv};
                    store_b16_4(a.out, a.Kb_out, run.x + first + tok, h * vt * 16 + v * 16 + 4 * g4, y);
                }
        }
        return;
    }
    // ---- single tokens: the waves' sums meet
    f4_t* s_acc = reinterpret_cast<f4_t*>(lds_win);                                  // [wave][VT][64]
    float2* s_ml = reinterpret_cast<float2*>(lds_win + (size_t)WAVES * VT * 1024);   // [wave][16]
#pragma unroll
    for (int v = 0; v < VT; v++) s_acc[(wave * VT + v) * 64 + lane] = acc[v][0];
    if (g4 == 0) s_ml[wave * 16 + x] = make_float2(CAP == 1 ? 0.f : m[0], lsum[0]);
    __syncthreads();
    float mx = -1e30f, f[WAVES], l = 0.f;
#pragma unroll
    for (int w = 0; w < WAVES; w++) mx = fmaxf(mx, s_ml[w * 16 + x].x);
#pragma unroll
    for (int w = 0; w < WAVES; w++) {
        f[w] = CAP == 1 ? 1.f : __builtin_amdgcn_exp2f(s_ml[w * 16 + x].x - mx);
        l = fmaf(f[w], s_ml[w * 16 + x].y, l);
    }
    const int hl = hg * a.HW + x, h = grp * a.rep + hl;   // (the column stays with the lane)
    if (hl >= a.rep || x >= a.HW) return;
    for (int v = wave; v < vt; v += WAVES) {
        f4_t sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < WAVES; w++) sum += f[w] * s_acc[(w * VT + v) * 64 + lane];
        if (a.nsplit == 1) {
            const float inv = 1.f / l;
            const float y[4] = {sum[0] * inv, sum[1] * inv, sum[2] * inv, sum[3] * inv};
            store_b16_4(a.out, a.Kb_out, run.x, h * vt * 16 + v * 16 + 4 * g4, y);
        } else {
            const size_t slice = ((size_t)run_id * a.H + h) * a.nsplit + split;
            *reinterpret_cast<f4_t*>(a.part_acc + slice * (16 * vt) + v * 16 + 4 * g4) = sum;
            if (v == 0 && g4 == 0) *reinterpret_cast<float2*>(a.part_ml + 2 * slice) = make_float2(mx, l);
        }
    }
}

__global__ __launch_bounds__(64) void k_window_merge(WindowKArgs a) {
    const int run_id = blockIdx.x, h = blockIdx.y, row = 16 * a.vt, t = a.runs[run_id].x;
    const size_t slice = ((size_t)run_id * a.H + h) * a.nsplit;
    float mx = -1e30f, l = 0.f;
    for (int s = 0; s < a.nsplit; s++) mx = fmaxf(mx, a.part_ml[2 * (slice + s)]);
    for (int s = 0; s < a.nsplit; s++) l += __builtin_amdgcn_exp2f(a.part_ml[2 * (slice + s)] - mx) * a.part_ml[2 * (slice + s) + 1];
    for (int d = 4 * threadIdx.x; d < row; d += 256) {
        f4_t sum = {0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < a.nsplit; s++)
            sum += __builtin_amdgcn_exp2f(a.part_ml[2 * (slice + s)] - mx) * *reinterpret_cast<const f4_t*>(a.part_acc + (slice + s) * row + d);
        const float y[4] = {sum[0] / l, sum[1] / l, sum[2] / l, sum[3] / l};
        store_b16_4(a.out, a.Kb_out, t, h * row + d, y);
    }
}

template <int KC, int VT, int C, bool SINGLE, int CAP, bool EXACT>
static void launch_win(const WindowKArgs& a, int grid) {
    constexpr int WAVES = window_waves(VT, SINGLE);
    const size_t shmem = SINGLE ? window_lds(VT, WAVES) : 0;
    static bool enabled = false;
    if (shmem > 64 * 1024 && !enabled) {
        HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_window_attn<KC, VT, C, SINGLE, CAP, EXACT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem));
        enabled = true;
    }
    NVLLM_LAUNCH((k_window_attn<KC, VT, C, SINGLE, CAP, EXACT>), dim3(grid), dim3(64 * WAVES), shmem, a);
}
template <int KC, int VT, int C, bool SINGLE, int CAP>
static void launch_win_exact(const WindowKArgs& a, int grid) {
    if (a.kc == KC && a.vt == VT) launch_win<KC, VT, C, SINGLE, CAP, true>(a, grid);
    else launch_win<KC, VT, C, SINGLE, CAP, false>(a, grid);
}
template <int KC, int VT, int C, bool SINGLE>
static void launch_win_cap(const WindowKArgs& a, int grid) {
    if (a.cap <= 0.f) launch_win_exact<KC, VT, C, SINGLE, 0>(a, grid);
    else if (a.cap <= CAP_FIXED) launch_win_exact<KC, VT, C, SINGLE, 1>(a, grid);
    else launch_win_exact<KC, VT, C, SINGLE, 2>(a, grid);
}

void launch_window_attention(const WindowAttn& w, const StepArrays& st) {
    if (st.n_runs <= 0) return;
    const KvPages& pool = w.pool;
    if (w.H % pool.G) NVLLM_FATAL("%d query heads do not divide over %d key/value heads", w.H, pool.G);
    if (w.size < 1 || w.keep_first < 0) NVLLM_FATAL("a window of %d tokens with %d kept", w.size, w.keep_first);
    const int kc = pool.dim_ld / 32, vt = pool.vdim_ld / 16, rep = w.H / pool.G;
    const int ppb = pool.block_size / KV_PAGE;
    const int Kb_out = w.H * pool.vdim_ld / 32;
    if (pool.elem_bytes == 4 || kc > 8 || vt > 16 || (ppb & (ppb - 1))) {
        const size_t lds = ((size_t)pool.dim_ld + pool.vdim_ld + 256 + 8 + 256) * 4;
        if (lds > 64 * 1024) NVLLM_FATAL("attention heads of %d and %d values are too wide", pool.dim, pool.vdim);
        ProfScope ps(PC_WINDOW_ATTN, 0, 0);
        const dim3 grid(st.T, w.H);
        if (pool.elem_bytes == 4)
            NVLLM_LAUNCH((k_window_attn_any<false>), grid, dim3(256), lds, pool, w.q, w.scale, w.cap, w.size, w.keep_first, st.d_pos, st.d_seq, st.d_tbl_off, st.d_tables, w.H,
                         w.out_f32, w.out_b16, Kb_out);
        else
            NVLLM_LAUNCH((k_window_attn_any<true>), grid, dim3(256), lds, pool, w.q, w.scale, w.cap, w.size, w.keep_first, st.d_pos, st.d_seq, st.d_tbl_off, st.d_tables, w.H,
                         w.out_f32, w.out_b16, Kb_out);
        return;
    }
    WindowKArgs a{};
    a.keys = (const __half*)pool.keys;
    a.values = (const __half*)pool.values;
    a.q = (const __half*)w.q;
    a.tables = st.d_tables;
    a.G = pool.G; a.rep = rep; a.H = w.H; a.kc = kc; a.vt = vt; a.size = w.size; a.keep = w.keep_first; a.scale = w.scale; a.cap = w.cap;
    a.page_shift = __builtin_ctz(ppb);
    a.out = w.out_b16;
    a.Kb_out = Kb_out;
    a.nsplit = 1;
    const int cls = kc <= 2 && vt <= 4 ? 0 : kc <= 4 && vt <= 8 ? 1 : 2;
    const long seen_cap = (long)w.size + w.keep_first;   // keys a token sees at most
    const double kv_bytes = (double)pool.G * (pool.dim_ld + pool.vdim_ld) * 2.0, io_bytes = (double)w.H * (pool.dim_ld + pool.vdim_ld) * 2.0;
    const double pair_flops = 2.0 * w.H * (pool.dim_ld + pool.vdim_ld);
    if (st.n_multi > 0) {
        a.runs = (const int4*)st.d_runs;
        a.n_runs = st.n_multi;
        // wide items share more of a page's load, narrow ones are more waves: the widest that still gives every SIMD one
        int C = cls == 0 ? 4 : cls == 1 ? 2 : 1, waves = 0;
        for (;; C /= 2) {
            a.HW = rep >= C ? C : rep >= 2 && C >= 2 ? 2 : 1;
            a.NHG = cdiv(rep, a.HW);
            a.n_sub = cdiv(std::min(st.max_run, WINDOW_RUN), 16 * C / a.HW);
            waves = a.G * a.n_runs * a.n_sub * a.NHG;
            if (C == 1 || waves >= 4 * rt().num_cus) break;
        }
        const int grid = cdiv(waves, 4);
        const double rows = (double)st.multi_rows(seen_cap), pairs = (double)st.multi_pairs(seen_cap);
        ProfScope ps(PC_WINDOW_ATTN, rows * kv_bytes + (double)(st.T - (st.n_runs - st.n_multi)) * io_bytes, pairs * pair_flops);
        if (cls == 0 && C == 4) launch_win_cap<2, 4, 4, false>(a, grid);
        else if (cls == 0 && C == 2) launch_win_cap<2, 4, 2, false>(a, grid);
        else if (cls == 0) launch_win_cap<2, 4, 1, false>(a, grid);
        else if (cls == 1 && C == 2) launch_win_cap<4, 8, 2, false>(a, grid);
        else if (cls == 1) launch_win_cap<4, 8, 1, false>(a, grid);
        else launch_win_cap<8, 16, 1, false>(a, grid);
    }
    const int n_single = st.n_runs - st.n_multi;
    if (n_single > 0) {
        a.runs = (const int4*)st.d_runs + st.n_multi;
        a.n_runs = n_single;
        a.n_sub = 1;
        a.HW = 16;
        a.NHG = cdiv(rep, 16);
        const int items = n_single * a.G * a.NHG, waves = window_waves(cls == 0 ? 4 : cls == 1 ? 8 : 16, true);
        const long longest = std::min<long>(st.max_pos + 1, seen_cap + 32);
        // slices until every CU has a workgroup, each wave of a slice with at least one pair of pages
        a.nsplit = (int)std::max<long>(1, std::min<long>(rt().num_cus / items, longest / 32 / waves));
        if (a.nsplit > 1) {
            const size_t slices = (size_t)n_single * w.H * a.nsplit;
            a.part_acc = (float*)ws_get(WS_ATT_PART, slices * (16 * vt + 2) * sizeof(float));
            a.part_ml = a.part_acc + slices * 16 * vt;
        }
        {
            const double rows = (double)st.single_rows(seen_cap);
            ProfScope ps(PC_WINDOW_ATTN_TOK, rows * kv_bytes + (double)n_single * io_bytes, rows * pair_flops);
            const int grid = items * a.nsplit;
            if (cls == 0) launch_win_cap<2, 4, 1, true>(a, grid);
            else if (cls == 1) launch_win_cap<4, 8, 1, true>(a, grid);
            else launch_win_cap<8, 16, 1, true>(a, grid);
        }
        if (a.nsplit > 1) {
            ProfScope ps(PC_ATTN_COMBINE, (double)n_single * w.H * (a.nsplit + 0.5) * vt * 64.0, 0);
            NVLLM_LAUNCH(k_window_merge, dim3(n_single, w.H), dim3(64), 0, a);
        }
    }
}

}  // namespace nvllm
