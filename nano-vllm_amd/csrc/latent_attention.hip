// latent_attention.hip -- attention over cached latents (latent_attention.h).
//
// k_latent_attn (bf16 pages).  A work item is up to CT consecutive tokens of one sequence x up to 16, 32 or 64
// (token, head) columns x a slice of the pages; all heads of a token share every cached row, so a row is read once per
// item.  The workgroup walks the item's positions in blocks of 64 (four pages); wave = page + 4 * column part:
//   copy    the waves bring the block global -> LDS with direct-to-LDS loads (pages are stored in operand order, so the
//           image is lane-linear), one block ahead of the multiplication, two buffers;
//   scores  S^T[key, col] = K Q^T over the whole row of the wave's page, for the columns of its part;
//   softmax block maxima meet in LDS; every wave turns its 16 keys into weights, bf16, in the operand order of the
//           next product (a score tile's registers ARE the k order that product uses, no shuffle);
//   values  O^T[d, col] += V^T P: the latents again, as the transposed operand, through the LDS transpose read; the
//           waves of a part split the latent's dims, and `col` stays on the lane, so rescaling needs no exchange.
// Two waves per SIMD (32 and 64 columns) alternate between LDS reads and multiplies.
// Scores, maxima and sums are fp32; queries, latents and weights enter the matrix cores as bf16.
// The sink joins the denominator once, after the last slice (here, or in k_latent_combine when pages are sliced
// across workgroups).
//
// k_latent_attn_any (fp32 rows, and bf16 rows wider than the kernel above has registers for): one workgroup per
// (token, head), fp32 arithmetic on the vector units.
#include "latent_attention.h"

#include "attn_tile.h"
#include "gemm_common.h"
#include "latent_kv.h"

namespace nvllm {

LatentPool latent_pool(void* base, int elem_bytes, int block_size, int rank, int rot) {
    LatentPool p{base, elem_bytes, block_size, rank, rot, rank, rot};
    if (elem_bytes == 2) {
        if (block_size % LATENT_PAGE) NVLLM_FATAL("bf16 latent pages hold 16 positions: block size %d is not a multiple of 16", block_size);
        p.rank_ld = (rank + 31) & ~31;
        p.rot_ld = (rot + 31) & ~31;
    }
    return p;
}

__device__ __forceinline__ float bf16_to_f32(unsigned short v) { return __builtin_bit_cast(float, (unsigned)v << 16); }

// ------------------------------------------------------------------ cache write
template <bool B16>
__global__ __launch_bounds__(256) void k_latent_kv(LatentKvRider a) {
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (B16) {
        latent_kv_ride(a, t, lane);
        return;
    }
    if (t >= a.T || a.kv_row[t] < 0) return;
    float* dst = reinterpret_cast<float*>(a.base) + (size_t)a.kv_row[t] * (a.rank_ld + a.rot_ld);
    latent_kv_token(a, t, lane, [&](int d, float v) { dst[d] = v; });
}

LatentKvRider latent_kv_rider(const LatentPool& pool, const float* raw, int raw_ld, int rot_at, const float* gain, float eps, const float2* rope,
                              const StepArrays& st) {
    LatentKvRider r;
    r.base = pool.base; r.raw = raw; r.gain = gain; r.rope = rope; r.pos = st.d_pos; r.kv_row = st.d_kv_row; r.eps = eps;
    r.raw_ld = raw_ld; r.rot_at = rot_at; r.T = st.T; r.rank = pool.rank; r.rot = pool.rot; r.rank_ld = pool.rank_ld; r.rot_ld = pool.rot_ld;
    return r;
}

void launch_latent_kv(const LatentPool& pool, const float* raw, int raw_ld, int rot_at, const float* gain, float eps, const float2* rope,
                      const StepArrays& st) {
    if (st.T <= 0) return;
    ProfScope ps(PC_LATENT_KV, (double)st.T * ((double)raw_ld * 4.0 + (double)pool.row() * pool.elem_bytes), 0);
    const LatentKvRider r = latent_kv_rider(pool, raw, raw_ld, rot_at, gain, eps, rope, st);
    if (pool.elem_bytes == 2) NVLLM_LAUNCH((k_latent_kv<true>), dim3(cdiv(st.T, 4)), dim3(256), 0, r);
    else NVLLM_LAUNCH((k_latent_kv<false>), dim3(cdiv(st.T, 4)), dim3(256), 0, r);
}

// ------------------------------------------------------------------ attention, any size
template <bool B16>
__device__ __forceinline__ float latent_elem(const void* base, long r, int d, int row) {
    if (B16) return bf16_to_f32(reinterpret_cast<const unsigned short*>(base)[latent_off(r, d, row)]);
    return reinterpret_cast<const float*>(base)[(size_t)r * row + d];
}

template <bool B16>
__global__ __launch_bounds__(256) void k_latent_attn_any(const void* base, const void* q, const float* __restrict__ sink, float scale,
                                                         const int* __restrict__ pos, const int* __restrict__ seq,
                                                         const int* __restrict__ tbl_off, const int* __restrict__ tables, int block_size, int H,
                                                         int rank, int rank_ld, int row, float* out_f32, __half* out_b16, int Kb_out) {
    extern __shared__ float lds_any[];   // q row [row], accumulators [rank_ld], weights [256], reductions [8]
    float* sq = lds_any;
    float* acc = sq + row;
    float* sp = acc + rank_ld;
    float* red = sp + 256;
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    for (int d = tid; d < row; d += 256) {
        const size_t i = ((size_t)t * H + h) * row + d;
        sq[d] = B16 ? bf16_to_f32(reinterpret_cast<const unsigned short*>(q)[i]) : reinterpret_cast<const float*>(q)[i];
    }
    for (int d = tid; d < rank_ld; d += 256) acc[d] = 0.f;
    const int p = pos[t];
    const int* table = tables + tbl_off[seq[t]];
    float m = -INFINITY, l = 0.f;   // the same in every thread
    __syncthreads();
    for (int k0 = 0; k0 <= p; k0 += 256) {
        const int key = k0 + tid;
        float s = -INFINITY;
        if (key <= p) {
            const long r = (long)table[key / block_size] * block_size + key % block_size;
            float dot = 0.f;
            for (int d = 0; d < row; d++) dot = fmaf(sq[d], latent_elem<B16>(base, r, d, row), dot);
            s = dot * scale;
        }
        float mx = s;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
        if (lane == 0) red[wave] = mx;
        __syncthreads();
        const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float e = key <= p ? expf(s - mn) : 0.f;
        sp[tid] = e;
        float sum = e;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
        if (lane == 0) red[4 + wave] = sum;
        __syncthreads();
        const float alpha = m == -INFINITY ? 0.f : expf(m - mn);
        l = l * alpha + ((red[4] + red[5]) + (red[6] + red[7]));
        m = mn;
        const int n = min(256, p - k0 + 1);
        for (int d = tid; d < rank; d += 256) {
            float a = acc[d] * alpha;
            for (int k = 0; k < n; k++) {
                const int kk = k0 + k;
                const long r = (long)table[kk / block_size] * block_size + kk % block_size;
                a = fmaf(sp[k], latent_elem<B16>(base, r, d, row), a);
            }
            acc[d] = a;
        }
        __syncthreads();   // weights and reductions are free again
    }
    const float top = fmaxf(m, sink[h]);
    const float f = expf(m - top), den = l * f + expf(sink[h] - top);
    for (int d = tid; d < rank_ld; d += 256) {
        const float o = d < rank ? acc[d] * f / den : 0.f;
        if (B16) {
            const int k = h * rank_ld + d;
            const __bf16 b = (__bf16)o;
            reinterpret_cast<__bf16*>(out_b16)[((size_t)(t >> 4) * Kb_out + (k >> 5)) * TILE_HALVES + (size_t)((t & 15) + 16 * ((k >> 3) & 3)) * 8 + (k & 7)] = b;
        } else {
            out_f32[((size_t)t * H + h) * rank + d] = o;
        }
    }
}

// ------------------------------------------------------------------ attention, bf16 pages
typedef short s4_t __attribute__((ext_vector_type(4)));
typedef short s8_t __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) s4_t lds_s4;

struct LatentKArgs {
    const __half* base;
    const __half* q;
    const float* sink;
    float scale;
    const int* tables;
    const int4* runs;     // (first token, count, last position, table offset)
    int n_sub;            // items of CT tokens per run
    int run_ld;           // tokens of the longest run: partial results are indexed [run][token of the run]
    int CT, HG, NG;       // tokens and heads per item; head groups
    int H, nsplit;
    int chunks;           // row / 32
    int n_tiles;          // rank_ld / 16
    int rank_ld;
    int page_shift;       // log2(pages per block)
    __half* out;
    int Kb_out;
    float* part_acc;      // [run][token of the run][head][slice][rank_ld]
    float* part_ml;       // [run][token of the run][head][slice][2], log2 domain
};

constexpr int LATENT_BLOCK_PAGES = 4;
static size_t latent_attn_lds(int chunks, int C) { return (size_t)2 * LATENT_BLOCK_PAGES * chunks * 1024 + (size_t)C * 2048 + (size_t)C * 2 * 4 * 16 * 4; }

// LDS stores of this wave are done, then everybody meets (copies to LDS in flight stay in flight)
__device__ __forceinline__ void latent_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}

typedef const __attribute__((address_space(4))) int* const_int_p;   // read-only for the whole launch: scalar loads

// RC: row chunks of 32 held as query fragments; NT: 16-dim value tiles per wave; C: column groups of 16 per wave; WC: waves
// side by side over the columns (4 * WC waves: wave = page of the block + 4 * column part).
// EXACT: the row has exactly RC chunks and 4 * NT value tiles.
template <int RC, int NT, int C, int WC, bool EXACT>
__global__ __launch_bounds__(256 * WC, WC) void k_latent_attn(LatentKArgs a) {
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_latent[];
    const int nc = EXACT ? RC : a.chunks;
    const int n_tiles = EXACT ? 4 * NT : a.n_tiles;
    __half* pages = reinterpret_cast<__half*>(lds_latent);                          // [2][4][nc][512]
    __half* s_p = pages + (size_t)2 * LATENT_BLOCK_PAGES * nc * TILE_HALVES;        // [C * WC][2][64][8]
    float* s_max = reinterpret_cast<float*>(s_p + C * WC * 2 * 64 * 8);             // [C * WC][4][16]
    float* s_sum = s_max + C * WC * 4 * 16;                                         // [C * WC][4][16]
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int x = lane & 15, g = lane >> 4;
    const int page = wave & 3, part = wave >> 2;   // this wave's page of a block, its part of the columns

    unsigned idx = blockIdx.x;
    const int split = (int)(idx % (unsigned)a.nsplit);
    idx /= (unsigned)a.nsplit;
    const int hg = (int)(idx % (unsigned)a.NG);
    idx /= (unsigned)a.NG;
    const int sub = (int)(idx % (unsigned)a.n_sub);
    const int run_id = (int)(idx / (unsigned)a.n_sub);
    const int4 run = a.runs[run_id];
    const int first = sub * a.CT;
    if (first >= run.y) return;
    const int ntok = min(a.CT, run.y - first), t0 = run.x + first;
    const int plast = run.z - (run.y - first - ntok);
    const int h0 = hg * a.HG;
    const const_int_p table = (const_int_p)(uintptr_t)(a.tables + __builtin_amdgcn_readfirstlane(run.w));
    // this slice's pages [p0, p1), in blocks of four
    const int npages = __builtin_amdgcn_readfirstlane((plast >> 4) + 1);
    const int per = (npages + a.nsplit - 1) / a.nsplit;
    const int p0 = split * per, p1 = min(npages, p0 + per);
    const int nblocks = p0 < p1 ? (p1 - p0 + LATENT_BLOCK_PAGES - 1) / LATENT_BLOCK_PAGES : 0;
    const int row = nc * 32;

    // this lane's columns: (token of the item, head); -1 where the item has none.  (Formed again where needed: the page loop
    // keeps only the last position each column sees.)
    auto column_of = [&](int j, int& tok, int& h) {
        // (tokens fastest: the 16 columns of a group are neighbouring rows of the output tiles)
        const int hl = j / a.CT;
        tok = j - hl * a.CT;
        h = h0 + hl;
        const bool valid = tok < ntok && hl < a.HG && h < a.H;
        tok = valid ? tok : 0;
        h = valid ? h : -1;
    };
    auto column = [&](int c, int& tok, int& h) { column_of(16 * (part * C + c) + (int)(threadIdx.x & 15), tok, h); };
    int plim[C];
#pragma unroll
    for (int c = 0; c < C; c++) {
        int tok, h;
        column(c, tok, h);
        plim[c] = h >= 0 ? min(plast - (ntok - 1 - tok), p1 * LATENT_PAGE - 1) : -1;
    }

    // the page id of a block's page `page`; past the slice's end its keys are masked, and the copy is the slice's last page
    // again, or nothing once the buffer holds an earlier block's (finite) rows
    auto page_of = [&](int b) {
        const int pg = min(p0 + b * LATENT_BLOCK_PAGES + page, npages - 1);
        return (table[pg >> a.page_shift] << a.page_shift) + (pg & ((1 << a.page_shift) - 1));
    };
    const unsigned lds0 = (unsigned)(size_t)(lds_void*)pages + (unsigned)(page * nc + part) * 1024u;
    auto issue = [&](int page_id, int b) {   // tiles part, part + WC, ... of the page
        if (b >= 2 && p0 + b * LATENT_BLOCK_PAGES + page >= p1) return;
        const int buf = b & 1;
        const __half* src = a.base + (size_t)page_id * (LATENT_PAGE * row) + (size_t)part * TILE_HALVES + lane * 8;
        const unsigned dst = lds0 + (unsigned)(buf * LATENT_BLOCK_PAGES * nc) * 1024u;
#pragma unroll
        for (int c = 0; c < RC; c += WC)
            if (EXACT ? c + WC <= RC || c + part < RC : c + part < nc)
                copy_tile_to_lds(src + (size_t)c * TILE_HALVES, __builtin_amdgcn_readfirstlane(dst + (unsigned)c * 1024u));
    };

    float m[C], lsum[C];
    f4_t acc[NT][C];
#pragma unroll
    for (int c = 0; c < C; c++) {
        m[c] = -INFINITY;
        lsum[c] = 0.f;
#pragma unroll
        for (int n = 0; n < NT; n++) acc[n][c] = f4_t{0.f, 0.f, 0.f, 0.f};
    }
    // Queries as the B operand: column x, dims 32k + 8g .. +7.  Every fragment is one direct-to-LDS copy whose lanes gather the
    // 16 columns' pieces, made once for the waves that share it, into the second page buffer (free until block 1 is
    // requested); from there it goes to registers.  (Columns nobody owns read a real row; their scores are masked.)
    const unsigned lds_q = (unsigned)(size_t)(lds_void*)pages + (unsigned)(LATENT_BLOCK_PAGES * nc) * 1024u;
    for (int f = wave; f < C * WC * nc; f += 4 * WC) {
        const int group = f / nc, k = f - group * nc;
        int tok, h;
        column_of(16 * group + x, tok, h);
        copy_tile_to_lds(a.q + ((size_t)(t0 + tok) * a.H + max(h, 0)) * row + 32 * k + 8 * g, __builtin_amdgcn_readfirstlane(lds_q + (unsigned)f * 1024u));
    }
    int next_page = page_of(1);
    if (nblocks > 0) issue(page_of(0), 0);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    latent_barrier();
    b8_t qf[C][RC];
#pragma unroll
    for (int c = 0; c < C; c++) {
        const b8_t* qs = reinterpret_cast<const b8_t*>(pages + (size_t)(LATENT_BLOCK_PAGES + part * C + c) * nc * TILE_HALVES) + lane;
#pragma unroll
        for (int k = 0; k < RC; k++) qf[c][k] = qs[(EXACT ? k : min(k, nc - 1)) * 64];
    }
    // (the fragments are in registers before the loop: inside it the compiler has no load of its own to wait for)
#pragma unroll
    for (int c = 0; c < C; c++)
#pragma unroll
        for (int k = 0; k < RC; k++) asm volatile("" : "+v"(qf[c][k]));
    const float sl2 = a.scale * 1.44269504088896340736f;   // scores in the log2 domain
    // transpose read: 16 lanes bring 4 keys x 16 dims, lane i gets dim i of the 4 keys
    const int tr_key = 4 * g + (x >> 2), tr_sub = (x & 3) >> 1, tr_off = 4 * (x & 1);

    // (no peeled iterations: their copies of the loop body would hold registers this one needs)
#pragma clang loop unroll(disable)
    for (int b = 0; b < nblocks; b++) {
        const int buf = b & 1;
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // this wave's tiles of block b are in LDS
        latent_barrier();                                   // ... and everybody's; block b - 1 has been consumed
        if (b + 1 < nblocks) {
            issue(next_page, b + 1);
            next_page = page_of(b + 2);
        }
        const __half* blk = pages + (size_t)buf * LATENT_BLOCK_PAGES * nc * TILE_HALVES;
        // ---- scores of this wave's page; key fragments a few chunks ahead of the multiplies
        constexpr int CH = C == 1 ? 2 : 1;   // independent accumulator chains per column group
        f4_t s[C], s2[CH][C];
#pragma unroll
        for (int c = 0; c < C; c++)
#pragma unroll
            for (int h = 0; h < CH; h++) s2[h][c] = f4_t{0.f, 0.f, 0.f, 0.f};
        const b8_t* kp = reinterpret_cast<const b8_t*>(blk + (size_t)page * nc * TILE_HALVES) + lane;
        constexpr int KA = C == 2 ? 3 : RC < 6 ? RC : 6;
        b8_t kf[KA];
#pragma unroll
        for (int k = 0; k < KA; k++) kf[k] = kp[(EXACT ? k : min(k, nc - 1)) * 64];
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int k = 0; k < RC; k++) {
            if (EXACT || k < nc) {
#pragma unroll
                for (int c = 0; c < C; c++) s2[k % CH][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[k % KA], qf[c][k], s2[k % CH][c], 0, 0, 0);
                if (k + KA < RC && (EXACT || k + KA < nc)) kf[k % KA] = kp[(k + KA) * 64];
            }
            __builtin_amdgcn_sched_barrier(0);
        }
#pragma unroll
        for (int c = 0; c < C; c++) s[c] = CH == 2 ? s2[0][c] + s2[CH - 1][c] : s2[0][c];
        const int kfirst = (p0 + b * LATENT_BLOCK_PAGES + page) * LATENT_PAGE + 4 * g;
#pragma unroll
        for (int c = 0; c < C; c++) {
            float mx = -INFINITY;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                s[c][r] = kfirst + r <= plim[c] ? s[c][r] * sl2 : -INFINITY;
                mx = fmaxf(mx, s[c][r]);
            }
            mx = rows_max(mx);
            if (g == 0) s_max[((part * C + c) * 4 + page) * 16 + x] = mx;
        }
        latent_barrier();
        // ---- weights
        float bm[C][4];
#pragma unroll
        for (int c = 0; c < C; c++)
#pragma unroll
            for (int w = 0; w < 4; w++) bm[c][w] = s_max[((part * C + c) * 4 + w) * 16 + x];
        float alpha[C];
        bool rises = false;
#pragma unroll
        for (int c = 0; c < C; c++) {
            const float mn = fmaxf(m[c], fmaxf(fmaxf(bm[c][0], bm[c][1]), fmaxf(bm[c][2], bm[c][3])));
            alpha[c] = mn == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m[c] - mn);
            rises |= mn > m[c];
            m[c] = mn;
            const float msafe = fmaxf(mn, -1.0e30f);   // nothing visible yet: exp2(-inf - finite) = 0, no NaN
            lsum[c] *= alpha[c];
            float p[4];
#pragma unroll
            for (int r = 0; r < 4; r++) {
                p[r] = __builtin_amdgcn_exp2f(s[c][r] - msafe);
                lsum[c] += p[r];
            }
            *reinterpret_cast<b4_t*>(s_p + ((size_t)((part * C + c) * 2 + (page >> 1)) * 64 + lane) * 8 + (page & 1) * 4) = to_b4(p);
        }
        if (__any(rises)) {
#pragma unroll
            for (int n = 0; n < NT; n++)
#pragma unroll
                for (int c = 0; c < C; c++)
#pragma unroll
                    for (int r = 0; r < 4; r++) acc[n][c][r] *= alpha[c];
        }
        latent_barrier();
        // ---- values: keys of pages (0, 1), then (2, 3)
        b8_t pf[C];
        auto load_weights = [&](int h) {
#pragma unroll
            for (int c = 0; c < C; c++) pf[c] = *reinterpret_cast<const b8_t*>(s_p + ((size_t)((part * C + c) * 2 + h) * 64 + lane) * 8);
        };
        load_weights(0);
        auto value_frag = [&](int i) {   // fragment i of 2 * NT: half i / NT of the block, value tile page + 4 * (i % NT)
            const int h = i / NT, n = EXACT ? page + 4 * (i % NT) : min(page + 4 * (i % NT), n_tiles - 1);
            const __half* v = blk + (size_t)(2 * h) * nc * TILE_HALVES + (n >> 1) * TILE_HALVES + (tr_key + 16 * (2 * (n & 1) + tr_sub)) * 8 + tr_off;
            const s4_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)v);
            const s4_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)(v + (size_t)nc * TILE_HALVES));
            const s8_t both = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
            return __builtin_bit_cast(b8_t, both);
        };
        constexpr int VA = C == 2 || NT == 1 ? 2 : 4;
        b8_t vf[VA];
#pragma unroll
        for (int i = 0; i < VA; i++) vf[i] = value_frag(i);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int i = 0; i < 2 * NT; i++) {
            // (a value tile past the end multiplies the last one again; its sums are never stored)
#pragma unroll
            for (int c = 0; c < C; c++) acc[i % NT][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[i % VA], pf[c], acc[i % NT][c], 0, 0, 0);
            if (i == NT - 1) load_weights(1);
            if (i + VA < 2 * NT) vf[i % VA] = value_frag(i + VA);
            __builtin_amdgcn_sched_barrier(0);
        }
    }
    // ---- the waves' partial sums meet; the sink; the result
#pragma unroll
    for (int c = 0; c < C; c++) {
        lsum[c] += __shfl_xor(lsum[c], 16, 64);
        lsum[c] += __shfl_xor(lsum[c], 32, 64);
        if (g == 0) s_sum[((part * C + c) * 4 + page) * 16 + x] = lsum[c];
    }
    latent_barrier();
#pragma unroll
    for (int c = 0; c < C; c++) {
        const float* bs = s_sum + (part * C + c) * 64 + x;
        const float L = (bs[0] + bs[16]) + (bs[32] + bs[48]);
        int tok, h;
        column(c, tok, h);
        if (h < 0) continue;
        float f = 1.f;
        const size_t th = ((size_t)run_id * a.run_ld + first + tok) * a.H + h;   // place among the partial results
        if (a.nsplit == 1) {
            const float sk = a.sink[h] * 1.44269504088896340736f, top = fmaxf(m[c], sk);
            const float w = __builtin_amdgcn_exp2f(m[c] - top);
            f = w / fmaf(L, w, __builtin_amdgcn_exp2f(sk - top));
        } else if (page == 0 && g == 0) {
            a.part_ml[(th * a.nsplit + split) * 2] = m[c];
            a.part_ml[(th * a.nsplit + split) * 2 + 1] = L;
        }
#pragma unroll
        for (int i = 0; i < NT; i++) {
            const int n = page + 4 * i;
            if (!(EXACT || n < n_tiles)) continue;
            const int d = 16 * n + 4 * g;
            if (a.nsplit == 1) {
                const float o[4] = {acc[i][c][0] * f, acc[i][c][1] * f, acc[i][c][2] * f, acc[i][c][3] * f};
                store_b16_4(a.out, a.Kb_out, t0 + tok, h * a.rank_ld + d, o);
            } else {
                *reinterpret_cast<f4_t*>(a.part_acc + (th * a.nsplit + split) * a.rank_ld + d) = acc[i][c];
            }
        }
    }
}

// slices of one (token, head) -> the attended latent, the sink in the denominator
__global__ __launch_bounds__(128) void k_latent_combine(const float* __restrict__ part_acc, const float* __restrict__ part_ml,
                                                        const float* __restrict__ sink, const int4* __restrict__ runs, int run_ld, int H, int nsplit,
                                                        int rank_ld, __half* out, int Kb_out) {
    const size_t th = blockIdx.x;
    const int h = blockIdx.x % H, slot = blockIdx.x / H;
    const int4 run = runs[slot / run_ld];
    if (slot % run_ld >= run.y) return;
    const int t = run.x + slot % run_ld;
    const float* ml = part_ml + th * nsplit * 2;
    const float sk = sink[h] * 1.44269504088896340736f;
    float top = sk;
    for (int s = 0; s < nsplit; s++) top = fmaxf(top, ml[2 * s]);
    float den = __builtin_amdgcn_exp2f(sk - top);
    for (int s = 0; s < nsplit; s++) den = fmaf(ml[2 * s + 1], __builtin_amdgcn_exp2f(ml[2 * s] - top), den);
    const float inv = 1.0f / den;
    for (int d = 4 * (int)threadIdx.x; d < rank_ld; d += 512) {
        f4_t o = {0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < nsplit; s++) {
            const float f = __builtin_amdgcn_exp2f(ml[2 * s] - top) * inv;   // a slice without pages: exp2(-inf) = 0, its sums are zeros
            const f4_t v = *reinterpret_cast<const f4_t*>(part_acc + (th * nsplit + s) * rank_ld + d);
#pragma unroll
            for (int r = 0; r < 4; r++) o[r] = fmaf(v[r], f, o[r]);
        }
        const float z[4] = {o[0], o[1], o[2], o[3]};
        store_b16_4(out, Kb_out, t, h * rank_ld + d, z);
    }
}

template <int RC, int NT, int C, int WC, bool EXACT_ONLY = false>
static void launch_latent_c(const LatentKArgs& k, long units) {
    const size_t lds = latent_attn_lds(k.chunks, C * WC);
    const bool exact = k.chunks == RC && k.n_tiles == 4 * NT;
    static bool ready = false;
    if (!ready) {
        const int most = (int)latent_attn_lds(RC, C * WC);
        if (most > 64 * 1024) {
            HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_latent_attn<RC, NT, C, WC, true>), hipFuncAttributeMaxDynamicSharedMemorySize, most));
            if constexpr (!EXACT_ONLY)
                HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_latent_attn<RC, NT, C, WC, false>), hipFuncAttributeMaxDynamicSharedMemorySize, most));
        }
        ready = true;
    }
    if (exact) NVLLM_LAUNCH((k_latent_attn<RC, NT, C, WC, true>), dim3((unsigned)units), dim3(256 * WC), lds, k);
    else if constexpr (!EXACT_ONLY) NVLLM_LAUNCH((k_latent_attn<RC, NT, C, WC, false>), dim3((unsigned)units), dim3(256 * WC), lds, k);
}
template <int RC, int NT>
static void launch_latent_rc(const LatentKArgs& k, long units, int columns) {
    if (columns == 16) launch_latent_c<RC, NT, 1, 1>(k, units);
    else if (columns == 32) launch_latent_c<RC, NT, 1, 2>(k, units);
    else launch_latent_c<RC, NT, 2, 2, (RC > 10)>(k, units);
}

void launch_latent_attention(const LatentAttn& a, const StepArrays& st) {
    if (st.T <= 0) return;
    const LatentPool& P = a.pool;
    const int row = P.row(), chunks = row / 32, vt = cdiv(P.rank_ld, 64);   // value tiles per wave
    // algorithmic work: every sequence's rows read once; per (token, key, head) the two products
    auto bytes_of = [&](double rows, double tokens) { return rows * row * P.elem_bytes + tokens * a.H * (row + P.rank_ld) * P.elem_bytes; };
    const double bytes = bytes_of((double)st.kv_rows, st.T);
    const double flops = 2.0 * (double)st.qk_pairs * a.H * (row + P.rank_ld);
    const bool tiled = P.elem_bytes == 2 && ((chunks <= 4 && vt <= 1) || (chunks <= 6 && vt <= 2) || (chunks <= 10 && vt <= 4) || (chunks <= 18 && vt <= 8));
    int pages_per_block = P.block_size / LATENT_PAGE, page_shift = 0;
    while ((1 << page_shift) < pages_per_block) page_shift++;
    if (!tiled || (1 << page_shift) != pages_per_block) {
        const size_t lds = ((size_t)row + P.rank_ld + 256 + 8) * sizeof(float);
        if (lds > 64 * 1024) NVLLM_FATAL("latent attention: a cached row of %d values is not supported", row);
        ProfScope ps(PC_LATENT_ATTN, bytes, flops);
        const dim3 grid(st.T, a.H);
        if (P.elem_bytes == 2)
            NVLLM_LAUNCH((k_latent_attn_any<true>), grid, dim3(256), lds, P.base, a.q, a.sink, a.scale, st.d_pos, st.d_seq, st.d_tbl_off, st.d_tables,
                         P.block_size, a.H, P.rank, P.rank_ld, row, a.out_f32, a.out_b16, a.H * P.rank_ld / 32);
        else
            NVLLM_LAUNCH((k_latent_attn_any<false>), grid, dim3(256), lds, P.base, a.q, a.sink, a.scale, st.d_pos, st.d_seq, st.d_tbl_off, st.d_tables,
                         P.block_size, a.H, P.rank, P.rank_ld, row, a.out_f32, a.out_b16, 0);
        return;
    }
    LatentKArgs k{};
    k.base = (const __half*)P.base;
    k.q = (const __half*)a.q;
    k.sink = a.sink;
    k.scale = a.scale;
    k.tables = st.d_tables;
    k.H = a.H;
    k.chunks = chunks;
    k.n_tiles = P.rank_ld / 16;
    k.rank_ld = P.rank_ld;
    k.page_shift = page_shift;
    k.out = a.out_b16;
    k.Kb_out = a.H * P.rank_ld / 32;
    // prompt portions and single tokens want differently shaped items: a launch each when the batch has both
    const int n_single = st.n_runs - st.n_multi;
    auto launch = [&](const int* runs, int n_runs, int max_run, double bytes, double flops) {
        if (n_runs <= 0) return;
        // columns per item: 64, or 32 or 16 when no item would fill more
        // (64 columns of the widest class fit the register file only when the row is exactly that class's)
        const bool wide = chunks > 10 || vt > 4, exact = chunks == 18 && vt * 64 == P.rank_ld;
        const int W = a.H * max_run <= 16 ? 16 : a.H * max_run <= 32 || (wide && !exact) ? 32 : 64;
        // up to 16 tokens per item (so that a column group is one head's neighbouring tokens), more only when there are few heads
        int ct = 1;
        while (ct < 16 && ct < max_run) ct *= 2;
        k.runs = (const int4*)runs;
        k.run_ld = max_run;
        k.HG = a.H < W / ct ? a.H : W / ct;
        k.NG = cdiv(a.H, k.HG);
        k.CT = W / k.HG;
        k.n_sub = cdiv(max_run, k.CT);
        // slices of pages until every CU has a workgroup, eight pages per slice at least
        const long items = (long)n_runs * k.n_sub * k.NG;
        const int npages = st.max_pos / LATENT_PAGE + 1;
        int nsplit = (int)((rt().num_cus + items / 2) / items);
        if (nsplit > cdiv(npages, 8)) nsplit = cdiv(npages, 8);
        if (nsplit > 64) nsplit = 64;
        if (nsplit < 1) nsplit = 1;
        k.nsplit = nsplit;
        const size_t rows = (size_t)n_runs * max_run * a.H * nsplit;
        if (nsplit > 1) {
            float* part = (float*)ws_get(WS_ATT_PART, rows * (P.rank_ld + 2) * sizeof(float));
            k.part_acc = part;
            k.part_ml = part + rows * P.rank_ld;
        }
        {
            ProfScope ps(max_run == 1 ? PC_LATENT_ATTN_TOK : PC_LATENT_ATTN, bytes, flops);
            const long units = items * nsplit;
            if (chunks <= 4 && vt <= 1) launch_latent_rc<4, 1>(k, units, W);
            else if (chunks <= 6 && vt <= 2) launch_latent_rc<6, 2>(k, units, W);
            else if (chunks <= 10 && vt <= 4) launch_latent_rc<10, 4>(k, units, W);
            else launch_latent_rc<18, 8>(k, units, W);
        }
        if (nsplit > 1) {
            ProfScope ps(PC_LATENT_COMBINE, (double)rows * (P.rank_ld + 2) * 4.0, 0);
            NVLLM_LAUNCH(k_latent_combine, dim3((unsigned)n_runs * max_run * a.H), dim3(128), 0, k.part_acc, k.part_ml, a.sink, k.runs, max_run, a.H, nsplit,
                         P.rank_ld, a.out_b16, k.Kb_out);
        }
    };
    const double single_bytes = bytes_of((double)st.kv_rows_single, n_single);
    const double single_flops = 2.0 * (double)st.kv_rows_single * a.H * (row + P.rank_ld);
    launch(st.d_runs, st.n_multi, st.max_run, bytes - single_bytes, flops - single_flops);
    launch(st.d_runs + 4 * st.n_multi, n_single, 1, single_bytes, single_flops);
}

// ------------------------------------------------------------------ fp32 head products
__global__ __launch_bounds__(256) void k_latent_q_f32(float* __restrict__ rows, const float* __restrict__ q, const float* __restrict__ uk,
                                                      const float2* __restrict__ rope, const int* __restrict__ pos, int H, int dim, int rot, int rank) {
    const int t = blockIdx.x, h = blockIdx.y;
    const float* qh = q + ((size_t)t * H + h) * (dim + rot);
    float* dst = rows + ((size_t)t * H + h) * (rank + rot);
    for (int j = threadIdx.x; j < rank; j += 256) {
        float s = 0.f;
        for (int d = 0; d < dim; d++) s = fmaf(qh[d], uk[((size_t)h * dim + d) * rank + j], s);
        dst[j] = s;
    }
    for (int i = threadIdx.x; i < rot / 2; i += 256) {
        const float2 cs = rope[(size_t)pos[t] * (rot / 2) + i];
        const float u = qh[dim + 2 * i], v = qh[dim + 2 * i + 1];
        dst[rank + 2 * i] = u * cs.x - v * cs.y;
        dst[rank + 2 * i + 1] = v * cs.x + u * cs.y;
    }
}
void launch_latent_q_f32(float* rows, const float* q, const float* uk, const float2* rope, const int* pos, int T, int H, int dim, int rot, int rank) {
    if (T <= 0) return;
    ProfScope ps(PC_GEMM_ABSORB, (double)H * dim * rank * 4.0 + (double)T * H * (dim + rank + 2 * rot) * 4.0, 2.0 * T * (double)H * dim * rank);
    NVLLM_LAUNCH(k_latent_q_f32, dim3(T, H), dim3(256), 0, rows, q, uk, rope, pos, H, dim, rot, rank);
}

__global__ __launch_bounds__(256) void k_latent_v_f32(float* __restrict__ out, const float* __restrict__ lat, const float* __restrict__ uv, int H, int vdim,
                                                      int rank) {
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63;
    const float* lh = lat + ((size_t)t * H + h) * rank;
    for (int v = threadIdx.x >> 6; v < vdim; v += 4) {   // a wave per output
        const float* w = uv + ((size_t)h * vdim + v) * rank;
        float s = 0.f;
        for (int c = lane; c < rank; c += 64) s = fmaf(lh[c], w[c], s);
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
        if (lane == 0) out[((size_t)t * H + h) * vdim + v] = s;
    }
}
void launch_latent_v_f32(float* out, const float* lat, const float* uv, int T, int H, int vdim, int rank) {
    if (T <= 0) return;
    ProfScope ps(PC_GEMM_VALUE, (double)H * vdim * rank * 4.0 + (double)T * H * (vdim + rank) * 4.0, 2.0 * T * (double)H * vdim * rank);
    NVLLM_LAUNCH(k_latent_v_f32, dim3(T, H), dim3(256), 0, out, lat, uv, H, vdim, rank);
}

// ------------------------------------------------------------------ converters
__global__ __launch_bounds__(256) void k_latent_rows_b16(__bf16* __restrict__ dst, const float* __restrict__ src, int rank, int rot, int rank_ld, int rot_ld) {
    const size_t r = blockIdx.x;
    for (int d = threadIdx.x; d < rank_ld + rot_ld; d += 256) {
        const int part = d >= rank_ld, i = part ? d - rank_ld : d;
        const float v = i < (part ? rot : rank) ? src[r * (rank + rot) + (part ? rank : 0) + i] : 0.f;
        dst[r * (rank_ld + rot_ld) + d] = (__bf16)v;
    }
}
void launch_latent_rows_b16(__half* dst, const float* src, int rows, const LatentPool& pool) {
    if (rows <= 0) return;
    NVLLM_LAUNCH(k_latent_rows_b16, dim3(rows), dim3(256), 0, (__bf16*)dst, src, pool.rank, pool.rot, pool.rank_ld, pool.rot_ld);
}

__global__ __launch_bounds__(256) void k_untile_b16(float* __restrict__ dst, const unsigned short* __restrict__ tiles, int H, int width, int width_ld, int Kb) {
    const int t = blockIdx.x, h = blockIdx.y;
    for (int d = threadIdx.x; d < width; d += 256) {
        const int k = h * width_ld + d;
        dst[((size_t)t * H + h) * width + d] =
            bf16_to_f32(tiles[((size_t)(t >> 4) * Kb + (k >> 5)) * TILE_HALVES + (size_t)((t & 15) + 16 * ((k >> 3) & 3)) * 8 + (k & 7)]);
    }
}
void launch_untile_b16(float* dst, const __half* tiles, int T, int H, int width, int width_ld) {
    if (T <= 0) return;
    NVLLM_LAUNCH(k_untile_b16, dim3(T, H), dim3(256), 0, dst, (const unsigned short*)tiles, H, width, width_ld, cdiv(H * width_ld, 32));
}

}  // namespace nvllm
