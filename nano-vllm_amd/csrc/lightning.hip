// lightning.hip -- linear attention with decay (lightning.h).
//
// k_lightning_chunk (bf16, portions of several tokens): a workgroup takes a portion's head x 64 value columns and walks
// the portion in chunks of 64 tokens, its four waves owning 16 columns of the state each, in registers:
//   P[s, t]  = decay^(t-s) (k_s . q_t), s <= t        one wave per 16 tokens t, to LDS as the operand of the next product
//   o_t      = decay^(t+1) S^T q_t + sum_s P[s, t] v_s
//   S        = decay^n S + sum_s k_s (decay^(n-1-s) v_s)^T
// q, k and v are bf16 values.  The 32-bit factors -- S, P and the decayed v -- enter the matrix cores as three bf16
// parts (truncations: 8 + 8 + 8 bits, together the exact value), so every product is that of the 32-bit numbers.
// The state's result registers are already in the k order of S^T q, P's in that of P v.
//
// k_lightning_step (single tokens, and everything in fp32): a workgroup per (portion, head), the state streamed once per
// token as float4 columns.
#include "lightning.h"

#include "gemm_common.h"

namespace nvllm {

typedef short s4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s4_t lds_s4;
typedef unsigned int u2_t __attribute__((ext_vector_type(2)));

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
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
constexpr int lightning_lds(int DC) { return 2 * CH * (DC * 32 + 8) * 2 + CH * VROW * 2 + 4 * 2 * 3 * 1024 + (CH + 1) * 4; }

template <int DC>
__global__ __launch_bounds__(256, 2) void k_lightning_chunk(Lightning a, const int4* __restrict__ spans, int vslices) {
    constexpr int QROW = DC * 32 + 8;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_l[];
    __half* s_q = reinterpret_cast<__half*>(lds_l);   // [CH][QROW]
    __half* s_k = s_q + CH * QROW;                    // [CH][QROW]
    __half* s_v = s_k + CH * QROW;                    // [CH][VROW]
    b8_t* s_p = reinterpret_cast<b8_t*>(s_v + CH * VROW);   // [t tile][s pair][part][64]
    float* s_dec = reinterpret_cast<float*>(s_p + 4 * 2 * 3 * 64);   // [CH + 1]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), x = lane & 15, g = lane >> 4;
    int idx = blockIdx.x;
    const int vs = idx % vslices;
    idx /= vslices;
    const int h = idx % a.H, span_id = idx / a.H;
    const int4 span = spans[span_id];
    const int n_tok = span.y;
    const int v0 = vs * 64, my_v = v0 + wave * 16;         // this wave's value columns
    const bool has_v = my_v < a.vdim_ld;
    if (tid <= CH) s_dec[tid] = a.decay[h * (CH + 1) + tid];

    // ---- the state's tiles: S[d = 16 i + 4 g + r][v = my_v + x]
    float* st = a.state + ((size_t)span.w * a.H + h) * a.dim * a.vdim;
    f4_t S[2 * DC];
#pragma unroll
    for (int i = 0; i < 2 * DC; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int d = 16 * i + 4 * g + r, v = my_v + x;
            S[i][r] = span.z > 0 && d < a.dim && v < a.vdim ? st[(size_t)d * a.vdim + v] : 0.f;
        }

    // ---- the chunk's rows, a chunk ahead in registers: 16-byte pieces, a row's pieces by neighbouring threads
    const int qk_pieces = a.dim_ld / 8;
    u4_t rq[DC], rk[DC], rv[2];
    u2_t rg[4];   // this lane's gates: columns my_v + 4 g .. + 3 of tokens 16 i + x
    auto fetch = [&](int c0) {
#pragma unroll
        for (int u = 0; u < DC; u++) {
            const int i = tid + 256 * u, row = i / (4 * DC), piece = i - row * (4 * DC);
            const bool live = c0 + row < n_tok && piece < qk_pieces;
            const __half* src = a.rows + (size_t)(span.x + c0 + row) * a.ld + h * a.dim_ld + piece * 8;
            rq[u] = live ? *reinterpret_cast<const u4_t*>(src) : u4_t{0, 0, 0, 0};
            rk[u] = live ? *reinterpret_cast<const u4_t*>(src + a.H * a.dim_ld) : u4_t{0, 0, 0, 0};
        }
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const int i = tid + 256 * u, row = i >> 3, piece = i & 7;
            const bool live = c0 + row < n_tok && v0 + piece * 8 < a.vdim_ld;
            const __half* src = a.rows + (size_t)(span.x + c0 + row) * a.ld + 2 * a.H * a.dim_ld + h * a.vdim_ld + v0 + piece * 8;
            rv[u] = live ? *reinterpret_cast<const u4_t*>(src) : u4_t{0, 0, 0, 0};
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int tok = min(c0 + 16 * i + x, n_tok - 1);
            rg[i] = has_v ? *reinterpret_cast<const u2_t*>(a.rows + (size_t)(span.x + tok) * a.ld + 2 * a.H * a.dim_ld + (a.H + h) * a.vdim_ld + my_v + 4 * g) : u2_t{0, 0};
        }
    };
    fetch(0);
    const int ss_ld = a.H * a.vdim_ld / 16, Kb_out = a.H * a.vdim_ld / 32;
    const f4_t gain = has_v ? *reinterpret_cast<const f4_t*>(a.gain + h * a.vdim_ld + my_v + 4 * g) : f4_t{0.f, 0.f, 0.f, 0.f};

    for (int c0 = 0; c0 < n_tok; c0 += CH) {
        const int n = min(CH, n_tok - c0);
#pragma unroll
        for (int u = 0; u < DC; u++) {
            const int i = tid + 256 * u, row = i / (4 * DC), piece = i - row * (4 * DC);
            *reinterpret_cast<u4_t*>(s_q + row * QROW + piece * 8) = rq[u];
            *reinterpret_cast<u4_t*>(s_k + row * QROW + piece * 8) = rk[u];
        }
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const int i = tid + 256 * u, row = i >> 3, piece = i & 7;
            *reinterpret_cast<u4_t*>(s_v + row * VROW + piece * 8) = rv[u];
        }
        u2_t gates[4];
#pragma unroll
        for (int i = 0; i < 4; i++) gates[i] = rg[i];
        __syncthreads();
        if (c0 + CH < n_tok) fetch(c0 + CH);
        // operands over dims in the order of the state's registers: {32 c + 4 g .., 32 c + 16 + 4 g ..} of row 16 i + x
        auto frag = [&](const __half* base, int i, int c) {
            const __half* p = base + (16 * i + x) * QROW + 32 * c + 4 * g;
            const u2_t lo = *reinterpret_cast<const u2_t*>(p), hi = *reinterpret_cast<const u2_t*>(p + 16);
            return __builtin_bit_cast(b8_t, u4_t{lo[0], lo[1], hi[0], hi[1]});
        };
        // ---- P of token tile `wave`: rows s (tiles 0 .. wave), columns t
        if (wave * 16 < n) {
            b8_t qf[DC];
#pragma unroll
            for (int c = 0; c < DC; c++) qf[c] = frag(s_q, wave, c);
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
                        for (int c = 0; c < DC; c++) p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(frag(s_k, i, c), qf[c], p, 0, 0, 0);
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
        __syncthreads();
        if (has_v) {
            // values of this wave's columns with tokens as k: {pair * 32 + 4 g .., pair * 32 + 16 + 4 g ..}, by the LDS transpose read
            // (16 lanes bring 4 rows x 16 columns, lane x receives column x of the four rows)
            s4_t vt[2][2];
#pragma unroll
            for (int pair = 0; pair < 2; pair++)
#pragma unroll
                for (int half = 0; half < 2; half++)
                    vt[pair][half] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                        (lds_s4*)(s_v + (32 * pair + 16 * half + 4 * g + (x >> 2)) * VROW + wave * 16 + 4 * (x & 3)));
            auto vfrag = [&](int pair) {
                const u2_t lo = __builtin_bit_cast(u2_t, vt[pair][0]), hi = __builtin_bit_cast(u2_t, vt[pair][1]);
                return __builtin_bit_cast(b8_t, u4_t{lo[0], lo[1], hi[0], hi[1]});
            };
            // the state as operand, three exact parts
            b8_t sf[DC][3];
#pragma unroll
            for (int c = 0; c < DC; c++) {
                const float e[8] = {S[2 * c][0], S[2 * c][1], S[2 * c][2], S[2 * c][3], S[2 * c + 1][0], S[2 * c + 1][1], S[2 * c + 1][2], S[2 * c + 1][3]};
                split3_frag(e, sf[c]);
            }
#pragma unroll
            for (int i = 0; i < 4; i++) {
                if (i * 16 >= n) break;
                f4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int c = 0; c < DC; c++) {
                    const b8_t qf = frag(s_q, i, c);
#pragma unroll
                    for (int k = 2; k >= 0; k--) o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sf[c][k], qf, o, 0, 0, 0);
                }
                const int tl = i * 16 + x, t = span.x + c0 + tl;
                o *= s_dec[tl + 1];
#pragma unroll
                for (int pair = 0; pair < 2; pair++) {
                    if (2 * pair > i) break;
#pragma unroll
                    for (int k = 2; k >= 0; k--)
                        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vfrag(pair), s_p[((i * 2 + pair) * 3 + k) * 64 + lane], o, 0, 0, 0);
                }
                float sq = o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
                sq += __shfl_xor(sq, 16, 64);
                sq += __shfl_xor(sq, 32, 64);
                if (tl < n) {
                    const int col = h * a.vdim_ld + my_v;
                    float y[4];
#pragma unroll
                    for (int r = 0; r < 4; r++) y[r] = o[r] * gain[r] * sigmoid_f(b16_f((unsigned short)(gates[i][r >> 1] >> (16 * (r & 1)))));
                    store_b16_4(a.out_b16, Kb_out, t, col + 4 * g, y);
                    if (g == 0) a.ss_out[(size_t)t * ss_ld + (col >> 4)] = sq;
                }
            }
            // ---- the state behind the chunk
            const float fade = s_dec[n];
#pragma unroll
            for (int i = 0; i < 2 * DC; i++) S[i] *= fade;
#pragma unroll
            for (int pair = 0; pair < 2; pair++) {
                float e[8];
                const b8_t vv = vfrag(pair);
#pragma unroll
                for (int i = 0; i < 8; i++) {
                    const int s = 32 * pair + 16 * (i >> 2) + 4 * g + (i & 3);
                    e[i] = s < n ? (float)vv[i] * s_dec[max(n - 1 - s, 0)] : 0.f;
                }
                b8_t parts[3];
                split3_frag(e, parts);
#pragma unroll
                for (int i = 0; i < 2 * DC; i++) {
                    const s4_t k0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)(s_k + (32 * pair + 4 * g + (x >> 2)) * QROW + 16 * i + 4 * (x & 3)));
                    const s4_t k1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)(s_k + (32 * pair + 16 + 4 * g + (x >> 2)) * QROW + 16 * i + 4 * (x & 3)));
                    const u2_t lo = __builtin_bit_cast(u2_t, k0), hi = __builtin_bit_cast(u2_t, k1);
                    const b8_t kt = __builtin_bit_cast(b8_t, u4_t{lo[0], lo[1], hi[0], hi[1]});
#pragma unroll
                    for (int k = 2; k >= 0; k--) S[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kt, parts[k], S[i], 0, 0, 0);
                }
            }
        }
        __syncthreads();   // the chunk's rows and P have been read
    }
    if (has_v && my_v + x < a.vdim)
#pragma unroll
        for (int i = 0; i < 2 * DC; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int d = 16 * i + 4 * g + r;
                if (d < a.dim) st[(size_t)d * a.vdim + my_v + x] = S[i][r];
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
static void launch_chunk(const Lightning& a, const StepArrays& st) {
    constexpr int shmem = lightning_lds(DC);
    static bool enabled = false;
    if (shmem > 64 * 1024 && !enabled) {
        HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_lightning_chunk<DC>), hipFuncAttributeMaxDynamicSharedMemorySize, shmem));
        enabled = true;
    }
    const int vslices = cdiv(a.vdim_ld, 64);
    NVLLM_LAUNCH((k_lightning_chunk<DC>), dim3(st.n_spans_multi * a.H * vslices), dim3(256), shmem, a, (const int4*)st.d_spans, vslices);
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
        ProfScope ps(PC_LIGHTNING, st.n_spans_multi * state_bytes + multi_tokens * token_bytes,
                     multi_tokens * (token_flops + pair * 0.5 * std::min(st.max_span, CH)));
        switch (DC) {
            case 1: launch_chunk<1>(a, st); break;
            case 2: launch_chunk<2>(a, st); break;
            case 3: launch_chunk<3>(a, st); break;
            case 4: launch_chunk<4>(a, st); break;
            default: launch_chunk<8>(a, st); break;
        }
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
