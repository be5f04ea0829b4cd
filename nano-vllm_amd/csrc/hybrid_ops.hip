// hybrid_ops.hip -- operator entry points (include/nvllm.h) of windowed attention, linear attention with decay and
// mixtures of experts.
#include <cmath>
#include <vector>

#include "gemm_common.h"
#include "latent_attention.h"
#include "lightning.h"
#include "model_dir.h"
#include "moe.h"
#include "step_arrays.h"
#include "window_attention.h"

namespace nvllm {

// fp32 rows of n values -> bf16 rows of ld (zeros behind)
__global__ __launch_bounds__(256) void k_rows_b16(__bf16* __restrict__ dst, const float* __restrict__ src, int n, int src_ld, int ld) {
    for (int i = threadIdx.x; i < ld; i += 256) dst[(size_t)blockIdx.x * ld + i] = (__bf16)(i < n ? src[(size_t)blockIdx.x * src_ld + i] : 0.f);
}
static void rows_b16(__half* dst, const float* src, int rows, int n, int src_ld, int ld) {
    if (rows > 0) NVLLM_LAUNCH(k_rows_b16, dim3(rows), dim3(256), 0, (__bf16*)dst, src, n, src_ld, ld);
}
// heads of `n` values at column `at` of rows of `ld`, padded to n_ld each
__global__ __launch_bounds__(256) void k_heads_b16(__bf16* __restrict__ dst, const float* __restrict__ src, int H, int n, int n_ld, int at, int ld) {
    const int t = blockIdx.x, h = blockIdx.y;
    for (int i = threadIdx.x; i < n_ld; i += 256) dst[(size_t)t * ld + at + h * n_ld + i] = (__bf16)(i < n ? src[((size_t)t * H + h) * n + i] : 0.f);
}
__global__ __launch_bounds__(256) void k_row_sums(float* __restrict__ out, const float* __restrict__ in, int T, int n) {
    const int t = blockIdx.x * 256 + threadIdx.x;
    if (t >= T) return;
    float s = 0.f;
    for (int i = 0; i < n; i++) s += in[(size_t)t * n + i];
    out[t] = s;
}
__global__ __launch_bounds__(256) void k_router_rows(float* __restrict__ out, const float* __restrict__ in, const int* __restrict__ row_of, int top, int D) {
    const int t = blockIdx.x;
    for (int n = threadIdx.x; n < D; n += 256) {
        float s = 0.f;
        for (int j = 0; j < top; j++) s += in[(size_t)row_of[t * top + j] * D + n];
        out[(size_t)t * D + n] = s;
    }
}

// a device buffer for the duration of a call
struct Temp {
    void* p = nullptr;
    explicit Temp(size_t bytes) {
        if (device_malloc(&p, bytes) != 0) NVLLM_FATAL("cannot allocate %zu bytes", bytes);
    }
    ~Temp() { device_free(p); }   // waits for the stream
    Temp(const Temp&) = delete;
    Temp& operator=(const Temp&) = delete;
    __half* h() const { return (__half*)p; }
    float* f() const { return (float*)p; }
};

static KvPages checked_pages(const KVCacheManager* mgr, int G, int dim, int vdim, int elem) {
    if (block_pool_bytes(mgr) != kv_pages_bytes(elem, mgr->block_size, mgr->num_blocks, G, dim, vdim))
        NVLLM_FATAL("this block pool does not hold %d heads of %d and %d values of %d bytes", G, dim, vdim, elem);
    return kv_pages(mgr->pool_k, elem, mgr->block_size, mgr->num_blocks, G, dim, vdim);
}

}  // namespace nvllm

using namespace nvllm;

extern "C" {

void nvllm_window_pool_init(KVCacheManager* mgr, int block_size, int num_blocks, int kv_heads, int dim, int vdim, int elem_bytes) {
    init_block_pool(mgr, block_size, num_blocks, kv_pages_bytes(elem_bytes, block_size, num_blocks, kv_heads, dim, vdim));
}

void nvllm_conv_rope(float* q, const float* raw, const float* taps, int n_taps, void* state, KVCacheManager* mgr, BlockTable** block_tables, int* seq_ids,
                     int* pos_arr, double base, int rot, int n_heads, int kv_heads, int dim, int vdim, int elem_bytes, int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    const KvPages pool = checked_pages(mgr, kv_heads, dim, vdim, elem_bytes);
    const StepArrays s = stage_step(nullptr, pos_arr, seq_ids, num_tokens, nullptr, 0, block_tables, nullptr, 0, mgr->block_size, WINDOW_RUN, nullptr, true, true);
    if (s.table_short || s.seq_split) NVLLM_FATAL("convolution over time: the batch does not fit its block tables, or a sequence's tokens are apart");
    ConvRope c{};
    const int channels = n_heads * dim + kv_heads * (dim + vdim);
    c.taps = taps; c.n_taps = n_taps; c.state = state; c.rot = rot; c.H = n_heads;
    c.rope = rot ? rotation_table(base, rot, s.max_pos + 1) : nullptr;
    if (elem_bytes == 4) {
        c.raw = raw; c.raw_ld = channels; c.q_out = q;
        launch_conv_rope(c, pool, s);
        return;
    }
    c.raw_ld = pad32(channels);
    const Temp rows((size_t)num_tokens * c.raw_ld * 2), q16((size_t)num_tokens * n_heads * pool.dim_ld * 2);
    rows_b16(rows.h(), raw, num_tokens, channels, channels, c.raw_ld);
    c.raw = rows.p; c.q_out = q16.p;
    launch_conv_rope(c, pool, s);
    // back to fp32 through tile order
    const int width = n_heads * pool.dim_ld;
    const Temp tiles(b16_halves(num_tokens, width) * 2);
    launch_tile_weights(tiles.h(), q16.h(), num_tokens, width, (long)(width / 32) * TILE_HALVES);
    launch_untile_b16(q, tiles.h(), num_tokens, n_heads, dim, pool.dim_ld);
}

void nvllm_window_attention(float* out, const float* q, KVCacheManager* mgr, BlockTable** block_tables, int* seq_ids, int* pos_arr, float scale, float cap, int size,
                            int keep_first, int n_heads, int kv_heads, int dim, int vdim, int elem_bytes, int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    const KvPages pool = checked_pages(mgr, kv_heads, dim, vdim, elem_bytes);
    const StepArrays s = stage_step(nullptr, pos_arr, seq_ids, num_tokens, nullptr, 0, block_tables, nullptr, 0, mgr->block_size, WINDOW_RUN, nullptr, true, true);
    if (s.table_short) NVLLM_FATAL("windowed attention: a position lies beyond its sequence's block table");
    WindowAttn a{};
    a.pool = pool; a.H = n_heads; a.scale = scale; a.cap = cap; a.size = size; a.keep_first = keep_first;
    if (elem_bytes == 4) {
        a.q = q; a.out_f32 = out;
        launch_window_attention(a, s);
        return;
    }
    const Temp rows((size_t)num_tokens * n_heads * pool.dim_ld * 2), tiles(b16_halves(num_tokens, n_heads * pool.vdim_ld) * 2);
    rows_b16(rows.h(), q, num_tokens * n_heads, dim, dim, pool.dim_ld);
    a.q = rows.p; a.out_b16 = tiles.h();
    launch_window_attention(a, s);
    launch_untile_b16(out, tiles.h(), num_tokens, n_heads, vdim, pool.vdim_ld);
}

void nvllm_lightning(float* out, float* ss, const float* q, const float* k, const float* v, const float* gate, const float* gain, const float* decay, float* state,
                     int* seq_ids, int* pos_arr, int heads, int dim, int vdim, int elem_bytes, int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    const StepArrays s = stage_step(nullptr, pos_arr, seq_ids, num_tokens, nullptr, 0, nullptr, nullptr, 0, 1, 0, nullptr, false, true, lightning_group(num_tokens, heads, vdim));
    if (s.seq_split) NVLLM_FATAL("linear attention: a sequence's tokens must lie side by side in the batch");
    std::vector<float> powers((size_t)heads * (LIGHTNING_CHUNK + 1));
    for (int h = 0; h < heads; h++)
        for (int n = 0; n <= LIGHTNING_CHUNK; n++) powers[(size_t)h * (LIGHTNING_CHUNK + 1) + n] = (float)std::pow((double)decay[h], n);
    const Temp table(powers.size() * 4);
    device_memcpy(table.p, powers.data(), powers.size() * 4, HOST_TO_DEVICE);
    Lightning a;
    a.H = heads; a.dim = dim; a.vdim = vdim; a.decay = table.f(); a.state = state;
    if (elem_bytes == 4) {
        a.q32 = q; a.k32 = k; a.v32 = v; a.out_f32 = out;
        launch_lightning(a, s);
        return;
    }
    a.dim_ld = pad32(dim); a.vdim_ld = pad32(vdim); a.ld = 2 * heads * (a.dim_ld + a.vdim_ld);
    const int vw = heads * a.vdim_ld;
    const Temp rows((size_t)num_tokens * a.ld * 2), tiles(b16_halves(num_tokens, vw) * 2), sums((size_t)num_tokens * (vw / 16) * 4);
    std::vector<float> padded((size_t)vw, 0.f), plain((size_t)heads * vdim);
    device_memcpy(plain.data(), gain, plain.size() * 4, DEVICE_TO_HOST);
    for (int h = 0; h < heads; h++)
        for (int i = 0; i < vdim; i++) padded[(size_t)h * a.vdim_ld + i] = plain[(size_t)h * vdim + i];
    const Temp gain_ld(padded.size() * 4);
    device_memcpy(gain_ld.p, padded.data(), padded.size() * 4, HOST_TO_DEVICE);
    auto put = [&](const float* src, int n, int n_ld, int at) { NVLLM_LAUNCH(k_heads_b16, dim3(num_tokens, heads), dim3(256), 0, (__bf16*)rows.p, src, heads, n, n_ld, at, a.ld); };
    put(q, dim, a.dim_ld, 0);
    put(k, dim, a.dim_ld, heads * a.dim_ld);
    put(v, vdim, a.vdim_ld, 2 * heads * a.dim_ld);
    put(gate, vdim, a.vdim_ld, 2 * heads * a.dim_ld + vw);
    a.rows = rows.h(); a.gain = gain_ld.f(); a.out_b16 = tiles.h(); a.ss_out = sums.f();
    launch_lightning(a, s);
    launch_untile_b16(out, tiles.h(), num_tokens, heads, vdim, a.vdim_ld);
    if (ss) NVLLM_LAUNCH(k_row_sums, dim3(cdiv(num_tokens, 256)), dim3(256), 0, ss, sums.f(), num_tokens, vw / 16);
}

void nvllm_expert_ff(float* out, int* choice, float* score, const float* in, const float* z, const float* gate, const float* up, const float* down, int dim, int ff,
                     int experts, int top, int elem_bytes, int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    const int pad = elem_bytes == 4 ? 16 : route_pad(num_tokens, experts, top);
    const Temp mem(route_ints(num_tokens, experts, top, pad) * 4);
    const RoutePlan plan = route_plan((int*)mem.p, num_tokens, experts, top, pad);
    launch_route(plan, z, experts);
    const size_t pairs = (size_t)num_tokens * top;
    if (choice) device_memcpy(choice, plan.choice, pairs * 4, DEVICE_TO_DEVICE);
    if (score) device_memcpy(score, plan.score, pairs * 4, DEVICE_TO_DEVICE);
    if (!out) return;
    if (elem_bytes == 4) {
        const Temp g(pairs * ff * 4), u(pairs * ff * 4), y(pairs * dim * 4);
        launch_matmul_experts_f32(g.f(), in, gate, plan, true, dim, ff);
        launch_matmul_experts_f32(u.f(), in, up, plan, true, dim, ff);
        launch_swiglu(g.f(), g.f(), u.f(), (long)pairs * ff);
        launch_matmul_experts_f32(y.f(), g.f(), down, plan, false, ff, dim);
        HIP_CHECK(hipMemsetAsync(out, 0, (size_t)num_tokens * dim * 4, rt().stream));
        MoeCombine c{};
        c.x = out; c.rows = y.f(); c.top = top; c.ld = dim;
        launch_moe_combine(c, num_tokens);
        return;
    }
    const int Dp = pad32(dim), Fp = pad32(ff);
    const long up_nb = (long)(Dp / 32) * TILE_HALVES, down_nb = (long)(Fp / 32) * TILE_HALVES;
    const Temp act(b16_halves(num_tokens, Dp) * 2), w_up((size_t)experts * (2 * Fp / 16) * up_nb * 2), w_down((size_t)experts * (Dp / 16) * down_nb * 2),
        hid(b16_halves(plan.capacity, Fp) * 2), y((size_t)plan.capacity * Dp * 4), y_sum((size_t)num_tokens * Dp * 4);
    HIP_CHECK(hipMemsetAsync(w_up.p, 0, (size_t)experts * (2 * Fp / 16) * up_nb * 2, rt().stream));   // rows of the padding
    HIP_CHECK(hipMemsetAsync(w_down.p, 0, (size_t)experts * (Dp / 16) * down_nb * 2, rt().stream));
    const Temp stage((size_t)std::max((long)num_tokens * dim, (long)ff * dim) * 2);
    rows_b16(stage.h(), in, num_tokens, dim, dim, dim);
    launch_tile_weights(act.h(), stage.h(), num_tokens, dim, up_nb);
    for (int e = 0; e < experts; e++) {
        for (int half = 0; half < 2; half++) {
            rows_b16(stage.h(), (half ? up : gate) + (size_t)e * ff * dim, ff, dim, dim, dim);
            launch_tile_weights(w_up.h() + ((size_t)e * (2 * Fp / 16) + half) * up_nb, stage.h(), ff, dim, 2 * up_nb);
        }
        rows_b16(stage.h(), down + (size_t)e * dim * ff, dim, ff, ff, ff);
        launch_tile_weights(w_down.h() + (size_t)e * (Dp / 16) * down_nb, stage.h(), dim, ff, down_nb);
    }
    B16Weight wu, wd;
    wu.tiles = w_up.h(); wu.N = 2 * Fp; wu.K = Dp;
    wd.tiles = w_down.h(); wd.N = Dp; wd.K = Fp;
    ExpertRows er{plan.block_expert, plan.source, plan.capacity, plan.pad, num_tokens * top};
    GemmEpilogue eu;
    eu.kind = GemmEpilogue::SWIGLU_A16;
    eu.row_weight = plan.weight; eu.a16_out = hid.h();
    launch_gemm_experts(wu, experts, act.h(), er, eu, PC_GEMM_EXPERT_UP);
    er.source = nullptr;
    GemmEpilogue ed;
    ed.kind = GemmEpilogue::F32;
    ed.out = y.f(); ed.ldo = Dp;
    launch_gemm_experts(wd, experts, hid.h(), er, ed, PC_GEMM_EXPERT_DOWN);
    NVLLM_LAUNCH(k_router_rows, dim3(num_tokens), dim3(256), 0, y_sum.f(), y.f(), plan.row_of, top, Dp);
    HIP_CHECK(hipMemcpy2DAsync(out, (size_t)dim * 4, y_sum.p, (size_t)Dp * 4, (size_t)dim * 4, num_tokens, hipMemcpyDeviceToDevice, rt().stream));
}

}  // extern "C"
