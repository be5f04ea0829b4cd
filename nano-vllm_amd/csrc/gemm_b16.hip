// gemm_b16.hip -- projections of bf16 models: the kernels of gemm.hip (decode-sized batches) and
// gemm_prefill.hip (hundreds of tokens) instantiated for bf16 weights and one bf16 activation plane, with
// fp32 accumulation, and the epilogues of latent attention and hyper-connections.  A block-diagonal product
// (one head per group of row blocks) is the same kernel with tiles that stay inside a group.
#include "gemm_prefill_tile.h"
#include "gemm_tile.h"
#include "latent_kv.h"

namespace nvllm {

namespace {

constexpr int NW = 8, RW = 4, RA = 2;

template <int NBW, int TB, int WAVES, int EPI, bool GRP, bool EXP = false>
__global__ __launch_bounds__(WAVES * 64) void k_gemm_b16(GemmArgs p) {
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_dyn[];
    if constexpr (EPI == GemmEpilogue::LATENT_Q) {
        if ((int)blockIdx.x >= p.ride_from) {
            if (blockIdx.y == 0 && blockIdx.z == 0) latent_kv_ride(p.ride, ((int)blockIdx.x - p.ride_from) * WAVES + (int)(threadIdx.x >> 6), threadIdx.x & 63);
            return;
        }
    }
    h8_t w[RW][NBW];
    const TileIdx ix{(int)blockIdx.x, (int)blockIdx.y, (int)blockIdx.z, EPI == GemmEpilogue::LATENT_Q ? p.ride_from : (int)gridDim.x};
    gemm_tile<NBW, TB, WAVES, RW, RA, EPI, float, false, 0, OpBf16, GRP, EXP>(p, ix, lds_dyn, w, [](int) {}, (int)threadIdx.x);
}

template <int NBW, int TB, int WAVES, int EPI, bool GRP, bool EXP = false>
void launch_stream(const GemmArgs& a, dim3 grid) {
    constexpr int shmem = gemm_tile_lds<NBW, TB, WAVES>();
    static_assert(shmem <= 160 * 1024, "partial tiles must fit the CU's LDS");
    static bool enabled = false;
    if (shmem > 64 * 1024 && !enabled) {
        HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_gemm_b16<NBW, TB, WAVES, EPI, GRP, EXP>),
                                      hipFuncAttributeMaxDynamicSharedMemorySize, shmem));
        enabled = true;
    }
    NVLLM_LAUNCH((k_gemm_b16<NBW, TB, WAVES, EPI, GRP, EXP>), grid, dim3(WAVES * 64), shmem, a);
}

template <int EPI, bool GRP>
void launch_stream_plan(const GemmArgs& a, const GemmPlan& pl) {
    const dim3 grid(pl.tiles_n + (EPI == GemmEpilogue::LATENT_Q && a.ride.base ? cdiv(a.ride.T, NW) : 0), pl.ks, pl.tiles_t);
    if constexpr (EPI == GemmEpilogue::SWIGLU_A16) {
        if (pl.nbw == 6) {
            launch_stream<6, 2, NW, EPI, GRP>(a, grid);
            return;
        }
    }
    if constexpr (EPI == GemmEpilogue::F32) {
        if (pl.nw == 4) {
            launch_stream<4, 4, 4, EPI, GRP>(a, grid);
            return;
        }
    }
    if (pl.nbw == 2) {
        if (pl.TB == 1) launch_stream<2, 1, NW, EPI, GRP>(a, grid);
        else launch_stream<2, 2, NW, EPI, GRP>(a, grid);
    } else if (pl.TB == 1) launch_stream<4, 1, NW, EPI, GRP>(a, grid);
    else if (pl.TB == 2) launch_stream<4, 2, NW, EPI, GRP>(a, grid);
    else launch_stream<4, 4, NW, EPI, GRP>(a, grid);
}

template <int EPI, bool GRP, int TW, bool EXP = false>
void launch_dense_tw(const GemmArgs& a, int tiles_n, int tiles_t, int nbuf) {
    using G = PfGeom<4, 1, 2, TW, 1>;
    const size_t shmem = (size_t)(G::RINV_HALVES + nbuf * G::STAGE_HALVES) * sizeof(__half);
    static size_t allowed = 0;
    if (shmem > allowed) {
        HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_gemm_prefill<4, 1, EPI, float, 2, TW, OpBf16, GRP, EXP>),
                                      hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem));
        allowed = shmem;
    }
    NVLLM_LAUNCH((k_gemm_prefill<4, 1, EPI, float, 2, TW, OpBf16, GRP, EXP>), dim3(tiles_n * tiles_t + (EPI == GemmEpilogue::LATENT_Q && a.ride.base ? cdiv(a.ride.T, 4) : 0)), dim3(256), shmem, a, tiles_n, tiles_t, nbuf,
                 tiles_n * tiles_t);
}

template <int EPI, bool GRP>
void launch_dense(GemmArgs a) {
    // 128-feature tiles, 128 tokens high, or 64 when the taller ones would leave CUs without a workgroup
    // (gemm_prefill.hip measures the same choice); a block-diagonal product pads every group to whole tiles
    const int cus = rt().num_cus;
    a.group_tiles = GRP ? cdiv(a.group_nb, 8) : 0;
    const int tiles_n = GRP ? a.group_tiles * (a.NB / a.group_nb) : cdiv(a.NB, 8);
    const int tall = tiles_n * cdiv(a.Tb, 8);
    const bool low = tall <= cus || tiles_n * cdiv(a.Tb, 4) <= 2 * cus;
    const int tiles_t = cdiv(a.Tb, low ? 4 : 8), total = tiles_n * tiles_t;
    const int per_cu = cdiv(total, cus);
    const int nbuf = per_cu >= 3 ? 3 : (per_cu == 2 ? 4 : 5);   // 16 KiB per stage (12 for the lower tiles)
    a.ksplit = 1;
    a.kb_per_split = a.Kb;
    a.ride_from = total;
    if (low) launch_dense_tw<EPI, GRP, 2>(a, tiles_n, tiles_t, nbuf);
    else launch_dense_tw<EPI, GRP, 4>(a, tiles_n, tiles_t, nbuf);
}

template <int EPI, bool GRP>
void launch_kind(GemmArgs a, int prof_cls, double bytes, double flops) {
    static const int pf_min_t = getenv("NVLLM_GEMM_PREFILL_T") ? atoi(getenv("NVLLM_GEMM_PREFILL_T")) : 256;
    // few features: the chip fills with token groups of 16 or 32, not with dense tiles
    const bool narrow = !GRP && EPI == GemmEpilogue::F32 && !a.e.amax_out && a.NB <= 8 && a.Tb <= 4 * rt().num_cus;
    if (a.T >= pf_min_t && !narrow) {
        {
            ProfScope ps(prof_cls, bytes, flops);
            a.e.amax_pairs = nullptr;   // the dense-tile kernel does not emit pairs: the rows are scanned afterwards
            launch_dense<EPI, GRP>(a);
        }
        if (EPI == GemmEpilogue::F32 && a.e.amax_out) launch_argmax_ld(a.e.amax_out, a.e.out, a.T, a.N, a.e.ldo, a.e.amax_out_host);
        return;
    }
    // a block-diagonal product has a short K and no K split; its plan is that of one group times the groups
    const int groups = GRP ? a.NB / a.group_nb : 1;
    GemmPlan pl = gemm_plan(GRP ? a.group_nb * 16 * groups : a.N, a.Kb * 32, a.T, EPI, GRP || narrow || (EPI == GemmEpilogue::F32 && a.e.amax_out) ? 1 : 0, 1 << 16, 0);
    if (narrow) {
        pl.nw = NW;
        pl.nbw = 2;
        pl.TB = a.Tb * cdiv(a.NB, 2) <= rt().num_cus ? 1 : 2;
        pl.tiles_n = cdiv(a.NB, 2);
        pl.tiles_t = cdiv(a.Tb, pl.TB);
    }
    if (GRP) {
        // a short K and no split: when 64-feature tiles leave half the CUs idle, 32-feature tiles x 32 or 16 tokens
        const int cus = rt().num_cus;
        if (cdiv(a.group_nb, pl.nbw) * groups * pl.tiles_t * 2 <= cus) {
            pl.nbw = 2;
            if (pl.TB > 1) pl.TB = cdiv(a.group_nb, 2) * groups * a.Tb > cus ? 2 : 1;
            pl.tiles_t = cdiv(a.Tb, pl.TB);
        }
        a.group_tiles = cdiv(a.group_nb, pl.nbw);
        pl.tiles_n = a.group_tiles * groups;
        pl.nw = NW;
    }
    a.ride_from = pl.tiles_n;
    a.ksplit = pl.ks;
    a.kb_per_split = pl.kb_per_split;
    const long wgs = (long)pl.tiles_n * pl.ks * pl.tiles_t;
    if (pl.ks > 1) a.slab = (float*)ws_get(WS_SLAB, (size_t)wgs * (pl.nbw / 2) * 2 * pl.TB * 64 * 16);
    a.close_sc1 = pl.ks > 1 && wgs <= rt().num_cus;
    {
        ProfScope ps(prof_cls, bytes, flops);
        launch_stream_plan<EPI, GRP>(a, pl);
    }
    if (EPI == GemmEpilogue::F32 && a.e.amax_out) {
        if (!a.e.amax_pairs || a.e.amax_ld < a.T) NVLLM_FATAL("fused arg-max needs a pair buffer of at least %d rows per tile", a.T);
        launch_argmax_tiles(a.e.amax_out, a.e.amax_pairs, cdiv(a.NB, pl.nbw), a.T, a.e.amax_ld, a.e.amax_out_host);
    }
}

template <int EPI>
void launch_experts_kind(GemmArgs a, int pad, bool dense, double bytes, double flops, int prof_cls) {
    const int cus = rt().num_cus;
    a.ksplit = 1;
    a.kb_per_split = a.Kb;
    ProfScope ps(prof_cls, bytes, flops);
    if (dense) {
        const int tiles_n = cdiv(a.NB, 8), tiles_t = a.Tb * 16 / pad, per_cu = cdiv(tiles_n * tiles_t, cus);
        const int nbuf = per_cu >= 3 ? 3 : (per_cu == 2 ? 4 : 5);
        a.ride_from = tiles_n * tiles_t;
        if (pad == 64) launch_dense_tw<EPI, false, 2, true>(a, tiles_n, tiles_t, nbuf);
        else launch_dense_tw<EPI, false, 4, true>(a, tiles_n, tiles_t, nbuf);
        return;
    }
    const int TB = pad / 16, tiles_t = a.Tb / TB;
    const bool narrow = cdiv(a.NB, 4) * tiles_t <= cus;   // (some of the row groups are empty)
    const dim3 grid(cdiv(a.NB, narrow ? 2 : 4), 1, tiles_t);
    a.ride_from = (int)grid.x;
    if (narrow) {
        if (TB == 1) launch_stream<2, 1, NW, EPI, false, true>(a, grid);
        else launch_stream<2, 2, NW, EPI, false, true>(a, grid);
    } else {
        if (TB == 1) launch_stream<4, 1, NW, EPI, false, true>(a, grid);
        else launch_stream<4, 2, NW, EPI, false, true>(a, grid);
    }
}

}  // namespace

void launch_gemm_experts(const B16Weight& w, int experts, const __half* act, const ExpertRows& rows, const GemmEpilogue& epi, int prof_cls) {
    if (rows.capacity <= 0) return;
    ensure_init();
    const bool dense = rows.pad >= 64;
    if (w.K % 32 || w.N % 32 || experts < 1 || rows.capacity % rows.pad || !(rows.pad == 16 || rows.pad == 32 || rows.pad == 64 || rows.pad == 128))
        NVLLM_FATAL("expert projection: [%d, %d] on %d rows in groups of %d is not supported", w.N, w.K, rows.capacity, rows.pad);
    GemmArgs a{};
    a.W = w.tiles;
    a.Kb = w.K / 32;
    a.nb_stride = (long)a.Kb * TILE_HALVES;
    a.NB = w.N / 16;
    a.expert_stride = a.NB * a.nb_stride;
    a.A = act;
    a.Tb = rows.capacity / 16;
    a.N = w.N;
    a.T = rows.capacity;
    a.act_Kb = a.Kb;
    a.block_expert = rows.block_expert;
    a.source = rows.source;
    a.counters = gemm_tile_counters();
    a.e = epi;
    const double touched = std::min(experts, rows.live);   // matrices read
    const double bytes = touched * w.N * w.K * 2.0 + (double)rows.live * w.K * 2.0 + (double)rows.live * w.N * (epi.kind == GemmEpilogue::F32 ? 4.0 : 1.0);
    const double flops = 2.0 * rows.live * (double)w.N * w.K;
    if (epi.kind == GemmEpilogue::SWIGLU_A16) {
        if (w.N % 64) NVLLM_FATAL("expert projection: a hidden width of %d is not padded to 32", w.N / 2);
        a.e.Kb_out = w.N / 64;
        launch_experts_kind<GemmEpilogue::SWIGLU_A16>(a, rows.pad, dense, bytes, flops, prof_cls);
    } else if (epi.kind == GemmEpilogue::F32) {
        launch_experts_kind<GemmEpilogue::F32>(a, rows.pad, dense, bytes, flops, prof_cls);
    } else {
        NVLLM_FATAL("this epilogue has no form for experts");
    }
}

void launch_gemm_b16(const B16Weight& w, const __half* act, int T, const GemmEpilogue& epi, int prof_cls, const LatentKvRider* ride) {
    if (T <= 0) return;
    ensure_init();
    if (w.K % 32) NVLLM_FATAL("bf16 projection: the input width %d is not padded to 32", w.K);
    const bool grp = w.groups > 1;
    GemmArgs a{};
    a.W = w.tiles;
    a.Kb = w.K / 32;
    a.nb_stride = (long)a.Kb * TILE_HALVES;
    a.NB = cdiv(w.N, 16);
    a.A = act;
    a.Tb = cdiv(T, 16);
    a.N = w.N;
    a.T = T;
    a.act_Kb = a.Kb * w.groups;
    if (grp) {
        if (w.N % w.groups || w.N / w.groups % 16) NVLLM_FATAL("block-diagonal projection: %d rows do not make %d groups of whole row blocks", w.N, w.groups);
        a.group_nb = a.NB / w.groups;
    }
    a.counters = gemm_tile_counters();
    a.e = epi;
    if (ride) {
        if (epi.kind != GemmEpilogue::LATENT_Q) NVLLM_FATAL("cache rows ride on the query projection only");
        a.ride = *ride;
    }
    auto need32 = [&](int n, const char* what) {
        if (n % 32) NVLLM_FATAL("bf16 projection: %s of %d is not padded to 32", what, n);
    };
    double out_bytes = (double)T * w.N * 2.0;
    switch (epi.kind) {
        case GemmEpilogue::F32: out_bytes = (double)T * w.N * 4.0; break;
        case GemmEpilogue::SWIGLU_A16:
            need32(w.N / 2, "a hidden width");
            a.e.Kb_out = w.N / 64;
            out_bytes = (double)T * w.N;
            break;
        case GemmEpilogue::TILE_B16: need32(w.N, "an output width"); a.e.Kb_out = w.N / 32; break;
        case GemmEpilogue::RESID_B16:
            need32(w.N, "a residual width");
            a.e.Kb_out = w.N / 32;
            out_bytes = (double)T * w.N * 10.0;
            break;
        case GemmEpilogue::LATENT_IN: need32(epi.latent_q, "a query latent"); a.e.Kb_out = epi.latent_q / 32; break;
        case GemmEpilogue::LATENT_Q: need32(epi.q_plain, "a query width"); a.e.Kb_out = epi.q_plain / 32; break;
        case GemmEpilogue::HYPER_2:
        case GemmEpilogue::HYPER_4:
            need32(w.N, "a residual width");
            a.e.Kb_out = w.N / 32;
            out_bytes = (double)T * w.N * (8.0 * epi.streams + 2.0);
            break;
        default: break;
    }
    const double bytes = (double)w.N * w.K * 2.0 + (double)T * w.K * w.groups * 2.0 + out_bytes;
    const double flops = 2.0 * T * (double)w.N * w.K;
    switch (epi.kind) {
        case GemmEpilogue::F32: launch_kind<GemmEpilogue::F32, false>(a, prof_cls, bytes, flops); break;
        case GemmEpilogue::SWIGLU_A16: launch_kind<GemmEpilogue::SWIGLU_A16, false>(a, prof_cls, bytes, flops); break;
        case GemmEpilogue::TILE_B16:
            if (grp) launch_kind<GemmEpilogue::TILE_B16, true>(a, prof_cls, bytes, flops);
            else launch_kind<GemmEpilogue::TILE_B16, false>(a, prof_cls, bytes, flops);
            break;
        case GemmEpilogue::ROWS_B16:
            if (grp) launch_kind<GemmEpilogue::ROWS_B16, true>(a, prof_cls, bytes, flops);
            else launch_kind<GemmEpilogue::ROWS_B16, false>(a, prof_cls, bytes, flops);
            break;
        case GemmEpilogue::LATENT_IN: launch_kind<GemmEpilogue::LATENT_IN, false>(a, prof_cls, bytes, flops); break;
        case GemmEpilogue::LATENT_Q: launch_kind<GemmEpilogue::LATENT_Q, false>(a, prof_cls, bytes, flops); break;
        case GemmEpilogue::RESID_B16: launch_kind<GemmEpilogue::RESID_B16, false>(a, prof_cls, bytes, flops); break;
        case GemmEpilogue::HYPER_2: launch_kind<GemmEpilogue::HYPER_2, false>(a, prof_cls, bytes, flops); break;
        case GemmEpilogue::HYPER_4: launch_kind<GemmEpilogue::HYPER_4, false>(a, prof_cls, bytes, flops); break;
        default: NVLLM_FATAL("this epilogue belongs to fp16 models");
    }
}

}  // namespace nvllm
