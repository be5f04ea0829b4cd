// gemm_prefill.hip -- launches of the dense-tile projection kernel (gemm_prefill_tile.h) for fp16 models.
#include "gemm_prefill_tile.h"

namespace nvllm {

namespace {

template <int FW, int KG, int EPI, typename KVT, int TW>
void launch_one(const GemmArgs& a, int tiles_n, int tiles_t, int nbuf, int split_from) {
    using G = PfGeom<FW, KG, 2, TW>;
    const size_t shmem = (size_t)(G::RINV_HALVES + (nbuf & 255) * G::STAGE_HALVES) * sizeof(__half);   // (a diagnostic build keeps flags above bit 8)
    static size_t allowed = 0;   // per instantiation: the largest dynamic LDS size enabled so far
    if (shmem > allowed) {
        HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_gemm_prefill<FW, KG, EPI, KVT, 2, TW>),
                                      hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem));
        allowed = shmem;
    }
    NVLLM_LAUNCH((k_gemm_prefill<FW, KG, EPI, KVT, 2, TW>), dim3(split_from + (tiles_n * tiles_t - split_from) * a.ksplit), dim3(256 * KG), shmem, a,
                 tiles_n, tiles_t, nbuf, split_from);
}

template <int FW, int KG, typename KVT, int TW = 4>
void launch_pf(const GemmArgs& a, int tiles_n, int tiles_t, int nbuf, int split_from) {
    switch (a.e.kind) {
        case GemmEpilogue::F32: launch_one<FW, KG, GemmEpilogue::F32, KVT, TW>(a, tiles_n, tiles_t, nbuf, split_from); break;
        case GemmEpilogue::SWIGLU_A16: launch_one<FW, KG, GemmEpilogue::SWIGLU_A16, KVT, TW>(a, tiles_n, tiles_t, nbuf, split_from); break;
        case GemmEpilogue::RESID_A16: launch_one<FW, KG, GemmEpilogue::RESID_A16, KVT, TW>(a, tiles_n, tiles_t, nbuf, split_from); break;
        default: launch_one<FW, KG, GemmEpilogue::ROPE_KV, KVT, TW>(a, tiles_n, tiles_t, nbuf, split_from); break;
    }
}

}  // namespace

// `a` is complete but for the K split: a.ksplit > 1 asks for every tile to be cut that many ways
// (wide decode batches; slab and counters are the library's own), otherwise none is.
void launch_gemm_prefill(GemmArgs a) {
    const int cus = rt().num_cus;
    static const int shape_env = getenv("NVLLM_GEMM_PREFILL_SHAPE") ? atoi(getenv("NVLLM_GEMM_PREFILL_SHAPE")) : 0;   // 2: 8 waves, 3: 4 waves
    static const int ring_env = getenv("NVLLM_GEMM_PREFILL_RING") ? atoi(getenv("NVLLM_GEMM_PREFILL_RING")) : 0;
    static const int ksplit_env = getenv("NVLLM_GEMM_PREFILL_KSPLIT") ? atoi(getenv("NVLLM_GEMM_PREFILL_KSPLIT")) : 0;   // cut every tile this many ways
    static const int tw_env = getenv("NVLLM_GEMM_PREFILL_TW") ? atoi(getenv("NVLLM_GEMM_PREFILL_TW")) : 0;               // token blocks per wave: 4, 3, 2
#ifdef NVLLM_PF_ABLATE
    static const int ablate_env = getenv("NVLLM_PF_ABLATE") ? atoi(getenv("NVLLM_PF_ABLATE")) << 8 : 0;
#else
    constexpr int ablate_env = 0;
#endif
    const bool kv16 = a.e.kind == GemmEpilogue::ROPE_KV && a.e.kv_elem_bytes == 2;
    int want_split = a.ksplit > 1 ? a.ksplit : 1;
    if (ksplit_env > 1) want_split = ksplit_env;
    const int tiles_n = cdiv(a.NB, 8);
    // 128-feature tiles, 128, 96 or 64 tokens high.  A launch runs in rounds of co-resident
    // workgroups (three per CU with two ring buffers) and a partly filled last round costs
    // nearly a full one, so the height is the one whose rounds waste least: 128 tokens unless
    // 96 needs fewer round-heights (TinyLlama's gate/up at 1,591 tokens: 1,144 tiles = 1.5 rounds
    // against 1,496 = 1.95 rounds of 3/4 the height, 150 -> 147 us; a projection half as wide
    // 88 -> 74 us).  Projections whose 128-token tiles would not even give every CU one
    // workgroup (wo, w_down: 208) take 64-token tiles, two workgroups per CU with three buffers
    // (35 -> 32 and 80 -> 77 us against the eight-wave form, which wide decode batches keep:
    // there every weight tile must still be read only once).
    const int tiles4 = tiles_n * cdiv(a.Tb, 8);
    const bool wide_decode = a.Tb <= 8 || want_split > 1;
    int shape = wide_decode && tiles4 * want_split <= cus ? 2 : 3;
    if (shape_env == 2 || shape_env == 3) shape = shape_env;
    int tw = 4;
    if (shape == 3 && !wide_decode) {
        if (tiles4 <= cus) {
            tw = 2;
        } else if (tiles_n * cdiv(a.Tb, 4) <= 2 * cus) {
            // a few more 128-token tiles than CUs: some CUs would run two tall tiles in a row (or side by side)
            // while the rest run one; 64-token tiles give every CU at most two short ones (TinyLlama's
            // q/k/v at 1,591 tokens: 340 tiles of 96 tokens -> 500 of 64, 52 -> 47 us)
            tw = 2;
        } else {
            const int slots = 3 * cus;
            const int tiles3 = tiles_n * cdiv(a.Tb, 6);
            if (cdiv(tiles3, slots) * 3 < cdiv(tiles4, slots) * 4) tw = 3;
        }
    }
    if (shape == 3 && tw_env >= 2 && tw_env <= 4) tw = tw_env;
    static const int tw_qkv_env = getenv("NVLLM_GEMM_PREFILL_TW_QKV") ? atoi(getenv("NVLLM_GEMM_PREFILL_TW_QKV")) : 0;   // the same for q/k/v only
    if (shape == 3 && a.e.kind == GemmEpilogue::ROPE_KV && tw_qkv_env >= 2 && tw_qkv_env <= 4) tw = tw_qkv_env;
    const int tiles_t = cdiv(a.Tb, 2 * tw);
    const int total = tiles_n * tiles_t;
    int nbuf;
    if (shape == 2) {   // 48 KiB per stage (two K-steps); a ring of three fills the LDS
        nbuf = 3;
        if (ring_env >= 2 && ring_env <= 3) nbuf = ring_env;
    } else {            // 24 KiB per stage (20, 16 for the lower tiles); three waves per SIMD fit the register file
        const int per_cu = cdiv(total * want_split, cus);
        nbuf = per_cu >= 3 ? 2 : (per_cu == 2 ? 3 : 5);
        if (ring_env >= 2 && ring_env <= 5) nbuf = ring_env;
    }
    // ---- the K split
    int split_from = total;
    a.ksplit = 1;
    a.kb_per_split = a.Kb;
    if (want_split > 1) {
        const int kg = shape == 2 ? 2 : 1;
        a.kb_per_split = cdiv(cdiv(a.Kb, want_split), kg) * kg;   // whole stages per slice
        a.ksplit = cdiv(a.Kb, a.kb_per_split);
        if (a.ksplit > 1 && total <= (1 << 16)) {   // (the counter array's size, gemm.hip)
            split_from = 0;
            a.slab = (float*)ws_get(WS_SLAB, (size_t)total * a.ksplit * 128 * (32 * tw) * sizeof(float));
        } else {
            a.ksplit = 1;
            a.kb_per_split = a.Kb;
        }
    }
    const int nb = nbuf | ablate_env;
    if (shape == 2) {
        if (kv16) launch_pf<4, 2, __half>(a, tiles_n, tiles_t, nb, split_from);
        else launch_pf<4, 2, float>(a, tiles_n, tiles_t, nb, split_from);
    } else if (tw == 4) {
        if (kv16) launch_pf<4, 1, __half, 4>(a, tiles_n, tiles_t, nb, split_from);
        else launch_pf<4, 1, float, 4>(a, tiles_n, tiles_t, nb, split_from);
    } else if (tw == 3) {
        if (kv16) launch_pf<4, 1, __half, 3>(a, tiles_n, tiles_t, nb, split_from);
        else launch_pf<4, 1, float, 3>(a, tiles_n, tiles_t, nb, split_from);
    } else {
        if (kv16) launch_pf<4, 1, __half, 2>(a, tiles_n, tiles_t, nb, split_from);
        else launch_pf<4, 1, float, 2>(a, tiles_n, tiles_t, nb, split_from);
    }
}

}  // namespace nvllm
