// ops_api.hip -- the operator entry points of include/ops.h on top of the kernel
// launchers: argument checking, host->HBM staging of the integer arrays and block
// tables, and the host-side KV block allocator.
#include <algorithm>
#include <cstring>
#include <unordered_map>
#include <vector>

#include "latent_attention.h"
#include "model_dir.h"
#include "nvllm_internal.h"
#include "step_arrays.h"

namespace nvllm {

// Pools created by init_kv_cache_manager, keyed by pool_k: element size and the
// geometry the reference passes again with every call.
struct PoolInfo {
    int elem_bytes;
    int n_layers, n_kv_heads, head_dim;
};
// Block pools of models that lay them out themselves: bytes behind pool_k.
static std::unordered_map<const void*, size_t>& block_pools() {
    static std::unordered_map<const void*, size_t> m;
    return m;
}
size_t block_pool_bytes(const KVCacheManager* mgr) {
    auto it = block_pools().find(mgr->pool_k);
    return it == block_pools().end() ? 0 : it->second;
}

static std::unordered_map<const void*, PoolInfo>& pools() {
    static std::unordered_map<const void*, PoolInfo> m;
    return m;
}

KvPoolView pool_view(const KVCacheManager* mgr, int n_kv_heads, int head_dim) {
    KvPoolView v;
    v.k = mgr->pool_k;
    v.v = mgr->pool_v;
    auto it = pools().find(mgr->pool_k);
    v.elem_bytes = it == pools().end() ? 4 : it->second.elem_bytes;
    v.block_size = mgr->block_size;
    v.num_blocks = mgr->num_blocks;
    v.layer_stride = (long)mgr->num_blocks * mgr->block_size * n_kv_heads * head_dim;
    return v;
}

// Flatten what the kernels need from the host-side batch description into one
// pinned region and upload it with a single copy.
StepArrays stage_step(const int* tokens, const int* pos_arr, const int* seq_ids, int T,
                      const int* output_indices, int B, BlockTable** tables, const BlockTable* single,
                      int pos0, int block_size, int attn_ct, const int* token_src, bool multi_first, bool spans, int chunk_len) {
    StepArrays s{};
    s.T = T;
    s.B = B;
    int n_seqs = 0;
    int max_pos = 0;
    for (int t = 0; t < T; t++) {
        const int p = pos_arr ? pos_arr[t] : pos0 + t;
        if (p > max_pos) max_pos = p;
        if (seq_ids && seq_ids[t] + 1 > n_seqs) n_seqs = seq_ids[t] + 1;
    }
    if (!seq_ids) n_seqs = 1;
    s.max_pos = max_pos;
    s.n_seqs = n_seqs;
    // blocks each sequence needs for this call = (largest position / block_size) + 1
    std::vector<int> need(n_seqs, 0);
    s.write_limit = T;
    if (tables || single) {
        for (int t = 0; t < T; t++) {
            const int p = pos_arr ? pos_arr[t] : pos0 + t;
            const int sid = seq_ids ? seq_ids[t] : 0;
            const int lb = p / block_size;
            const BlockTable* bt = single ? single : tables[sid];
            // never read the caller's table past its num_blocks entries
            const int have = lb + 1 < bt->num_blocks ? lb + 1 : bt->num_blocks;
            if (have > need[sid]) need[sid] = have;
            if (lb >= bt->num_blocks) s.table_short = true;
            if (s.write_limit == T && lb >= bt->num_blocks) {
                // reference attention.c:159-162 (and :123-126): report and stop writing
                printf("Error: Block table too small! logical_idx=%d, num_blocks=%d\n", lb, bt->num_blocks);
                s.write_limit = t;
            }
        }
    }
    size_t total_tbl = 0;
    for (int i = 0; i < n_seqs; i++) total_tbl += (size_t)need[i];
    std::vector<int> tbl_off(n_seqs, 0);
    for (int i = 1; i < n_seqs; i++) tbl_off[i] = tbl_off[i - 1] + need[i - 1];
    // attention work items: (first token, token count, last position, offset of the
    // sequence's block table) -- everything a wave needs in one 16-byte load
    std::vector<int> runs;
    s.kv_positions = 0;
    if (attn_ct > 0) {
        auto pos_of = [&](int t) { return pos_arr ? pos_arr[t] : pos0 + t; };
        auto seq_of = [&](int t) { return seq_ids ? seq_ids[t] : 0; };
        for (int t = 0; t < T;) {
            int n = 1;
            while (t + n < T && n < attn_ct && seq_of(t + n) == seq_of(t) && pos_of(t + n) == pos_of(t + n - 1) + 1) n++;
            runs.push_back(t);
            runs.push_back(n);
            runs.push_back(pos_of(t + n - 1));
            runs.push_back(tbl_off[seq_of(t)]);
            s.kv_positions += pos_of(t + n - 1) + 1;
            for (int i = 0; i < n; i++) s.qk_pairs += pos_of(t + i) + 1;
            if (n > s.max_run) s.max_run = n;
            for (int tb = t >> 4; tb <= (t + n - 1) >> 4; tb++)
                if (tb < 4) s.runs_in_tb[tb]++;
            t += n;
        }
        if (multi_first) {
            std::vector<int> singles;
            size_t keep = 0;
            for (size_t i = 0; i < runs.size(); i += 4) {
                if (runs[i + 1] == 1) {
                    singles.insert(singles.end(), runs.begin() + (long)i, runs.begin() + (long)i + 4);
                    s.kv_rows_single += runs[i + 2] + 1;
                } else {
                    std::copy(runs.begin() + (long)i, runs.begin() + (long)i + 4, runs.begin() + (long)keep);
                    keep += 4;
                }
            }
            std::copy(singles.begin(), singles.end(), runs.begin() + (long)keep);
            s.n_multi = (int)(keep / 4);
        }
    }
    if (attn_ct > 0) {
        std::vector<int> seen_to(n_seqs, 0);
        for (int t = 0; t < T; t++) {
            int& last = seen_to[seq_ids ? seq_ids[t] : 0];
            const int p = (pos_arr ? pos_arr[t] : pos0 + t) + 1;
            if (p > last) last = p;
        }
        for (int v : seen_to) s.kv_rows += v;
    }
    {   // does any sequence occur twice?
        std::vector<char> seen(n_seqs, 0);
        s.one_token_per_seq = true;
        for (int t = 0; t < T && s.one_token_per_seq; t++) {
            const int sid = seq_ids ? seq_ids[t] : 0;
            if (seen[sid]) s.one_token_per_seq = false;
            seen[sid] = 1;
        }
    }
    s.n_runs = (int)runs.size() / 4;
    std::vector<int> span, span_of;
    if (spans) {
        auto pos_of = [&](int t) { return pos_arr ? pos_arr[t] : pos0 + t; };
        auto seq_of = [&](int t) { return seq_ids ? seq_ids[t] : 0; };
        std::vector<char> seen(n_seqs, 0);
        span_of.resize(T);
        for (int pass = 0; pass < 2; pass++)   // portions of several tokens, then single tokens
            for (int t = 0; t < T;) {
                int n = 1;
                while (t + n < T && seq_of(t + n) == seq_of(t) && pos_of(t + n) == pos_of(t + n - 1) + 1) n++;
                if ((n > 1) == (pass == 0)) {
                    if (seen[seq_of(t)]) s.seq_split = true;
                    seen[seq_of(t)] = 1;
                    for (int i = 0; i < n; i++) span_of[t + i] = (int)span.size() / 4;
                    span.insert(span.end(), {t, n, pos_of(t), seq_of(t)});
                    if (n > s.max_span) s.max_span = n;
                }
                t += n;
                if (pass == 0) s.n_spans_multi = (int)span.size() / 4;
            }
        s.n_spans = (int)span.size() / 4;
        s.host_spans = span;
    }
    std::vector<int> chunks, first_chunk;
    if (spans && chunk_len > 0) {
        s.chunk_len = chunk_len;
        for (int i = 0; i < s.n_spans_multi; i++) {
            first_chunk.push_back((int)chunks.size() / 2);
            for (int c = 0; c * chunk_len < span[4 * i + 1]; c++) chunks.insert(chunks.end(), {i, c});
        }
        s.n_chunks = (int)chunks.size() / 2;
    }
    // where each token's K/V row goes: resolves position -> (block table entry, slot) on
    // the host so the kernels that store K/V need one load instead of a chain of three
    std::vector<int> kv_row;
    if (tables || single) {
        kv_row.resize(T);
        for (int t = 0; t < T; t++) {
            const int p = pos_arr ? pos_arr[t] : pos0 + t;
            const BlockTable* bt = single ? single : tables[seq_ids ? seq_ids[t] : 0];
            kv_row[t] = t < s.write_limit ? bt->block_indices[p / block_size] * block_size + p % block_size : -1;
        }
    }
    const size_t n_ints = (size_t)(tokens ? T : 0) + (token_src ? T : 0) + (pos_arr ? T : 0) + (seq_ids ? T : 0) + kv_row.size() +
                          (output_indices ? B : 0) + n_seqs + total_tbl + runs.size() + span.size() + span_of.size() + chunks.size() + first_chunk.size() + 64;
    int* host = pinned_ints(n_ints);
    int* dev = (int*)ws_get(WS_STEP, n_ints * sizeof(int));
    size_t o = 0;
    auto put = [&](const int* src, size_t n) -> int* {
        if (!src || n == 0) return nullptr;
        memcpy(host + o, src, n * sizeof(int));
        int* d = dev + o;
        o += n;
        return d;
    };
    s.d_tokens = put(tokens, T);
    s.d_tok_src = put(token_src, T);
    s.d_pos = put(pos_arr, T);
    s.d_seq = put(seq_ids, T);
    s.d_out_idx = put(output_indices, B);
    s.d_kv_row = kv_row.empty() ? nullptr : put(kv_row.data(), kv_row.size());
    s.d_tbl_off = nullptr;
    s.d_tables = nullptr;
    if (tables || single) {
        s.d_tbl_off = dev + o;
        int* off_host = host + o;
        o += n_seqs;
        s.d_tables = dev + o;
        size_t run = 0;
        for (int i = 0; i < n_seqs; i++) {
            off_host[i] = tbl_off[i];
            if (need[i] > 0) {
                const BlockTable* bt = single ? single : tables[i];
                memcpy(host + o + run, bt->block_indices, (size_t)need[i] * sizeof(int));
                run += (size_t)need[i];
            }
        }
        o += run;
    }
    o = (o + 3) & ~(size_t)3;  // int4 alignment
    s.d_runs = runs.empty() ? nullptr : put(runs.data(), runs.size());
    s.d_spans = span.empty() ? nullptr : put(span.data(), span.size());
    s.d_chunks = chunks.empty() ? nullptr : put(chunks.data(), chunks.size());   // (pairs, behind quadruples)
    s.d_first_chunk = first_chunk.empty() ? nullptr : put(first_chunk.data(), first_chunk.size());
    s.d_span_of = span_of.empty() ? nullptr : put(span_of.data(), span_of.size());
    if (o > 0) {
        static const int by_kernel = getenv("NVLLM_STAGE_COPY") ? atoi(getenv("NVLLM_STAGE_COPY")) == 0 : 1;
        if (by_kernel && o <= (1u << 16)) launch_copy_ints(dev, host, o);   // small: a kernel reads the pinned region itself
        else HIP_CHECK(hipMemcpyAsync(dev, host, o * sizeof(int), hipMemcpyHostToDevice, rt().stream));
    }
    return s;
}

}  // namespace nvllm

using namespace nvllm;

extern "C" {

// ------------------------------------------------------------- dense ops
void rms_norm(float* o, float* x, float* weight, int size, int num_tokens, float eps) {
    ensure_init();
    launch_rmsnorm_f32(o, x, weight, size, num_tokens, eps);
}

void matmul(float* out, float* in, float* weight, int num_tokens, int in_dim, int out_dim) {
    ensure_init();
    const WeightEntry* w = find_weight(weight);
    if (!w) {  // a plain fp32 [out_dim, in_dim] device buffer
        launch_matmul_f32w(out, in, weight, num_tokens, in_dim, out_dim);
        return;
    }
    if (w->rowmajor && !w->tiles) NVLLM_FATAL("matmul: the embedding table handle is not a projection weight");
    if (w->K != in_dim || w->N != out_dim)
        NVLLM_FATAL("matmul: handle is [%d, %d] but the call says [%d, %d]", w->N, w->K, out_dim, in_dim);
    __half* a16 = (__half*)ws_get(WS_MISC, a16_halves(num_tokens, in_dim) * sizeof(__half));
    launch_pack_a16(a16, in, num_tokens, in_dim);
    GemmEpilogue e;
    e.kind = GemmEpilogue::F32;
    e.out = out;
    e.ldo = out_dim;
    launch_gemm(*w, w->tiles, out_dim, a16, num_tokens, e, 0, PC_GEMM_OTHER);
}

void apply_rope(float* q, float* k, int pos, float theta, int head_dim, int num_tokens, int n_heads,
                int n_kv_heads) {
    ensure_init();
    if (num_tokens <= 0) return;
    const float2* tab = rope_table(theta, head_dim, pos + num_tokens);
    launch_rope(q, k, nullptr, pos, tab, num_tokens, n_heads, n_kv_heads, head_dim);
}

void apply_rope_batch(float* q, float* k, int* pos_arr, float theta, int head_dim, int num_tokens,
                      int n_heads, int n_kv_heads) {
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, pos_arr, nullptr, num_tokens, nullptr, 0, nullptr, nullptr, 0, 1);
    const float2* tab = rope_table(theta, head_dim, s.max_pos + 1);
    launch_rope(q, k, s.d_pos, 0, tab, num_tokens, n_heads, n_kv_heads, head_dim);
}

void swiglu(float* hb, float* h_gate, float* h_up, int hidden_dim, int num_tokens) {
    ensure_init();
    launch_swiglu(hb, h_gate, h_up, (long)hidden_dim * num_tokens);
}

void softmax(float* x, int size) {
    ensure_init();
    launch_softmax(x, size);
}

void accum(float* a, float* b, int size) {
    ensure_init();
    launch_accum(a, b, size);
}

// ------------------------------------------------------- KV block pool
// Host bookkeeping exactly as reference memory.c:8-82; the two pools are HBM.
static void init_free_stack(KVCacheManager* mgr, int block_size, int num_blocks) {
    mgr->block_size = block_size;
    mgr->num_blocks = num_blocks;
    mgr->free_blocks_count = num_blocks;
    mgr->free_block_indices = (int*)malloc((size_t)num_blocks * sizeof(int));
    for (int slot = 0; slot < num_blocks; slot++) mgr->free_block_indices[slot] = num_blocks - 1 - slot;
}

void init_kv_cache_manager(KVCacheManager* mgr, int block_size, int num_blocks, int n_layers,
                           int n_kv_heads, int head_dim) {
    ensure_init();
    // a driver that knows only this entry point, with a folder model loaded: the pool is that model's own
    if (DirModel* m = current_dir_model(n_layers, n_kv_heads, head_dim)) {
        m->init_kv(mgr, block_size, num_blocks);
        return;
    }
    // tensor parallelism: the caller passes the model's head count (it sizes the pool from Config);
    // this process stores and reads the K/V of its own heads only
    if (tp().active && tp().world > 1) {
        if (n_kv_heads % tp().world) NVLLM_FATAL("%d kv heads do not divide over %d tensor-parallel ranks", n_kv_heads, tp().world);
        n_kv_heads /= tp().world;
    }
    init_free_stack(mgr, block_size, num_blocks);
    const size_t elems = (size_t)n_layers * num_blocks * block_size * n_kv_heads * head_dim;
    const int eb = rt().kv_elem_bytes;
    if (eb == 2 && (block_size != KV16_PAGE_KEYS || head_dim % 16 != 0))
        NVLLM_FATAL("an fp16 KV pool stores 16-position pages: block_size must be 16 (got %d) and head_dim a "
                    "multiple of 16 (got %d)", block_size, head_dim);
    void *pk = nullptr, *pv = nullptr;
    if (device_malloc(&pk, elems * eb) != 0 || device_malloc(&pv, elems * eb) != 0)
        NVLLM_FATAL("cannot allocate the KV pool (2 x %zu bytes)", elems * eb);
    // fresh pool reads as zeros, so attention over never-written rows is at least defined
    HIP_CHECK(hipMemsetAsync(pk, 0, elems * eb, rt().stream));
    HIP_CHECK(hipMemsetAsync(pv, 0, elems * eb, rt().stream));
    mgr->pool_k = (float*)pk;
    mgr->pool_v = (float*)pv;
    pools()[pk] = PoolInfo{eb, n_layers, n_kv_heads, head_dim};
}

}  // extern "C"
void nvllm::init_block_pool(KVCacheManager* mgr, int block_size, int num_blocks, size_t bytes) {
    ensure_init();
    init_free_stack(mgr, block_size, num_blocks);
    void* pool = nullptr;
    if (device_malloc(&pool, bytes) != 0) NVLLM_FATAL("cannot allocate the block pool (%zu bytes)", bytes);
    HIP_CHECK(hipMemsetAsync(pool, 0, bytes, rt().stream));   // rows nobody has written are finite
    mgr->pool_k = (float*)pool;
    mgr->pool_v = nullptr;
    block_pools()[pool] = bytes;
}
extern "C" {

void free_kv_cache_manager(KVCacheManager* mgr) {
    if (mgr->free_block_indices) free(mgr->free_block_indices);
    mgr->free_block_indices = nullptr;
    if (mgr->pool_k) {
        pools().erase(mgr->pool_k);
        block_pools().erase(mgr->pool_k);
        device_free(mgr->pool_k);
    }
    if (mgr->pool_v) device_free(mgr->pool_v);
    mgr->pool_k = mgr->pool_v = nullptr;
}

int alloc_block(KVCacheManager* mgr) {
    if (mgr->free_blocks_count <= 0) return -1;
    mgr->free_blocks_count -= 1;
    return mgr->free_block_indices[mgr->free_blocks_count];
}

void free_block(KVCacheManager* mgr, int block_idx) {
    if (mgr->free_blocks_count >= mgr->num_blocks) return;
    mgr->free_block_indices[mgr->free_blocks_count] = block_idx;
    mgr->free_blocks_count += 1;
}

long get_physical_offset(KVCacheManager* mgr, int layer, int block_idx, int block_offset, int n_kv_heads,
                         int head_dim) {
    const long row = (long)n_kv_heads * head_dim;
    const long blk = (long)mgr->block_size * row;
    const long lay = (long)mgr->num_blocks * blk;
    return (long)layer * lay + (long)block_idx * blk + (long)block_offset * row;
}

// --------------------------------------------------------------- KV writes
static KvPoolView contiguous_view(float* kc, float* vc, int max_seq_len, int n_kv_heads, int head_dim) {
    KvPoolView v;
    v.k = kc;
    v.v = vc;
    v.elem_bytes = 4;
    v.block_size = 1;
    v.num_blocks = max_seq_len;
    v.layer_stride = (long)max_seq_len * n_kv_heads * head_dim;
    return v;
}

void update_kv_cache(float* key_cache, float* value_cache, float* k, float* v, int layer, int pos,
                     int max_seq_len, int n_kv_heads, int head_dim, int num_tokens) {
    ensure_init();
    const KvPoolView pv = contiguous_view(key_cache, value_cache, max_seq_len, n_kv_heads, head_dim);
    launch_kv_write(k, v, nullptr, pos, nullptr, nullptr, nullptr, pv, layer, num_tokens, n_kv_heads, head_dim);
}

void update_kv_cache_paged(KVCacheManager* mgr, BlockTable* block_table, float* k, float* v, int layer,
                           int pos, int n_kv_heads, int head_dim, int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, nullptr, nullptr, num_tokens, nullptr, 0, nullptr, block_table, pos,
                              mgr->block_size);
    launch_kv_write(k, v, nullptr, pos, nullptr, s.d_tbl_off, s.d_tables, pool_view(mgr, n_kv_heads, head_dim),
                    layer, s.write_limit, n_kv_heads, head_dim);
}

void update_kv_cache_paged_batch(KVCacheManager* mgr, BlockTable** block_tables, int* seq_ids, float* k,
                                 float* v, int layer, int* pos_arr, int n_kv_heads, int head_dim,
                                 int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, pos_arr, seq_ids, num_tokens, nullptr, 0, block_tables, nullptr, 0,
                              mgr->block_size);
    launch_kv_write(k, v, s.d_pos, 0, s.d_seq, s.d_tbl_off, s.d_tables, pool_view(mgr, n_kv_heads, head_dim),
                    layer, s.write_limit, n_kv_heads, head_dim);
}

// --------------------------------------------------------------- attention
void multi_head_attention(float* out, float* q, float* key_cache, float* value_cache, float* att, int layer,
                          int pos, int max_seq_len, int n_heads, int n_kv_heads, int head_dim,
                          int num_tokens) {
    (void)att;
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, nullptr, nullptr, num_tokens, nullptr, 0, nullptr, nullptr, pos, 16,
                              attn_tokens_per_item(n_heads, n_kv_heads));
    AttnArgs a{};
    a.q = q;
    a.out_f32 = out;
    a.pool = contiguous_view(key_cache, value_cache, max_seq_len, n_kv_heads, head_dim);
    a.layer = layer;
    a.T = num_tokens;
    a.H = n_heads;
    a.KVH = n_kv_heads;
    a.hd = head_dim;
    a.max_pos = s.max_pos;
    a.runs = s.d_runs;
    a.n_runs = s.n_runs;
    a.kv_positions = s.kv_positions;
    launch_paged_attention(a);
}

void paged_attention(float* out, float* q, KVCacheManager* mgr, BlockTable* block_table, float* att,
                     int layer, int pos, int max_seq_len, int n_heads, int n_kv_heads, int head_dim,
                     int num_tokens) {
    (void)att;
    (void)max_seq_len;
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, nullptr, nullptr, num_tokens, nullptr, 0, nullptr, block_table, pos,
                              mgr->block_size, attn_tokens_per_item(n_heads, n_kv_heads));
    // the reference reads block ids past the table here (attention.c:285 has no bounds check);
    // on the GPU that would be a wild read of the pool, so it ends the process instead
    if (s.table_short) NVLLM_FATAL("paged attention: a position lies beyond its sequence's block table");
    AttnArgs a{};
    a.q = q;
    a.out_f32 = out;
    a.pool = pool_view(mgr, n_kv_heads, head_dim);
    a.layer = layer;
    a.tables = s.d_tables;
    a.T = num_tokens;
    a.H = n_heads;
    a.KVH = n_kv_heads;
    a.hd = head_dim;
    a.max_pos = s.max_pos;
    a.runs = s.d_runs;
    a.n_runs = s.n_runs;
    a.kv_positions = s.kv_positions;
    launch_paged_attention(a);
}

void paged_attention_batch(float* out, float* q, KVCacheManager* mgr, BlockTable** block_tables, int* seq_ids,
                           float* att, int layer, int* pos_arr, int max_seq_len, int n_heads, int n_kv_heads,
                           int head_dim, int num_tokens) {
    (void)att;
    (void)max_seq_len;
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, pos_arr, seq_ids, num_tokens, nullptr, 0, block_tables, nullptr, 0,
                              mgr->block_size, attn_tokens_per_item(n_heads, n_kv_heads));
    // the reference reads block ids past the table here (attention.c:285 has no bounds check);
    // on the GPU that would be a wild read of the pool, so it ends the process instead
    if (s.table_short) NVLLM_FATAL("paged attention: a position lies beyond its sequence's block table");
    AttnArgs a{};
    a.q = q;
    a.out_f32 = out;
    a.pool = pool_view(mgr, n_kv_heads, head_dim);
    a.layer = layer;
    a.tables = s.d_tables;
    a.T = num_tokens;
    a.H = n_heads;
    a.KVH = n_kv_heads;
    a.hd = head_dim;
    a.max_pos = s.max_pos;
    a.runs = s.d_runs;
    a.n_runs = s.n_runs;
    a.kv_positions = s.kv_positions;
    launch_paged_attention(a);
}

}  // extern "C"

// -------------------------------------------------- operators of folder models (include/nvllm.h)
extern "C" {

void nvllm_hyper_step(float* x, const float* y, const float* bias, const float* scale, const float* record, const float* norm_w,
                      const float* norm_b, float* out, int streams, int dim, int num_tokens) {
    ensure_init();
    HyperStep h{};
    h.x = x; h.y = y; h.bias = bias; h.scale = scale; h.record = record; h.norm_w = norm_w; h.norm_b = norm_b; h.out_f32 = out;
    h.streams = streams; h.ld = dim;
    launch_hyper_step(h, num_tokens);
}

void nvllm_swiglu_bias(float* out, const float* g, const float* u, const float* bg, const float* bu, int hidden_dim, int num_tokens) {
    ensure_init();
    launch_swiglu_bias(out, g, u, bg, bu, num_tokens, hidden_dim);
}

void nvllm_softcap(float* x, float cap, long n) {
    ensure_init();
    launch_softcap(x, cap, n);
}

void nvllm_latent_pool_init(KVCacheManager* mgr, int block_size, int num_blocks, int rank, int rot, int elem_bytes) {
    init_block_pool(mgr, block_size, num_blocks, latent_pool_bytes(latent_pool(nullptr, elem_bytes, block_size, rank, rot), num_blocks));
}

static void check_latent_pool(const KVCacheManager* mgr, int rank, int rot, int elem_bytes) {
    if (block_pool_bytes(mgr) != latent_pool_bytes(latent_pool(nullptr, elem_bytes, mgr->block_size, rank, rot), mgr->num_blocks))
        NVLLM_FATAL("this block pool does not hold rows of %d + %d values of %d bytes", rank, rot, elem_bytes);
}

void nvllm_latent_cache_write(KVCacheManager* mgr, BlockTable** block_tables, int* seq_ids, int* pos_arr, const float* kv, const float* gain,
                              float eps, double base, int rank, int rot, int elem_bytes, int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, pos_arr, seq_ids, num_tokens, nullptr, 0, block_tables, nullptr, 0, mgr->block_size);
    if (s.table_short) NVLLM_FATAL("latent cache write: a position lies beyond its sequence's block table");
    check_latent_pool(mgr, rank, rot, elem_bytes);
    launch_latent_kv(latent_pool(mgr->pool_k, elem_bytes, mgr->block_size, rank, rot), kv, rank + rot, rank, gain, eps,
                     rotation_table(base, rot, s.max_pos + 1), s);
}

void nvllm_latent_attention(float* out, const float* q, KVCacheManager* mgr, BlockTable** block_tables, int* seq_ids, int* pos_arr,
                            const float* sink, float scale, int n_heads, int rank, int rot, int elem_bytes, int num_tokens) {
    ensure_init();
    if (num_tokens <= 0) return;
    StepArrays s = stage_step(nullptr, pos_arr, seq_ids, num_tokens, nullptr, 0, block_tables, nullptr, 0, mgr->block_size, LATENT_RUN,
                              nullptr, true);
    if (s.table_short) NVLLM_FATAL("latent attention: a position lies beyond its sequence's block table");
    check_latent_pool(mgr, rank, rot, elem_bytes);
    LatentAttn a{};
    a.pool = latent_pool(mgr->pool_k, elem_bytes, mgr->block_size, rank, rot);
    a.sink = sink;
    a.scale = scale;
    a.H = n_heads;
    if (elem_bytes == 4) {
        a.q = q;
        a.out_f32 = out;
        launch_latent_attention(a, s);
        return;
    }
    __half* rows = (__half*)ws_get(WS_Q_ROWS, (size_t)num_tokens * n_heads * a.pool.row() * sizeof(__half));
    launch_latent_rows_b16(rows, q, num_tokens * n_heads, a.pool);
    a.q = rows;
    a.out_b16 = (__half*)ws_get(WS_LATENT, b16_halves(num_tokens, n_heads * a.pool.rank_ld) * sizeof(__half));
    launch_latent_attention(a, s);
    launch_untile_b16(out, a.out_b16, num_tokens, n_heads, rank, a.pool.rank_ld);
}

}  // extern "C"
