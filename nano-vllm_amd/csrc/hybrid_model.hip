// hybrid_model.hip -- the "Simivik" design: a decoder whose layers mix tokens either by linear attention with a decaying
// state ("lightning") or by grouped-query attention with a short convolution over time, half-split rotation, capped scores
// and a sliding window that keeps the first tokens; feed-forwards are dense (squared relu) or mixtures of experts with a
// sigmoid router and a gated shared expert; norms are RMS with weights around zero; layers may borrow another layer's
// tensors (with a cache and state of their own); embeddings are tied.
//
// Two forms of the forward pass:
//   bf16  RMS norms are folded into the projections as elsewhere: x * gain goes into the tiles, 1/rms is applied to the sums.
//           lightning   [q; k; v; gate] with silu on the first three -> rows;  state;  W_o with the residual step
//           attention   [q; k; v] -> rows;  convolution, rotation, cache write;  attention;  W_o with the residual step
//           dense       up with relu^2;  down with the residual step
//           experts     [router; shared gate];  choice and sorting;  gate/up and down of the chosen experts (rows gathered
//                       by the first product);  the shared expert's two;  sum with the residual step
//   fp32  one plain operator per step of the design (weights expanded to fp32).
// Every width is padded to 32 with zero weights where the tiles need it, so no size is special.
#include <algorithm>
#include <cmath>
#include <cstring>

#include "gemm_common.h"
#include "lightning.h"
#include "model_dir.h"
#include "moe.h"
#include "window_attention.h"

namespace nvllm {

namespace {

struct MixerSizes {
    bool lightning = false;
    int heads = 0, dim = 0, vdim = 0;
    // attention
    int groups = 0, taps = 0;   // taps 0: no convolution
    int rot = 0, window = 0, keep_first = 0;
    double base = 1.0;
    float scale = 1.f, cap = 0.f;
    int channels() const { return heads * dim + groups * (dim + vdim); }
    int state_taps() const { return taps > 1 ? taps - 1 : 0; }
};

struct FfSizes {
    int dense = 0;              // width of a dense feed-forward; 0: none or experts
    int experts = 0, top = 0, expert_ff = 0, shared_ff = 0;
    bool any() const { return dense > 0 || experts > 0; }
};

struct HybridLayer {
    MixerSizes m;
    FfSizes f;
    // bf16
    B16Weight in, o, up, down, router, experts_up, experts_down, shared_up, shared_down;
    // fp32 (row-major, unpadded)
    float *in32[4] = {nullptr, nullptr, nullptr, nullptr}, *o32 = nullptr, *up32 = nullptr, *gate32 = nullptr, *down32 = nullptr, *router32 = nullptr;
    float *shared_gate32 = nullptr, *shared_up32 = nullptr, *shared_down32 = nullptr;
    // both
    float *norm[2] = {nullptr, nullptr};   // 1 + stored weight
    float *head_norm = nullptr, *decay = nullptr, *conv = nullptr;
};

// What a layer run keeps of its own between passes.
struct RunMemory {
    size_t slot_bytes = 0;
    void* mem = nullptr;
};

class HybridModel : public HbmModel {
public:
    HybridModel(const ModelDir& dir, Config* p);
    ~HybridModel() override {
        for (auto& r : states_) device_free(r.mem);
    }
    void init_kv(KVCacheManager* mgr, int block_size, int num_blocks) override;
    void init_states(int slots) override;
    void forward(const PassArgs& a) override;

private:
    bool f32_;
    int D_, Dp_, V_;
    float eps_;
    std::vector<HybridLayer> layers_;   // by index in config.json; borrowed ones stay empty
    std::vector<int> source_;           // layer run -> layer whose tensors it uses
    std::vector<RunMemory> states_;
    int slots_ = 0;
    const void* embed_ = nullptr;
    B16Weight head_;
    float* final_norm_ = nullptr;

    void load_layer(const ModelDir& dir, int i, const Json& cfg);
    void load_mixer(const ModelDir& dir, HybridLayer& w, const std::string& M);
    void load_ff(const ModelDir& dir, HybridLayer& w, const std::string& P);
    float* norm_gain(const ModelDir& dir, const std::string& name);
    size_t pool_bytes(int run, int block_size, int num_blocks) const;
    KvPages pages(const KVCacheManager* mgr, int run) const;
    const float* next_gain(size_t run, int part) const;
    Lightning lightning(const HybridLayer& w, int run) const;
    ConvRope conv_rope(const HybridLayer& w, int run, const StepArrays& st) const;
    WindowAttn attention(const HybridLayer& w, const KvPages& pool) const;
    void forward_b16(const PassArgs& a, const StepArrays& st);
    void forward_f32(const PassArgs& a, const StepArrays& st);
};

// ------------------------------------------------------------------ configuration
const Json* given(const Json& o, const char* key) {   // null and absent are the same
    const Json* j = o.find(key);
    return j && !j->is_null() ? j : nullptr;
}

MixerSizes read_mixer(const Json& cfg, const std::string& at) {
    const std::string am = at + ".mixer";
    const char* where = am.c_str();
    const std::string& type = json_get(cfg, "type", Json::STRING, at.c_str()).text;
    const Json& c = json_get(cfg, "mixer", Json::OBJECT, at.c_str());
    MixerSizes m;
    m.heads = json_int(c, "heads", where);
    m.dim = json_int(c, "dim", where);
    m.vdim = json_int(c, "vdim", where);
    if (m.heads < 1 || m.dim < 1 || m.vdim < 1) bad_config((am + ": heads, dim and vdim must be positive").c_str());
    if (type == "lightning") {
        m.lightning = true;
        if ((int)json_get(c, "decay", Json::ARRAY, where).items.size() != m.heads) bad_config((am + ".decay does not name one number per head").c_str());
        return m;
    }
    if (type != "attention") bad_config((at + " has the unknown mixer '" + type + "'").c_str());
    m.groups = json_int(c, "kv_heads", where);
    m.scale = (float)json_num(c, "scale", where);
    if (given(c, "conv")) m.taps = json_int(c, "conv", where);
    if (given(c, "softcap")) m.cap = (float)json_num(c, "softcap", where);
    if (const Json* r = given(c, "rot")) {
        m.rot = json_int(*r, "dims", (am + ".rot").c_str());
        m.base = json_num(*r, "base", (am + ".rot").c_str());
    }
    m.window = 1 << 30;
    if (const Json* k = given(c, "mask")) {
        if (given(*k, "size")) m.window = json_int(*k, "size", (am + ".mask").c_str());
        if (given(*k, "keep_first")) m.keep_first = json_int(*k, "keep_first", (am + ".mask").c_str());
    }
    if (m.groups < 1 || m.heads % m.groups || m.taps < 0 || m.cap < 0.f || m.rot < 0 || m.rot % 2 || m.rot > m.dim || !(m.base > 0.0) || m.window < 1 || m.keep_first < 0)
        bad_config(("the sizes of " + am + " are inconsistent").c_str());
    return m;
}

FfSizes read_ff(const Json& cfg, const std::string& at) {
    FfSizes f;
    const Json* c = given(cfg, "mlp");
    if (!c) return f;
    const std::string af = at + ".mlp";
    const std::string& kind = json_get(*c, "kind", Json::STRING, af.c_str()).text;
    if (kind == "dense") {
        f.dense = json_int(*c, "ff", af.c_str());
        if (f.dense < 1) bad_config((af + ".ff is not positive").c_str());
    } else if (kind == "moe") {
        const Json& router = json_get(*c, "router", Json::OBJECT, af.c_str());
        f.experts = json_int(router, "experts", (af + ".router").c_str());
        f.top = json_int(router, "top", (af + ".router").c_str());
        f.expert_ff = json_int(json_get(*c, "expert", Json::OBJECT, af.c_str()), "ff", (af + ".expert").c_str());
        if (const Json* s = given(*c, "shared")) {
            f.shared_ff = json_int(*s, "ff", (af + ".shared").c_str());
            if (f.shared_ff < 1) bad_config((af + ".shared.ff is not positive").c_str());
        }
        if (f.experts < 1 || f.top < 1 || f.top > f.experts || f.expert_ff < 1) bad_config(("the sizes of " + af + " are inconsistent").c_str());
    } else {
        bad_config((af + " has the unknown kind '" + kind + "'").c_str());
    }
    return f;
}

// ------------------------------------------------------------------ weights
// A row-major bf16 matrix under construction.
struct HostMatrix {
    const ModelDir& dir;
    int K;   // columns as stored
    std::vector<uint16_t> out, src;
    HostMatrix(const ModelDir& d, size_t rows, int cols) : dir(d), K(cols), out(rows * (size_t)cols, 0) {}
    void read(const std::string& name, int rows, int cols) {
        src.resize((size_t)rows * cols);
        dir.read_bf16(name, {rows, cols}, src.data());
    }
    // n rows of the last tensor, from row r0, to row d0
    void rows(size_t d0, int r0, int n) { memcpy(out.data() + d0 * K, src.data() + (size_t)r0 * K, (size_t)n * K * 2); }
    // [heads * per, K] to rows of `ld` per head
    void heads(size_t d0, const std::string& name, int n, int per, int ld) {
        read(name, n * per, K);
        for (int h = 0; h < n; h++) rows(d0 + (size_t)h * ld, h * per, per);
    }
    // gate and up rows in alternating blocks of 16
    void gate_up(size_t d0, const std::string& prefix, int ff) {
        for (int half = 0; half < 2; half++) {
            read(prefix + (half ? "up" : "gate"), ff, K);
            for (int r = 0; r < ff; r++) rows(d0 + (size_t)(r / 16) * 32 + half * 16 + r % 16, r, 1);
        }
    }
};

float* HybridModel::norm_gain(const ModelDir& dir, const std::string& name) {
    std::vector<float> v((size_t)Dp_, 0.f);
    dir.read_f32(name, {D_}, v.data());
    for (int i = 0; i < D_; i++) v[i] += 1.f;
    return upload(v);
}

void HybridModel::load_mixer(const ModelDir& dir, HybridLayer& w, const std::string& M) {
    const MixerSizes& m = w.m;
    const int H = m.heads, G = m.lightning ? H : m.groups, dp = pad32(m.dim), vp = pad32(m.vdim);
    const char* names[4] = {"q", "k", "v", "g"};
    const int parts = m.lightning ? 4 : 3, count[4] = {H, G, G, H}, per[4] = {m.dim, m.dim, m.vdim, m.vdim};
    if (m.lightning) {
        std::vector<float> gain((size_t)H * (f32_ ? m.vdim : vp), 0.f), file((size_t)H * m.vdim);
        dir.read_f32(M + "norm", {H * m.vdim}, file.data());
        for (int h = 0; h < H; h++) memcpy(gain.data() + (size_t)h * (f32_ ? m.vdim : vp), file.data() + (size_t)h * m.vdim, m.vdim * sizeof(float));
        w.head_norm = upload(gain);
    } else if (m.taps > 0) {
        // [taps][channels], channels in the order q, k, v
        std::vector<float> taps((size_t)m.taps * m.channels()), file;
        int at = 0;
        for (int i = 0; i < 3; i++) {
            const int n = count[i] * per[i];
            file.resize((size_t)n * m.taps);
            dir.read_f32(M + names[i] + ".conv", {n, m.taps}, file.data());
            for (int c = 0; c < n; c++)
                for (int j = 0; j < m.taps; j++) taps[(size_t)j * m.channels() + at + c] = file[(size_t)c * m.taps + j];
            at += n;
        }
        w.conv = upload(taps);
    }
    if (f32_) {
        if (m.lightning) {
            for (int i = 0; i < 4; i++) w.in32[i] = matrix_f32(dir, M + names[i], count[i] * per[i], D_);
        } else {   // one matrix: the channels of a token side by side
            std::vector<float> all((size_t)m.channels() * D_);
            size_t at = 0;
            for (int i = 0; i < 3; i++) {
                dir.read_f32(M + names[i], {count[i] * per[i], D_}, all.data() + at);
                at += (size_t)count[i] * per[i] * D_;
            }
            w.in32[0] = upload(all);
        }
        w.o32 = matrix_f32(dir, M + "o", D_, H * m.vdim);
        return;
    }
    if (m.lightning) {   // every head padded
        const int rows = 2 * H * (dp + vp), ld[4] = {dp, dp, vp, vp};
        HostMatrix in(dir, rows, D_);
        size_t at = 0;
        for (int i = 0; i < 4; i++) {
            in.heads(at, M + names[i], H, per[i], ld[i]);
            at += (size_t)H * ld[i];
        }
        w.in = tile(in.out, rows, D_);
    } else {
        const int rows = pad32(m.channels());
        HostMatrix in(dir, rows, D_);
        size_t at = 0;
        for (int i = 0; i < parts; i++) {
            in.heads(at, M + names[i], count[i], per[i], per[i]);
            at += (size_t)count[i] * per[i];
        }
        w.in = tile(in.out, rows, D_);
    }
    // W_o: columns padded head by head
    HostMatrix o(dir, Dp_, H * vp);
    o.read(M + "o", D_, H * m.vdim);
    for (int n = 0; n < D_; n++)
        for (int h = 0; h < H; h++) memcpy(o.out.data() + ((size_t)n * H + h) * vp, o.src.data() + ((size_t)n * H + h) * m.vdim, (size_t)m.vdim * 2);
    w.o = tile(o.out, Dp_, H * vp);
}

void HybridModel::load_ff(const ModelDir& dir, HybridLayer& w, const std::string& P) {
    const FfSizes& f = w.f;
    auto expert = [&](int e) { return P + "e" + std::to_string(e) + "."; };
    if (f32_) {
        if (f.dense) {
            w.up32 = matrix_f32(dir, P + "up", f.dense, D_);
            w.down32 = matrix_f32(dir, P + "down", D_, f.dense);
            return;
        }
        const size_t one = (size_t)f.expert_ff * D_;
        std::vector<float> all(one * f.experts);
        auto stack = [&](const char* name, long rows, long cols) {
            for (int e = 0; e < f.experts; e++) dir.read_f32(expert(e) + name, {rows, cols}, all.data() + one * e);
            return upload(all);
        };
        w.gate32 = stack("gate", f.expert_ff, D_);
        w.up32 = stack("up", f.expert_ff, D_);
        w.down32 = stack("down", D_, f.expert_ff);
        std::vector<float> router((size_t)(f.experts + 1) * D_, 0.f);
        dir.read_f32(P + "router", {f.experts, D_}, router.data());
        if (f.shared_ff) {
            dir.read_f32(P + "shared.sg", {1, D_}, router.data() + (size_t)f.experts * D_);
            w.shared_gate32 = matrix_f32(dir, P + "shared.gate", f.shared_ff, D_);
            w.shared_up32 = matrix_f32(dir, P + "shared.up", f.shared_ff, D_);
            w.shared_down32 = matrix_f32(dir, P + "shared.down", D_, f.shared_ff);
        }
        w.router32 = upload(router);
        return;
    }
    auto down_matrix = [&](const std::string& name, int ff) {
        HostMatrix d(dir, Dp_, ff);
        d.read(name, D_, ff);
        d.rows(0, 0, D_);
        return tile(d.out, Dp_, ff);
    };
    if (f.dense) {
        HostMatrix up(dir, pad32(f.dense), D_);
        up.read(P + "up", f.dense, D_);
        up.rows(0, 0, f.dense);
        w.up = tile(up.out, pad32(f.dense), D_);
        w.down = down_matrix(P + "down", f.dense);
        return;
    }
    const int Fp = pad32(f.expert_ff);
    {
        HostMatrix gu(dir, (size_t)f.experts * 2 * Fp, D_);
        for (int e = 0; e < f.experts; e++) gu.gate_up((size_t)e * 2 * Fp, expert(e), f.expert_ff);
        w.experts_up = tile(gu.out, f.experts * 2 * Fp, D_);
        w.experts_up.N = 2 * Fp;   // of one expert
    }
    {
        HostMatrix d(dir, (size_t)f.experts * Dp_, f.expert_ff);
        for (int e = 0; e < f.experts; e++) {
            d.read(expert(e) + "down", D_, f.expert_ff);
            d.rows((size_t)e * Dp_, 0, D_);
        }
        w.experts_down = tile(d.out, f.experts * Dp_, f.expert_ff);
        w.experts_down.N = Dp_;
    }
    HostMatrix router(dir, f.experts + 1, D_);
    router.read(P + "router", f.experts, D_);
    router.rows(0, 0, f.experts);
    if (f.shared_ff) {
        router.read(P + "shared.sg", 1, D_);
        router.rows(f.experts, 0, 1);
        const int Sp = pad32(f.shared_ff);
        HostMatrix gu(dir, (size_t)2 * Sp, D_);
        gu.gate_up(0, P + "shared.", f.shared_ff);
        w.shared_up = tile(gu.out, 2 * Sp, D_);
        w.shared_down = down_matrix(P + "shared.down", f.shared_ff);
    }
    w.router = tile(router.out, f.experts + 1, D_);
}

void HybridModel::load_layer(const ModelDir& dir, int i, const Json& cfg) {
    const std::string at = "layers[" + std::to_string(i) + "]", L = "l" + std::to_string(i) + ".";
    HybridLayer& w = layers_[i];
    w.m = read_mixer(cfg, at);
    w.f = read_ff(cfg, at);
    w.norm[0] = norm_gain(dir, L + "norm1");
    if (w.f.any()) w.norm[1] = norm_gain(dir, L + "norm2");
    if (w.m.lightning) {   // powers of the decay, formed in double
        const Json& d = json_get(json_get(cfg, "mixer", Json::OBJECT, at.c_str()), "decay", Json::ARRAY, at.c_str());
        std::vector<float> pow_tab((size_t)w.m.heads * (LIGHTNING_CHUNK + 1));
        for (int h = 0; h < w.m.heads; h++) {
            const double v = d.items[h].number;
            if (d.items[h].type != Json::NUMBER || !(v >= 0.0 && v <= 1.0)) bad_config((at + ".mixer.decay: a decay lies between 0 and 1").c_str());
            for (int n = 0; n <= LIGHTNING_CHUNK; n++) pow_tab[(size_t)h * (LIGHTNING_CHUNK + 1) + n] = (float)std::pow(v, n);
        }
        w.decay = upload(pow_tab);
    }
    load_mixer(dir, w, L + "mix.");
    if (w.f.any()) load_ff(dir, w, L + "mlp.");
}

HybridModel::HybridModel(const ModelDir& dir, Config* p) {
    const Json& c = dir.config;
    f32_ = rt().compute_dtype == NVLLM_COMPUTE_F32;
    D_ = json_int(c, "width", "config");
    V_ = json_int(c, "vocab", "config");
    eps_ = (float)json_num(json_get(c, "norm", Json::OBJECT, "config"), "eps", "config.norm");
    if (D_ < 1 || V_ < 1) bad_config("width or vocab is out of range");
    Dp_ = f32_ ? D_ : pad32(D_);
    const Json& list = json_get(c, "layers", Json::ARRAY, "config");
    const int n = (int)list.items.size();
    if (n < 1) bad_config("it lists no layers");
    layers_.resize(n);
    for (int i = 0; i < n; i++) {
        int s = i;
        for (int hops = 0; given(list.items[s], "weights_of"); hops++) {
            s = json_int(list.items[s], "weights_of", "a layer");
            if (s < 0 || s >= n || hops > n) bad_config("a layer's weights_of leads to no layer");
        }
        source_.push_back(s);
        if (s == i) load_layer(dir, i, list.items[i]);
    }
    if (f32_) {
        embed_ = matrix_f32(dir, "embed", V_, D_);
    } else {
        std::vector<uint16_t> table((size_t)V_ * D_), padded((size_t)V_ * Dp_, 0);
        dir.read_bf16("embed", {V_, D_}, table.data());
        for (int v = 0; v < V_; v++) memcpy(padded.data() + (size_t)v * Dp_, table.data() + (size_t)v * D_, (size_t)D_ * 2);
        void* d = alloc(padded.size() * 2, "the embedding table");
        device_memcpy(d, padded.data(), padded.size() * 2, HOST_TO_DEVICE);
        embed_ = d;
        head_ = tile(table, V_, D_);
    }
    final_norm_ = norm_gain(dir, "final.norm");
    states_.resize(n);
    for (int r = 0; r < n; r++) {
        const MixerSizes& m = layers_[source_[r]].m;
        states_[r].slot_bytes = m.lightning ? lightning_state_floats(m.heads, m.dim, m.vdim) * 4 : (size_t)m.state_taps() * m.channels() * (f32_ ? 4 : 2);
    }
    const MixerSizes& m0 = layers_[source_[0]].m;
    p->dim = D_;
    p->hidden_dim = 1;
    for (const auto& l : layers_) p->hidden_dim = std::max(p->hidden_dim, std::max(l.f.dense, l.f.expert_ff));
    p->n_layers = n;
    p->n_heads = m0.heads;
    p->n_kv_heads = m0.lightning ? m0.heads : m0.groups;
    p->vocab_size = V_;
    p->max_seq_len = 2048;
    p->head_dim = m0.dim;
    p->rope_theta = (float)m0.base;
}

// ------------------------------------------------------------------ cache and state
size_t HybridModel::pool_bytes(int run, int block_size, int num_blocks) const {
    const MixerSizes& m = layers_[source_[run]].m;
    return m.lightning ? 0 : kv_pages_bytes(f32_ ? 4 : 2, block_size, num_blocks, m.groups, m.dim, m.vdim);
}
KvPages HybridModel::pages(const KVCacheManager* mgr, int run) const {
    const MixerSizes& m = layers_[source_[run]].m;
    size_t off = 0;
    for (int r = 0; r < run; r++) off += pool_bytes(r, mgr->block_size, mgr->num_blocks);
    return kv_pages((char*)mgr->pool_k + off, f32_ ? 4 : 2, mgr->block_size, mgr->num_blocks, m.groups, m.dim, m.vdim);
}
void HybridModel::init_kv(KVCacheManager* mgr, int block_size, int num_blocks) {
    size_t bytes = 0;
    for (size_t r = 0; r < source_.size(); r++) bytes += pool_bytes((int)r, block_size, num_blocks);
    init_block_pool(mgr, block_size, num_blocks, bytes);
}

void HybridModel::init_states(int slots) {
    if (slots <= slots_) return;
    for (auto& r : states_) {
        if (!r.slot_bytes) continue;
        void* d = nullptr;
        if (device_malloc(&d, r.slot_bytes * slots) != 0) NVLLM_FATAL("cannot allocate the states of %d sequences (%zu bytes)", slots, r.slot_bytes * slots);
        HIP_CHECK(hipMemsetAsync(d, 0, r.slot_bytes * slots, rt().stream));   // slots nobody has written are finite
        if (r.mem) {
            device_memcpy(d, r.mem, r.slot_bytes * slots_, DEVICE_TO_DEVICE);
            device_free(r.mem);
        }
        r.mem = d;
    }
    slots_ = slots;
}

// ------------------------------------------------------------------ the pass
const float* HybridModel::next_gain(size_t run, int part) const {   // of the norm that follows sublayer `part` of a run
    if (part == 0 && layers_[source_[run]].f.any()) return layers_[source_[run]].norm[1];
    return run + 1 < source_.size() ? layers_[source_[run + 1]].norm[0] : final_norm_;
}
Lightning HybridModel::lightning(const HybridLayer& w, int run) const {
    Lightning l;
    l.H = w.m.heads; l.dim = w.m.dim; l.vdim = w.m.vdim; l.decay = w.decay; l.state = (float*)states_[run].mem;
    return l;
}
ConvRope HybridModel::conv_rope(const HybridLayer& w, int run, const StepArrays& st) const {
    ConvRope c{};
    c.taps = w.conv; c.n_taps = std::max(1, w.m.taps); c.state = states_[run].mem; c.rot = w.m.rot; c.H = w.m.heads;
    c.rope = w.m.rot ? rotation_table(w.m.base, w.m.rot, st.max_pos + 1) : nullptr;
    return c;
}
WindowAttn HybridModel::attention(const HybridLayer& w, const KvPages& pool) const {
    WindowAttn t{};
    t.pool = pool; t.H = w.m.heads; t.scale = w.m.scale; t.cap = w.m.cap; t.size = w.m.window; t.keep_first = w.m.keep_first;
    return t;
}

void HybridModel::forward(const PassArgs& a) {
    size_t bytes = 0;
    for (size_t r = 0; r < source_.size(); r++) bytes += pool_bytes((int)r, a.mgr->block_size, a.mgr->num_blocks);
    if (block_pool_bytes(a.mgr) != bytes) NVLLM_FATAL("transformer_batch: the block pool was not made for this model (nvllm_init_model_kv)");
    int slots = 0;
    for (int t = 0; t < a.T; t++) {
        if (a.pos[t] < 0 || a.seq_ids[t] < 0 || a.tokens[t] < 0 || a.tokens[t] >= V_)
            NVLLM_FATAL("transformer_batch: token %d (id %d, position %d) is out of range", t, a.tokens[t], a.pos[t]);
        slots = std::max(slots, a.seq_ids[t] + 1);
    }
    init_states(slots);
    int group = LIGHTNING_CHUNK;
    for (const auto& l : layers_)
        if (l.m.lightning) group = std::max(group, lightning_group(a.T, l.m.heads, l.m.vdim));
    const StepArrays st = stage_step(a.tokens, a.pos, a.seq_ids, a.T, a.output_indices, a.B, a.tables, nullptr, 0, a.mgr->block_size, WINDOW_RUN, a.token_src, true, true,
                                     group);
    if (st.table_short) NVLLM_FATAL("transformer_batch: a position lies beyond its sequence's block table (allocate the block first)");
    if (st.seq_split) NVLLM_FATAL("transformer_batch: the tokens of a sequence must lie side by side in the batch");
    if (f32_) forward_f32(a, st);
    else forward_b16(a, st);
}

void HybridModel::forward_b16(const PassArgs& a, const StepArrays& st) {
    const int T = a.T, B = a.B, x_tiles = Dp_ / 32;
    // workspaces of the widest layer
    size_t sorted = 0, rows = 0, raw = 0, hid = 0, heads_ss = 0, shared_hid = 0, y_rows = 0, z_ld = 0, ints = 0;
    for (const auto& l : layers_) {
        const MixerSizes& m = l.m;
        const FfSizes& f = l.f;
        const size_t dp = pad32(m.dim), vp = pad32(m.vdim), H = m.heads;
        rows = std::max(rows, m.lightning ? 2 * H * (dp + vp) : H * dp);
        if (!m.lightning) raw = std::max(raw, (size_t)pad32(m.channels()));
        else heads_ss = std::max(heads_ss, H * vp / 16);
        hid = std::max(hid, b16_halves(T, (int)(H * vp)));
        hid = std::max(hid, b16_halves(T, pad32(f.dense)));
        if (f.experts) {
            const int pad = route_pad(T, f.experts, f.top);
            const size_t w = route_ints(T, f.experts, f.top, pad);
            const int cap = route_plan(nullptr, T, f.experts, f.top, pad).capacity;
            hid = std::max(hid, b16_halves(cap, pad32(f.expert_ff)));
            y_rows = std::max(y_rows, (size_t)cap);
            if (pad >= 64) sorted = std::max(sorted, b16_halves(cap, Dp_));
            shared_hid = std::max(shared_hid, b16_halves(T, pad32(f.shared_ff)));
            z_ld = std::max(z_ld, (size_t)pad32(f.experts + 1));
            ints = std::max(ints, w);
        }
    }
    float* x = (float*)ws_get(WS_STREAMS, (size_t)T * Dp_ * sizeof(float));
    __half* act = (__half*)ws_get(WS_A16_X, b16_halves(T, Dp_) * sizeof(__half));
    __half* wide = (__half*)ws_get(WS_A16_H, hid * sizeof(__half));   // mixer results, hidden units: never two at once
    float* ss = (float*)ws_get(WS_MISC, (size_t)T * x_tiles * sizeof(float));
    float* ss_heads = (float*)ws_get(WS_MISC2, (size_t)T * heads_ss * sizeof(float));
    __half* q_rows = (__half*)ws_get(WS_Q_ROWS, (size_t)T * rows * sizeof(__half));
    __half* raw_rows = (__half*)ws_get(WS_KV_RAW, (size_t)T * raw * sizeof(__half));
    __half* hid_shared = (__half*)ws_get(WS_A16_ATT, std::max(shared_hid, b16_halves(B, Dp_)) * sizeof(__half));
    float* y_experts = (float*)ws_get(WS_F32_A, y_rows * Dp_ * sizeof(float));
    float* y_shared = (float*)ws_get(WS_F32_B, (shared_hid ? (size_t)T * Dp_ : 0) * sizeof(float));
    float* z = (float*)ws_get(WS_F32_C, (size_t)T * z_ld * sizeof(float));
    int* route_mem = (int*)ws_get(WS_LATENT, ints * sizeof(int));
    __half* act_sorted = (__half*)ws_get(WS_A16_SORTED, sorted * sizeof(__half));

    launch_embed_norm_b16(x, act, ss, embed_, st.d_tokens, layers_[source_[0]].norm[0], T, Dp_, st.d_tok_src, a.d_argmax);
    auto normed = [&](GemmEpilogue::Kind kind) {   // a projection of the normed residual
        GemmEpilogue e;
        e.kind = kind;
        e.ss_in = ss; e.ss_tiles = x_tiles; e.d_in = D_; e.eps = eps_;
        return e;
    };
    auto to_rows = [&](GemmEpilogue e, __half* out, int ld) {
        e.q_rows = (__bf16*)out; e.q_heads = 1; e.q_row = ld; e.head_ld = ld;
        return e;
    };
    auto residual = [&](const B16Weight& w, const __half* in, GemmEpilogue e, const float* gain, int cls) {
        e.kind = GemmEpilogue::RESID_B16;
        e.x = x; e.gain_next = gain; e.a16_out = act; e.ss_out = ss;
        launch_gemm_b16(w, in, T, e, cls);
    };
    for (size_t run = 0; run < source_.size(); run++) {
        const HybridLayer& w = layers_[source_[run]];
        const MixerSizes& m = w.m;
        const FfSizes& f = w.f;
        const int H = m.heads, dp = pad32(m.dim), vp = pad32(m.vdim);
        if (m.lightning) {
            GemmEpilogue e = to_rows(normed(GemmEpilogue::ROWS_B16), q_rows, w.in.N);
            e.silu_to = H * (2 * dp + vp);
            launch_gemm_b16(w.in, act, T, e, PC_GEMM_QKV);
            Lightning l = lightning(w, (int)run);
            l.rows = q_rows; l.ld = w.in.N; l.dim_ld = dp; l.vdim_ld = vp; l.gain = w.head_norm; l.out_b16 = wide; l.ss_out = ss_heads;
            launch_lightning(l, st);
            GemmEpilogue r;   // the norm over all heads: 1/rms of what the state gave
            r.ss_in = ss_heads; r.ss_tiles = H * vp / 16; r.d_in = H * m.vdim; r.eps = eps_;
            residual(w.o, wide, r, next_gain(run, 0), PC_GEMM_WO);
        } else {
            launch_gemm_b16(w.in, act, T, to_rows(normed(GemmEpilogue::ROWS_B16), raw_rows, w.in.N), PC_GEMM_QKV);
            const KvPages pool = pages(a.mgr, (int)run);
            ConvRope c = conv_rope(w, (int)run, st);
            c.raw = raw_rows; c.raw_ld = w.in.N; c.q_out = q_rows;
            launch_conv_rope(c, pool, st);
            WindowAttn t = attention(w, pool);
            t.q = q_rows; t.out_b16 = wide;
            launch_window_attention(t, st);
            residual(w.o, wide, GemmEpilogue(), next_gain(run, 0), PC_GEMM_WO);
        }
        if (f.dense) {
            GemmEpilogue e = normed(GemmEpilogue::TILE_B16);
            e.relu2 = true; e.a16_out = wide;
            launch_gemm_b16(w.up, act, T, e, PC_GEMM_GATEUP);
            residual(w.down, wide, GemmEpilogue(), next_gain(run, 1), PC_GEMM_DOWN);
        } else if (f.experts) {
            const int ldz = pad32(f.experts + 1);
            GemmEpilogue ez = normed(GemmEpilogue::F32);
            ez.out = z; ez.ldo = ldz;
            launch_gemm_b16(w.router, act, T, ez, PC_GEMM_ROUTER);
            const RoutePlan plan = route_plan(route_mem, T, f.experts, f.top, route_pad(T, f.experts, f.top));
            launch_route(plan, z, ldz);
            ExpertRows er{plan.block_expert, plan.source, plan.capacity, plan.pad, T * f.top};
            GemmEpilogue eu = normed(GemmEpilogue::SWIGLU_A16);
            eu.ss_gather = plan.source; eu.row_weight = plan.weight; eu.a16_out = wide;
            if (plan.pad >= 64) {   // many rows per expert: sorted once (a gathering tile copy touches a cache line per 16 bytes)
                launch_expert_rows(act_sorted, x, w.norm[1], plan, Dp_);
                er.source = nullptr;
            }
            launch_gemm_experts(w.experts_up, f.experts, er.source ? act : act_sorted, er, eu, PC_GEMM_EXPERT_UP);
            er.source = nullptr;
            GemmEpilogue ed;
            ed.kind = GemmEpilogue::F32;
            ed.out = y_experts; ed.ldo = Dp_;
            launch_gemm_experts(w.experts_down, f.experts, wide, er, ed, PC_GEMM_EXPERT_DOWN);
            if (f.shared_ff) {
                GemmEpilogue su = normed(GemmEpilogue::SWIGLU_A16);
                su.a16_out = hid_shared;
                launch_gemm_b16(w.shared_up, act, T, su, PC_GEMM_SHARED_UP);
                GemmEpilogue sd;
                sd.kind = GemmEpilogue::F32;
                sd.out = y_shared; sd.ldo = Dp_;
                launch_gemm_b16(w.shared_down, hid_shared, T, sd, PC_GEMM_SHARED_DOWN);
            }
            MoeCombine c{};
            c.x = x; c.rows = y_experts; c.row_of = plan.row_of; c.top = f.top; c.shared = f.shared_ff ? y_shared : nullptr;
            c.z = z; c.ldz = ldz; c.z_col = f.experts; c.gain = next_gain(run, 1); c.out_b16 = act; c.ss = ss; c.ld = Dp_;
            launch_moe_combine(c, T);
        }
    }
    if (B <= 0) return;
    wait_for_row_copies();
    bool identity = B == T;
    for (int k = 0; identity && k < B; k++) identity = a.output_indices[k] == k;
    GemmEpilogue e = normed(GemmEpilogue::F32);
    const __half* rows_out = act;
    if (!identity) {
        launch_gather_b16(hid_shared, act, st.d_out_idx, B, Dp_);
        rows_out = hid_shared;
        e.ss_gather = st.d_out_idx;
    }
    e.out = a.d_logits; e.ldo = V_;
    e.amax_out = a.d_argmax;
    e.amax_out_host = a.argmax_host;
    e.amax_ld = (B + 63) & ~63;
    e.amax_pairs = (float2*)ws_get(WS_AMAX_PAIRS, (size_t)cdiv(V_, 32) * e.amax_ld * sizeof(float2));
    launch_gemm_b16(head_, rows_out, B, e, PC_GEMM_HEAD);
}

void HybridModel::forward_f32(const PassArgs& a, const StepArrays& st) {
    const int T = a.T, B = a.B;
    size_t wide = D_, q_row = 0, z_ld = 0, ints = 0;
    for (const auto& l : layers_) {
        const MixerSizes& m = l.m;
        const FfSizes& f = l.f;
        const size_t H = m.heads;
        wide = std::max({wide, H * m.vdim, (size_t)f.dense, (size_t)f.top * std::max(f.expert_ff, D_), (size_t)f.shared_ff});
        if (m.lightning) wide = std::max(wide, H * m.dim);
        else wide = std::max(wide, (size_t)m.channels());
        q_row = std::max(q_row, H * m.dim);
        if (f.experts) {
            z_ld = std::max(z_ld, (size_t)f.experts + 1);
            ints = std::max(ints, route_ints(T, f.experts, f.top, 16));
        }
    }
    auto rows = [&](WsSlot slot, size_t n) { return (float*)ws_get(slot, (size_t)T * n * sizeof(float)); };
    float *x = rows(WS_STREAMS, D_), *act = rows(WS_A16_X, D_), *b = rows(WS_F32_A, wide), *c = rows(WS_F32_B, wide), *d = rows(WS_F32_C, wide);
    float *q = rows(WS_Q_ROWS, q_row), *z = rows(WS_MISC, z_ld);
    int* route_mem = (int*)ws_get(WS_LATENT, ints * sizeof(int));
    launch_embed_streams(x, embed_, false, st.d_tokens, T, 1, D_, st.d_tok_src, a.d_argmax);
    for (size_t run = 0; run < source_.size(); run++) {
        const HybridLayer& w = layers_[source_[run]];
        const MixerSizes& m = w.m;
        const FfSizes& f = w.f;
        const int H = m.heads;
        launch_rmsnorm_f32(act, x, w.norm[0], D_, T, eps_);
        if (m.lightning) {
            const int qn = H * m.dim, vn = H * m.vdim;
            launch_matmul_f32w(q, act, w.in32[0], T, D_, qn);
            launch_matmul_f32w(b, act, w.in32[1], T, D_, qn);
            launch_matmul_f32w(c, act, w.in32[2], T, D_, vn);
            launch_silu(q, (long)T * qn);
            launch_silu(b, (long)T * qn);
            launch_silu(c, (long)T * vn);
            Lightning l = lightning(w, (int)run);
            l.q32 = q; l.k32 = b; l.v32 = c; l.out_f32 = d;
            launch_lightning(l, st);
            launch_rmsnorm_f32(d, d, w.head_norm, vn, T, eps_);
            launch_matmul_f32w(b, act, w.in32[3], T, D_, vn);
            launch_sigmoid_gate(d, d, b, (long)T * vn);
            launch_matmul_f32w(b, d, w.o32, T, vn, D_);
        } else {
            launch_matmul_f32w(c, act, w.in32[0], T, D_, m.channels());
            const KvPages pool = pages(a.mgr, (int)run);
            ConvRope r = conv_rope(w, (int)run, st);
            r.raw = c; r.raw_ld = m.channels(); r.q_out = q;
            launch_conv_rope(r, pool, st);
            WindowAttn t = attention(w, pool);
            t.q = q; t.out_f32 = d;
            launch_window_attention(t, st);
            launch_matmul_f32w(b, d, w.o32, T, H * m.vdim, D_);
        }
        launch_accum(x, b, (long)T * D_);
        if (!f.any()) continue;
        launch_rmsnorm_f32(act, x, w.norm[1], D_, T, eps_);
        if (f.dense) {
            launch_matmul_f32w(b, act, w.up32, T, D_, f.dense);
            launch_relu2(b, (long)T * f.dense);
            launch_matmul_f32w(c, b, w.down32, T, f.dense, D_);
            launch_accum(x, c, (long)T * D_);
            continue;
        }
        const int ldz = f.experts + 1;
        launch_matmul_f32w(z, act, w.router32, T, D_, ldz);
        const RoutePlan plan = route_plan(route_mem, T, f.experts, f.top, 16);
        launch_route(plan, z, ldz);
        launch_matmul_experts_f32(b, act, w.gate32, plan, true, D_, f.expert_ff);
        launch_matmul_experts_f32(c, act, w.up32, plan, true, D_, f.expert_ff);
        launch_swiglu(b, b, c, (long)T * f.top * f.expert_ff);
        launch_matmul_experts_f32(d, b, w.down32, plan, false, f.expert_ff, D_);
        if (f.shared_ff) {
            launch_matmul_f32w(b, act, w.shared_gate32, T, D_, f.shared_ff);
            launch_matmul_f32w(c, act, w.shared_up32, T, D_, f.shared_ff);
            launch_swiglu(b, b, c, (long)T * f.shared_ff);
            launch_matmul_f32w(c, b, w.shared_down32, T, f.shared_ff, D_);
        }
        MoeCombine mc{};
        mc.x = x; mc.rows = d; mc.top = f.top; mc.shared = f.shared_ff ? c : nullptr; mc.z = z; mc.ldz = ldz; mc.z_col = f.experts; mc.ld = D_;
        launch_moe_combine(mc, T);
    }
    if (B <= 0) return;
    wait_for_row_copies();
    launch_rmsnorm_f32(act, x, final_norm_, D_, T, eps_);
    launch_gather_rows_f32(b, act, st.d_out_idx, B, D_);
    launch_matmul_f32w(a.d_logits, b, (const float*)embed_, B, D_, V_);
    launch_argmax_ld(a.d_argmax, a.d_logits, B, V_, V_, a.argmax_host);
}

}  // namespace

DirModel* load_hybrid_model(const ModelDir& dir, Config* p) { return new HybridModel(dir, p); }

}  // namespace nvllm
