// latent_model.hip -- the "Suselorn" design: a decoder whose layers are latent attention (queries and
// keys/values through low-rank latents, one rotated key part shared by all heads, a sink per head) and a
// gated feed-forward with biases, on several hyper-connected residual streams, with Dynamic Tanh norms,
// layer scale, a span of layers that runs several times with the same weights (a cache slice per run), tied
// embeddings and soft-capped logits.
//
// Two forms of the forward pass:
//   bf16  eight launches per layer run (nine when attention is cut into slices).  The Dynamic Tanh norm needs no statistics, so the residual projections'
//         epilogues do the whole step between two sublayers: bias, layer scale, stream mixing, the next
//         sublayer's input and its norm, stored as activation tiles.
//           latent_in   [W_dq ; W_dkv]       query latent (x gain) -> tiles + sums of squares; rest -> fp32 rows
//           latent_q    W_uq (rows reordered: unrotated parts of all heads, then rotated parts)  1/rms, rotation;
//                       extra workgroups norm, rotate and write the new cache rows
//           absorb      W_uk^T head by head  -> query rows over the latent
//           attention   (+ merge of slices)
//           value       W_uv head by head
//           o           W_o, hyper epilogue;  gate/up (interleaved, biased SwiGLU);  down, hyper epilogue
//   fp32  one plain operator per step of the design (weights expanded to fp32).
// Every width is padded to 32 with zero weights where the tiles need it, so no size is special.
#include <algorithm>
#include <memory>

#include "gemm_common.h"
#include "latent_attention.h"
#include "model_dir.h"

namespace nvllm {

namespace {

struct Mixer {
    int heads, dim, rot, vdim, rank, q_rank;
    double base;
    float scale;
};

struct LayerWeightsDir {
    Mixer m;
    int ff = 0;   // 0: the layer has no feed-forward
    // bf16
    B16Weight in, uq, uk, uv, o, gateup, down;
    // fp32 (row-major, unpadded)
    float *dq = nullptr, *dkv = nullptr, *uq32 = nullptr, *uk32 = nullptr, *uv32 = nullptr, *o32 = nullptr, *gate = nullptr, *up = nullptr, *down32 = nullptr;
    // both: fp32 vectors, zero-padded in the bf16 form
    float *gain_q = nullptr, *gain_kv = nullptr, *sink = nullptr;
    float *ls[2] = {nullptr, nullptr}, *norm_w[2] = {nullptr, nullptr}, *norm_b[2] = {nullptr, nullptr};
    float *bias_gate = nullptr, *bias_up = nullptr, *bias_gu = nullptr, *bias_down = nullptr;
};

// One sublayer of the pass: what it is, and the record its residual update uses (mixing of this sublayer, input and
// norm of the one after it).
struct Sublayer {
    int layer, part, run;   // part 0: mixer, 1: feed-forward; run: which cache slice (mixers)
    const float* record;
    const float *next_w, *next_b;   // norm of the next sublayer, or the final norm
};

class LatentHyperModel : public HbmModel {
public:
    LatentHyperModel(const ModelDir& dir, Config* p);
    void init_kv(KVCacheManager* mgr, int block_size, int num_blocks) override;
    void forward(const PassArgs& a) override;

private:
    bool f32_;
    int D_, Dp_, V_, S_;     // width, padded width, vocabulary, streams
    float eps_, softcap_;
    std::vector<LayerWeightsDir> layers_;
    std::vector<int> runs_;  // layer of every run, in order
    std::vector<Sublayer> subs_;
    const float* first_record_ = nullptr;   // input weights and alpha of the first sublayer
    const void* embed_ = nullptr;
    B16Weight head_;

    LatentPool pool(const KVCacheManager* mgr, int run) const;
    size_t pool_bytes(int block_size, int num_blocks, int runs) const;   // of the first `runs` cache slices
    void load_layer(const ModelDir& dir, int i, const Json& cfg);
    void forward_b16(const PassArgs& a, const StepArrays& st);
    void forward_f32(const PassArgs& a, const StepArrays& st);
};

void LatentHyperModel::load_layer(const ModelDir& dir, int i, const Json& cfg) {
    const std::string at = "layers[" + std::to_string(i) + "]", L = "l" + std::to_string(i) + ".", M = L + "mix.", P = L + "mlp.";
    const Json& type = json_get(cfg, "type", Json::STRING, at.c_str());
    if (type.text != "latent_attention") {
        fprintf(stderr, "nvllm: config.json: %s has the unknown mixer '%s'\n", at.c_str(), type.text.c_str());
        exit(1);
    }
    const Json& mc = json_get(cfg, "mixer", Json::OBJECT, at.c_str());
    const std::string am = at + ".mixer";
    const Json& rot = json_get(mc, "rot", Json::OBJECT, am.c_str());
    LayerWeightsDir w;
    Mixer& m = w.m;
    m.heads = json_int(mc, "heads", am.c_str());
    m.dim = json_int(mc, "dim", am.c_str());
    m.rot = json_int(mc, "rot_dim", am.c_str());
    m.vdim = json_int(mc, "vdim", am.c_str());
    m.rank = json_int(mc, "kv_rank", am.c_str());
    m.q_rank = json_int(mc, "q_rank", am.c_str());
    m.scale = (float)json_num(mc, "scale", am.c_str());
    m.base = json_num(rot, "base", (am + ".rot").c_str());
    if (m.heads < 1 || m.dim < 1 || m.rot < 2 || m.rot % 2 || m.vdim < 1 || m.rank < 1 || m.q_rank < 1 || m.base <= 0.0 ||
        json_int(rot, "dims", (am + ".rot").c_str()) != m.rot) {
        fprintf(stderr, "nvllm: config.json: the sizes of %s are inconsistent\n", am.c_str());
        exit(1);
    }
    const Json* mlp = cfg.find("mlp");
    if (mlp && !mlp->is_null()) {
        const std::string af = at + ".mlp";
        if (json_get(*mlp, "kind", Json::STRING, af.c_str()).text != "dense") {
            fprintf(stderr, "nvllm: config.json: %s has an unknown kind\n", af.c_str());
            exit(1);
        }
        w.ff = json_int(*mlp, "ff", af.c_str());
        if (w.ff < 1) bad_config((af + ".ff is not positive").c_str());
    }
    const int H = m.heads, QD = m.dim + m.rot;
    w.sink = vec(dir, M + "sink", H, H);
    for (int q = 0; q < (w.ff ? 2 : 1); q++) {
        const std::string n = std::to_string(q + 1);
        w.norm_w[q] = vec(dir, L + "norm" + n, D_, Dp_);
        w.norm_b[q] = vec(dir, L + "norm" + n + ".b", D_, Dp_);
        w.ls[q] = vec(dir, L + "ls" + n, D_, Dp_);
    }
    if (f32_) {
        w.gain_q = vec(dir, M + "dq.norm", m.q_rank, m.q_rank);
        w.gain_kv = vec(dir, M + "dkv.norm", m.rank, m.rank);
        w.dq = matrix_f32(dir, M + "dq", m.q_rank, D_);
        w.dkv = matrix_f32(dir, M + "dkv", m.rank + m.rot, D_);
        w.uq32 = matrix_f32(dir, M + "uq", H * QD, m.q_rank);
        w.uk32 = matrix_f32(dir, M + "uk", H * m.dim, m.rank);
        w.uv32 = matrix_f32(dir, M + "uv", H * m.vdim, m.rank);
        w.o32 = matrix_f32(dir, M + "o", D_, H * m.vdim);
        if (w.ff) {
            w.gate = matrix_f32(dir, P + "gate", w.ff, D_);
            w.up = matrix_f32(dir, P + "up", w.ff, D_);
            w.down32 = matrix_f32(dir, P + "down", D_, w.ff);
            w.bias_gate = vec(dir, P + "gate.b", w.ff, w.ff);
            w.bias_up = vec(dir, P + "up.b", w.ff, w.ff);
            w.bias_down = vec(dir, P + "down.b", D_, D_);
        }
        layers_.push_back(w);
        return;
    }
    const int Qp = pad32(m.q_rank), Cp = pad32(m.rank), Rp = pad32(m.rot), dimp = pad32(m.dim), vp = pad32(m.vdim);
    w.gain_q = vec(dir, M + "dq.norm", m.q_rank, Qp);
    w.gain_kv = vec(dir, M + "dkv.norm", m.rank, Cp);
    std::vector<uint16_t> src, dst;
    auto read = [&](const std::string& name, int rows, int cols) {
        src.resize((size_t)rows * cols);
        dir.read_bf16(name, {rows, cols}, src.data());
    };
    // rows [r0, r0 + n) of `src` (width K) to row d0 of `dst`
    auto rows_to = [&](int d0, int r0, int n, int K) { memcpy(dst.data() + (size_t)d0 * K, src.data() + (size_t)r0 * K, (size_t)n * K * 2); };
    // [W_dq ; latent rows of W_dkv ; rotated rows of W_dkv], each padded
    dst.assign((size_t)(Qp + Cp + Rp) * D_, 0);
    read(M + "dq", m.q_rank, D_);
    rows_to(0, 0, m.q_rank, D_);
    read(M + "dkv", m.rank + m.rot, D_);
    rows_to(Qp, 0, m.rank, D_);
    rows_to(Qp + Cp, m.rank, m.rot, D_);
    w.in = tile(dst, Qp + Cp + Rp, D_);
    // W_uq: every head's unrotated rows, then every head's rotated rows
    read(M + "uq", H * QD, m.q_rank);
    dst.assign((size_t)H * (dimp + Rp) * m.q_rank, 0);
    for (int h = 0; h < H; h++) {
        rows_to(h * dimp, h * QD, m.dim, m.q_rank);
        rows_to(H * dimp + h * Rp, h * QD + m.dim, m.rot, m.q_rank);
    }
    w.uq = tile(dst, H * (dimp + Rp), m.q_rank);
    // W_uk transposed head by head: [rank, dim] per head
    read(M + "uk", H * m.dim, m.rank);
    dst.assign((size_t)H * Cp * m.dim, 0);
    for (int h = 0; h < H; h++)
        for (int d = 0; d < m.dim; d++) {
            const uint16_t* s = src.data() + ((size_t)h * m.dim + d) * m.rank;
            uint16_t* o = dst.data() + (size_t)h * Cp * m.dim + d;
            for (int c = 0; c < m.rank; c++) o[(size_t)c * m.dim] = s[c];
        }
    w.uk = tile(dst, H * Cp, m.dim, H);
    // W_uv head by head: [vdim, rank] per head
    read(M + "uv", H * m.vdim, m.rank);
    dst.assign((size_t)H * vp * m.rank, 0);
    for (int h = 0; h < H; h++) rows_to(h * vp, h * m.vdim, m.vdim, m.rank);
    w.uv = tile(dst, H * vp, m.rank, H);
    // W_o: columns padded head by head
    read(M + "o", D_, H * m.vdim);
    dst.assign((size_t)Dp_ * H * vp, 0);
    for (int n = 0; n < D_; n++)
        for (int h = 0; h < H; h++)
            memcpy(dst.data() + ((size_t)n * H + h) * vp, src.data() + ((size_t)n * H + h) * m.vdim, (size_t)m.vdim * 2);
    w.o = tile(dst, Dp_, H * vp);
    if (w.ff) {
        const int Fp = pad32(w.ff);
        // 16-row blocks alternating gate, up
        dst.assign((size_t)2 * Fp * D_, 0);
        std::vector<float> bias((size_t)2 * Fp, 0.f), b((size_t)w.ff);
        for (int half = 0; half < 2; half++) {
            const char* name = half ? "up" : "gate";
            read(P + name, w.ff, D_);
            dir.read_f32(P + name + ".b", {w.ff}, b.data());
            for (int r = 0; r < w.ff; r++) {
                const int to = (r / 16) * 32 + half * 16 + r % 16;
                rows_to(to, r, 1, D_);
                bias[to] = b[r];
            }
        }
        w.gateup = tile(dst, 2 * Fp, D_);
        w.bias_gu = upload(bias);
        read(P + "down", D_, w.ff);
        dst.assign((size_t)Dp_ * w.ff, 0);
        rows_to(0, 0, D_, w.ff);
        w.down = tile(dst, Dp_, w.ff);
        w.bias_down = vec(dir, P + "down.b", D_, Dp_);
    }
    layers_.push_back(w);
}

LatentHyperModel::LatentHyperModel(const ModelDir& dir, Config* p) {
    const Json& c = dir.config;
    f32_ = rt().compute_dtype == NVLLM_COMPUTE_F32;
    D_ = json_int(c, "width", "config");
    V_ = json_int(c, "vocab", "config");
    S_ = json_int(c, "streams", "config");
    eps_ = (float)json_num(json_get(c, "norm", Json::OBJECT, "config"), "eps", "config.norm");
    softcap_ = (float)json_num(c, "logit_softcap", "config");
    if (D_ < 1 || V_ < 1 || S_ < 1 || S_ > 64 || !(softcap_ > 0.f)) bad_config("width, vocab, streams or logit_softcap is out of range");
    Dp_ = f32_ ? D_ : pad32(D_);
    const Json& list = json_get(c, "layers", Json::ARRAY, "config");
    const int n_layers = (int)list.items.size();
    if (n_layers < 1) bad_config("it lists no layers");
    int start = 0, stop = 0, times = 1;
    const Json* loop = c.find("loop");
    if (loop && !loop->is_null()) {
        start = json_int(*loop, "start", "config.loop");
        stop = json_int(*loop, "stop", "config.loop");
        times = json_int(*loop, "times", "config.loop");
        if (start < 0 || stop < start || stop > n_layers || times < 0) bad_config("the loop does not fit the layers");
    }
    for (int i = 0; i < start; i++) runs_.push_back(i);
    for (int r = 0; r < times; r++)
        for (int i = start; i < stop; i++) runs_.push_back(i);
    for (int i = stop; i < n_layers; i++) runs_.push_back(i);
    for (int i = 0; i < n_layers; i++) load_layer(dir, i, list.items[i]);

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
    const float* final_w = vec(dir, "final.norm", D_, Dp_);
    const float* final_b = vec(dir, "final.norm.b", D_, Dp_);
    float final_alpha = 0.f;
    dir.read_f32("final.norm.alpha", {}, &final_alpha);

    // the sublayers in order, then their records
    int run = 0;
    for (int l : runs_) {
        subs_.push_back(Sublayer{l, 0, run, nullptr, nullptr, nullptr});
        if (layers_[l].ff) subs_.push_back(Sublayer{l, 1, run, nullptr, nullptr, nullptr});
        run++;
    }
    auto numbers = [&](const Sublayer& s, const char* what, const std::vector<long>& shape, float* out) {
        dir.read_f32("l" + std::to_string(s.layer) + ".hc" + std::to_string(s.part + 1) + "." + what, shape, out);
    };
    auto input_of = [&](size_t i, float* in) {   // in[s], then alpha, of sublayer i (past the last: the sum of the streams, final norm)
        if (i < subs_.size()) {
            numbers(subs_[i], "in", {S_}, in);
            dir.read_f32("l" + std::to_string(subs_[i].layer) + ".norm" + std::to_string(subs_[i].part + 1) + ".alpha", {}, in + S_);
        } else {
            for (int s = 0; s < S_; s++) in[s] = 1.f;
            in[S_] = final_alpha;
        }
    };
    std::vector<float> rec((size_t)hyper_record_floats(S_), 0.f);
    input_of(0, rec.data() + S_ * S_ + S_);
    first_record_ = upload(rec);
    for (size_t i = 0; i < subs_.size(); i++) {
        Sublayer& s = subs_[i];
        numbers(s, "mix", {S_, S_}, rec.data());
        numbers(s, "out", {S_}, rec.data() + S_ * S_);
        input_of(i + 1, rec.data() + S_ * S_ + S_);
        s.record = upload(rec);
        const bool last = i + 1 == subs_.size();
        s.next_w = last ? final_w : layers_[subs_[i + 1].layer].norm_w[subs_[i + 1].part];
        s.next_b = last ? final_b : layers_[subs_[i + 1].layer].norm_b[subs_[i + 1].part];
    }
    if (subs_.empty()) bad_config("no layer runs");

    const Mixer& m0 = layers_[0].m;
    p->dim = D_;
    p->hidden_dim = 1;
    for (const auto& l : layers_) p->hidden_dim = std::max(p->hidden_dim, l.ff);
    p->n_layers = (int)runs_.size();
    p->n_heads = m0.heads;
    p->n_kv_heads = 1;
    p->vocab_size = V_;
    p->max_seq_len = 2048;
    p->head_dim = m0.rank + m0.rot;
    p->rope_theta = (float)m0.base;
}

size_t LatentHyperModel::pool_bytes(int block_size, int num_blocks, int runs) const {
    size_t bytes = 0;
    for (int r = 0; r < runs; r++) {
        const Mixer& m = layers_[runs_[r]].m;
        bytes += latent_pool_bytes(latent_pool(nullptr, f32_ ? 4 : 2, block_size, m.rank, m.rot), num_blocks);
    }
    return bytes;
}

LatentPool LatentHyperModel::pool(const KVCacheManager* mgr, int run) const {
    const Mixer& m = layers_[runs_[run]].m;
    return latent_pool((char*)mgr->pool_k + pool_bytes(mgr->block_size, mgr->num_blocks, run), f32_ ? 4 : 2, mgr->block_size, m.rank, m.rot);
}

void LatentHyperModel::init_kv(KVCacheManager* mgr, int block_size, int num_blocks) {
    init_block_pool(mgr, block_size, num_blocks, pool_bytes(block_size, num_blocks, (int)runs_.size()));
}

void LatentHyperModel::forward(const PassArgs& a) {
    if (block_pool_bytes(a.mgr) != pool_bytes(a.mgr->block_size, a.mgr->num_blocks, (int)runs_.size()))
        NVLLM_FATAL("transformer_batch: the block pool was not made for this model (nvllm_init_model_kv)");
    for (int t = 0; t < a.T; t++)
        if (a.pos[t] < 0 || a.tokens[t] < 0 || a.tokens[t] >= V_) NVLLM_FATAL("transformer_batch: token %d (id %d, position %d) is out of range", t, a.tokens[t], a.pos[t]);
    const StepArrays st = stage_step(a.tokens, a.pos, a.seq_ids, a.T, a.output_indices, a.B, a.tables, nullptr, 0, a.mgr->block_size, LATENT_RUN, a.token_src, true);
    if (st.table_short) NVLLM_FATAL("transformer_batch: a position lies beyond its sequence's block table (allocate the block first)");
    if (f32_) forward_f32(a, st);
    else forward_b16(a, st);
}

void LatentHyperModel::forward_b16(const PassArgs& a, const StepArrays& st) {
    const int T = a.T, B = a.B;
    // workspaces of the widest layer
    int raw_ld = 0, q_row = 0, q_plain = 0, lat = 0, val = 0, ffp = 0, qlat = 0;
    for (const auto& l : layers_) {
        const Mixer& m = l.m;
        raw_ld = std::max(raw_ld, pad32(m.rank) + pad32(m.rot));
        q_row = std::max(q_row, m.heads * (pad32(m.rank) + pad32(m.rot)));
        q_plain = std::max(q_plain, m.heads * pad32(m.dim));
        lat = std::max(lat, m.heads * pad32(m.rank));
        val = std::max(val, m.heads * pad32(m.vdim));
        ffp = std::max(ffp, pad32(l.ff));
        qlat = std::max(qlat, pad32(m.q_rank));
    }
    float* x = (float*)ws_get(WS_STREAMS, (size_t)T * S_ * Dp_ * sizeof(float));
    __half* act = (__half*)ws_get(WS_A16_X, b16_halves(T, Dp_) * sizeof(__half));
    __half* hid = (__half*)ws_get(WS_A16_H, b16_halves(T, std::max(std::max(q_plain, val), ffp)) * sizeof(__half));   // unrotated queries, values, MLP: never two at once
    __half* qt = (__half*)ws_get(WS_A16_ATT, b16_halves(T, qlat) * sizeof(__half));
    float* ss = (float*)ws_get(WS_MISC, (size_t)T * (qlat / 32) * sizeof(float));
    float* raw = (float*)ws_get(WS_KV_RAW, (size_t)T * raw_ld * sizeof(float));
    __bf16* q = (__bf16*)ws_get(WS_Q_ROWS, (size_t)T * q_row * sizeof(__bf16));
    __half* latents = (__half*)ws_get(WS_LATENT, b16_halves(T, lat) * sizeof(__half));
    const bool fused = S_ <= 4;
    float* y = fused ? nullptr : (float*)ws_get(WS_F32_A, (size_t)T * Dp_ * sizeof(float));

    launch_embed_streams(x, embed_, true, st.d_tokens, T, S_, Dp_, st.d_tok_src, a.d_argmax);
    {
        HyperStep h{};
        h.x = x; h.record = first_record_; h.streams = S_; h.ld = Dp_; h.out_b16 = act;
        h.norm_w = layers_[subs_[0].layer].norm_w[0];
        h.norm_b = layers_[subs_[0].layer].norm_b[0];
        launch_hyper_step(h, T);
    }
    // a residual projection and the step to the next sublayer
    auto residual = [&](const B16Weight& w, const __half* in, const Sublayer& s, const float* bias, int cls) {
        const float* scale = layers_[s.layer].ls[s.part];
        GemmEpilogue e;
        if (fused) {
            e.kind = S_ <= 2 ? GemmEpilogue::HYPER_2 : GemmEpilogue::HYPER_4;
            e.x = x; e.bias = bias; e.hyper = s.record; e.hyper_scale = scale; e.norm_w = s.next_w; e.norm_b = s.next_b; e.streams = S_;
            e.a16_out = act;
            launch_gemm_b16(w, in, T, e, cls);
            return;
        }
        e.kind = GemmEpilogue::F32;
        e.out = y; e.ldo = Dp_;
        launch_gemm_b16(w, in, T, e, cls);
        HyperStep h{};
        h.x = x; h.y = y; h.bias = bias; h.scale = scale; h.record = s.record; h.norm_w = s.next_w; h.norm_b = s.next_b; h.out_b16 = act;
        h.streams = S_; h.ld = Dp_;
        launch_hyper_step(h, T);
    };
    for (const Sublayer& s : subs_) {
        const LayerWeightsDir& w = layers_[s.layer];
        const Mixer& m = w.m;
        if (s.part == 1) {
            GemmEpilogue e;
            e.kind = GemmEpilogue::SWIGLU_A16;
            e.bias = w.bias_gu;
            e.a16_out = hid;
            launch_gemm_b16(w.gateup, act, T, e, PC_GEMM_GATEUP);
            residual(w.down, hid, s, w.bias_down, PC_GEMM_DOWN);
            continue;
        }
        const float2* rope = rotation_table(m.base, m.rot, st.max_pos + 1);
        const int Qp = pad32(m.q_rank), Cp = pad32(m.rank), Rp = pad32(m.rot), dimp = pad32(m.dim);
        GemmEpilogue e1;
        e1.kind = GemmEpilogue::LATENT_IN;
        e1.latent_q = Qp; e1.gain_next = w.gain_q; e1.a16_out = qt; e1.ss_out = ss;
        e1.out = raw; e1.ldo = Cp + Rp;
        launch_gemm_b16(w.in, act, T, e1, PC_GEMM_LATENT_IN);
        const LatentPool pl = pool(a.mgr, s.run);
        const LatentKvRider ride = latent_kv_rider(pl, raw, Cp + Rp, Cp, w.gain_kv, eps_, rope, st);
        GemmEpilogue e2;
        e2.kind = GemmEpilogue::LATENT_Q;
        e2.ss_in = ss; e2.ss_tiles = Qp / 32; e2.d_in = m.q_rank; e2.eps = eps_;
        e2.q_plain = m.heads * dimp; e2.rot_ld = Rp; e2.rot_dim = m.rot; e2.rope = rope; e2.pos = st.d_pos;
        e2.a16_out = hid; e2.q_rows = q; e2.q_heads = m.heads; e2.q_row = Cp + Rp; e2.head_ld = Cp;
        launch_gemm_b16(w.uq, qt, T, e2, PC_GEMM_LATENT_Q, &ride);
        GemmEpilogue e3;
        e3.kind = GemmEpilogue::ROWS_B16;
        e3.q_rows = q; e3.q_heads = m.heads; e3.q_row = Cp + Rp; e3.head_ld = Cp;
        launch_gemm_b16(w.uk, hid, T, e3, PC_GEMM_ABSORB);
        LatentAttn at{};
        at.pool = pl; at.q = q; at.sink = w.sink; at.scale = m.scale; at.H = m.heads; at.out_b16 = latents;
        launch_latent_attention(at, st);
        GemmEpilogue e4;
        e4.kind = GemmEpilogue::TILE_B16;
        e4.a16_out = hid;
        launch_gemm_b16(w.uv, latents, T, e4, PC_GEMM_VALUE);
        residual(w.o, hid, s, nullptr, PC_GEMM_WO);
    }
    if (B <= 0) return;
    wait_for_row_copies();
    bool identity = B == T;
    for (int k = 0; identity && k < B; k++) identity = a.output_indices[k] == k;
    const __half* rows = act;
    if (!identity) {
        __half* g = (__half*)ws_get(WS_A16_ATT, b16_halves(B, std::max(Dp_, qlat)) * sizeof(__half));
        launch_gather_b16(g, act, st.d_out_idx, B, Dp_);
        rows = g;
    }
    GemmEpilogue e;
    e.kind = GemmEpilogue::F32;
    e.out = a.d_logits; e.ldo = V_; e.softcap = softcap_;
    e.amax_out = a.d_argmax;
    e.amax_out_host = a.argmax_host;
    e.amax_ld = (B + 63) & ~63;
    e.amax_pairs = (float2*)ws_get(WS_AMAX_PAIRS, (size_t)cdiv(V_, 32) * e.amax_ld * sizeof(float2));
    launch_gemm_b16(head_, rows, B, e, PC_GEMM_HEAD);
}

void LatentHyperModel::forward_f32(const PassArgs& a, const StepArrays& st) {
    const int T = a.T, B = a.B;
    size_t wide = D_, kv = 0, q_row = 0, lat = 0;
    for (const auto& l : layers_) {
        const Mixer& m = l.m;
        wide = std::max(wide, (size_t)std::max(std::max(m.heads * (m.dim + m.rot), m.heads * m.vdim), std::max(l.ff, m.q_rank)));
        kv = std::max(kv, (size_t)m.rank + m.rot);
        q_row = std::max(q_row, (size_t)m.heads * (m.rank + m.rot));
        lat = std::max(lat, (size_t)m.heads * m.rank);
    }
    auto rows = [&](WsSlot slot, size_t n) { return (float*)ws_get(slot, (size_t)T * n * sizeof(float)); };
    float *x = rows(WS_STREAMS, (size_t)S_ * D_), *act = rows(WS_F32_A, D_), *b = rows(WS_F32_B, wide), *c = rows(WS_F32_C, wide);
    float *raw = rows(WS_KV_RAW, kv), *q = rows(WS_Q_ROWS, q_row), *latents = rows(WS_LATENT, lat);
    launch_embed_streams(x, embed_, false, st.d_tokens, T, S_, D_, st.d_tok_src, a.d_argmax);
    auto step = [&](const float* y, const float* bias, const float* scale, const float* record, const float* nw, const float* nb) {
        HyperStep h{};
        h.x = x; h.y = y; h.bias = bias; h.scale = scale; h.record = record; h.norm_w = nw; h.norm_b = nb; h.out_f32 = act;
        h.streams = S_; h.ld = D_;
        launch_hyper_step(h, T);
    };
    step(nullptr, nullptr, nullptr, first_record_, layers_[subs_[0].layer].norm_w[0], layers_[subs_[0].layer].norm_b[0]);
    for (const Sublayer& s : subs_) {
        const LayerWeightsDir& w = layers_[s.layer];
        const Mixer& m = w.m;
        const int H = m.heads;
        if (s.part == 1) {
            launch_matmul_f32w(b, act, w.gate, T, D_, w.ff);
            launch_matmul_f32w(c, act, w.up, T, D_, w.ff);
            launch_swiglu_bias(b, b, c, w.bias_gate, w.bias_up, T, w.ff);
            launch_matmul_f32w(c, b, w.down32, T, w.ff, D_);
            step(c, w.bias_down, w.ls[1], s.record, s.next_w, s.next_b);
            continue;
        }
        const float2* rope = rotation_table(m.base, m.rot, st.max_pos + 1);
        launch_matmul_f32w(b, act, w.dq, T, D_, m.q_rank);
        launch_rmsnorm_f32(b, b, w.gain_q, m.q_rank, T, eps_);
        launch_matmul_f32w(c, b, w.uq32, T, m.q_rank, H * (m.dim + m.rot));
        launch_latent_q_f32(q, c, w.uk32, rope, st.d_pos, T, H, m.dim, m.rot, m.rank);
        launch_matmul_f32w(raw, act, w.dkv, T, D_, m.rank + m.rot);
        const LatentPool pl = pool(a.mgr, s.run);
        launch_latent_kv(pl, raw, m.rank + m.rot, m.rank, w.gain_kv, eps_, rope, st);
        LatentAttn at{};
        at.pool = pl; at.q = q; at.sink = w.sink; at.scale = m.scale; at.H = H; at.out_f32 = latents;
        launch_latent_attention(at, st);
        launch_latent_v_f32(b, latents, w.uv32, T, H, m.vdim, m.rank);
        launch_matmul_f32w(c, b, w.o32, T, H * m.vdim, D_);
        step(c, nullptr, w.ls[0], s.record, s.next_w, s.next_b);
    }
    if (B <= 0) return;
    wait_for_row_copies();
    launch_gather_rows_f32(b, act, st.d_out_idx, B, D_);
    launch_matmul_f32w(a.d_logits, b, (const float*)embed_, B, D_, V_);
    launch_softcap(a.d_logits, softcap_, (long)B * V_);
    launch_argmax_ld(a.d_argmax, a.d_logits, B, V_, V_, a.argmax_host);
}

}  // namespace

DirModel* load_latent_hyper_model(const ModelDir& dir, Config* p) { return new LatentHyperModel(dir, p); }

}  // namespace nvllm
