// model_dir.hip -- reading a model folder, and its tensors' way to HBM (model_dir.h).
#include "model_dir.h"

#include <cstring>
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace nvllm {

[[noreturn]] static void die(const std::string& what) {
    fprintf(stderr, "nvllm: %s\n", what.c_str());
    exit(1);
}

static std::string shape_text(const std::vector<long>& s) {
    std::string t = "[";
    for (size_t i = 0; i < s.size(); i++) t += (i ? ", " : "") + std::to_string(s[i]);
    return t + "]";
}

ModelDir::ModelDir(const char* path) {
    const std::string dir(path), cfg = dir + "/config.json", st = dir + "/model.safetensors";
    FILE* f = fopen(cfg.c_str(), "rb");
    if (!f) die("cannot open " + cfg);
    std::string text;
    char buf[4096];
    for (size_t n; (n = fread(buf, 1, sizeof buf, f)) > 0;) text.append(buf, n);
    fclose(f);
    config = JsonReader(text.data(), text.size(), "config.json").document();

    const int fd = open(st.c_str(), O_RDONLY);
    if (fd < 0) die("cannot open " + st);
    struct stat info;
    if (fstat(fd, &info) != 0 || info.st_size < 8) die(st + " is too short");
    map_bytes_ = (size_t)info.st_size;
    map_ = mmap(nullptr, map_bytes_, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (map_ == MAP_FAILED) die("cannot map " + st);
    const unsigned char* base = (const unsigned char*)map_;
    uint64_t header = 0;
    for (int i = 7; i >= 0; i--) header = header << 8 | base[i];
    if (header > map_bytes_ - 8) die(st + ": the header runs past the end of the file");
    const size_t data0 = 8 + (size_t)header, data_bytes = map_bytes_ - data0;
    const Json h = JsonReader((const char*)base + 8, (size_t)header, "the safetensors header").document();
    for (const auto& m : h.members) {
        if (m.first == "__metadata__") continue;
        const Json* dt = m.second.find("dtype");
        const Json* sh = m.second.find("shape");
        const Json* off = m.second.find("data_offsets");
        if (!dt || !sh || !off || off->items.size() != 2) die(st + ": tensor '" + m.first + "' is not described");
        TensorRef t;
        t.dtype = dt->text;
        for (const Json& d : sh->items) t.shape.push_back((long)d.number);
        const int esz = t.dtype == "BF16" || t.dtype == "F16" ? 2 : t.dtype == "F32" || t.dtype == "I32" ? 4 : 0;
        if (!esz) die(st + ": tensor '" + m.first + "' has the unknown type " + t.dtype);
        const size_t b = (size_t)off->items[0].number, e = (size_t)off->items[1].number;
        if (b > e || e > data_bytes || e - b != (size_t)t.count() * esz) die(st + ": tensor '" + m.first + "' does not fit its bytes");
        t.data = base + data0 + b;
        tensors_.emplace(m.first, std::move(t));
    }
}

ModelDir::~ModelDir() {
    if (map_) munmap(map_, map_bytes_);
}

const TensorRef& ModelDir::tensor(const std::string& name, const std::vector<long>& shape) const {
    auto it = tensors_.find(name);
    if (it == tensors_.end()) die("model.safetensors has no tensor '" + name + "'");
    if (it->second.shape != shape) die("tensor '" + name + "' is " + shape_text(it->second.shape) + ", config.json asks for " + shape_text(shape));
    return it->second;
}

void ModelDir::read_f32(const std::string& name, const std::vector<long>& shape, float* out) const {
    const TensorRef& t = tensor(name, shape);
    const long n = t.count();
    if (t.dtype == "F32") {
        memcpy(out, t.data, (size_t)n * 4);
    } else if (t.dtype == "BF16") {
        for (long i = 0; i < n; i++) {
            uint16_t v;
            memcpy(&v, t.data + 2 * i, 2);
            const uint32_t u = (uint32_t)v << 16;
            memcpy(out + i, &u, 4);
        }
    } else {
        die("tensor '" + name + "' has type " + t.dtype + ", a bf16 or fp32 tensor was expected");
    }
}

void ModelDir::read_bf16(const std::string& name, const std::vector<long>& shape, uint16_t* out) const {
    const TensorRef& t = tensor(name, shape);
    const long n = t.count();
    if (t.dtype == "BF16") {
        memcpy(out, t.data, (size_t)n * 2);
    } else if (t.dtype == "F32") {
        for (long i = 0; i < n; i++) {
            uint32_t u;
            memcpy(&u, t.data + 4 * i, 4);
            out[i] = (u & 0x7fffffffu) > 0x7f800000u ? (uint16_t)0x7fc0 : (uint16_t)((u + 0x7fffu + ((u >> 16) & 1u)) >> 16);
        }
    } else {
        die("tensor '" + name + "' has type " + t.dtype + ", a bf16 or fp32 tensor was expected");
    }
}

void bad_config(const char* what) {
    fprintf(stderr, "nvllm: config.json: %s\n", what);
    exit(1);
}

void* HbmModel::alloc(size_t bytes, const char* what) {
    void* d = nullptr;
    if (device_malloc(&d, bytes) != 0) NVLLM_FATAL("cannot allocate %zu bytes of HBM for %s", bytes, what);
    bufs_.push_back(d);
    return d;
}
float* HbmModel::upload(const std::vector<float>& v) {
    float* d = (float*)alloc(v.size() * sizeof(float), "a vector");
    device_memcpy(d, v.data(), v.size() * sizeof(float), HOST_TO_DEVICE);
    return d;
}
float* HbmModel::vec(const ModelDir& dir, const std::string& name, int n, int n_pad) {
    std::vector<float> v((size_t)n_pad, 0.f);
    dir.read_f32(name, {n}, v.data());
    return upload(v);
}
float* HbmModel::matrix_f32(const ModelDir& dir, const std::string& name, int rows, int cols) {
    std::vector<float> v((size_t)rows * cols);
    dir.read_f32(name, {rows, cols}, v.data());
    return upload(v);
}
B16Weight HbmModel::tile(const std::vector<uint16_t>& rm, int N, int K, int groups) {
    const int Kp = pad32(K), Nb = cdiv(N, 16);
    B16Weight w;
    w.N = N;
    w.K = Kp;
    w.groups = groups;
    __half* tiles = (__half*)alloc((size_t)Nb * (Kp / 32) * TILE_HALVES * 2, "a projection");
    void* stage = nullptr;
    if (device_malloc(&stage, rm.size() * 2) != 0) NVLLM_FATAL("no memory for a load buffer of %zu bytes", rm.size() * 2);
    device_memcpy(stage, rm.data(), rm.size() * 2, HOST_TO_DEVICE);
    launch_tile_weights(tiles, (const __half*)stage, N, K, (long)(Kp / 32) * TILE_HALVES);   // moves 16-bit patterns
    device_free(stage);
    w.tiles = tiles;
    return w;
}

}  // namespace nvllm
