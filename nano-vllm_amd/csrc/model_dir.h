// model_dir.h -- a model that comes as a folder: config.json (its "architecture" names the design) and
// model.safetensors (an 8-byte little-endian length, that many bytes of JSON: name -> dtype, shape,
// data_offsets, then the data).  The tensor file is mapped, not read: a loader touches each tensor once,
// on its way to HBM.  The registry at the end of model.hip maps architecture names to loaders.
#pragma once

#include <cstdint>
#include <string>
#include <unordered_map>
#include <vector>

#include "json.h"
#include "nvllm_internal.h"
#include "step_arrays.h"

namespace nvllm {

struct TensorRef {
    std::string dtype;            // "BF16", "F32", "F16", "I32"
    std::vector<long> shape;      // empty: a scalar
    const unsigned char* data = nullptr;
    long count() const {
        long n = 1;
        for (long d : shape) n *= d;
        return n;
    }
};

class ModelDir {
public:
    explicit ModelDir(const char* path);   // ends the process with a message when a file is missing or malformed
    ~ModelDir();
    ModelDir(const ModelDir&) = delete;
    ModelDir& operator=(const ModelDir&) = delete;

    Json config;
    // the tensor, or an end with a message when it is missing or its shape differs
    const TensorRef& tensor(const std::string& name, const std::vector<long>& shape) const;
    // its elements as fp32 (exact) or as bf16 bit patterns (rounded to nearest even if the file holds a wider type)
    void read_f32(const std::string& name, const std::vector<long>& shape, float* out) const;
    void read_bf16(const std::string& name, const std::vector<long>& shape, uint16_t* out) const;

private:
    std::unordered_map<std::string, TensorRef> tensors_;
    void* map_ = nullptr;
    size_t map_bytes_ = 0;
};

// One forward pass over one ragged batch, as a design's forward() sees it.
struct PassArgs {
    const int* tokens;            // host arrays of the batch (T entries; output rows: B entries)
    const int* pos;
    const int* seq_ids;
    const int* output_indices;
    const int* token_src;         // optional: >= 0 names the output row of the previous pass that the token continues
    int T, B;
    BlockTable** tables;
    KVCacheManager* mgr;
    float* d_logits;              // [B, vocab] in HBM: to be filled
    int* d_argmax;                // [B] in HBM: to be filled; holds the previous pass's indices on entry
    int* argmax_host;             // optional: the indices also go to this page-locked array
};

// A design loaded from a folder.  One subclass per design; everything a subclass needs from the rest of
// the library goes through this interface and the kernel launchers.
class DirModel {
public:
    virtual ~DirModel() {}
    virtual void init_kv(KVCacheManager* mgr, int block_size, int num_blocks) = 0;
    // room for the state that `slots` sequences carry from token to token (a sequence's slot is its id)
    virtual void init_states(int slots) { (void)slots; }
    virtual void forward(const PassArgs& a) = 0;
};

// What designs share: tensors on their way from the file to HBM.
class HbmModel : public DirModel {
public:
    ~HbmModel() override {
        for (void* b : bufs_) device_free(b);
    }

protected:
    void* alloc(size_t bytes, const char* what);
    float* upload(const std::vector<float>& v);
    float* vec(const ModelDir& dir, const std::string& name, int n, int n_pad);   // padded with zeros
    float* matrix_f32(const ModelDir& dir, const std::string& name, int rows, int cols);
    // row-major bf16 [N][K] on the host -> tiles in HBM, K padded to 32
    B16Weight tile(const std::vector<uint16_t>& rm, int N, int K, int groups = 1);

private:
    std::vector<void*> bufs_;
};
[[noreturn]] void bad_config(const char* what);   // ends the process with a message about config.json
inline int pad32(int n) { return (n + 31) & ~31; }
typedef DirModel* (*DirModelLoader)(const ModelDir& dir, Config* p);
DirModel* load_latent_hyper_model(const ModelDir& dir, Config* p);   // latent_model.hip
DirModel* load_hybrid_model(const ModelDir& dir, Config* p);         // hybrid_model.hip

// ops_api.hip: host bookkeeping of a block pool whose storage is ONE HBM buffer of `bytes` bytes (pool_v stays null)
void init_block_pool(KVCacheManager* mgr, int block_size, int num_blocks, size_t bytes);
size_t block_pool_bytes(const KVCacheManager* mgr);   // of such a pool; 0 for any other
// model.hip: the folder model loaded last, if its Config says these numbers
DirModel* current_dir_model(int n_layers, int n_kv_heads, int head_dim);

// model.hip: the previous pass's result rows have left the workspaces the classifier writes
void wait_for_row_copies();

}  // namespace nvllm
