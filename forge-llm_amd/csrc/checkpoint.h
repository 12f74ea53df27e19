// A model folder: config.json (which names the architecture) and model.safetensors.  The registry turns the configuration of
// any known architecture into a BlockSpec, the description block_model.hip builds a network from.  Host code, no GPU.
#pragma once

#include <stdint.h>

#include <map>
#include <memory>
#include <string>
#include <tuple>
#include <vector>

namespace fh {

// ---- JSON ------------------------------------------------------------------------------------
struct Json {
    enum Kind { Null, Bool, Number, String, Array, Object } kind = Null;
    bool b = false;
    double num = 0;
    std::string str;
    std::vector<Json> arr;
    std::map<std::string, Json> obj;
    const Json* get(const std::string& key) const {          // nullptr: no such member
        const auto it = obj.find(key);
        return kind == Object && it != obj.end() ? &it->second : nullptr;
    }
};
// FORGE_HIP_OK, or FORGE_HIP_ERR_INVALID with a message that says where the text goes wrong.
int32_t json_parse(const char* text, size_t n, Json* out);

// ---- safetensors -------------------------------------------------------------------------------
struct TensorView {
    enum Type { BF16, F16, F32, I32 } type = BF16;
    std::vector<uint64_t> shape;
    const uint8_t* data = nullptr;
    uint64_t numel() const { uint64_t n = 1; for (uint64_t d : shape) n *= d; return n; }
    float at(uint64_t i) const;                              // element i as a float (not for I32)
    // elements [first, first + n) as floats / as bfloat16 bits (rounded to nearest even)
    void read_f32(uint64_t first, uint64_t n, float* out) const;
    void read_bf16(uint64_t first, uint64_t n, uint16_t* out) const;
};

class SafeTensors {
public:
    SafeTensors() = default;
    SafeTensors(const SafeTensors&) = delete;
    SafeTensors& operator=(const SafeTensors&) = delete;
    ~SafeTensors();
    int32_t open(const std::string& path);
    const TensorView* find(const std::string& name) const {
        const auto it = tensors_.find(name);
        return it == tensors_.end() ? nullptr : &it->second;
    }
    // The tensor, which must have exactly this shape.
    int32_t get(const std::string& name, const std::vector<uint64_t>& shape, const TensorView** out) const;

private:
    std::map<std::string, TensorView> tensors_;
    void* map_ = nullptr;
    size_t map_bytes_ = 0;
};

// ---- network description -------------------------------------------------------------------------
struct RotarySpec {
    uint32_t dims = 0;                   // dimension i turns against i + dims / 2 by position * frequency(i)
    double base = 0;
    // Stretched frequencies: waves longer than original / low turn `factor` times slower, those shorter than original / high as they
    // are, with a blend between.  factor = 0: none.
    double factor = 0, low = 0, high = 0, original = 0;
    double frequency(uint32_t i) const;  // base^(-2 i / dims), stretched
    bool operator<(const RotarySpec& o) const {
        return std::tie(dims, base, factor, low, high, original) < std::tie(o.dims, o.base, o.factor, o.low, o.high, o.original);
    }
};
struct LatentAttentionSpec {
    uint32_t heads = 0, dim = 0, rot_dim = 0, vdim = 0, q_rank = 0, kv_rank = 0;
    uint32_t window = 0;                 // a position sees itself and the window - 1 before it; 0: all of them
    double scale = 0;
    RotarySpec rot;
};
// Grouped-query attention: queries and keys normed per head (RMS) and rotated, a sigmoid gate on the heads' output.
struct GroupedAttentionSpec {
    uint32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    double scale = 0;
    RotarySpec rot;
};
// Gated linear attention: a decay per key channel, sigmoid(low-rank map)^(1 / tau); the map's rank is its tensors'.
struct LinearAttentionSpec {
    uint32_t heads = 0, dim = 0, vdim = 0;
    double tau = 0;
};
enum class MixerKind { LatentAttention, GroupedAttention, LinearAttention };
enum class FeedForwardKind { None, SiluGated, GeluTanhGated };
enum class NormKind { DynTanh, LayerNorm };
struct LayerSpec {
    MixerKind mixer = MixerKind::LatentAttention;
    LatentAttentionSpec latent;
    GroupedAttentionSpec grouped;
    LinearAttentionSpec linear;
    FeedForwardKind ff = FeedForwardKind::None;
    uint32_t ff_size = 0;
    uint32_t weights = 0;                // the layer whose tensors this one runs with (its own index, or another's)
};
struct BlockSpec {
    std::string architecture;
    uint32_t width = 0, vocab = 0;
    double embedding_scale = 1, eps = 0;
    NormKind norm = NormKind::DynTanh;
    bool post_norms = false;             // a norm behind each sublayer, ahead of the residual sum
    bool tied_head = false;              // the embedding table is the output matrix
    double logit_cap = 0;                // logits <- cap tanh(logits / cap); 0: as they are
    std::vector<LayerSpec> layers;
    // layers [loop_start, loop_stop) run loop_times times in a row with the same weights and a cache per pass; ahead of each
    // pass x <- W [x; embedding output].  loop_times = 0: no loop.
    uint32_t loop_start = 0, loop_stop = 0, loop_times = 0;
};
// Whether `architecture` is in the registry.
bool architecture_known(const std::string& architecture);
// config.json's text -> spec, by its "architecture".
int32_t block_spec_from_config(const Json& config, BlockSpec* out);
int32_t block_spec_from_folder(const std::string& dir, BlockSpec* out);

}  // namespace fh
