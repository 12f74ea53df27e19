// The mixers of a BlockSpec's layers (block_mixers.hip): what a layer does between its norm and its output product.  A mixer owns its
// packed weights; its cache or state belongs to the layer run and is handed in.
#pragma once

#include <map>
#include <memory>
#include <string>
#include <utility>
#include <vector>

#include "checkpoint.h"
#include "model.h"

namespace fh {

inline uint32_t pad_to(uint32_t n, uint32_t to) { return (n + to - 1) / to * to; }

// A matrix put together on the host, then uploaded.
struct MatrixBuilder {
    DType t;
    uint32_t N, K;
    std::vector<uint8_t> bytes;
    MatrixBuilder(DType type, uint32_t n, uint32_t k) : t(type), N(n), K(k), bytes((size_t)n * k * dtype_size(type)) {}
    // row `row`, columns col.. <- n elements of tensor row src_row from src_col on
    void put(uint32_t row, uint32_t col, const TensorView& v, uint32_t src_row, uint32_t src_col, uint32_t n) {
        uint8_t* dst = bytes.data() + ((size_t)row * K + col) * dtype_size(t);
        const uint64_t first = (uint64_t)src_row * v.shape[1] + src_col;
        if (t == DType::BF16) v.read_bf16(first, n, (uint16_t*)dst);
        else v.read_f32(first, n, (float*)dst);
    }
    int32_t upload(DevBuf* buf, DenseWeight* w) const;
};

// Angle tables, one per kind of rotation: cos and sin [max_seq][dims / 2].
struct RotaryTables {
    std::map<RotarySpec, std::pair<DevBuf, DevBuf>> tables;
    int32_t get(const RotarySpec& r, uint32_t max_seq, const float** cos_t, const float** sin_t);
};
// Place of rotated dimension j of a head in the packed matrices: pairs side by side, what does not turn behind them.
inline uint32_t rotated_place(uint32_t j, uint32_t dims) { return j < dims / 2 ? 2 * j : j < dims ? 2 * (j - dims / 2) + 1 : j; }

// What loading a layer's parts needs.
struct BlockLoad {
    const SafeTensors& st;
    DType t;
    uint32_t spec_width, width;          // of the stream: real, padded
    uint32_t max_seq;
    double eps;
    RotaryTables& rotary;
};

// Scratch areas that all layers share: every layer says what it wants, the largest wish is granted.
struct BlockScratch {
    enum Area { RAW, GATE, OUT, Q, K, V, CQ, QL, PARTS, WORK, AREAS };
    size_t want[AREAS] = {};
    DevBuf buf[AREAS];
    void need(Area a, size_t bytes) { want[a] = std::max(want[a], bytes); }
    int32_t alloc();
    void* p(Area a) const { return buf[a].p; }
    float* f(Area a) const { return buf[a].as<float>(); }
};

// M rows at base_pos (or, one row, at *pos_dev); `in` is the layer's input for the mixer's first product.
struct MixerCall {
    forge_hip_model* model;
    DenseIn in;
    void* cache;
    uint32_t M, base_pos;
    const uint32_t* pos_dev;
    const BlockScratch& scratch;
};

struct Mixer {
    DType t = DType::BF16;
    uint32_t max_seq = 0;
    DenseWeight o;                       // the output product
    DevBuf b_o;

    virtual ~Mixer() = default;
    virtual size_t cache_bytes() const = 0;
    virtual void plan(BlockScratch* s, uint32_t rows) const = 0;
    // Everything up to the output product; returns that product's input.
    virtual DenseIn enqueue(const MixerCall& c) const = 0;
    virtual int decode_launches() const = 0;

    // W_o [width][heads * vdim] with each head's columns padded to `head` and their number to a multiple of 64
    int32_t load_output(const BlockLoad& l, const std::string& name, uint32_t heads, uint32_t vdim, uint32_t head);
};

// `name`: the prefix of the mixer's tensors; `at`: the layer, for messages.
int32_t load_mixer(const BlockLoad& l, const LayerSpec& spec, const std::string& name, const std::string& at, std::unique_ptr<Mixer>* out);
// The fields of forge_hip_config that come from a layer's mixer.
void describe_mixer(const LayerSpec& spec, forge_hip_config* c);

}  // namespace fh
