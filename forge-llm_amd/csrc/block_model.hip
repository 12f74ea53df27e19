// The network of a BlockSpec (checkpoint.h): a residual stream in 32-bit, layers of a mixer (block_mixer.h) and an optional gated
// feed-forward, norms ahead of (and, where the design has them, behind) each sublayer, a run of layers that may be looped, layers
// that may run with another layer's weights.  Weights, activations and cache are bfloat16 or 32-bit (DType), dense.
//
// One routine enqueues the layers for M rows: a prompt chunk, or the one row of a decode step (position in device memory, so
// that the step can be a graph).  Norms:
//   Dynamic Tanh is elementwise, so no kernel is its own: the product that ends a sublayer carries "post-norm, residual, next norm" in
//   its epilogue and leaves the next sublayer's input beside the stream.
//   A layer norm needs the whole row: a prompt's rows go through a kernel of their own, a decode step's row is normed on its way
//   into the product that reads it.
// Per layer run: the mixer, W_o + residual, [gate; up] + activation, down + residual.
#include <math.h>
#include <stdlib.h>
#include <string.h>

#include "block_mixer.h"

using namespace fh;

namespace {

constexpr uint32_t HEAD_ROWS = 64;           // rows of one lm_head product of a prompt
constexpr uint32_t DEFAULT_MAX_SEQ = 4096;   // config.json names no context length

// The fields of forge_hip_config that a spec fills (per-layer sizes: the first attention layer's, or the first layer's; inter: the largest).
void describe(const BlockSpec& s, forge_hip_config* c) {
    *c = forge_hip_config{};
    c->hidden = s.width;
    c->layers = (uint32_t)s.layers.size();
    c->vocab = s.vocab;
    c->rms_eps = (float)s.eps;
    const LayerSpec* first = &s.layers[0];
    for (size_t i = s.layers.size(); i-- > 0;)
        if (s.layers[i].mixer != MixerKind::LinearAttention) first = &s.layers[i];
    describe_mixer(*first, c);
    for (const LayerSpec& l : s.layers) c->inter = std::max(c->inter, l.ff_size);
}

// A norm of the stream; neither: the stream itself.
struct BlockNorm {
    DynTanh tanh;
    LayerNorm ln;
};

struct BlockLayer {
    std::unique_ptr<Mixer> mixer;
    DenseWeight gate_up, down;
    DevBuf b_gate_up, b_down, b_norms;
    BlockNorm norm1, norm1b, norm2, norm2b;
    uint32_t ff = 0;                         // 0: no feed-forward
    Act act = Act::Silu;
};

struct LayerRun {
    uint32_t layer;                          // index of the layer whose tensors it runs with
    bool pass_start;                         // the loop's input product comes first
    size_t cache;                            // byte offset of this run's cache or state
};

struct BlockModel : forge_hip_model {
    BlockSpec spec;
    DType t = DType::BF16;
    uint32_t width = 0;                      // padded width of the stream
    std::vector<std::unique_ptr<BlockLayer>> layers;      // null: a layer without tensors of its own
    std::vector<LayerRun> runs;
    RotaryTables rotary;
    DenseWeight loop_in, head;
    BlockNorm final_norm;
    const void* table = nullptr;             // embedding rows of table_ld elements
    uint32_t table_ld = 0;
    DevBuf b_embed, b_loop, b_head, b_final, b_cache;
    DevBuf x, h, xcat, act, rows_sel, h_sel; // of one prompt chunk
    BlockScratch scratch;

    uint32_t logits_rows_max() const override { return HEAD_ROWS; }
    uint32_t layer_runs() const override { return (uint32_t)runs.size(); }

    int32_t load(const std::string& dir, uint32_t max_seq, uint32_t flags);
    int32_t load_layer(const BlockLoad& l, uint32_t i);
    int32_t load_norm(const SafeTensors& st, const std::string& name, DevBuf* buf, uint32_t slot, BlockNorm* out);
    int32_t alloc_scratch();

    bool elementwise_norms() const { return spec.norm == NormKind::DynTanh; }
    // Where the input of run i goes and how it is made from the stream, for elementwise norms.
    struct Next { DynTanh norm; void* out; uint32_t ld; };
    Next next_input(size_t i) const {
        if (!elementwise_norms()) return {DynTanh{}, nullptr, 0};
        if (i == runs.size()) return {final_norm.tanh, h.p, width};
        if (runs[i].pass_start) return {DynTanh{}, xcat.p, 2 * width};
        return {layers[runs[i].layer]->norm1.tanh, h.p, width};
    }
    Next next_ff(const BlockLayer& L) const { return elementwise_norms() ? Next{L.norm2.tanh, h.p, width} : Next{DynTanh{}, nullptr, 0}; }
    // The stream behind `n` as a product's input.  Elementwise norms: the last epilogue has made it.
    DenseIn normed(const BlockNorm& n, uint32_t M) {
        if (elementwise_norms()) return dense_rows(h.p, width);
        if (M == 1) {
            DenseIn in;
            in.kind = DenseIn::Normed;
            in.f32 = x.as<float>();
            in.ln = n.ln;
            return in;
        }
        enqueue_layer_norm(n, M);
        return dense_rows(h.p, width);
    }
    void enqueue_layer_norm(const BlockNorm& n, uint32_t M) {
        StageMark m(this, ST_RMSNORM);
        launch_layer_norm(t, x.as<float>(), width, n.ln, width, M, h.p, width, stream);
    }
    void enqueue_embedding(const uint32_t* tokens, uint32_t M);
    void enqueue_run(size_t i, uint32_t M, uint32_t base_pos, const uint32_t* pos_dev);
    void enqueue_final_norm(uint32_t M) {
        if (!elementwise_norms()) enqueue_layer_norm(final_norm, M);
    }

    void enqueue_decode_step() override {
        enqueue_embedding(d_token(), 1);
        for (size_t i = 0; i < runs.size(); i++) enqueue_run(i, 1, 0, d_pos());
        enqueue_final_norm(1);
        enqueue_row_logits(0);
        enqueue_argmax(true, true);
    }
    int32_t enqueue_prompt_rows(uint32_t rows, uint32_t base_pos) override {
        enqueue_embedding(ptok.as<uint32_t>(), rows);
        for (size_t i = 0; i < runs.size(); i++) enqueue_run(i, rows, base_pos, nullptr);
        enqueue_final_norm(rows);
        return FORGE_HIP_OK;
    }
    void enqueue_logits(const void* rows, uint32_t n) {
        DenseEpiArgs e;
        e.f32 = logits.as<float>();
        e.ld_f32 = cfg.vocab;
        e.cap = (float)spec.logit_cap;
        launch_dense(t, head, dense_rows(rows, width), n, DenseEpi::F32, e, stream);
    }
    void enqueue_row_logits(uint32_t row) override {
        StageMark m(this, ST_LM_HEAD);
        enqueue_logits(h.as<uint8_t>() + (size_t)row * width * dtype_size(t), 1);
    }
    void enqueue_rows_logits(const uint32_t* rows, uint32_t n) override {
        if (n == 1) { enqueue_row_logits(rows[0]); return; }
        StageMark m(this, ST_LM_HEAD);
        (void)hipMemcpyAsync(rows_sel.p, rows, n * 4, hipMemcpyHostToDevice, stream);       // pageable source: staged when the call returns
        launch_gather_rows(t, h.p, width, rows_sel.as<uint32_t>(), n, width, h_sel.p, width, stream);
        enqueue_logits(h_sel.p, n);
    }
    int32_t decode_launches() const override {
        int n = 1 + (elementwise_norms() ? 0 : 1) + 1 + 2;       // embedding, final norm, lm_head, argmax
        for (const LayerRun& r : runs) n += (r.pass_start ? 1 : 0) + layers[r.layer]->mixer->decode_launches() + 1 + (layers[r.layer]->ff ? 2 : 0);
        return n;
    }
    int32_t prompt_residuals(uint32_t rows, float* out_host) override {
        enqueue_embedding(ptok.as<uint32_t>(), rows);
        for (size_t i = 0; i < runs.size(); i++) {
            enqueue_run(i, rows, 0, nullptr);
            FH_HIP(hipStreamSynchronize(stream));
            FH_HIP(hipMemcpy2D(out_host + i * rows * spec.width, (size_t)spec.width * 4, x.p, (size_t)width * 4, (size_t)spec.width * 4, rows,
                               hipMemcpyDeviceToHost));
        }
        return FORGE_HIP_OK;
    }
};

void BlockModel::enqueue_embedding(const uint32_t* tokens, uint32_t M) {
    StageMark m(this, ST_EMBED);
    const Next nx = next_input(0);
    // the embedding output is the second half of the loop product's input for the whole chunk
    void* x0 = loop_in.p ? xcat.as<uint8_t>() + width * dtype_size(t) : nullptr;
    launch_dense_embedding(t, table, table_ld, spec.width, (float)spec.embedding_scale, tokens, M, x.as<float>(), width, nx.norm, nx.out, nx.ld, x0,
                           2 * width, counts.as<uint32_t>(), stream);
}

void BlockModel::enqueue_run(size_t i, uint32_t M, uint32_t base_pos, const uint32_t* pos_dev) {
    const LayerRun& r = runs[i];
    const BlockLayer& L = *layers[r.layer];
    // what ends a sublayer: stream = post(product) (+ stream), next input = norm(stream)
    auto residual = [&](const DenseWeight& w, const DenseIn& in, const DynTanh& post, bool add, const Next& nx, int stage) {
        StageMark m(this, stage);
        DenseEpiArgs e;
        e.f32 = x.as<float>();
        e.ld_f32 = width;
        e.post = post;
        e.add = add;
        e.next = nx.norm;
        e.out = nx.out;
        e.ld_out = nx.ld;
        launch_dense(t, w, in, M, DenseEpi::Residual, e, stream);
    };
    if (r.pass_start) residual(loop_in, dense_rows(xcat.p, 2 * width), DynTanh{}, false, Next{L.norm1.tanh, h.p, width}, ST_QKV);
    const DenseIn heads = L.mixer->enqueue({this, normed(L.norm1, M), b_cache.as<uint8_t>() + r.cache, M, base_pos, pos_dev, scratch});
    residual(L.mixer->o, heads, L.norm1b.tanh, true, L.ff ? next_ff(L) : next_input(i + 1), ST_O);
    if (!L.ff) return;
    const DenseIn in = normed(L.norm2, M);
    {
        StageMark m(this, ST_GATE_UP);
        DenseEpiArgs e;
        e.out = act.p;
        e.ld_out = L.ff;
        e.act = L.act;
        launch_dense(t, L.gate_up, in, M, DenseEpi::ActPair, e, stream);
    }
    residual(L.down, dense_rows(act.p, L.ff), L.norm2b.tanh, true, next_input(i + 1), ST_DOWN);
}

int32_t BlockModel::load_norm(const SafeTensors& st, const std::string& name, DevBuf* buf, uint32_t slot, BlockNorm* out) {
    const TensorView *w, *b, *a = nullptr;
    int32_t rc;
    if ((rc = st.get(name, {spec.width}, &w)) || (rc = st.get(name + ".b", {spec.width}, &b))) return rc;
    if (elementwise_norms() && (rc = st.get(name + ".alpha", {}, &a))) return rc;
    std::vector<float> v(2 * (size_t)width, 0.f);
    w->read_f32(0, spec.width, v.data());
    b->read_f32(0, spec.width, v.data() + width);
    float* d = buf->as<float>() + (size_t)slot * 2 * width;
    FH_HIP(hipMemcpy(d, v.data(), v.size() * 4, hipMemcpyHostToDevice));
    if (elementwise_norms()) out->tanh = DynTanh{d, d + width, a->at(0)};
    else out->ln = LayerNorm{d, d + width, spec.width, (float)spec.eps};
    return FORGE_HIP_OK;
}

int32_t BlockModel::load_layer(const BlockLoad& l, uint32_t i) {
    const LayerSpec& ls = spec.layers[i];
    layers.emplace_back();
    if (ls.weights != i) return FORGE_HIP_OK;
    layers.back().reset(new BlockLayer());
    BlockLayer& L = *layers.back();
    L.ff = ls.ff == FeedForwardKind::None ? 0 : pad_to(ls.ff_size, 64);
    L.act = ls.ff == FeedForwardKind::GeluTanhGated ? Act::GeluTanh : Act::Silu;
    const std::string at = "layer " + std::to_string(i) + ": ", n = "l" + std::to_string(i) + ".";
    FH_CHECK(L.ff <= dense_k_max(), at + "ff is at most 32768");
    int32_t rc = load_mixer(l, ls, n + "mix.", at, &L.mixer);
    if (rc) return rc;
    const uint32_t W = spec.width;
    const TensorView *v, *g;
    if (L.ff) {
        const std::string ff = n + "mlp.";
        MatrixBuilder m(t, 2 * L.ff, width);
        if ((rc = l.st.get(ff + "gate", {ls.ff_size, W}, &g)) || (rc = l.st.get(ff + "up", {ls.ff_size, W}, &v))) return rc;
        for (uint32_t r = 0; r < ls.ff_size; r++) { m.put(2 * r, 0, *g, r, 0, W); m.put(2 * r + 1, 0, *v, r, 0, W); }
        if ((rc = m.upload(&L.b_gate_up, &L.gate_up))) return rc;
        MatrixBuilder d(t, width, L.ff);
        if ((rc = l.st.get(ff + "down", {W, ls.ff_size}, &v))) return rc;
        for (uint32_t r = 0; r < W; r++) d.put(r, 0, *v, r, 0, ls.ff_size);
        if ((rc = d.upload(&L.b_down, &L.down))) return rc;
    }
    if ((rc = L.b_norms.alloc((size_t)8 * width * 4)) || (rc = load_norm(l.st, n + "norm1", &L.b_norms, 0, &L.norm1))) return rc;
    if (L.ff && (rc = load_norm(l.st, n + "norm2", &L.b_norms, 2, &L.norm2))) return rc;
    if (spec.post_norms && (rc = load_norm(l.st, n + "norm1b", &L.b_norms, 1, &L.norm1b))) return rc;
    if (spec.post_norms && L.ff && (rc = load_norm(l.st, n + "norm2b", &L.b_norms, 3, &L.norm2b))) return rc;
    return FORGE_HIP_OK;
}

int32_t BlockModel::alloc_scratch() {
    const size_t es = dtype_size(t), R = chunk_rows;
    size_t ff = 0, cache_bytes = 0;
    for (const auto& l : layers) {
        if (!l) continue;
        ff = std::max<size_t>(ff, l->ff);
        l->mixer->plan(&scratch, (uint32_t)R);
    }
    for (LayerRun& r : runs) {
        r.cache = cache_bytes;
        cache_bytes += (layers[r.layer]->mixer->cache_bytes() + 255) / 256 * 256;
    }
    int32_t rc;
    if ((rc = b_cache.alloc(cache_bytes)) || (rc = x.alloc(R * width * 4)) || (rc = h.alloc(R * width * es)) || (rc = act.alloc(R * ff * es)) ||
        (rc = rows_sel.alloc(HEAD_ROWS * 4)) || (rc = h_sel.alloc(HEAD_ROWS * width * es)) || (rc = scratch.alloc()))
        return rc;
    if (loop_in.p && (rc = xcat.alloc(R * 2 * width * es))) return rc;
    return FORGE_HIP_OK;
}

int32_t BlockModel::load(const std::string& dir, uint32_t max_seq, uint32_t flags) {
    int32_t rc = block_spec_from_folder(dir, &spec);
    if (rc) return rc;
    FH_CHECK(flags == 0, "model folder: flags must be 0");
    FH_CHECK(elementwise_norms() || (!spec.loop_times && !spec.post_norms), "model folder: loops and post-norms need elementwise norms");
    SafeTensors st;
    if ((rc = st.open(dir + "/model.safetensors"))) return rc;
    if (forge_hip_device_count() < 1) return fail(FORGE_HIP_ERR_NO_DEVICE, "no HIP device");
    width = pad_to(spec.width, 64);
    FH_CHECK(2 * (uint64_t)width <= dense_k_max(), "width is at most 16384");
    describe(spec, &cfg);
    cfg.max_seq = max_seq ? max_seq : DEFAULT_MAX_SEQ;
    cfg.wdtype = cfg.lm_head_dtype = (uint32_t)t;
    if ((rc = init_shared())) return rc;
    const BlockLoad from{st, t, spec.width, width, cfg.max_seq, spec.eps, rotary};
    for (uint32_t i = 0; i < cfg.layers; i++)
        if ((rc = load_layer(from, i))) return rc;
    auto run = [&](uint32_t i, bool pass_start) { runs.push_back({spec.layers[i].weights, pass_start, 0}); };
    const uint32_t body = spec.loop_times ? spec.loop_stop : 0;
    for (uint32_t i = 0; i < (spec.loop_times ? spec.loop_start : cfg.layers); i++) run(i, false);
    for (uint32_t p = 0; p < spec.loop_times; p++)
        for (uint32_t i = spec.loop_start; i < spec.loop_stop; i++) run(i, i == spec.loop_start);
    if (spec.loop_times)
        for (uint32_t i = body; i < cfg.layers; i++) run(i, false);

    const TensorView* v;
    auto rows_of = [&](const TensorView& from, uint32_t ld, DevBuf* buf, DenseWeight* w) {
        MatrixBuilder m(t, spec.vocab, ld);
        for (uint32_t r = 0; r < spec.vocab; r++) m.put(r, 0, from, r, 0, spec.width);
        return m.upload(buf, w);
    };
    if ((rc = st.get(spec.tied_head ? "embed" : "head", {spec.vocab, spec.width}, &v)) || (rc = rows_of(*v, width, &b_head, &head))) return rc;
    table = head.p;
    table_ld = width;
    if (!spec.tied_head) {
        DenseWeight w;
        if ((rc = st.get("embed", {spec.vocab, spec.width}, &v)) || (rc = rows_of(*v, spec.width, &b_embed, &w))) return rc;
        table = w.p;
        table_ld = spec.width;
    }
    if (spec.loop_times) {
        if ((rc = st.get("loop.in", {spec.width, 2 * (uint64_t)spec.width}, &v))) return rc;
        MatrixBuilder m(t, width, 2 * width);
        for (uint32_t r = 0; r < spec.width; r++) { m.put(r, 0, *v, r, 0, spec.width); m.put(r, width, *v, r, spec.width, spec.width); }
        if ((rc = m.upload(&b_loop, &loop_in))) return rc;
    }
    if ((rc = b_final.alloc((size_t)2 * width * 4)) || (rc = load_norm(st, "final.norm", &b_final, 0, &final_norm))) return rc;
    if ((rc = alloc_scratch())) return rc;
    FH_HIP(hipDeviceSynchronize());
    return FORGE_HIP_OK;
}

}  // namespace

extern "C" {

int32_t forge_hip_folder_config(const char* dir, forge_hip_config* out) {
    FH_CHECK(dir && out, "folder_config: null pointer");
    BlockSpec s;
    const int32_t rc = block_spec_from_folder(dir, &s);
    if (rc) return rc;
    describe(s, out);
    return FORGE_HIP_OK;
}

int32_t forge_hip_model_create_from_folder(const char* dir, uint32_t max_seq, uint32_t dtype, uint32_t flags, forge_hip_model** out) {
    FH_CHECK(out, "model_create_from_folder: null out");
    *out = nullptr;
    FH_CHECK(dir, "model_create_from_folder: null path");
    FH_CHECK(dtype == FORGE_HIP_BF16 || dtype == FORGE_HIP_F32, "model_create_from_folder: dtype must be BF16 (30) or F32 (0)");
    std::unique_ptr<BlockModel> m(new BlockModel());
    m->t = (DType)dtype;
    const int32_t rc = m->load(dir, max_seq, flags);
    if (rc) return rc;
    *out = m.release();
    return FORGE_HIP_OK;
}

}  // extern "C"
