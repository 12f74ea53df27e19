// The network of a BlockSpec (checkpoint.h): a residual stream in 32-bit, layers of a mixer and an optional gated feed-forward,
// Dynamic Tanh ahead of and behind each sublayer, a run of layers that may be looped.  Weights, activations and cache are
// bfloat16 or 32-bit (DType), dense.
//
// One routine enqueues the layers for M rows: a prompt chunk, or the one row of a decode step (position in device memory, so
// that the step can be a graph).  The norms are elementwise, so no kernel is theirs: the product that ends a sublayer carries
// "post-norm, residual, next norm" in its epilogue and leaves the next sublayer's input beside the stream.  Per layer run:
//   prompt: [W_dq; W_dkv; W_g], norms + cache rows, W_uq + rotation, [W_uk; W_uv] over the visible cache rows, attention * gate,
//           W_o + residual, [gate; up] + SiLU, down + residual;
//   decode: [W_dq; W_dkv; W_g], norm + W_uq + rotation beside the cache row, W_uk^T q, attention over latents, merge + W_uv * gate,
//           W_o + residual, [gate; up] + SiLU, down + residual.
//
// Every size is padded with zeros to what the kernels take (a head's parts to 32, depths of products to 64), in the weights'
// rows and columns, so that the padding of every activation is zero.  Rotary pairs (i, i + dims / 2) are laid side by side in
// the rows of W_uq and W_dkv: scores do not depend on the order of a key's dimensions.
#include <math.h>
#include <stdlib.h>
#include <string.h>

#include <map>
#include <utility>

#include "checkpoint.h"
#include "model.h"

using namespace fh;

namespace {

constexpr uint32_t HEAD_ROWS = 64;           // rows of one lm_head product of a prompt
constexpr uint32_t DEFAULT_MAX_SEQ = 4096;   // config.json names no context length

uint32_t up(uint32_t n, uint32_t to) { return (n + to - 1) / to * to; }

// The fields of forge_hip_config that a spec fills (per-layer sizes: the first layer's; inter: the largest).
void describe(const BlockSpec& s, forge_hip_config* c) {
    *c = forge_hip_config{};
    const LatentAttentionSpec& a = s.layers[0].latent;
    c->hidden = s.width;
    c->layers = (uint32_t)s.layers.size();
    c->vocab = s.vocab;
    c->heads = a.heads;
    c->kv_heads = 1;                         // one cached row for all heads
    c->head_dim = a.dim + a.rot_dim;
    c->rms_eps = (float)s.eps;
    c->rope_theta = (float)a.rot.base;
    c->sliding_window = a.window;
    for (const LayerSpec& l : s.layers) c->inter = std::max(c->inter, l.ff_size);
}

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
    int32_t upload(DevBuf* buf, DenseWeight* w) const {
        const int32_t rc = buf->alloc(bytes.size());
        if (rc) return rc;
        FH_HIP(hipMemcpy(buf->p, bytes.data(), bytes.size(), hipMemcpyHostToDevice));
        *w = DenseWeight{buf->p, N, K};
        return FORGE_HIP_OK;
    }
};

struct BlockLayer {
    LatentShape sh;
    DenseWeight in;                          // [W_dq; W_dkv; W_g]
    DenseWeight uq, ukv, o, gate_up, down;
    DevBuf b_in, b_uq, b_ukv, b_o, b_gate_up, b_down, b_norms;
    const float *q_norm = nullptr, *kv_norm = nullptr;
    const float *cos_t = nullptr, *sin_t = nullptr;
    DynTanh norm1, norm1b, norm2, norm2b;
    uint32_t hv = 0;                         // columns of the concatenated heads
    uint32_t ff = 0;                         // 0: no feed-forward
};

struct LayerRun {
    uint32_t layer;
    bool pass_start;                         // the loop's input product comes first
    size_t cache;                            // byte offset of this run's cache
};

struct BlockModel : forge_hip_model {
    BlockSpec spec;
    DType t = DType::BF16;
    uint32_t width = 0;                      // padded width of the stream
    std::vector<std::unique_ptr<BlockLayer>> layers;
    std::vector<LayerRun> runs;
    std::map<std::pair<double, uint32_t>, std::pair<DevBuf, DevBuf>> rotary;      // (base, dims) -> cos, sin [max_seq][dims / 2]
    DenseWeight loop_in, head;
    DynTanh final_norm;
    DevBuf b_embed, b_loop, b_head, b_final, b_cache;
    // scratch of one prompt chunk
    DevBuf x, h, xcat, raw, cq, q, kbuf, vbuf, gate, attn, act, ql, parts, rows_sel, h_sel;

    uint32_t logits_rows_max() const override { return HEAD_ROWS; }
    uint32_t layer_runs() const override { return (uint32_t)runs.size(); }

    int32_t load(const std::string& dir, uint32_t max_seq, uint32_t flags);
    int32_t load_layer(const SafeTensors& st, uint32_t i);
    int32_t load_norm(const SafeTensors& st, const std::string& name, DevBuf* buf, uint32_t slot, DynTanh* out);
    int32_t alloc_scratch();

    // The rows' input product of run i: where it lies, and how to make it from the stream.
    struct Next { DynTanh norm; void* out; uint32_t ld; };
    Next next_input(size_t i) const {
        if (i == runs.size()) return {final_norm, h.p, width};
        if (runs[i].pass_start) return {DynTanh{}, xcat.p, 2 * width};
        return {layers[runs[i].layer]->norm1, h.p, width};
    }
    void enqueue_embedding(const uint32_t* tokens, uint32_t M);
    void enqueue_run(size_t i, uint32_t M, uint32_t base_pos, const uint32_t* pos_dev);
    void enqueue_mixer(const BlockLayer& L, void* cache, uint32_t M, uint32_t base_pos, const uint32_t* pos_dev);

    void enqueue_decode_step() override {
        enqueue_embedding(d_token(), 1);
        for (size_t i = 0; i < runs.size(); i++) enqueue_run(i, 1, 0, d_pos());
        enqueue_row_logits(0);
        enqueue_argmax(true, true);
    }
    int32_t enqueue_prompt_rows(uint32_t rows, uint32_t base_pos) override {
        enqueue_embedding(ptok.as<uint32_t>(), rows);
        for (size_t i = 0; i < runs.size(); i++) enqueue_run(i, rows, base_pos, nullptr);
        return FORGE_HIP_OK;
    }
    void enqueue_row_logits(uint32_t row) override {
        StageMark m(this, ST_LM_HEAD);
        DenseEpiArgs e;
        e.f32 = logits.as<float>();
        e.ld_f32 = cfg.vocab;
        launch_dense(t, head, h.as<uint8_t>() + (size_t)row * width * dtype_size(t), width, 1, DenseEpi::F32, e, stream);
    }
    void enqueue_rows_logits(const uint32_t* rows, uint32_t n) override {
        if (n == 1) { enqueue_row_logits(rows[0]); return; }
        StageMark m(this, ST_LM_HEAD);
        (void)hipMemcpyAsync(rows_sel.p, rows, n * 4, hipMemcpyHostToDevice, stream);       // pageable source: staged when the call returns
        launch_gather_rows(t, h.p, width, rows_sel.as<uint32_t>(), n, width, h_sel.p, width, stream);
        DenseEpiArgs e;
        e.f32 = logits.as<float>();
        e.ld_f32 = cfg.vocab;
        launch_dense(t, head, h_sel.p, width, n, DenseEpi::F32, e, stream);
    }
    int32_t decode_launches() const override {
        int n = 1 + 1 + 2;                   // embedding, lm_head, argmax
        for (const LayerRun& r : runs) n += (r.pass_start ? 1 : 0) + 6 + (layers[r.layer]->ff ? 2 : 0);
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
    launch_dense_embedding(t, b_embed.p, spec.width, (float)spec.embedding_scale, tokens, M, x.as<float>(), width, nx.norm, nx.out, nx.ld, x0,
                           2 * width, counts.as<uint32_t>(), stream);
}

void BlockModel::enqueue_mixer(const BlockLayer& L, void* cache, uint32_t M, uint32_t base_pos, const uint32_t* pos_dev) {
    const LatentShape& sh = L.sh;
    const size_t es = dtype_size(t);
    {
        StageMark m(this, ST_QKV);
        DenseEpiArgs e;
        e.f32 = raw.as<float>();
        e.ld_f32 = e.split = sh.raw_row();
        e.out = gate.p;
        e.ld_out = L.hv;
        launch_dense(t, L.in, h.p, width, M, DenseEpi::RawGate, e, stream);
    }
    if (M == 1) {
        LatentDecodeIo io{raw.as<float>(), L.q_norm, L.kv_norm, L.cos_t, L.sin_t, L.uq, L.ukv, q.p, ql.p, cache, parts.as<float>(), gate.p, attn.p,
                          cfg.max_seq, base_pos, pos_dev};
        { StageMark m(this, ST_QKV); launch_latent_query(t, sh, io, stream); }
        StageMark m(this, ST_ATTN);
        launch_latent_attn_decode(t, sh, io, stream);
        return;
    }
    {
        StageMark m(this, ST_ROPE);
        launch_latent_norm_store(t, sh, raw.as<float>(), L.q_norm, L.kv_norm, L.cos_t, L.sin_t, M, base_pos, cq.p, cache, stream);
    }
    // keys and values of every position some row sees, from a multiple of 64 on
    const uint32_t lo = sh.window && base_pos >= sh.window ? (base_pos - sh.window + 1) / 64 * 64 : 0;
    {
        StageMark m(this, ST_QKV);
        DenseEpiArgs e;
        e.out = q.p;
        e.ld_out = sh.q_row();
        e.cos_t = L.cos_t;
        e.sin_t = L.sin_t;
        e.base_pos = base_pos;
        e.head_stride = sh.dim + sh.rot;
        e.rot_off = sh.dim;
        e.rot_pairs = sh.rot_pairs;
        launch_dense(t, L.uq, cq.p, sh.q_rank, M, DenseEpi::Rope, e, stream);
        DenseEpiArgs k;
        k.out = kbuf.p;
        k.ld_out = k.split = sh.heads * sh.dim;
        k.out2 = vbuf.p;
        k.ld_out2 = sh.heads * sh.vdim;
        launch_dense(t, L.ukv, (const uint8_t*)cache + (size_t)lo * sh.cache_row() * es, sh.cache_row(), base_pos + M - lo, DenseEpi::Split, k, stream);
    }
    StageMark m(this, ST_ATTN);
    launch_latent_attn_prefill(t, sh, q.p, kbuf.p, vbuf.p, cache, lo, gate.p, attn.p, L.hv, M, base_pos, stream);
}

void BlockModel::enqueue_run(size_t i, uint32_t M, uint32_t base_pos, const uint32_t* pos_dev) {
    const LayerRun& r = runs[i];
    const BlockLayer& L = *layers[r.layer];
    // what ends a sublayer: stream = post(product) (+ stream), next input = norm(stream)
    auto residual = [&](const DenseWeight& w, const void* a, uint32_t lda, const DynTanh& post, bool add, const Next& nx, int stage) {
        StageMark m(this, stage);
        DenseEpiArgs e;
        e.f32 = x.as<float>();
        e.ld_f32 = width;
        e.post = post;
        e.add = add;
        e.next = nx.norm;
        e.out = nx.out;
        e.ld_out = nx.ld;
        launch_dense(t, w, a, lda, M, DenseEpi::Residual, e, stream);
    };
    if (r.pass_start) residual(loop_in, xcat.p, 2 * width, DynTanh{}, false, Next{L.norm1, h.p, width}, ST_QKV);
    enqueue_mixer(L, b_cache.as<uint8_t>() + r.cache, M, base_pos, pos_dev);
    residual(L.o, attn.p, L.hv, L.norm1b, true, L.ff ? Next{L.norm2, h.p, width} : next_input(i + 1), ST_O);
    if (!L.ff) return;
    {
        StageMark m(this, ST_GATE_UP);
        DenseEpiArgs e;
        e.out = act.p;
        e.ld_out = L.ff;
        launch_dense(t, L.gate_up, h.p, width, M, DenseEpi::SiluPair, e, stream);
    }
    residual(L.down, act.p, L.ff, L.norm2b, true, next_input(i + 1), ST_DOWN);
}

int32_t BlockModel::load_norm(const SafeTensors& st, const std::string& name, DevBuf* buf, uint32_t slot, DynTanh* out) {
    const TensorView *w, *b, *a;
    int32_t rc;
    if ((rc = st.get(name, {spec.width}, &w)) || (rc = st.get(name + ".b", {spec.width}, &b)) || (rc = st.get(name + ".alpha", {}, &a))) return rc;
    std::vector<float> v(2 * (size_t)width, 0.f);
    w->read_f32(0, spec.width, v.data());
    b->read_f32(0, spec.width, v.data() + width);
    float* d = buf->as<float>() + (size_t)slot * 2 * width;
    FH_HIP(hipMemcpy(d, v.data(), v.size() * 4, hipMemcpyHostToDevice));
    *out = DynTanh{d, d + width, a->at(0)};
    return FORGE_HIP_OK;
}

int32_t BlockModel::load_layer(const SafeTensors& st, uint32_t i) {
    const LayerSpec& ls = spec.layers[i];
    const LatentAttentionSpec& a = ls.latent;
    layers.emplace_back(new BlockLayer());
    BlockLayer& L = *layers.back();
    LatentShape& sh = L.sh;
    sh.heads = a.heads;
    sh.dim = up(a.dim, 32);
    sh.rot = up(a.rot_dim, 32);
    sh.vdim = up(a.vdim, 32);
    sh.rank = up(a.kv_rank, 64);
    sh.q_rank = up(a.q_rank, 64);
    sh.rank_n = a.kv_rank;
    sh.q_rank_n = a.q_rank;
    sh.rot_pairs = a.rot.dims / 2;
    sh.window = a.window;
    sh.scale = (float)a.scale;
    sh.eps = (float)spec.eps;
    L.hv = up(a.heads * sh.vdim, 64);
    L.ff = ls.ff == FeedForwardKind::None ? 0 : up(ls.ff_size, 64);
    const std::string at = "layer " + std::to_string(i) + ": ";
    FH_CHECK(latent_shape_supported(t, sh), at + "the kernels take dim + rot_dim and vdim up to 256 and kv_rank up to 1024 (each rounded up to its padding)");
    FH_CHECK(L.hv <= dense_k_max() && L.ff <= dense_k_max(), at + "heads * vdim and ff are at most 32768");

    const std::string n = "l" + std::to_string(i) + ".", mx = n + "mix.";
    const uint32_t W = spec.width, H = a.heads, dq = a.dim + a.rot_dim, half = a.rot.dims / 2;
    // place of rotated dimension j in the padded layout: pairs side by side, what does not turn behind them
    auto rot_place = [&](uint32_t j) { return j < half ? 2 * j : j < a.rot.dims ? 2 * (j - half) + 1 : j; };
    int32_t rc;
    const TensorView *v, *g;
    {
        MatrixBuilder m(t, sh.raw_row() + L.hv, width);
        if ((rc = st.get(mx + "dq", {a.q_rank, W}, &v))) return rc;
        for (uint32_t r = 0; r < a.q_rank; r++) m.put(r, 0, *v, r, 0, W);
        if ((rc = st.get(mx + "dkv", {a.kv_rank + a.rot_dim, W}, &v))) return rc;
        for (uint32_t r = 0; r < a.kv_rank; r++) m.put(sh.q_rank + r, 0, *v, r, 0, W);
        for (uint32_t j = 0; j < a.rot_dim; j++) m.put(sh.q_rank + sh.rank + rot_place(j), 0, *v, a.kv_rank + j, 0, W);
        if ((rc = st.get(mx + "g", {(uint64_t)H * a.vdim, W}, &g))) return rc;
        for (uint32_t k = 0; k < H; k++)
            for (uint32_t d = 0; d < a.vdim; d++) m.put(sh.raw_row() + k * sh.vdim + d, 0, *g, k * a.vdim + d, 0, W);
        if ((rc = m.upload(&L.b_in, &L.in))) return rc;
    }
    {
        MatrixBuilder m(t, sh.q_row(), sh.q_rank);
        if ((rc = st.get(mx + "uq", {(uint64_t)H * dq, a.q_rank}, &v))) return rc;
        for (uint32_t k = 0; k < H; k++)
            for (uint32_t d = 0; d < dq; d++)
                m.put(k * (sh.dim + sh.rot) + (d < a.dim ? d : sh.dim + rot_place(d - a.dim)), 0, *v, k * dq + d, 0, a.q_rank);
        if ((rc = m.upload(&L.b_uq, &L.uq))) return rc;
    }
    {
        MatrixBuilder m(t, H * (sh.dim + sh.vdim), sh.rank);
        if ((rc = st.get(mx + "uk", {(uint64_t)H * a.dim, a.kv_rank}, &v)) || (rc = st.get(mx + "uv", {(uint64_t)H * a.vdim, a.kv_rank}, &g))) return rc;
        for (uint32_t k = 0; k < H; k++) {
            for (uint32_t d = 0; d < a.dim; d++) m.put(k * sh.dim + d, 0, *v, k * a.dim + d, 0, a.kv_rank);
            for (uint32_t d = 0; d < a.vdim; d++) m.put(H * sh.dim + k * sh.vdim + d, 0, *g, k * a.vdim + d, 0, a.kv_rank);
        }
        if ((rc = m.upload(&L.b_ukv, &L.ukv))) return rc;
    }
    {
        MatrixBuilder m(t, width, L.hv);
        if ((rc = st.get(mx + "o", {W, (uint64_t)H * a.vdim}, &v))) return rc;
        for (uint32_t r = 0; r < W; r++)
            for (uint32_t k = 0; k < H; k++) m.put(r, k * sh.vdim, *v, r, k * a.vdim, a.vdim);
        if ((rc = m.upload(&L.b_o, &L.o))) return rc;
    }
    if (L.ff) {
        const std::string ff = n + "mlp.";
        MatrixBuilder m(t, 2 * L.ff, width);
        if ((rc = st.get(ff + "gate", {ls.ff_size, W}, &g)) || (rc = st.get(ff + "up", {ls.ff_size, W}, &v))) return rc;
        for (uint32_t r = 0; r < ls.ff_size; r++) { m.put(2 * r, 0, *g, r, 0, W); m.put(2 * r + 1, 0, *v, r, 0, W); }
        if ((rc = m.upload(&L.b_gate_up, &L.gate_up))) return rc;
        MatrixBuilder d(t, width, L.ff);
        if ((rc = st.get(ff + "down", {W, ls.ff_size}, &v))) return rc;
        for (uint32_t r = 0; r < W; r++) d.put(r, 0, *v, r, 0, ls.ff_size);
        if ((rc = d.upload(&L.b_down, &L.down))) return rc;
    }
    if ((rc = L.b_norms.alloc(((size_t)8 * width + sh.q_rank + sh.rank) * 4))) return rc;
    if ((rc = load_norm(st, n + "norm1", &L.b_norms, 0, &L.norm1)) || (rc = load_norm(st, n + "norm1b", &L.b_norms, 1, &L.norm1b))) return rc;
    if (L.ff && ((rc = load_norm(st, n + "norm2", &L.b_norms, 2, &L.norm2)) || (rc = load_norm(st, n + "norm2b", &L.b_norms, 3, &L.norm2b)))) return rc;
    {
        std::vector<float> w(sh.q_rank + sh.rank, 0.f);
        if ((rc = st.get(mx + "dq.norm", {a.q_rank}, &v)) || (rc = st.get(mx + "dkv.norm", {a.kv_rank}, &g))) return rc;
        v->read_f32(0, a.q_rank, w.data());
        g->read_f32(0, a.kv_rank, w.data() + sh.q_rank);
        float* d = L.b_norms.as<float>() + (size_t)8 * width;
        FH_HIP(hipMemcpy(d, w.data(), w.size() * 4, hipMemcpyHostToDevice));
        L.q_norm = d;
        L.kv_norm = d + sh.q_rank;
    }
    auto& tab = rotary[{a.rot.base, a.rot.dims}];
    if (!tab.first.p) {
        std::vector<float> ct((size_t)cfg.max_seq * half), sn(ct.size());
        for (uint32_t k = 0; k < half; k++) {
            const double f = pow(a.rot.base, -2.0 * k / a.rot.dims);
            for (uint32_t p = 0; p < cfg.max_seq; p++) {
                ct[(size_t)p * half + k] = (float)cos(p * f);
                sn[(size_t)p * half + k] = (float)sin(p * f);
            }
        }
        if ((rc = tab.first.alloc(ct.size() * 4)) || (rc = tab.second.alloc(ct.size() * 4))) return rc;
        FH_HIP(hipMemcpy(tab.first.p, ct.data(), ct.size() * 4, hipMemcpyHostToDevice));
        FH_HIP(hipMemcpy(tab.second.p, sn.data(), sn.size() * 4, hipMemcpyHostToDevice));
    }
    L.cos_t = tab.first.as<float>();
    L.sin_t = tab.second.as<float>();
    return FORGE_HIP_OK;
}

int32_t BlockModel::alloc_scratch() {
    const size_t es = dtype_size(t), R = chunk_rows;
    size_t raw_n = 0, hv = 0, qrank = 0, qrow = 0, ff = 0, kb = 0, vb = 0, lat = 0, pb = 0, cache_bytes = 0;
    for (const auto& l : layers) {
        const LatentShape& sh = l->sh;
        const size_t kv_rows = sh.window ? std::min<size_t>(cfg.max_seq, R + sh.window + 64) : cfg.max_seq;
        raw_n = std::max<size_t>(raw_n, sh.raw_row());
        hv = std::max<size_t>(hv, l->hv);
        qrank = std::max<size_t>(qrank, sh.q_rank);
        qrow = std::max<size_t>(qrow, sh.q_row());
        ff = std::max<size_t>(ff, l->ff);
        kb = std::max<size_t>(kb, kv_rows * sh.heads * sh.dim);
        vb = std::max<size_t>(vb, kv_rows * sh.heads * sh.vdim);
        lat = std::max<size_t>(lat, (size_t)sh.heads * sh.rank);
        pb = std::max<size_t>(pb, latent_parts_bytes(sh, cfg.max_seq));
    }
    for (LayerRun& r : runs) {
        r.cache = cache_bytes;
        cache_bytes += (size_t)cfg.max_seq * layers[r.layer]->sh.cache_row() * es;
    }
    int32_t rc;
    if ((rc = b_cache.alloc(cache_bytes)) || (rc = x.alloc(R * width * 4)) || (rc = h.alloc(R * width * es)) || (rc = raw.alloc(R * raw_n * 4)) ||
        (rc = cq.alloc(R * qrank * es)) || (rc = q.alloc(R * qrow * es)) || (rc = kbuf.alloc(kb * es)) || (rc = vbuf.alloc(vb * es)) ||
        (rc = gate.alloc(R * hv * es)) || (rc = attn.alloc(R * hv * es)) || (rc = act.alloc(R * ff * es)) || (rc = ql.alloc(lat * es)) ||
        (rc = parts.alloc(pb)) || (rc = rows_sel.alloc(HEAD_ROWS * 4)) || (rc = h_sel.alloc(HEAD_ROWS * width * es)))
        return rc;
    if (loop_in.p && (rc = xcat.alloc(R * 2 * width * es))) return rc;
    // parts without keys keep what they held: weighted with 0, which needs a finite number
    FH_HIP(hipMemset(parts.p, 0, pb));
    // columns that pad the concatenated heads are read (against zero weights) and never written
    FH_HIP(hipMemset(attn.p, 0, R * hv * es));
    return FORGE_HIP_OK;
}

int32_t BlockModel::load(const std::string& dir, uint32_t max_seq, uint32_t flags) {
    int32_t rc = block_spec_from_folder(dir, &spec);
    if (rc) return rc;
    FH_CHECK(flags == 0, "model folder: flags must be 0");
    SafeTensors st;
    if ((rc = st.open(dir + "/model.safetensors"))) return rc;
    if (forge_hip_device_count() < 1) return fail(FORGE_HIP_ERR_NO_DEVICE, "no HIP device");
    width = up(spec.width, 64);
    FH_CHECK(2 * (uint64_t)width <= dense_k_max(), "width is at most 16384");
    describe(spec, &cfg);
    cfg.max_seq = max_seq ? max_seq : DEFAULT_MAX_SEQ;
    cfg.wdtype = cfg.lm_head_dtype = (uint32_t)t;
    if ((rc = init_shared())) return rc;
    for (uint32_t i = 0; i < cfg.layers; i++)
        if ((rc = load_layer(st, i))) return rc;
    const uint32_t body = spec.loop_times ? spec.loop_stop : 0;
    for (uint32_t i = 0; i < (spec.loop_times ? spec.loop_start : cfg.layers); i++) runs.push_back({i, false, 0});
    for (uint32_t p = 0; p < spec.loop_times; p++)
        for (uint32_t i = spec.loop_start; i < spec.loop_stop; i++) runs.push_back({i, i == spec.loop_start, 0});
    if (spec.loop_times)
        for (uint32_t i = body; i < cfg.layers; i++) runs.push_back({i, false, 0});

    const TensorView* v;
    if ((rc = st.get("embed", {spec.vocab, spec.width}, &v))) return rc;
    {
        MatrixBuilder m(t, spec.vocab, spec.width);
        for (uint32_t r = 0; r < spec.vocab; r++) m.put(r, 0, *v, r, 0, spec.width);
        DenseWeight table;
        if ((rc = m.upload(&b_embed, &table))) return rc;
    }
    if (spec.loop_times) {
        if ((rc = st.get("loop.in", {spec.width, 2 * (uint64_t)spec.width}, &v))) return rc;
        MatrixBuilder m(t, width, 2 * width);
        for (uint32_t r = 0; r < spec.width; r++) { m.put(r, 0, *v, r, 0, spec.width); m.put(r, width, *v, r, spec.width, spec.width); }
        if ((rc = m.upload(&b_loop, &loop_in))) return rc;
    }
    if ((rc = st.get("head", {spec.vocab, spec.width}, &v))) return rc;
    {
        MatrixBuilder m(t, spec.vocab, width);
        for (uint32_t r = 0; r < spec.vocab; r++) m.put(r, 0, *v, r, 0, spec.width);
        if ((rc = m.upload(&b_head, &head))) return rc;
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
