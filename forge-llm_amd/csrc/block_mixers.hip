// The mixers of block networks: latent attention, grouped-query attention, gated linear attention.
//
// Every size is padded with zeros to what the kernels take (a head's parts to 32, depths of products to 64), in the weights'
// rows and columns, so that the padding of every activation is zero.  Rotary pairs (i, i + dims / 2) are laid side by side in
// the rows of the query and key matrices: scores do not depend on the order of a key's dimensions.
#include <math.h>
#include <string.h>

#include "block_mixer.h"

namespace fh {

int32_t MatrixBuilder::upload(DevBuf* buf, DenseWeight* w) const {
    const int32_t rc = buf->alloc(bytes.size());
    if (rc) return rc;
    FH_HIP(hipMemcpy(buf->p, bytes.data(), bytes.size(), hipMemcpyHostToDevice));
    *w = DenseWeight{buf->p, N, K};
    return FORGE_HIP_OK;
}

int32_t RotaryTables::get(const RotarySpec& r, uint32_t max_seq, const float** cos_t, const float** sin_t) {
    auto& tab = tables[r];
    if (!tab.first.p) {
        const uint32_t half = r.dims / 2;
        std::vector<float> ct((size_t)max_seq * half), sn(ct.size());
        for (uint32_t k = 0; k < half; k++) {
            const double f = r.frequency(k);
            for (uint32_t p = 0; p < max_seq; p++) {
                ct[(size_t)p * half + k] = (float)cos(p * f);
                sn[(size_t)p * half + k] = (float)sin(p * f);
            }
        }
        int32_t rc;
        if ((rc = tab.first.alloc(ct.size() * 4)) || (rc = tab.second.alloc(ct.size() * 4))) return rc;
        FH_HIP(hipMemcpy(tab.first.p, ct.data(), ct.size() * 4, hipMemcpyHostToDevice));
        FH_HIP(hipMemcpy(tab.second.p, sn.data(), sn.size() * 4, hipMemcpyHostToDevice));
    }
    *cos_t = tab.first.as<float>();
    *sin_t = tab.second.as<float>();
    return FORGE_HIP_OK;
}

int32_t BlockScratch::alloc() {
    for (int a = 0; a < AREAS; a++) {
        if (!want[a]) continue;
        const int32_t rc = buf[a].alloc(want[a]);
        if (rc) return rc;
        // what is never written is read against zero weights (columns that pad the concatenated heads, attention parts without
        // keys), which needs finite numbers
        FH_HIP(hipMemset(buf[a].p, 0, want[a]));
    }
    return FORGE_HIP_OK;
}

int32_t Mixer::load_output(const BlockLoad& l, const std::string& name, uint32_t heads, uint32_t vdim, uint32_t head) {
    const TensorView* v;
    int32_t rc;
    if ((rc = l.st.get(name, {l.spec_width, (uint64_t)heads * vdim}, &v))) return rc;
    MatrixBuilder m(l.t, l.width, pad_to(heads * head, 64));
    for (uint32_t r = 0; r < l.spec_width; r++)
        for (uint32_t k = 0; k < heads; k++) m.put(r, k * head, *v, r, k * vdim, vdim);
    return m.upload(&b_o, &o);
}

namespace {

// Packs the rows of several projections of the same input, head by head with each head's rows padded.
struct InputPacker {
    const BlockLoad& l;
    MatrixBuilder m;
    InputPacker(const BlockLoad& load, uint32_t rows) : l(load), m(load.t, rows, load.width) {}
    // tensor [heads * dim][width] -> rows row0 + head * pad + place(d)
    template <typename F>
    int32_t heads(const std::string& name, uint32_t row0, uint32_t n, uint32_t dim, uint32_t pad, F place) {
        const TensorView* v;
        const int32_t rc = l.st.get(name, {(uint64_t)n * dim, l.spec_width}, &v);
        if (rc) return rc;
        for (uint32_t k = 0; k < n; k++)
            for (uint32_t d = 0; d < dim; d++) m.put(row0 + k * pad + place(d), 0, *v, k * dim + d, 0, l.spec_width);
        return FORGE_HIP_OK;
    }
    int32_t heads(const std::string& name, uint32_t row0, uint32_t n, uint32_t dim, uint32_t pad) {
        return heads(name, row0, n, dim, pad, [](uint32_t d) { return d; });
    }
};

// A vector of n elements in 32-bit, each at its place in the padded layout.
template <typename F>
int32_t read_vector(const BlockLoad& l, const std::string& name, uint32_t n, float* out, F place) {
    const TensorView* v;
    const int32_t rc = l.st.get(name, {n}, &v);
    if (rc) return rc;
    for (uint32_t i = 0; i < n; i++) out[place(i)] = v->at(i);
    return FORGE_HIP_OK;
}
uint32_t in_order(uint32_t i) { return i; }

int32_t upload_floats(const std::vector<float>& v, DevBuf* buf) {
    const int32_t rc = buf->alloc(v.size() * 4);
    if (rc) return rc;
    FH_HIP(hipMemcpy(buf->p, v.data(), v.size() * 4, hipMemcpyHostToDevice));
    return FORGE_HIP_OK;
}

// The input product [raw part | gate]: raw columns in 32-bit, act(gate) beside them.
void enqueue_raw_gate(const MixerCall& c, DType t, const DenseWeight& w, uint32_t raw, uint32_t gate, Act act) {
    StageMark m(c.model, ST_QKV);
    DenseEpiArgs e;
    e.f32 = c.scratch.f(BlockScratch::RAW);
    e.ld_f32 = e.split = raw;
    e.out = c.scratch.p(BlockScratch::GATE);
    e.ld_out = gate;
    e.act = act;
    launch_dense(t, w, c.in, c.M, DenseEpi::RawGate, e, c.model->stream);
}

// ---- latent attention ------------------------------------------------------------------------------------------------------
// prompt: [W_dq; W_dkv; W_g], norms + cache rows, W_uq + rotation, [W_uk; W_uv] over the visible cache rows, attention * gate;
// decode: [W_dq; W_dkv; W_g], norm + W_uq + rotation beside the cache row, W_uk^T q, attention over latents, merge + W_uv * gate.
struct LatentMixer : Mixer {
    LatentShape sh;
    DenseWeight in, uq, ukv;                 // in: [W_dq; W_dkv; W_g]
    DevBuf b_in, b_uq, b_ukv, b_norms;
    const float *q_norm = nullptr, *kv_norm = nullptr, *cos_t = nullptr, *sin_t = nullptr;
    uint32_t hv = 0;                         // columns of the concatenated heads

    int32_t load(const BlockLoad& l, const LatentAttentionSpec& a, const std::string& mx, const std::string& at) {
        sh.heads = a.heads;
        sh.dim = pad_to(a.dim, 32);
        sh.rot = pad_to(a.rot_dim, 32);
        sh.vdim = pad_to(a.vdim, 32);
        sh.rank = pad_to(a.kv_rank, 64);
        sh.q_rank = pad_to(a.q_rank, 64);
        sh.rank_n = a.kv_rank;
        sh.q_rank_n = a.q_rank;
        sh.rot_pairs = a.rot.dims / 2;
        sh.window = a.window;
        sh.scale = (float)a.scale;
        sh.eps = (float)l.eps;
        hv = pad_to(a.heads * sh.vdim, 64);
        FH_CHECK(latent_shape_supported(t, sh), at + "the kernels take dim + rot_dim and vdim up to 256 and kv_rank up to 1024 (each rounded up to its padding)");
        FH_CHECK(hv <= dense_k_max(), at + "heads * vdim is at most 32768");
        const uint32_t H = a.heads, dq = a.dim + a.rot_dim;
        auto rot_place = [&](uint32_t j) { return rotated_place(j, a.rot.dims); };
        int32_t rc;
        const TensorView *v, *g;
        {
            InputPacker m(l, sh.raw_row() + hv);
            if ((rc = m.heads(mx + "dq", 0, 1, a.q_rank, a.q_rank))) return rc;
            if ((rc = m.heads(mx + "dkv", sh.q_rank, 1, a.kv_rank + a.rot_dim, 0,
                              [&](uint32_t j) { return j < a.kv_rank ? j : sh.rank + rot_place(j - a.kv_rank); })))
                return rc;
            if ((rc = m.heads(mx + "g", sh.raw_row(), H, a.vdim, sh.vdim)) || (rc = m.m.upload(&b_in, &in))) return rc;
        }
        {
            MatrixBuilder m(t, sh.q_row(), sh.q_rank);
            if ((rc = l.st.get(mx + "uq", {(uint64_t)H * dq, a.q_rank}, &v))) return rc;
            for (uint32_t k = 0; k < H; k++)
                for (uint32_t d = 0; d < dq; d++)
                    m.put(k * (sh.dim + sh.rot) + (d < a.dim ? d : sh.dim + rot_place(d - a.dim)), 0, *v, k * dq + d, 0, a.q_rank);
            if ((rc = m.upload(&b_uq, &uq))) return rc;
        }
        {
            MatrixBuilder m(t, H * (sh.dim + sh.vdim), sh.rank);
            if ((rc = l.st.get(mx + "uk", {(uint64_t)H * a.dim, a.kv_rank}, &v)) || (rc = l.st.get(mx + "uv", {(uint64_t)H * a.vdim, a.kv_rank}, &g))) return rc;
            for (uint32_t k = 0; k < H; k++) {
                for (uint32_t d = 0; d < a.dim; d++) m.put(k * sh.dim + d, 0, *v, k * a.dim + d, 0, a.kv_rank);
                for (uint32_t d = 0; d < a.vdim; d++) m.put(H * sh.dim + k * sh.vdim + d, 0, *g, k * a.vdim + d, 0, a.kv_rank);
            }
            if ((rc = m.upload(&b_ukv, &ukv))) return rc;
        }
        if ((rc = load_output(l, mx + "o", H, a.vdim, sh.vdim))) return rc;
        std::vector<float> w(sh.q_rank + sh.rank, 0.f);
        if ((rc = read_vector(l, mx + "dq.norm", a.q_rank, w.data(), in_order)) || (rc = read_vector(l, mx + "dkv.norm", a.kv_rank, w.data() + sh.q_rank, in_order)) ||
            (rc = upload_floats(w, &b_norms)))
            return rc;
        q_norm = b_norms.as<float>();
        kv_norm = q_norm + sh.q_rank;
        return l.rotary.get(a.rot, max_seq, &cos_t, &sin_t);
    }
    size_t cache_bytes() const override { return (size_t)max_seq * sh.cache_row() * dtype_size(t); }
    void plan(BlockScratch* s, uint32_t R) const override {
        const size_t es = dtype_size(t), kv_rows = sh.window ? std::min<size_t>(max_seq, R + sh.window + 64) : max_seq;
        s->need(BlockScratch::RAW, (size_t)R * sh.raw_row() * 4);
        s->need(BlockScratch::GATE, (size_t)R * hv * es);
        s->need(BlockScratch::OUT, (size_t)R * hv * es);
        s->need(BlockScratch::CQ, (size_t)R * sh.q_rank * es);
        s->need(BlockScratch::Q, (size_t)R * sh.q_row() * es);
        s->need(BlockScratch::K, kv_rows * sh.heads * sh.dim * es);
        s->need(BlockScratch::V, kv_rows * sh.heads * sh.vdim * es);
        s->need(BlockScratch::QL, (size_t)sh.heads * sh.rank * es);
        s->need(BlockScratch::PARTS, latent_parts_bytes(sh, max_seq));
    }
    DenseIn enqueue(const MixerCall& c) const override {
        const BlockScratch& sc = c.scratch;
        hipStream_t stream = c.model->stream;
        const float* raw = sc.f(BlockScratch::RAW);
        void* out = sc.p(BlockScratch::OUT);
        enqueue_raw_gate(c, t, in, sh.raw_row(), hv, Act::Sigmoid);
        if (c.M == 1) {
            LatentDecodeIo io{raw, q_norm, kv_norm, cos_t, sin_t, uq, ukv, sc.p(BlockScratch::Q), sc.p(BlockScratch::QL), c.cache, sc.f(BlockScratch::PARTS),
                              sc.p(BlockScratch::GATE), out, max_seq, c.base_pos, c.pos_dev};
            { StageMark m(c.model, ST_QKV); launch_latent_query(t, sh, io, stream); }
            StageMark m(c.model, ST_ATTN);
            launch_latent_attn_decode(t, sh, io, stream);
            return dense_rows(out, hv);
        }
        {
            StageMark m(c.model, ST_ROPE);
            launch_latent_norm_store(t, sh, raw, q_norm, kv_norm, cos_t, sin_t, c.M, c.base_pos, sc.p(BlockScratch::CQ), c.cache, stream);
        }
        // keys and values of every position some row sees, from a multiple of 64 on
        const uint32_t lo = sh.window && c.base_pos >= sh.window ? (c.base_pos - sh.window + 1) / 64 * 64 : 0;
        {
            StageMark m(c.model, ST_QKV);
            DenseEpiArgs e;
            e.out = sc.p(BlockScratch::Q);
            e.ld_out = sh.q_row();
            e.cos_t = cos_t;
            e.sin_t = sin_t;
            e.base_pos = c.base_pos;
            e.head_stride = sh.dim + sh.rot;
            e.rot_off = sh.dim;
            e.rot_pairs = sh.rot_pairs;
            launch_dense(t, uq, dense_rows(sc.p(BlockScratch::CQ), sh.q_rank), c.M, DenseEpi::Rope, e, stream);
            DenseEpiArgs k;
            k.out = sc.p(BlockScratch::K);
            k.ld_out = k.split = sh.heads * sh.dim;
            k.out2 = sc.p(BlockScratch::V);
            k.ld_out2 = sh.heads * sh.vdim;
            launch_dense(t, ukv, dense_rows((const uint8_t*)c.cache + (size_t)lo * sh.cache_row() * dtype_size(t), sh.cache_row()), c.base_pos + c.M - lo,
                         DenseEpi::Split, k, stream);
        }
        StageMark m(c.model, ST_ATTN);
        PromptAttn p;
        p.heads = sh.heads;
        p.dim = sh.dim;
        p.rot = sh.rot;
        p.vdim = sh.vdim;
        p.window = sh.window;
        p.scale = sh.scale;
        p.q = sc.p(BlockScratch::Q);
        p.k = sc.p(BlockScratch::K);
        p.k_row = sh.heads * sh.dim;
        p.v = sc.p(BlockScratch::V);
        p.v_row = sh.heads * sh.vdim;
        p.shared = (const uint8_t*)c.cache + sh.rank * dtype_size(t);
        p.shared_row = sh.cache_row();
        p.kv_lo = lo;
        p.gate = sc.p(BlockScratch::GATE);
        p.out = out;
        p.ld_out = hv;
        launch_attn_prompt(t, p, c.M, c.base_pos, stream);
        return dense_rows(out, hv);
    }
    int decode_launches() const override { return 5; }
};

// ---- grouped-query attention -----------------------------------------------------------------------------------------------
// prompt: [W_q; W_k; W_v; W_g], norms + rotation + cache rows, attention * gate;
// decode: [W_q; W_k; W_v; W_g], norms + rotation + cache row + attention, merge * gate.
struct GroupedMixer : Mixer {
    GroupedShape sh;
    DenseWeight in;
    DevBuf b_in, b_norms;
    const float *q_norm = nullptr, *k_norm = nullptr, *cos_t = nullptr, *sin_t = nullptr;
    uint32_t hv = 0;

    int32_t load(const BlockLoad& l, const GroupedAttentionSpec& a, const std::string& mx, const std::string& at) {
        sh.heads = a.heads;
        sh.kv_heads = a.kv_heads;
        sh.dim = pad_to(a.dim, 32);
        sh.vdim = pad_to(a.vdim, 32);
        sh.dim_n = a.dim;
        sh.rot_pairs = a.rot.dims / 2;
        sh.scale = (float)a.scale;
        sh.eps = (float)l.eps;
        hv = pad_to(a.heads * sh.vdim, 64);
        FH_CHECK(sh.dim <= DENSE_HEAD_MAX && sh.vdim <= DENSE_HEAD_MAX, at + "dim and vdim are at most 256");
        FH_CHECK(hv <= dense_k_max(), at + "heads * vdim is at most 32768");
        auto place = [&](uint32_t j) { return rotated_place(j, a.rot.dims); };
        int32_t rc;
        const uint32_t k0 = a.heads * sh.dim, v0 = k0 + sh.k_row();
        InputPacker m(l, sh.raw_row() + hv);
        if ((rc = m.heads(mx + "q", 0, a.heads, a.dim, sh.dim, place)) || (rc = m.heads(mx + "k", k0, a.kv_heads, a.dim, sh.dim, place)) ||
            (rc = m.heads(mx + "v", v0, a.kv_heads, a.vdim, sh.vdim)) || (rc = m.heads(mx + "g", sh.raw_row(), a.heads, a.vdim, sh.vdim)) ||
            (rc = m.m.upload(&b_in, &in)) || (rc = load_output(l, mx + "o", a.heads, a.vdim, sh.vdim)))
            return rc;
        std::vector<float> w(2 * sh.dim, 0.f);
        if ((rc = read_vector(l, mx + "q.norm", a.dim, w.data(), place)) || (rc = read_vector(l, mx + "k.norm", a.dim, w.data() + sh.dim, place)) ||
            (rc = upload_floats(w, &b_norms)))
            return rc;
        q_norm = b_norms.as<float>();
        k_norm = q_norm + sh.dim;
        return l.rotary.get(a.rot, max_seq, &cos_t, &sin_t);
    }
    size_t k_bytes() const { return (size_t)max_seq * sh.k_row() * dtype_size(t); }
    size_t cache_bytes() const override { return k_bytes() + (size_t)max_seq * sh.v_row() * dtype_size(t); }
    void plan(BlockScratch* s, uint32_t R) const override {
        const size_t es = dtype_size(t);
        s->need(BlockScratch::RAW, (size_t)R * sh.raw_row() * 4);
        s->need(BlockScratch::GATE, (size_t)R * hv * es);
        s->need(BlockScratch::OUT, (size_t)R * hv * es);
        s->need(BlockScratch::Q, (size_t)R * sh.heads * sh.dim * es);
        s->need(BlockScratch::PARTS, grouped_parts_bytes(sh, max_seq));
    }
    DenseIn enqueue(const MixerCall& c) const override {
        const BlockScratch& sc = c.scratch;
        hipStream_t stream = c.model->stream;
        void* out = sc.p(BlockScratch::OUT);
        enqueue_raw_gate(c, t, in, sh.raw_row(), hv, Act::Sigmoid);
        const GroupedIo io{sc.f(BlockScratch::RAW), q_norm, k_norm, cos_t, sin_t, c.cache, (uint8_t*)c.cache + k_bytes(), max_seq, c.base_pos, c.pos_dev};
        if (c.M == 1) {
            StageMark m(c.model, ST_ATTN);
            launch_grouped_decode(t, sh, io, sc.f(BlockScratch::PARTS), sc.p(BlockScratch::GATE), out, stream);
            return dense_rows(out, hv);
        }
        {
            StageMark m(c.model, ST_ROPE);
            launch_grouped_norm_store(t, sh, io, c.M, sc.p(BlockScratch::Q), stream);
        }
        StageMark m(c.model, ST_ATTN);
        PromptAttn p;
        p.heads = sh.heads;
        p.group = sh.group();
        p.dim = sh.dim;
        p.vdim = sh.vdim;
        p.scale = sh.scale;
        p.q = sc.p(BlockScratch::Q);
        p.k = io.k_cache;
        p.k_row = sh.k_row();
        p.v = io.v_cache;
        p.v_row = sh.v_row();
        p.gate = sc.p(BlockScratch::GATE);
        p.out = out;
        p.ld_out = hv;
        launch_attn_prompt(t, p, c.M, c.base_pos, stream);
        return dense_rows(out, hv);
    }
    int decode_launches() const override { return 3; }
};

// ---- gated linear attention --------------------------------------------------------------------------------------------------
// prompt: [W_q; W_k; W_v; W_a1; W_g], chunks, scan, output (norm, gate);
// decode: [W_q; W_k; W_v; W_a1; W_g], state; the heads' norm and the gate go with the output product.
struct LinearMixer : Mixer {
    LinearShape sh;
    DenseWeight in;
    DevBuf b_in, b_vec;
    const float *w2 = nullptr, *b2 = nullptr, *norm = nullptr;
    uint32_t hv = 0;

    int32_t load(const BlockLoad& l, const LinearAttentionSpec& a, const std::string& mx, const std::string& at) {
        const TensorView* v = l.st.find(mx + "a1");
        FH_CHECK(v && v->shape.size() == 2 && v->shape[0] >= 1, "tensor '" + mx + "a1' is missing or no matrix");
        FH_CHECK(v->shape[0] <= 128, at + "the decay's rank is at most 128");
        const uint32_t rank = (uint32_t)v->shape[0];
        sh.heads = a.heads;
        sh.dim = pad_to(a.dim, 32);
        sh.vdim = pad_to(a.vdim, 32);
        sh.rank = pad_to(rank, 16);
        sh.vdim_n = a.vdim;
        sh.q_scale = (float)(1.0 / sqrt((double)a.dim));
        sh.inv_tau = (float)(1.0 / a.tau);
        sh.eps = (float)l.eps;
        hv = pad_to(a.heads * sh.vdim, 64);
        FH_CHECK(linear_shape_supported(sh), at + "dim and vdim are at most 256");
        FH_CHECK(hv <= dense_k_max(), at + "heads * vdim is at most 32768");
        int32_t rc;
        const uint32_t v0 = 2 * sh.qk(), low = v0 + a.heads * sh.vdim;
        InputPacker m(l, sh.raw_row() + hv);
        if ((rc = m.heads(mx + "q", 0, a.heads, a.dim, sh.dim)) || (rc = m.heads(mx + "k", sh.qk(), a.heads, a.dim, sh.dim)) ||
            (rc = m.heads(mx + "v", v0, a.heads, a.vdim, sh.vdim)) || (rc = m.heads(mx + "a1", low, 1, rank, sh.rank)) ||
            (rc = m.heads(mx + "g", sh.raw_row(), a.heads, a.vdim, sh.vdim)) || (rc = m.m.upload(&b_in, &in)) ||
            (rc = load_output(l, mx + "o", a.heads, a.vdim, sh.vdim)))
            return rc;
        // the second map transposed, its bias, the heads' norm: 32-bit
        const size_t n = (size_t)sh.rank * sh.qk();
        std::vector<float> w(n + sh.qk() + sh.vdim, 0.f);
        auto channel = [&](uint32_t i) { return i / a.dim * sh.dim + i % a.dim; };
        if ((rc = l.st.get(mx + "a2", {(uint64_t)a.heads * a.dim, rank}, &v))) return rc;
        for (uint32_t i = 0; i < a.heads * a.dim; i++)
            for (uint32_t r = 0; r < rank; r++) w[(size_t)r * sh.qk() + channel(i)] = v->at((uint64_t)i * rank + r);
        if ((rc = read_vector(l, mx + "a2.b", a.heads * a.dim, w.data() + n, channel)) || (rc = read_vector(l, mx + "norm", a.vdim, w.data() + n + sh.qk(), in_order)) ||
            (rc = upload_floats(w, &b_vec)))
            return rc;
        w2 = b_vec.as<float>();
        b2 = w2 + n;
        norm = b2 + sh.qk();
        return FORGE_HIP_OK;
    }
    size_t cache_bytes() const override { return sh.state() * 4; }
    void plan(BlockScratch* s, uint32_t R) const override {
        s->need(BlockScratch::RAW, (size_t)R * sh.raw_row() * 4);
        s->need(BlockScratch::GATE, (size_t)R * hv * dtype_size(t));
        s->need(BlockScratch::OUT, (size_t)R * hv * dtype_size(t));
        s->need(BlockScratch::WORK, linear_work_bytes(sh, R));
    }
    DenseIn enqueue(const MixerCall& c) const override {
        const BlockScratch& sc = c.scratch;
        enqueue_raw_gate(c, t, in, sh.raw_row(), hv, Act::Silu);
        const LinearIo io{sc.f(BlockScratch::RAW), w2, b2, (float*)c.cache, c.base_pos, c.pos_dev};
        StageMark m(c.model, ST_ATTN);
        if (c.M == 1) {
            launch_linear_step(sh, io, sc.f(BlockScratch::WORK), c.model->stream);
            DenseIn o;
            o.kind = DenseIn::HeadGate;
            o.f32 = sc.f(BlockScratch::WORK);
            o.heads = sh.heads;
            o.head = sh.vdim;
            o.head_n = sh.vdim_n;
            o.w = norm;
            o.gate = sc.p(BlockScratch::GATE);
            o.eps = sh.eps;
            return o;
        }
        launch_linear_prompt(t, sh, io, c.M, sc.f(BlockScratch::WORK), norm, sc.p(BlockScratch::GATE), sc.p(BlockScratch::OUT), hv, c.model->stream);
        return dense_rows(sc.p(BlockScratch::OUT), hv);
    }
    int decode_launches() const override { return 2; }
};

template <typename M, typename S>
int32_t load_as(const BlockLoad& l, const S& spec, const std::string& name, const std::string& at, std::unique_ptr<Mixer>* out) {
    std::unique_ptr<M> m(new M());
    m->t = l.t;
    m->max_seq = l.max_seq;
    const int32_t rc = m->load(l, spec, name, at);
    if (!rc) *out = std::move(m);
    return rc;
}

}  // namespace

int32_t load_mixer(const BlockLoad& l, const LayerSpec& s, const std::string& name, const std::string& at, std::unique_ptr<Mixer>* out) {
    switch (s.mixer) {
        case MixerKind::LatentAttention: return load_as<LatentMixer>(l, s.latent, name, at, out);
        case MixerKind::GroupedAttention: return load_as<GroupedMixer>(l, s.grouped, name, at, out);
        case MixerKind::LinearAttention: return load_as<LinearMixer>(l, s.linear, name, at, out);
    }
    return fail(FORGE_HIP_ERR_INVALID, at + "unknown mixer");
}

void describe_mixer(const LayerSpec& s, forge_hip_config* c) {
    switch (s.mixer) {
        case MixerKind::LatentAttention:
            c->heads = s.latent.heads;
            c->kv_heads = 1;                         // one cached row for all heads
            c->head_dim = s.latent.dim + s.latent.rot_dim;
            c->rope_theta = (float)s.latent.rot.base;
            c->sliding_window = s.latent.window;
            break;
        case MixerKind::GroupedAttention:
            c->heads = s.grouped.heads;
            c->kv_heads = s.grouped.kv_heads;
            c->head_dim = s.grouped.dim;
            c->rope_theta = (float)s.grouped.rot.base;
            break;
        case MixerKind::LinearAttention:
            c->heads = c->kv_heads = s.linear.heads; // a state per head
            c->head_dim = s.linear.dim;
            break;
    }
}

}  // namespace fh
