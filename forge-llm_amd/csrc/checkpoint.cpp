// Model folders (config.json + model.safetensors): JSON and safetensors readers, the registry of architectures.
#include "checkpoint.h"

#include <errno.h>
#include <fcntl.h>
#include <math.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cmath>

#include "common.h"

namespace fh {

// ---- JSON ------------------------------------------------------------------------------------
namespace {

struct Parser {
    const char* p;
    const char* end;
    const char* start;
    std::string err;
    int depth = 0;

    bool bad(const std::string& what) {
        if (err.empty()) err = what + " at byte " + std::to_string(p - start);
        return false;
    }
    void space() { while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++; }
    bool word(const char* w) {
        const size_t n = strlen(w);
        if ((size_t)(end - p) < n || memcmp(p, w, n) != 0) return bad("unknown word");
        p += n;
        return true;
    }
    static void utf8(uint32_t c, std::string* s) {
        if (c < 0x80) s->push_back((char)c);
        else if (c < 0x800) { s->push_back((char)(0xC0 | c >> 6)); s->push_back((char)(0x80 | (c & 63))); }
        else if (c < 0x10000) { s->push_back((char)(0xE0 | c >> 12)); s->push_back((char)(0x80 | (c >> 6 & 63))); s->push_back((char)(0x80 | (c & 63))); }
        else { s->push_back((char)(0xF0 | c >> 18)); s->push_back((char)(0x80 | (c >> 12 & 63))); s->push_back((char)(0x80 | (c >> 6 & 63))); s->push_back((char)(0x80 | (c & 63))); }
    }
    bool hex4(uint32_t* out) {
        if (end - p < 4) return bad("short \\u escape");
        uint32_t v = 0;
        for (int i = 0; i < 4; i++) {
            const char c = *p++;
            v = v * 16 + (c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : 99);
            if (v > 0xFFFF) return bad("bad \\u escape");
        }
        *out = v;
        return true;
    }
    bool string(std::string* s) {
        p++;                                     // the quote
        s->clear();
        for (;;) {
            if (p >= end) return bad("string without an end");
            const char c = *p++;
            if (c == '"') return true;
            if ((unsigned char)c < 0x20) return bad("control character in a string");
            if (c != '\\') { s->push_back(c); continue; }
            if (p >= end) return bad("string without an end");
            const char x = *p++;
            switch (x) {
                case '"': case '\\': case '/': s->push_back(x); break;
                case 'b': s->push_back('\b'); break;
                case 'f': s->push_back('\f'); break;
                case 'n': s->push_back('\n'); break;
                case 'r': s->push_back('\r'); break;
                case 't': s->push_back('\t'); break;
                case 'u': {
                    uint32_t u;
                    if (!hex4(&u)) return false;
                    if (u >= 0xD800 && u < 0xDC00 && end - p >= 6 && p[0] == '\\' && p[1] == 'u') {
                        p += 2;
                        uint32_t lo;
                        if (!hex4(&lo)) return false;
                        if (lo < 0xDC00 || lo > 0xDFFF) return bad("bad surrogate pair");
                        u = 0x10000 + ((u - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    utf8(u, s);
                    break;
                }
                default: return bad("bad escape");
            }
        }
    }
    bool value(Json* v) {
        space();
        if (p >= end) return bad("text ends early");
        if (++depth > 64) return bad("nested too deeply");
        bool ok = true;
        switch (*p) {
            case '{': {
                v->kind = Json::Object;
                p++;
                space();
                if (p < end && *p == '}') { p++; break; }
                for (;;) {
                    space();
                    std::string key;
                    if (p >= end || *p != '"') { ok = bad("expected a member name"); break; }
                    if (!(ok = string(&key))) break;
                    space();
                    if (p >= end || *p != ':') { ok = bad("expected ':'"); break; }
                    p++;
                    if (!(ok = value(&v->obj[key]))) break;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == '}') { p++; break; }
                    ok = bad("expected ',' or '}'");
                    break;
                }
                break;
            }
            case '[': {
                v->kind = Json::Array;
                p++;
                space();
                if (p < end && *p == ']') { p++; break; }
                for (;;) {
                    v->arr.emplace_back();
                    if (!(ok = value(&v->arr.back()))) break;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == ']') { p++; break; }
                    ok = bad("expected ',' or ']'");
                    break;
                }
                break;
            }
            case '"': v->kind = Json::String; ok = string(&v->str); break;
            case 't': v->kind = Json::Bool; v->b = true; ok = word("true"); break;
            case 'f': v->kind = Json::Bool; v->b = false; ok = word("false"); break;
            case 'n': v->kind = Json::Null; ok = word("null"); break;
            default: {
                const char* q = p;
                while (q < end && (strchr("+-.eE", *q) ? *q != 0 : (*q >= '0' && *q <= '9'))) q++;
                const std::string t(p, q);
                char* stop = nullptr;
                v->kind = Json::Number;
                v->num = t.empty() ? 0 : strtod(t.c_str(), &stop);
                if (t.empty() || *stop) ok = bad("not a value");
                else p = q;
            }
        }
        depth--;
        return ok;
    }
};

}  // namespace

int32_t json_parse(const char* text, size_t n, Json* out) {
    Parser ps{text, text + n, text, {}};
    *out = Json{};
    bool ok = ps.value(out);
    if (ok) {
        ps.space();
        if (ps.p != ps.end) ok = ps.bad("text after the value");
    }
    return ok ? FORGE_HIP_OK : fail(FORGE_HIP_ERR_INVALID, "JSON: " + ps.err);
}

// ---- safetensors -------------------------------------------------------------------------------
namespace {

inline float bf16_value(uint16_t b) {
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}
inline uint16_t bf16_round(float f) {
    uint32_t u;
    memcpy(&u, &f, 4);
    if ((u & 0x7FFFFFFFu) > 0x7F800000u) return (uint16_t)(u >> 16 | 0x40u);        // NaN stays NaN
    return (uint16_t)((u + 0x7FFFu + (u >> 16 & 1u)) >> 16);
}

}  // namespace

float TensorView::at(uint64_t i) const {
    float f = 0.f;
    read_f32(i, 1, &f);
    return f;
}

void TensorView::read_f32(uint64_t first, uint64_t n, float* out) const {
    if (type == F32 || type == I32) { memcpy(out, data + first * 4, n * 4); return; }
    for (uint64_t i = 0; i < n; i++) {
        uint16_t b;
        memcpy(&b, data + (first + i) * 2, 2);
        out[i] = type == BF16 ? bf16_value(b) : f16_to_f32_host(b);
    }
}

void TensorView::read_bf16(uint64_t first, uint64_t n, uint16_t* out) const {
    if (type == BF16) { memcpy(out, data + first * 2, n * 2); return; }
    for (uint64_t i = 0; i < n; i++) {
        float f;
        read_f32(first + i, 1, &f);
        out[i] = bf16_round(f);
    }
}

SafeTensors::~SafeTensors() {
    if (map_) munmap(map_, map_bytes_);
}

int32_t SafeTensors::open(const std::string& path) {
    const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
    if (fd < 0) return fail(FORGE_HIP_ERR_INVALID, path + ": " + strerror(errno));
    struct stat st;
    if (fstat(fd, &st) != 0 || st.st_size < 8) { ::close(fd); return fail(FORGE_HIP_ERR_INVALID, path + ": too short for a safetensors file"); }
    map_bytes_ = (size_t)st.st_size;
    void* m = mmap(nullptr, map_bytes_, PROT_READ, MAP_PRIVATE, fd, 0);
    ::close(fd);
    if (m == MAP_FAILED) return fail(FORGE_HIP_ERR_INVALID, path + ": cannot be mapped");
    map_ = m;
    const uint8_t* base = (const uint8_t*)m;
    uint64_t header = 0;
    memcpy(&header, base, 8);
    FH_CHECK(header <= map_bytes_ - 8, path + ": the header is longer than the file");
    Json j;
    const int32_t rc = json_parse((const char*)base + 8, header, &j);
    if (rc) return rc;
    FH_CHECK(j.kind == Json::Object, path + ": the header is not an object");
    const uint64_t room = map_bytes_ - 8 - header;
    for (const auto& [name, t] : j.obj) {
        if (name == "__metadata__") continue;
        const Json *dt = t.get("dtype"), *sh = t.get("shape"), *off = t.get("data_offsets");
        FH_CHECK(dt && dt->kind == Json::String && sh && sh->kind == Json::Array && off && off->kind == Json::Array && off->arr.size() == 2,
                 path + ": tensor '" + name + "' is not described");
        TensorView v;
        uint64_t es = 2;
        if (dt->str == "BF16") v.type = TensorView::BF16;
        else if (dt->str == "F16") v.type = TensorView::F16;
        else if (dt->str == "F32") { v.type = TensorView::F32; es = 4; }
        else if (dt->str == "I32") { v.type = TensorView::I32; es = 4; }
        else return fail(FORGE_HIP_ERR_INVALID, path + ": tensor '" + name + "' has the type " + dt->str + " (BF16, F16, F32 and I32 are read)");
        uint64_t bytes = es;
        for (const Json& d : sh->arr) {
            FH_CHECK(d.kind == Json::Number && d.num >= 0 && d.num < 4294967296.0, path + ": tensor '" + name + "' has an impossible shape");
            v.shape.push_back((uint64_t)d.num);
            FH_CHECK(!__builtin_mul_overflow(bytes, (uint64_t)d.num, &bytes), path + ": tensor '" + name + "' has an impossible shape");
        }
        const double a = off->arr[0].num, b = off->arr[1].num;
        FH_CHECK(a >= 0 && b >= a && b <= (double)room && (uint64_t)b - (uint64_t)a == bytes, path + ": tensor '" + name + "' does not lie in the file");
        v.data = base + 8 + header + (uint64_t)a;
        tensors_[name] = v;
    }
    return FORGE_HIP_OK;
}

int32_t SafeTensors::get(const std::string& name, const std::vector<uint64_t>& shape, const TensorView** out) const {
    const TensorView* v = find(name);
    FH_CHECK(v, "tensor '" + name + "' is missing");
    auto text = [](const std::vector<uint64_t>& s) {
        std::string t = "[";
        for (size_t i = 0; i < s.size(); i++) t += (i ? ", " : "") + std::to_string(s[i]);
        return t + "]";
    };
    FH_CHECK(v->shape == shape, "tensor '" + name + "' has the shape " + text(v->shape) + ", the configuration needs " + text(shape));
    FH_CHECK(v->type != TensorView::I32, "tensor '" + name + "' holds integers");
    *out = v;
    return FORGE_HIP_OK;
}

// ---- registry --------------------------------------------------------------------------------------
namespace {

// Members of a configuration object; the first failure is kept.
struct Reader {
    int32_t rc = FORGE_HIP_OK;
    bool fail_at(const std::string& where, const char* what) {
        if (!rc) rc = fail(FORGE_HIP_ERR_INVALID, "config.json: " + where + " " + what);
        return false;
    }
    const Json* object(const Json& j, const char* key, const std::string& at) {
        const Json* v = j.get(key);
        if (!v || v->kind != Json::Object) { fail_at(at + key, "must be an object"); return nullptr; }
        return v;
    }
    uint32_t size(const Json& j, const char* key, const std::string& at, uint32_t least = 1) {
        const Json* v = j.get(key);
        if (!v || v->kind != Json::Number || v->num != floor(v->num) || v->num < least || v->num > 2147483647.0) {
            fail_at(at + key, "must be a whole number in range");
            return 0;
        }
        return (uint32_t)v->num;
    }
    double number(const Json& j, const char* key, const std::string& at) {
        const Json* v = j.get(key);
        if (!v || v->kind != Json::Number || !std::isfinite(v->num)) { fail_at(at + key, "must be a number"); return 0; }
        return v->num;
    }
};

// "rot": base, dims (even, at most `limit`) and, where the design has it, "scaling".
void read_rotation(Reader& r, const Json& m, const std::string& at, uint32_t limit, bool scaling, RotarySpec* s) {
    const Json* rot = r.object(m, "rot", at);
    if (!rot) return;
    const std::string in = at + "rot.";
    s->dims = r.size(*rot, "dims", in);
    s->base = r.number(*rot, "base", in);
    if (!r.rc && (s->dims % 2 || s->dims > limit || s->base <= 0)) r.fail_at(at + "rot", "does not fit the head");
    const Json* sc = scaling ? rot->get("scaling") : nullptr;
    if (!sc || sc->kind == Json::Null) return;
    if (sc->kind != Json::Object) { r.fail_at(in + "scaling", "must be an object"); return; }
    s->factor = r.number(*sc, "factor", in + "scaling.");
    s->low = r.number(*sc, "low", in + "scaling.");
    s->high = r.number(*sc, "high", in + "scaling.");
    s->original = r.number(*sc, "original", in + "scaling.");
    if (!r.rc && (s->factor <= 0 || s->low <= 0 || s->high < s->low || s->original <= 0)) r.fail_at(in + "scaling", "makes no sense");
}

void read_latent_attention(Reader& r, const Json& m, const std::string& at, LatentAttentionSpec* s) {
    s->heads = r.size(m, "heads", at);
    s->dim = r.size(m, "dim", at);
    s->rot_dim = r.size(m, "rot_dim", at);
    s->vdim = r.size(m, "vdim", at);
    s->q_rank = r.size(m, "q_rank", at);
    s->kv_rank = r.size(m, "kv_rank", at);
    s->scale = r.number(m, "scale", at);
    read_rotation(r, m, at, s->rot_dim, false, &s->rot);
    const Json* mask = m.get("mask");
    if (mask && mask->kind != Json::Null) {
        const Json* size = mask->get("size");
        if (mask->kind != Json::Object) r.fail_at(at + "mask", "must be an object");
        else if (size && size->kind != Json::Null) s->window = r.size(*mask, "size", at + "mask.");
    }
}

void read_grouped_attention(Reader& r, const Json& m, const std::string& at, GroupedAttentionSpec* s) {
    s->heads = r.size(m, "heads", at);
    s->kv_heads = r.size(m, "kv_heads", at);
    s->dim = r.size(m, "dim", at);
    s->vdim = r.size(m, "vdim", at);
    s->scale = r.number(m, "scale", at);
    if (!r.rc && s->heads % s->kv_heads) r.fail_at(at + "kv_heads", "must divide heads");
    read_rotation(r, m, at, s->dim, true, &s->rot);
}

void read_linear_attention(Reader& r, const Json& m, const std::string& at, LinearAttentionSpec* s) {
    s->heads = r.size(m, "heads", at);
    s->dim = r.size(m, "dim", at);
    s->vdim = r.size(m, "vdim", at);
    s->tau = r.number(m, "tau", at);
    if (!r.rc && s->tau <= 0) r.fail_at(at + "tau", "must be positive");
}

// What every architecture's configuration starts with.
void read_frame(Reader& r, const Json& c, BlockSpec* s) {
    s->width = r.size(c, "width", "");
    s->vocab = r.size(c, "vocab", "");
    if (const Json* e = r.object(c, "embedding", "")) s->embedding_scale = r.number(*e, "scale", "embedding.");
    if (const Json* n = r.object(c, "norm", "")) s->eps = r.number(*n, "eps", "norm.");
}

// "layers": a list of {type, mixer, mlp}; `mixer` reads a layer's mixer by its type and says whether it knows it.
template <typename F>
void read_layers(Reader& r, const Json& c, FeedForwardKind dense, BlockSpec* s, F mixer) {
    const Json* layers = c.get("layers");
    if (!layers || layers->kind != Json::Array || layers->arr.empty()) { r.fail_at("layers", "must be a list"); return; }
    for (size_t i = 0; i < layers->arr.size() && !r.rc; i++) {
        const Json& l = layers->arr[i];
        const std::string at = "layers[" + std::to_string(i) + "].";
        LayerSpec ls;
        ls.weights = (uint32_t)i;
        const Json* type = l.get("type");
        if (!type || type->kind != Json::String) { r.fail_at(at + "type", "must be a string"); break; }
        const Json* m = r.object(l, "mixer", at);
        if (!m) break;
        if (!mixer(type->str, *m, at + "mixer.", &ls)) { r.fail_at(at + "type", "is no mixer of this architecture"); break; }
        const Json* mlp = l.get("mlp");
        if (mlp && mlp->kind != Json::Null) {
            const Json* kind = mlp->get("kind");
            if (!kind || kind->kind != Json::String || kind->str != "dense") { r.fail_at(at + "mlp.kind", "must be \"dense\""); break; }
            ls.ff = dense;
            ls.ff_size = r.size(*mlp, "ff", at + "mlp.");
        }
        s->layers.push_back(ls);
    }
}

// "weights_of": j in a layer's entry: the layer runs with layer j's tensors, and the rest of its entry equals j's.
void read_shared_weights(Reader& r, const Json& c, BlockSpec* s) {
    auto same = [](const LayerSpec& a, const LayerSpec& b) {
        auto rot = [](const RotarySpec& x, const RotarySpec& y) { return !(x < y) && !(y < x); };
        const GroupedAttentionSpec &g = a.grouped, &h = b.grouped;
        const LinearAttentionSpec &l = a.linear, &m = b.linear;
        return a.mixer == b.mixer && a.ff == b.ff && a.ff_size == b.ff_size && g.heads == h.heads && g.kv_heads == h.kv_heads && g.dim == h.dim &&
               g.vdim == h.vdim && g.scale == h.scale && rot(g.rot, h.rot) && l.heads == m.heads && l.dim == m.dim && l.vdim == m.vdim && l.tau == m.tau;
    };
    const size_t n = s->layers.size();
    for (size_t i = 0; i < n && !r.rc; i++) {
        const Json& l = c.get("layers")->arr[i];
        const std::string at = "layers[" + std::to_string(i) + "].";
        const Json* of = l.get("weights_of");
        if (!of || of->kind == Json::Null) continue;
        s->layers[i].weights = r.size(l, "weights_of", at, 0);
        if (!r.rc && s->layers[i].weights >= n) r.fail_at(at + "weights_of", "names no layer");
    }
    // a layer named may itself borrow: follow to the one that has tensors
    for (size_t i = 0; i < n && !r.rc; i++) {
        uint32_t j = s->layers[i].weights;
        for (size_t hops = 0; j != s->layers[j].weights && hops <= n; hops++) j = s->layers[j].weights;
        const std::string at = "layers[" + std::to_string(i) + "].weights_of";
        if (j != s->layers[j].weights) r.fail_at(at, "goes round in a circle");
        else if (!same(s->layers[i], s->layers[j])) r.fail_at(at, "names a layer of another shape");
        s->layers[i].weights = j;
    }
}

// "Vabirax": looped decoder of latent-attention layers, Dynamic Tanh ahead of and behind every sublayer.
int32_t parse_vabirax(const Json& c, BlockSpec* s) {
    Reader r;
    s->post_norms = true;
    read_frame(r, c, s);
    read_layers(r, c, FeedForwardKind::SiluGated, s, [&](const std::string& type, const Json& m, const std::string& at, LayerSpec* l) {
        if (type != "latent_attention") return false;
        l->mixer = MixerKind::LatentAttention;
        read_latent_attention(r, m, at, &l->latent);
        return true;
    });
    const Json* loop = c.get("loop");
    if (loop && loop->kind != Json::Null && !r.rc) {
        s->loop_start = r.size(*loop, "start", "loop.", 0);
        s->loop_stop = r.size(*loop, "stop", "loop.");
        s->loop_times = r.size(*loop, "times", "loop.");
        if (!r.rc && (s->loop_start >= s->loop_stop || s->loop_stop > s->layers.size())) r.fail_at("loop", "does not fit the layers");
    }
    return r.rc;
}

// "Kakirax": decoder that mixes gated linear attention and grouped-query attention layers, a layer norm ahead of every sublayer;
// layers may share weights, the output matrix is the embedding table, logits are capped.
int32_t parse_kakirax(const Json& c, BlockSpec* s) {
    Reader r;
    s->norm = NormKind::LayerNorm;
    s->tied_head = true;
    read_frame(r, c, s);
    const Json* cap = c.get("logit_softcap");
    if (cap && cap->kind != Json::Null) {
        s->logit_cap = r.number(c, "logit_softcap", "");
        if (!r.rc && s->logit_cap <= 0) r.fail_at("logit_softcap", "must be positive");
    }
    read_layers(r, c, FeedForwardKind::GeluTanhGated, s, [&](const std::string& type, const Json& m, const std::string& at, LayerSpec* l) {
        if (type == "attention") {
            l->mixer = MixerKind::GroupedAttention;
            read_grouped_attention(r, m, at, &l->grouped);
        } else if (type == "gla") {
            l->mixer = MixerKind::LinearAttention;
            read_linear_attention(r, m, at, &l->linear);
        } else {
            return false;
        }
        return true;
    });
    if (!r.rc) read_shared_weights(r, c, s);
    return r.rc;
}

struct Architecture {
    const char* name;
    int32_t (*parse)(const Json& config, BlockSpec* out);
};
const Architecture ARCHITECTURES[] = {
    {"Vabirax", parse_vabirax},
    {"Kakirax", parse_kakirax},
};

}  // namespace

double RotarySpec::frequency(uint32_t i) const {
    const double f = pow(base, -2.0 * i / dims);
    if (factor == 0) return f;
    const double length = 2 * M_PI / f;
    if (length < original / high) return f;
    if (length > original / low) return f / factor;
    const double s = high > low ? (original / length - low) / (high - low) : 1.0;
    return (1 - s) * f / factor + s * f;
}

bool architecture_known(const std::string& architecture) {
    for (const Architecture& a : ARCHITECTURES)
        if (architecture == a.name) return true;
    return false;
}

int32_t block_spec_from_config(const Json& config, BlockSpec* out) {
    *out = BlockSpec{};
    const Json* name = config.get("architecture");
    FH_CHECK(name && name->kind == Json::String, "config.json: \"architecture\" is missing");
    out->architecture = name->str;
    for (const Architecture& a : ARCHITECTURES)
        if (name->str == a.name) return a.parse(config, out);
    return fail(FORGE_HIP_ERR_INVALID, "config.json: unknown architecture \"" + name->str + "\"");
}

int32_t block_spec_from_folder(const std::string& dir, BlockSpec* out) {
    const std::string path = dir + "/config.json";
    FILE* f = fopen(path.c_str(), "rb");
    if (!f) return fail(FORGE_HIP_ERR_INVALID, path + ": " + strerror(errno));
    std::string text;
    char buf[65536];
    size_t n;
    while ((n = fread(buf, 1, sizeof(buf), f)) > 0) text.append(buf, n);
    fclose(f);
    Json j;
    const int32_t rc = json_parse(text.data(), text.size(), &j);
    return rc ? rc : block_spec_from_config(j, out);
}

}  // namespace fh
