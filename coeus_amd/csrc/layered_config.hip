// Configuration of the layered models: a small JSON reader, the registry of designs, and the list of
// tensors a configuration needs.  Host code only.
#include "layered.hpp"

#include <cmath>
#include <cstdlib>
#include <initializer_list>

namespace coeus {

// ---------------------------------------------------------------- JSON
namespace {

constexpr int kMaxDepth = 64;

struct Parser {
    const char *p, *end;
    std::string err;

    bool bad(const char *what) {
        if (err.empty()) err = what;
        return false;
    }
    void space() {
        while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++;
    }
    bool word(const char *w) {
        const size_t n = std::strlen(w);
        if ((size_t)(end - p) < n || std::memcmp(p, w, n) != 0) return bad("unexpected character");
        p += n;
        return true;
    }
    static void put_utf8(std::string &s, uint32_t c) {
        if (c < 0x80) s += (char)c;
        else if (c < 0x800) { s += (char)(0xC0 | c >> 6); s += (char)(0x80 | (c & 63)); }
        else if (c < 0x10000) { s += (char)(0xE0 | c >> 12); s += (char)(0x80 | ((c >> 6) & 63)); s += (char)(0x80 | (c & 63)); }
        else { s += (char)(0xF0 | c >> 18); s += (char)(0x80 | ((c >> 12) & 63)); s += (char)(0x80 | ((c >> 6) & 63)); s += (char)(0x80 | (c & 63)); }
    }
    bool hex4(uint32_t &v) {
        if (end - p < 4) return bad("short \\u escape");
        v = 0;
        for (int i = 0; i < 4; i++) {
            const char c = *p++;
            v <<= 4;
            if (c >= '0' && c <= '9') v |= (uint32_t)(c - '0');
            else if (c >= 'a' && c <= 'f') v |= (uint32_t)(c - 'a' + 10);
            else if (c >= 'A' && c <= 'F') v |= (uint32_t)(c - 'A' + 10);
            else return bad("bad \\u escape");
        }
        return true;
    }
    bool string(std::string &s) {
        if (p >= end || *p != '"') return bad("expected a string");
        p++;
        while (p < end && *p != '"') {
            if ((unsigned char)*p < 0x20) return bad("control character in a string");
            if (*p != '\\') { s += *p++; continue; }
            if (++p >= end) break;
            const char c = *p++;
            switch (c) {
                case '"': case '\\': case '/': s += c; break;
                case 'b': s += '\b'; break;
                case 'f': s += '\f'; break;
                case 'n': s += '\n'; break;
                case 'r': s += '\r'; break;
                case 't': s += '\t'; break;
                case 'u': {
                    uint32_t v = 0, lo = 0;
                    if (!hex4(v)) return false;
                    if (v >= 0xD800 && v < 0xDC00) {  // the first half of a surrogate pair
                        if (end - p < 2 || p[0] != '\\' || p[1] != 'u') return bad("lone surrogate");
                        p += 2;
                        if (!hex4(lo)) return false;
                        if (lo < 0xDC00 || lo >= 0xE000) return bad("lone surrogate");
                        v = 0x10000 + ((v - 0xD800) << 10) + (lo - 0xDC00);
                    } else if (v >= 0xDC00 && v < 0xE000) {
                        return bad("lone surrogate");
                    }
                    put_utf8(s, v);
                    break;
                }
                default: return bad("bad escape");
            }
        }
        if (p >= end) return bad("unterminated string");
        p++;
        return true;
    }
    bool number(double &v) {
        const char *b = p;
        if (p < end && *p == '-') p++;
        if (p >= end || *p < '0' || *p > '9') return bad("unexpected character");
        if (*p == '0') p++;  // no leading zeros
        else while (p < end && *p >= '0' && *p <= '9') p++;
        if (p < end && *p == '.') {
            if (++p >= end || *p < '0' || *p > '9') return bad("bad number");
            while (p < end && *p >= '0' && *p <= '9') p++;
        }
        if (p < end && (*p == 'e' || *p == 'E')) {
            p++;
            if (p < end && (*p == '+' || *p == '-')) p++;
            if (p >= end || *p < '0' || *p > '9') return bad("bad number");
            while (p < end && *p >= '0' && *p <= '9') p++;
        }
        const std::string s(b, p);
        v = std::strtod(s.c_str(), nullptr);
        return true;
    }
    bool value(Json &j, int depth) {
        if (depth > kMaxDepth) return bad("nested too deeply");
        space();
        if (p >= end) return bad("unexpected end");
        switch (*p) {
            case 'n': j.type = Json::Null; return word("null");
            case 't': j.type = Json::Bool; j.b = true; return word("true");
            case 'f': j.type = Json::Bool; j.b = false; return word("false");
            case '"': j.type = Json::String; return string(j.str);
            case '[':
                j.type = Json::Array;
                p++;
                space();
                if (p < end && *p == ']') { p++; return true; }
                for (;;) {
                    j.items.emplace_back();
                    if (!value(j.items.back(), depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == ']') { p++; return true; }
                    return bad("expected , or ]");
                }
            case '{':
                j.type = Json::Object;
                p++;
                space();
                if (p < end && *p == '}') { p++; return true; }
                for (;;) {
                    space();
                    std::string key;
                    if (!string(key)) return false;
                    space();
                    if (p >= end || *p != ':') return bad("expected :");
                    p++;
                    j.fields.emplace_back(std::move(key), Json());
                    if (!value(j.fields.back().second, depth + 1)) return false;
                    space();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == '}') { p++; return true; }
                    return bad("expected , or }");
                }
            default: j.type = Json::Number; return number(j.num);
        }
    }
};

}  // namespace

const Json *Json::get(const char *key) const {
    const Json *hit = nullptr;
    if (type == Object)
        for (const auto &kv : fields)
            if (kv.first == key) hit = &kv.second;  // the last of repeated keys counts
    return hit;
}

bool json_parse(const char *text, uint64_t len, Json &out, std::string &err) {
    Parser ps{text, text + len, {}};
    bool ok = ps.value(out, 0);
    if (ok) {
        ps.space();
        if (ps.p != ps.end) ok = ps.bad("text after the value");
    }
    err = ps.err;
    return ok;
}

// ---------------------------------------------------------------- reading a configuration
namespace {

int bad_config(const std::string &key, const char *why) {
    return fail(COEUS_INVALID_CONFIG, "Invalid configuration: %s: %s", key.c_str(), why);
}

constexpr uint64_t kMaxSize = 1ull << 24;  // any width, rank, head count or vocabulary

int get_size(const Json &o, const std::string &path, const char *key, uint64_t &out) {
    const Json *j = o.get(key);
    if (!j || j->type != Json::Number) return bad_config(path + key, "expected a number");
    if (!(j->num >= 1.0) || j->num > (double)kMaxSize || j->num != std::floor(j->num))
        return bad_config(path + key, "must be a whole number of at least 1");
    out = (uint64_t)j->num;
    return COEUS_OK;
}

int get_real(const Json &o, const std::string &path, const char *key, float &out) {
    const Json *j = o.get(key);
    if (!j || j->type != Json::Number || !std::isfinite((float)j->num)) return bad_config(path + key, "expected a number");
    out = (float)j->num;
    return COEUS_OK;
}

int read_gated_delta(const Json &m, const std::string &path, MixerSpec &s) {
    s.kind = MixerKind::GatedDelta;
    COEUS_TRY(get_size(m, path, "heads", s.heads));
    COEUS_TRY(get_size(m, path, "kv_heads", s.kv_heads));
    COEUS_TRY(get_size(m, path, "dim", s.dim));
    COEUS_TRY(get_size(m, path, "vdim", s.vdim));
    COEUS_TRY(get_size(m, path, "conv", s.conv));
    if (s.heads % s.kv_heads) return bad_config(path + "kv_heads", "heads must be a multiple of kv_heads");
    if (s.dim > 256) return bad_config(path + "dim", "more than 256 is not supported");
    if (s.vdim > 1024) return bad_config(path + "vdim", "more than 1024 is not supported");
    if (s.conv > 16) return bad_config(path + "conv", "more than 16 taps are not supported");
    return COEUS_OK;
}

int read_mask(const Json &m, const std::string &path, MixerSpec &s) {
    const Json *mask = m.get("mask");
    if (!mask || mask->type == Json::Null) return COEUS_OK;
    if (mask->type != Json::Object) return bad_config(path + "mask", "expected an object");
    return get_size(*mask, path + "mask.", "size", s.window);
}

int read_latent_attention(const Json &m, const std::string &path, MixerSpec &s) {
    s.kind = MixerKind::LatentAttention;
    COEUS_TRY(get_size(m, path, "heads", s.heads));
    COEUS_TRY(get_size(m, path, "dim", s.dim));
    COEUS_TRY(get_size(m, path, "vdim", s.vdim));
    COEUS_TRY(get_size(m, path, "q_rank", s.q_rank));
    COEUS_TRY(get_size(m, path, "kv_rank", s.kv_rank));
    COEUS_TRY(get_real(m, path, "scale", s.scale));
    if (s.dim > 256) return bad_config(path + "dim", "more than 256 is not supported");
    if (s.vdim > 256) return bad_config(path + "vdim", "more than 256 is not supported");
    if (s.kv_rank > 2048) return bad_config(path + "kv_rank", "more than 2048 is not supported");
    return read_mask(m, path, s);
}

int read_matrix_memory(const Json &m, const std::string &path, MixerSpec &s) {
    s.kind = MixerKind::MatrixMemory;
    COEUS_TRY(get_size(m, path, "heads", s.heads));
    COEUS_TRY(get_size(m, path, "dim", s.dim));
    COEUS_TRY(get_size(m, path, "vdim", s.vdim));
    COEUS_TRY(get_real(m, path, "gate_cap", s.gate_cap));
    if (!(s.gate_cap > 0.f)) return bad_config(path + "gate_cap", "must be positive");
    if (s.dim > 512) return bad_config(path + "dim", "more than 512 is not supported");
    if (s.vdim > 1024) return bad_config(path + "vdim", "more than 1024 is not supported");
    return COEUS_OK;
}

int read_shared_kv(const Json &m, const std::string &path, MixerSpec &s) {
    s.kind = MixerKind::SharedKv;
    COEUS_TRY(get_size(m, path, "heads", s.heads));
    COEUS_TRY(get_size(m, path, "kv_heads", s.kv_heads));
    COEUS_TRY(get_size(m, path, "dim", s.dim));
    COEUS_TRY(get_size(m, path, "vdim", s.vdim));
    COEUS_TRY(get_real(m, path, "scale", s.scale));
    if (s.heads % s.kv_heads) return bad_config(path + "kv_heads", "heads must be a multiple of kv_heads");
    if (s.vdim != s.dim) return bad_config(path + "vdim", "must equal dim where the values are the keys");
    if (s.dim > 256) return bad_config(path + "dim", "more than 256 is not supported");
    return read_mask(m, path, s);
}

// A mixer's reader by the layer's type.  A design may have several variants of one mixer, told apart
// by a number at the end ("delta", "delta_2"): they share a reader, their sizes differ.
struct MixerType {
    const char *name;
    int (*read)(const Json &, const std::string &, MixerSpec &);
};
int read_mixer(const std::string &type, const Json &m, const std::string &path, std::initializer_list<MixerType> types, MixerSpec &s) {
    std::string base = type;
    const size_t us = base.rfind('_');
    if (us != std::string::npos && us + 1 < base.size() &&
        base.find_first_not_of("0123456789", us + 1) == std::string::npos)
        base.resize(us);
    for (const MixerType &t : types)
        if (base == t.name) return t.read(m, path, s);
    return fail(COEUS_INVALID_CONFIG, "Invalid configuration: %stype = %s: unknown layer type", path.c_str(), type.c_str());
}

// What every design's configuration has: width, vocabulary, the norms' eps, and the list of layers, whose
// mixers are of the given types.  read_gate (nullable) reads what a feed-forward has besides its width.
int read_stack(const Json &j, std::initializer_list<MixerType> types, int (*read_gate)(const Json &, const std::string &, LayerSpec &),
               LayeredConfig &c) {
    COEUS_TRY(get_size(j, "", "width", c.width));
    COEUS_TRY(get_size(j, "", "vocab", c.vocab));
    const Json *norm = j.get("norm"), *layers = j.get("layers");
    if (!norm || norm->type != Json::Object) return bad_config("norm", "expected an object");
    COEUS_TRY(get_real(*norm, "norm.", "eps", c.eps));
    if (!layers || layers->type != Json::Array || layers->items.empty())
        return bad_config("layers", "expected a list of layers");
    if (layers->items.size() > 4096) return bad_config("layers", "too many layers");
    for (size_t i = 0; i < layers->items.size(); i++) {
        const Json &lj = layers->items[i];
        const std::string path = "layers[" + std::to_string(i) + "].";
        const Json *type = lj.get("type"), *mixer = lj.get("mixer"), *mlp = lj.get("mlp");
        if (!type || type->type != Json::String) return bad_config(path + "type", "expected a string");
        if (!mixer || mixer->type != Json::Object) return bad_config(path + "mixer", "expected an object");
        LayerSpec l;
        l.source = i;
        COEUS_TRY(read_mixer(type->str, *mixer, path + "mixer.", types, l.mixer));
        if (mlp && mlp->type != Json::Null) {
            const Json *kind = mlp->get("kind");
            if (!kind || kind->type != Json::String || kind->str != "dense")
                return bad_config(path + "mlp.kind", "unknown feed-forward");
            COEUS_TRY(get_size(*mlp, path + "mlp.", "ff", l.ff));
            if (read_gate) COEUS_TRY(read_gate(*mlp, path + "mlp.", l));
        }
        c.layers.push_back(l);
    }
    return COEUS_OK;
}

// "weights_of": j makes a layer use layer j's tensors (which may be another layer's in turn).
int read_shared_layers(const Json &j, LayeredConfig &c) {
    const std::vector<Json> &items = j.get("layers")->items;
    const size_t n = items.size();
    for (size_t i = 0; i < n; i++) {
        const Json *of = items[i].get("weights_of");
        if (!of || of->type == Json::Null) continue;
        const std::string path = "layers[" + std::to_string(i) + "].weights_of";
        if (of->type != Json::Number || !(of->num >= 0.0) || of->num >= (double)n || of->num != std::floor(of->num))
            return bad_config(path, "must be the number of a layer");
        c.layers[i].source = (uint64_t)of->num;
        if (c.layers[i].source == i) return bad_config(path, "a layer cannot take its own tensors from itself");
    }
    for (size_t i = 0; i < n; i++) {
        const std::string path = "layers[" + std::to_string(i) + "].weights_of";
        uint64_t at = i;
        for (size_t hop = 0; c.layers[at].source != at; hop++) {
            if (hop == n) return bad_config(path, "no layer of this chain has tensors");
            at = c.layers[at].source;
        }
        LayerSpec &l = c.layers[i];
        const LayerSpec &o = c.layers[at];
        if (!(l.mixer == o.mixer) || l.ff != o.ff || l.gate != o.gate || l.limit != o.limit)
            return bad_config(path, "the two layers differ");
        l.source = at;
    }
    return COEUS_OK;
}

// Bofirax: each sublayer reads the residual stream itself, its output is RMS-normalised and scaled per
// channel before it is added; embedding table and output projection are one tensor.
int read_bofirax(const Json &j, LayeredConfig &c) {
    return read_stack(j, {{"delta", read_gated_delta}, {"latent_attention", read_latent_attention}}, nullptr, c);
}

int read_clamped_gate(const Json &mlp, const std::string &path, LayerSpec &l) {
    l.gate = GateKind::Clamped;
    return get_real(mlp, path, "limit", l.limit);
}

// Zekilix: hyper-connections around sublayers with a layer norm in front; matrix memories and windowed
// attention whose values are its keys; layers may share tensors; scaled embeddings, an output projection of
// its own, capped logits.
int read_zekilix(const Json &j, LayeredConfig &c) {
    COEUS_TRY(read_stack(j, {{"mlstm", read_matrix_memory}, {"attention", read_shared_kv}}, read_clamped_gate, c));
    COEUS_TRY(read_shared_layers(j, c));
    c.tied = false;
    const Json *emb = j.get("embedding");
    if (!emb || emb->type != Json::Object) return bad_config("embedding", "expected an object");
    COEUS_TRY(get_real(*emb, "embedding.", "scale", c.embed_scale));
    COEUS_TRY(get_size(j, "", "streams", c.streams));
    if (c.streams > kMaxHyperStreams) return bad_config("streams", "more than 8 are not supported");
    COEUS_TRY(get_real(j, "", "residual_mult", c.residual_mult));
    COEUS_TRY(get_real(j, "", "logit_softcap", c.logit_softcap));
    if (!(c.logit_softcap > 0.f)) return bad_config("logit_softcap", "must be positive");
    return COEUS_OK;
}

struct Architecture {
    const char *name;
    int (*read)(const Json &, LayeredConfig &);
};
constexpr Architecture kArchitectures[] = {{"Bofirax", read_bofirax}, {"Zekilix", read_zekilix}};

}  // namespace

int layered_config_parse(const char *text, uint64_t len, LayeredConfig &out) {
    Json j;
    std::string err;
    if (!json_parse(text, len, j, err)) return fail(COEUS_INVALID_CONFIG, "Invalid configuration: not JSON: %s", err.c_str());
    const Json *arch = j.get("architecture");
    if (!arch || arch->type != Json::String) return bad_config("architecture", "expected a string");
    for (const Architecture &a : kArchitectures)
        if (arch->str == a.name) {
            out = LayeredConfig{};
            out.architecture = a.name;
            return a.read(j, out);
        }
    return fail(COEUS_INVALID_CONFIG, "Invalid configuration: architecture = %s: unknown architecture", arch->str.c_str());
}

// ---------------------------------------------------------------- tensors
std::string layer_tensor(uint64_t layer, const char *suffix) { return "l" + std::to_string(layer) + "." + suffix; }

std::vector<TensorSpec> layered_tensors(const LayeredConfig &c) {
    std::vector<TensorSpec> t;
    t.push_back({"embed", c.vocab, c.width, 0.f});
    for (uint64_t l = 0; l < c.layers.size(); l++) {
        const LayerSpec &s = c.layers[l];
        const MixerSpec &m = s.mixer;
        if (s.source != l) continue;
        auto mat = [&](const char *suffix, uint64_t rows, uint64_t cols, float mean = 0.f) {
            t.push_back({layer_tensor(l, suffix), rows, cols, mean});
        };
        auto vec = [&](const char *suffix, uint64_t n, float mean) { t.push_back({layer_tensor(l, suffix), n, 0, mean}); };
        const uint64_t qk = m.heads * m.dim, v = m.inner();
        switch (m.kind) {
            case MixerKind::GatedDelta: {
                const uint64_t kqk = m.kv_heads * m.dim;
                const float tap = 1.0f / (float)m.conv;
                mat("mix.q", kqk, c.width); mat("mix.q.conv", kqk, m.conv, tap);
                mat("mix.k", kqk, c.width); mat("mix.k.conv", kqk, m.conv, tap);
                mat("mix.v", v, c.width); mat("mix.v.conv", v, m.conv, tap);
                mat("mix.g", v, c.width);
                mat("mix.b", m.heads, c.width); mat("mix.a", m.heads, c.width);
                vec("mix.A_log", m.heads, -2.f); vec("mix.dt_bias", m.heads, -2.f);
                vec("mix.norm", m.vdim, 1.f);
                break;
            }
            case MixerKind::LatentAttention:
                mat("mix.dq", m.q_rank, c.width); vec("mix.dq.norm", m.q_rank, 1.f);
                mat("mix.uq", qk, m.q_rank);
                mat("mix.dkv", m.kv_rank, c.width); vec("mix.dkv.norm", m.kv_rank, 1.f);
                mat("mix.uk", qk, m.kv_rank); mat("mix.uv", v, m.kv_rank);
                break;
            case MixerKind::MatrixMemory:
                mat("mix.q", qk, c.width); mat("mix.k", qk, c.width); mat("mix.v", v, c.width); mat("mix.g", v, c.width);
                mat("mix.i", m.heads, c.width); vec("mix.i.b", m.heads, 0.f);
                mat("mix.f", m.heads, c.width); vec("mix.f.b", m.heads, 4.f);
                vec("mix.norm", v, 1.f);
                break;
            case MixerKind::SharedKv:
                mat("mix.q", qk, c.width); vec("mix.q.norm", qk, 1.f);
                mat("mix.k", m.kv_heads * m.dim, c.width); vec("mix.k.norm", m.kv_heads * m.dim, 1.f);
                mat("mix.g", v, c.width);
                break;
        }
        mat("mix.o", c.width, v);
        // what stands around a sublayer
        auto around = [&](const char *norm, const char *ls, const std::string &hc) {
            vec(norm, c.width, 1.f);
            if (!c.streams) { vec(ls, c.width, 1.f); return; }
            vec((hc + ".in").c_str(), c.streams, 1.0f / (float)c.streams);
            vec((hc + ".out").c_str(), c.streams, 1.f);
            mat((hc + ".mix").c_str(), c.streams, c.streams, 1.0f / (float)c.streams);
        };
        around("norm1", "ls1", "hc1");
        if (s.ff) {
            mat("mlp.gate", s.ff, c.width); mat("mlp.up", s.ff, c.width); mat("mlp.down", c.width, s.ff);
            around("norm2", "ls2", "hc2");
        }
    }
    t.push_back({"final.norm", c.width, 0, 1.f});
    if (!c.tied) t.push_back({"head", c.vocab, c.width, 0.f});
    return t;
}

}  // namespace coeus
