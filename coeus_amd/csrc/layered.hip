// Layered decoder models on the device: construction from a folder (config.json + model.safetensors) or
// from a seed, the state a session carries, and the layers of a prompt pass and of a decode step.
//
// Two forms of the residual: norms behind the sublayers (a sublayer reads the f32 residual stream itself, and
// norm_residual adds its normalised, scaled output to it), and hyper-connections (several f32 streams; one
// launch takes a sublayer's output into them and makes the next one's normalised input).
#include "model.hpp"

#include <cmath>
#include <initializer_list>

namespace coeus {

DeltaDims LayeredLayer::delta_dims() const {
    const MixerSpec &m = spec.mixer;
    return DeltaDims{(uint32_t)m.heads, (uint32_t)m.kv_heads, (uint32_t)m.dim, (uint32_t)m.vdim, (uint32_t)m.conv, (uint32_t)in.n};
}
LatentDims LayeredLayer::latent_dims() const {
    const MixerSpec &m = spec.mixer;
    return LatentDims{(uint32_t)m.heads, (uint32_t)m.dim, (uint32_t)m.vdim, (uint32_t)m.q_rank, (uint32_t)m.kv_rank,
                      (uint32_t)m.window, (uint32_t)in.n, m.scale};
}
MemoryDims LayeredLayer::memory_dims() const {
    const MixerSpec &m = spec.mixer;
    return MemoryDims{(uint32_t)m.heads, (uint32_t)m.dim, (uint32_t)m.vdim, (uint32_t)in.n, m.gate_cap};
}
SharedKvDims LayeredLayer::shared_dims() const {
    constexpr float kSlopeRange = 8.0f;  // distance slopes 2^(-8 (h + 1) / heads)
    const MixerSpec &m = spec.mixer;
    return SharedKvDims{(uint32_t)m.heads, (uint32_t)m.kv_heads, (uint32_t)m.dim, (uint32_t)m.window, (uint32_t)in.n, m.scale, kSlopeRange};
}

LayeredStack::~LayeredStack() {
    for (LayeredLayer &l : layers)
        for (Weight *w : {&l.in, &l.o, &l.up, &l.down, &l.uq, &l.ukv}) weight_free(*w);
    if (small) (void)hipFree(small);
    if (folds) (void)hipFree(folds);
}

// ---------------------------------------------------------------- state
// Offsets are counted first, then assigned: the recurrent part of every layer, then the rings of cached
// rows.  Those start as zeros and are not cleared again: a position that is not written yet has no weight,
// but its slot may be read, so it has to hold finite values.
int LayeredState::create(const LayeredStack &stack, bool bf16, uint64_t batch_, uint64_t max_ctx, hipStream_t st) {
    batch = batch_;
    layers.assign(stack.layers.size(), Layer{});
    uint64_t off = 0;
    std::vector<std::pair<void **, uint64_t>> fix;
    auto take = [&](auto *where, uint64_t bytes) { fix.emplace_back((void **)where, off); off += round_up(bytes, 256); };
    for (size_t l = 0; l < layers.size(); l++) {
        const MixerSpec &m = stack.weights(l).spec.mixer;
        if (m.kind == MixerKind::GatedDelta) {
            take(&layers[l].delta.s, batch * m.heads * m.dim * m.vdim * 4);
            take(&layers[l].delta.ring, batch * m.conv * m.conv_channels() * 4);
        } else if (m.kind == MixerKind::MatrixMemory) {
            take(&layers[l].memory.s, batch * m.heads * m.dim * m.vdim * 4);
            take(&layers[l].memory.n, batch * m.heads * m.dim * 4);
            take(&layers[l].memory.m, batch * m.heads * 4);
        }
    }
    recurrent_bytes = off;
    for (size_t l = 0; l < layers.size(); l++) {
        const LayeredLayer &ly = stack.weights(l);
        const MixerSpec &m = ly.spec.mixer;
        uint64_t len = 0;
        if (m.kind == MixerKind::LatentAttention) len = m.kv_rank;
        else if (m.kind == MixerKind::SharedKv) len = ly.shared_dims().row_len();
        else continue;
        const uint64_t cap = m.window && m.window < max_ctx ? m.window : max_ctx;
        layers[l].ring.cap = (uint32_t)cap;
        layers[l].ring.bf16 = bf16;
        take(&layers[l].ring.c, batch * cap * len * (bf16 ? 2 : 4));
    }
    COEUS_TRY(mem.ensure(off ? off : 256));
    COEUS_HIP(hipMemsetAsync(mem.p, 0, mem.bytes, st));
    for (auto &f : fix) *f.first = (char *)mem.p + f.second;
    return COEUS_OK;
}

int LayeredState::clear(hipStream_t st) {
    if (recurrent_bytes) COEUS_HIP(hipMemsetAsync(mem.p, 0, recurrent_bytes, st));
    return COEUS_OK;
}

// ---------------------------------------------------------------- construction
namespace {

uint16_t bf16_bits_host(float x) {
    uint32_t u;
    std::memcpy(&u, &x, 4);
    if ((u & 0x7f800000u) == 0x7f800000u && (u & 0x007fffffu)) return (uint16_t)((u | 0x00400000u) >> 16);
    return (uint16_t)((u + 0x7fffu + ((u >> 16) & 1u)) >> 16);
}

// Where the values come from: a weight file, or the synthetic generator (tensor i of the list draws
// from indices behind those of the tensors before it).
struct Source {
    const SafeTensors *file = nullptr;
    uint64_t seed = 0;
    std::vector<TensorSpec> specs;
    std::vector<uint64_t> first;

    int index(const std::string &name, size_t &out) const {
        for (size_t i = 0; i < specs.size(); i++)
            if (specs[i].name == name) { out = i; return COEUS_OK; }
        return fail(COEUS_INVALID_INPUT, "unknown tensor %s", name.c_str());
    }
    // f32 on the host (small tensors)
    int host(const std::string &name, std::vector<float> &out) const {
        size_t i = 0;
        COEUS_TRY(index(name, i));
        out.resize(specs[i].elems());
        if (!file) {
            for (size_t j = 0; j < out.size(); j++) out[j] = specs[i].mean + synth_value_host(seed, first[i] + j);
            return COEUS_OK;
        }
        const SafeTensor *t = file->find(name);
        if (t->dtype == "F32") {
            std::memcpy(out.data(), t->data, out.size() * 4);
        } else {
            for (size_t j = 0; j < out.size(); j++) {
                const uint32_t u = ((uint32_t)t->data[2 * j] | (uint32_t)t->data[2 * j + 1] << 8) << 16;
                std::memcpy(&out[j], &u, 4);
            }
        }
        return COEUS_OK;
    }
    // rows of a matrix into rows row0, row0 + stride, .. of a dense device weight
    int rows(const std::string &name, Weight &w, uint64_t row0, uint64_t stride, hipStream_t st) const {
        size_t i = 0;
        COEUS_TRY(index(name, i));
        const TensorSpec &s = specs[i];
        if (s.cols != w.k || row0 + (s.rows - 1) * stride >= w.n)
            return fail(COEUS_INVALID_INPUT, "tensor %s does not fit its place", name.c_str());
        const uint64_t es = w.dtype == COEUS_W_F32 ? 4 : 2, row = s.cols * es;
        char *dst = (char *)w.data + row0 * row;
        if (file) {
            const SafeTensor *t = file->find(name);
            std::vector<uint8_t> conv;
            const uint8_t *src = t->data;
            if ((t->dtype == "BF16") != (w.dtype == COEUS_W_BF16)) {
                std::vector<float> f;
                COEUS_TRY(host(name, f));
                conv.resize(f.size() * es);
                if (w.dtype == COEUS_W_F32) std::memcpy(conv.data(), f.data(), conv.size());
                else for (size_t j = 0; j < f.size(); j++) { const uint16_t u = bf16_bits_host(f[j]); std::memcpy(&conv[2 * j], &u, 2); }
                src = conv.data();
            }
            COEUS_HIP(hipMemcpy2D(dst, row * stride, src, row, row, s.rows, hipMemcpyHostToDevice));
            return COEUS_OK;
        }
        DeviceBuf f, h;
        struct Drop { DeviceBuf &a, &b; ~Drop() { a.release(); b.release(); } } drop{f, h};
        COEUS_TRY(f.ensure(s.elems() * 4));
        COEUS_TRY(launch_fill_seeded((float *)f.p, s.elems(), seed, first[i], s.mean, st));
        const void *src = f.p;
        if (es == 2) {
            COEUS_TRY(h.ensure(s.elems() * 2));
            COEUS_TRY(launch_f32_to_bf16((const float *)f.p, (uint16_t *)h.p, s.elems(), st));
            src = h.p;
        }
        COEUS_HIP(hipMemcpy2DAsync(dst, row * stride, src, row, row, s.rows, hipMemcpyDeviceToDevice, st));
        COEUS_HIP(hipStreamSynchronize(st));
        return COEUS_OK;
    }
};

// The records that decode steps fold hyper-connections with, in the order of the sublayers.
int make_folds(LayeredStack &stack, hipStream_t st) {
    const LayeredConfig &cfg = stack.cfg;
    if (!cfg.streams || cfg.streams > kMaxFoldedStreams) return COEUS_OK;
    COEUS_HIP(hipMalloc((void **)&stack.folds, 2 * cfg.layers.size() * kHyperFoldFloats * 4));
    const Around *from = nullptr;
    float *at = stack.folds;
    auto next = [&](const Around &to) -> int {
        COEUS_TRY(launch_hyper_fold(from ? from->mix : nullptr, from ? from->out : nullptr, to.in, cfg.residual_mult, (uint32_t)cfg.streams,
                                    at, st));
        from = &to;
        at += kHyperFoldFloats;
        return COEUS_OK;
    };
    for (size_t l = 0; l < cfg.layers.size(); l++) {
        COEUS_TRY(next(stack.weights(l).around_mixer));
        if (cfg.layers[l].ff) COEUS_TRY(next(stack.weights(l).around_ff));
    }
    return COEUS_OK;
}

int build(const LayeredConfig &cfg, const SafeTensors *file, uint64_t seed, const coeus_load_options &opt, Model **out) {
    if (opt.weight_dtype != COEUS_W_F32 && opt.weight_dtype != COEUS_W_BF16)
        return fail(COEUS_INVALID_CONFIG, "Invalid configuration: weight_dtype = %u: layered models take f32 or bf16 weights",
                    opt.weight_dtype);
    const uint64_t max_seq = opt.max_seq_len ? opt.max_seq_len : 1048576, max_batch = opt.max_batch ? opt.max_batch : 1;
    if (max_seq >= (1ull << 31)) return fail(COEUS_INVALID_CONFIG, "Invalid configuration: max_seq_len = %llu: too large", (unsigned long long)max_seq);
    if (max_batch > 16)
        return fail(COEUS_INVALID_CONFIG, "Invalid configuration: max_batch = %llu: at most 16 sequences per session", (unsigned long long)max_batch);
    COEUS_TRY(check_device());
    const bool bf16 = opt.weight_dtype == COEUS_W_BF16;
    const uint32_t wd = opt.weight_dtype;

    Source src;
    src.file = file;
    src.seed = seed;
    src.specs = layered_tensors(cfg);
    uint64_t total = 0;
    for (const TensorSpec &t : src.specs) { src.first.push_back(total); total += t.elems(); }

    std::unique_ptr<Model> m(new Model());
    m->stack.reset(new LayeredStack());
    LayeredStack &stack = *m->stack;
    stack.cfg = cfg;
    coeus_config &c = m->cfg;  // what the family-independent code and coeus_model_config read
    c.hidden_dim = cfg.width;
    c.num_layers = cfg.layers.size();
    c.num_heads = cfg.layers[0].mixer.heads;
    c.head_dim = cfg.layers[0].mixer.dim;
    for (const LayerSpec &l : cfg.layers) c.intermediate_dim = std::max(c.intermediate_dim, l.ff);
    c.vocab_size = cfg.vocab;
    c.max_seq_len = max_seq;
    c.layer_norm_eps = cfg.eps;
    c.activation = COEUS_ACT_SILU_GATED;
    c.norm = cfg.streams ? COEUS_NORM_LAYERNORM : COEUS_NORM_RMSNORM;
    c.norm_scope = COEUS_SCOPE_TOKEN;
    c.weight_dtype = wd;
    c.kv_dtype = bf16 ? COEUS_KV_BF16 : COEUS_KV_F32;
    c.max_batch = max_batch;
    m->n_params = total;
    m->embed_scale = cfg.embed_scale;
    m->logit_softcap = cfg.logit_softcap;
    COEUS_HIP(hipStreamCreateWithFlags(&m->stream, hipStreamNonBlocking));
    hipStream_t st = m->stream;

    // ---- f32 vectors of all layers, one allocation
    std::vector<float> small, tmp;
    std::vector<std::pair<const float **, uint64_t>> fix;  // pointers to set once the allocation exists
    auto put = [&](const float **where, const std::vector<float> &v) {
        fix.emplace_back(where, small.size());
        small.insert(small.end(), v.begin(), v.end());
        small.resize(round_up(small.size(), 4), 0.f);  // 16-byte loads
    };
    auto put_tensor = [&](const float **where, const std::string &name) -> int {
        COEUS_TRY(src.host(name, tmp));
        put(where, tmp);
        return COEUS_OK;
    };
    stack.layers.resize(cfg.layers.size());
    for (uint64_t l = 0; l < cfg.layers.size(); l++) {
        LayeredLayer &ly = stack.layers[l];
        ly.spec = cfg.layers[l];
        if (ly.spec.source != l) continue;
        const MixerSpec &mx = ly.spec.mixer;
        auto name = [&](const char *s) { return layer_tensor(l, s); };
        // rows behind the last projection pad the row length to a multiple of 4 (16-byte stores); zero weights
        const uint64_t in_rows = round_up(mx.in_rows(), 4);
        COEUS_TRY(weight_alloc(ly.in, wd, cfg.width, in_rows));
        COEUS_HIP(hipMemset(ly.in.data, 0, ly.in.bytes));
        COEUS_TRY(weight_alloc(ly.o, wd, mx.inner(), cfg.width));
        COEUS_TRY(src.rows(name("mix.o"), ly.o, 0, 1, st));
        // the parts of the fused input projection, one behind the other
        auto project = [&](std::initializer_list<std::pair<const char *, uint64_t>> parts) -> int {
            uint64_t r = 0;
            for (const auto &part : parts) {
                COEUS_TRY(src.rows(name(part.first), ly.in, r, 1, st));
                r += part.second;
            }
            return COEUS_OK;
        };
        switch (mx.kind) {
            case MixerKind::GatedDelta: {
                COEUS_TRY(project({{"mix.q", mx.kv_heads * mx.dim}, {"mix.k", mx.kv_heads * mx.dim}, {"mix.v", mx.inner()},
                                   {"mix.g", mx.inner()}, {"mix.b", mx.heads}, {"mix.a", mx.heads}}));
                // taps of q, k, v, [tap][channel]
                const uint64_t C = mx.conv_channels();
                std::vector<float> taps(mx.conv * C);
                uint64_t c0 = 0;
                for (const char *s : {"mix.q.conv", "mix.k.conv", "mix.v.conv"}) {
                    COEUS_TRY(src.host(name(s), tmp));
                    const uint64_t n = tmp.size() / mx.conv;
                    for (uint64_t ch = 0; ch < n; ch++)
                        for (uint64_t j = 0; j < mx.conv; j++) taps[j * C + c0 + ch] = tmp[ch * mx.conv + j];
                    c0 += n;
                }
                put(&ly.delta.conv, taps);
                COEUS_TRY(src.host(name("mix.A_log"), tmp));
                for (float &v : tmp) v = expf(v);
                put(&ly.delta.exp_a, tmp);
                COEUS_TRY(put_tensor(&ly.delta.dt_bias, name("mix.dt_bias")));
                COEUS_TRY(put_tensor(&ly.delta.norm, name("mix.norm")));
                ly.delta.eps = cfg.eps;
                break;
            }
            case MixerKind::LatentAttention:
                COEUS_TRY(project({{"mix.dq", mx.q_rank}, {"mix.dkv", mx.kv_rank}}));
                COEUS_TRY(weight_alloc(ly.uq, wd, mx.q_rank, mx.heads * mx.dim));
                COEUS_TRY(src.rows(name("mix.uq"), ly.uq, 0, 1, st));
                COEUS_TRY(weight_alloc(ly.ukv, wd, mx.kv_rank, mx.heads * (mx.dim + mx.vdim)));
                COEUS_TRY(src.rows(name("mix.uk"), ly.ukv, 0, 1, st));
                COEUS_TRY(src.rows(name("mix.uv"), ly.ukv, mx.heads * mx.dim, 1, st));
                COEUS_TRY(put_tensor(&ly.dq_norm, name("mix.dq.norm")));
                COEUS_TRY(put_tensor(&ly.dkv_norm, name("mix.dkv.norm")));
                break;
            case MixerKind::MatrixMemory:
                COEUS_TRY(project({{"mix.q", mx.heads * mx.dim}, {"mix.k", mx.heads * mx.dim}, {"mix.v", mx.inner()},
                                   {"mix.g", mx.inner()}, {"mix.i", mx.heads}, {"mix.f", mx.heads}}));
                COEUS_TRY(put_tensor(&ly.memory.in_bias, name("mix.i.b")));
                COEUS_TRY(put_tensor(&ly.memory.forget_bias, name("mix.f.b")));
                COEUS_TRY(put_tensor(&ly.memory.norm, name("mix.norm")));
                ly.memory.eps = cfg.eps;
                break;
            case MixerKind::SharedKv: {
                COEUS_TRY(project({{"mix.q", mx.heads * mx.dim}, {"mix.k", mx.kv_heads * mx.dim}, {"mix.g", mx.inner()}}));
                std::vector<float> wq;
                COEUS_TRY(src.host(name("mix.q.norm"), wq));
                COEUS_TRY(src.host(name("mix.k.norm"), tmp));
                const uint64_t per = mx.heads / mx.kv_heads;
                for (uint64_t h = 0; h < mx.heads; h++)
                    for (uint64_t t = 0; t < mx.dim; t++) wq[h * mx.dim + t] *= tmp[h / per * mx.dim + t];
                put(&ly.wqk, wq);
                break;
            }
        }
        auto around = [&](Around &a, const char *norm, const char *ls, const std::string &hc) -> int {
            COEUS_TRY(put_tensor(&a.norm, name(norm)));
            if (!cfg.streams) return put_tensor(&a.ls, name(ls));
            COEUS_TRY(put_tensor(&a.in, name((hc + ".in").c_str())));
            COEUS_TRY(put_tensor(&a.out, name((hc + ".out").c_str())));
            return put_tensor(&a.mix, name((hc + ".mix").c_str()));
        };
        COEUS_TRY(around(ly.around_mixer, "norm1", "ls1", "hc1"));
        if (ly.spec.ff) {
            COEUS_TRY(weight_alloc(ly.up, wd, cfg.width, 2 * ly.spec.ff));  // rows gate_0, up_0, gate_1, ..
            COEUS_TRY(src.rows(name("mlp.gate"), ly.up, 0, 2, st));
            COEUS_TRY(src.rows(name("mlp.up"), ly.up, 1, 2, st));
            COEUS_TRY(weight_alloc(ly.down, wd, ly.spec.ff, cfg.width));
            COEUS_TRY(src.rows(name("mlp.down"), ly.down, 0, 1, st));
            COEUS_TRY(around(ly.around_ff, "norm2", "ls2", "hc2"));
        }
        for (const Weight *w : {&ly.in, &ly.o, &ly.up, &ly.down, &ly.uq, &ly.ukv}) m->weight_bytes += w->bytes;
    }
    COEUS_TRY(put_tensor(&m->fin_s, "final.norm"));
    COEUS_HIP(hipMalloc((void **)&stack.small, small.size() * 4));
    COEUS_HIP(hipMemcpy(stack.small, small.data(), small.size() * 4, hipMemcpyHostToDevice));
    for (auto &f : fix) *f.first = stack.small + f.second;
    m->weight_bytes += small.size() * 4;
    COEUS_TRY(make_folds(stack, st));

    // ---- output projection, which may be the embedding table
    COEUS_TRY(weight_alloc(m->out, wd, cfg.width, cfg.vocab));
    COEUS_TRY(src.rows(cfg.tied ? "embed" : "head", m->out, 0, 1, st));
    m->weight_bytes += m->out.bytes;
    m->embed = m->out.data;
    m->embed_bf16 = bf16;
    if (!cfg.tied) {
        Weight table;
        const int rc = weight_alloc(table, wd, cfg.width, cfg.vocab);
        m->embed = table.data;  // (freed with the model)
        COEUS_TRY(rc);
        COEUS_TRY(src.rows("embed", table, 0, 1, st));
        m->weight_bytes += table.bytes;
    }
    COEUS_HIP(hipDeviceSynchronize());
    *out = m.release();
    return COEUS_OK;
}

}  // namespace

int layered_load(const char *dir, const coeus_load_options &opt, Model **out) {
    std::string text;
    LayeredConfig cfg;
    COEUS_TRY(read_text_file(std::string(dir) + "/config.json", text));
    COEUS_TRY(layered_config_parse(text.data(), text.size(), cfg));
    SafeTensors file;
    COEUS_TRY(file.open(std::string(dir) + "/model.safetensors"));
    COEUS_TRY(check_tensors(file, layered_tensors(cfg)));
    return build(cfg, &file, 0, opt, out);
}

int layered_create_seeded(const char *json, uint64_t len, const coeus_load_options &opt, uint64_t seed, Model **out) {
    LayeredConfig cfg;
    COEUS_TRY(layered_config_parse(json, len, cfg));
    return build(cfg, nullptr, seed, opt, out);
}

// ---------------------------------------------------------------- prompt pass
// Positions in front of pos0 that an attention layer's rows can still see.
static uint64_t visible_history(const MixerSpec &m, uint64_t pos0) {
    return m.window && m.window - 1 < pos0 ? m.window - 1 : pos0;
}

int layered_workspace(const Model &m, Workspace &ws, uint64_t batch, uint64_t n, uint64_t pos0) {
    const LayeredStack &stack = *m.stack;
    const bool bf16 = m.cfg.weight_dtype == COEUS_W_BF16;
    const uint64_t rows = batch * n, W = stack.cfg.width;
    uint64_t in = 0, att = 0, ff = 0, mix = 0, lat = 0, q = 0, kv = 0, lp = 0, part = 0;
    auto up = [](uint64_t &v, uint64_t x) { if (x > v) v = x; };
    auto split = [&](const Weight &w, uint64_t r) { up(part, gemm_split_scratch_bytes(w, r)); };
    for (const LayeredLayer &l : stack.layers) {
        const MixerSpec &mx = l.spec.mixer;
        if (!l.in.data) continue;  // (another layer's tensors)
        up(in, rows * l.in.n * 4);
        up(att, rows * mx.inner() * 4);
        up(lp, rows * gemm_ld(mx.inner()) * 2);
        split(l.in, rows); split(l.o, rows);
        const uint64_t lrows = batch * (visible_history(mx, pos0) + n), es = bf16 ? 2 : 4;
        switch (mx.kind) {
            case MixerKind::GatedDelta: {
                const DeltaDims dm = l.delta_dims();
                const uint64_t qk = round_up(rows * mx.kv_heads * delta_padded_dim(dm.d), 4), g = round_up(rows * mx.heads, 4);
                up(mix, (2 * qk + round_up(rows * mx.inner(), 4) + 2 * g) * 4 + delta_prompt_scratch_bytes(dm, batch, n));
                break;
            }
            case MixerKind::LatentAttention:
                up(mix, rows * (bf16 ? gemm_ld(mx.q_rank) * 2 : mx.q_rank * 4));
                up(lat, lrows * (bf16 ? gemm_ld(mx.kv_rank) : mx.kv_rank) * es);
                up(q, rows * mx.heads * mx.dim * es);
                up(kv, lrows * mx.heads * (mx.dim + mx.vdim) * es);
                split(l.uq, rows); split(l.ukv, lrows);
                break;
            case MixerKind::MatrixMemory:
                up(mix, memory_prompt_scratch_bytes(l.memory_dims(), batch, n));
                break;
            case MixerKind::SharedKv:
                up(q, rows * mx.heads * mx.dim * es);
                up(kv, lrows * l.shared_dims().row_len() * es);
                break;
        }
        if (l.spec.ff) {
            up(ff, rows * l.spec.ff * 4);
            up(lp, rows * gemm_ld(l.spec.ff) * 2);
            split(l.up, rows); split(l.down, rows);
        }
    }
    COEUS_TRY(ws.h.ensure(rows * W * 4));
    COEUS_TRY(ws.x.ensure(rows * W * 4));
    COEUS_TRY(ws.qkv.ensure(in));
    COEUS_TRY(ws.att.ensure(att));
    COEUS_TRY(ws.ids.ensure(rows * 8));
    COEUS_TRY(ws.mix.ensure(mix));
    COEUS_TRY(ws.norm_part.ensure(norm_sequence_scratch_bytes()));
    if (lat) COEUS_TRY(ws.lat.ensure(lat));
    if (q) COEUS_TRY(ws.q_lp.ensure(q));
    if (kv) COEUS_TRY(ws.kv_lp.ensure(kv));
    if (stack.cfg.streams) COEUS_TRY(ws.streams.ensure(rows * stack.cfg.streams * W * 4));
    if (bf16) {
        COEUS_TRY(ws.a_lp.ensure(rows * gemm_ld(W) * 2));
        COEUS_TRY(ws.b_lp.ensure(lp));
    } else if (ff) {
        COEUS_TRY(ws.ff.ensure(ff));
    }
    if (part) COEUS_TRY(ws.gemm_part.ensure(part));
    ws.gs.partials = (float *)ws.gemm_part.p; ws.gs.partials_bytes = ws.gemm_part.bytes;
    ws.gs.a_lp = ws.a_lp.p; ws.gs.a_lp_bytes = ws.a_lp.bytes;
    ws.gs.w_lp = nullptr; ws.gs.w_lp_bytes = 0;
    return COEUS_OK;
}

namespace {

// A step of hyper-connections: the pending output of a sublayer (behind `from`; null: none) into the streams,
// and what `to` puts in front of the next one (null: the plain sum).
HyperStep hyper_step(const LayeredConfig &cfg, const Around *from, const float *y, const Around *to) {
    HyperStep h;
    h.streams = (uint32_t)cfg.streams;
    h.mult = cfg.residual_mult;
    h.eps = cfg.eps;
    if (from) { h.y = y; h.mix = from->mix; h.out = from->out; }
    if (to) { h.in = to->in; h.norm = to->norm; }
    return h;
}

// What the layers of one prompt pass share.  x() is what a sublayer reads as a matmul operand: 16-bit rows
// (bf16), or f32 rows.  With one stream that is the residual stream itself; with hyper-connections the streams
// have a buffer of their own and `pending` is the sublayer whose output (y) they have not taken in yet.
struct Pass {
    Model &m;
    Workspace &ws;
    uint64_t batch, n, pos0, rows;
    bool bf16;
    hipStream_t st;
    const Around *pending = nullptr;
    float *h() const { return (float *)ws.h.p; }
    float *y() const { return (float *)ws.x.p; }
    float *proj() const { return (float *)ws.qkv.p; }
    float *att() const { return (float *)ws.att.p; }
    float *streams() const { return (float *)ws.streams.p; }
    const void *x() const { return bf16 ? (const void *)ws.a_lp.p : (const void *)ws.h.p; }
    LpOut x_lp() const { return LpOut{ws.a_lp.p, gemm_ld(m.stack->cfg.width), true}; }
    int gemm(const Weight &w, const void *a, uint64_t r, const Epilogue &e) const { return launch_gemm(w, a, r, e, ws.gs, st, bf16); }
    int gemm_f32_out(const Weight &w, const void *a, uint64_t r, float *dst) const {
        Epilogue e;
        e.out_f32 = dst;
        return gemm(w, a, r, e);
    }
    int begin() const {
        const uint64_t W = m.stack->cfg.width;
        const bool hyper = m.stack->cfg.streams != 0;
        COEUS_TRY(launch_embed(m.embed, m.embed_bf16, nullptr, (const uint64_t *)ws.ids.p, rows, n, pos0, nullptr, W,
                               hyper ? streams() : h(), nullptr, st, nullptr, nullptr, m.embed_scale, m.streams()));
        return bf16 && !hyper ? launch_f32_to_16(h(), ws.a_lp.p, rows, W, gemm_ld(W), true, st) : COEUS_OK;
    }
    // makes x(), in front of a sublayer
    int enter(const Around &a) {
        const LayeredConfig &cfg = m.stack->cfg;
        if (!cfg.streams) return COEUS_OK;
        const LpOut lp = x_lp();
        const HyperStep step = hyper_step(cfg, pending, y(), &a);
        pending = nullptr;
        return launch_hyper(streams(), rows, cfg.width, step, bf16 ? nullptr : h(), bf16 ? &lp : nullptr, st);
    }
    // behind a sublayer, whose output is y()
    int leave(const Around &a) {
        const LayeredConfig &cfg = m.stack->cfg;
        if (cfg.streams) { pending = &a; return COEUS_OK; }
        const LpOut lp = x_lp();
        return launch_norm_residual(y(), rows, cfg.width, a.norm, a.ls, cfg.eps, h(), st, bf16 ? &lp : nullptr);
    }
    // the residual stream (the sum of the streams) in h()
    int settle() {
        const LayeredConfig &cfg = m.stack->cfg;
        if (!cfg.streams) return COEUS_OK;
        const HyperStep step = hyper_step(cfg, pending, y(), nullptr);
        pending = nullptr;
        return launch_hyper(streams(), rows, cfg.width, step, h(), nullptr, st);
    }
};

int prefill_delta(const Pass &p, const LayeredLayer &l, const DeltaState &state) {
    const MixerSpec &mx = l.spec.mixer;
    const DeltaDims dm = l.delta_dims();
    COEUS_TRY(p.gemm_f32_out(l.in, p.x(), p.rows, p.proj()));
    float *base = (float *)p.ws.mix.p;
    auto take = [&](uint64_t n) { float *r = base; base += round_up(n, 4); return r; };
    DeltaOperands op;
    op.q = take(p.rows * mx.kv_heads * delta_padded_dim(dm.d));
    op.k = take(p.rows * mx.kv_heads * delta_padded_dim(dm.d));
    op.v = take(p.rows * mx.inner());
    op.beta = take(p.rows * mx.heads);
    op.lg = take(p.rows * mx.heads);
    COEUS_TRY(launch_delta_prepare(p.proj(), dm, l.delta, state, p.batch, p.n, p.pos0, op, p.st));
    COEUS_TRY(launch_delta_ring(p.proj(), dm, state, p.batch, p.n, p.pos0, p.st));
    COEUS_TRY(launch_delta_prompt(dm, op, state, p.batch, p.n, p.att(), base, p.ws.mix.bytes - ((char *)base - (char *)p.ws.mix.p), p.st));
    const LpOut lp{p.ws.b_lp.p, gemm_ld(mx.inner()), true};
    COEUS_TRY(launch_delta_gate(p.att(), p.proj(), dm, l.delta, p.rows, p.bf16 ? nullptr : p.att(), p.bf16 ? &lp : nullptr, p.st));
    return p.gemm_f32_out(l.o, p.bf16 ? (const void *)p.ws.b_lp.p : (const void *)p.att(), p.rows, p.y());
}

int prefill_latent(const Pass &p, const LayeredLayer &l, const RowRing &cache) {
    const MixerSpec &mx = l.spec.mixer;
    const LatentDims dm = l.latent_dims();
    const uint64_t hist = visible_history(mx, p.pos0), lrows = hist + p.n;
    const uint64_t lat_ld = p.bf16 ? gemm_ld(mx.kv_rank) : mx.kv_rank;
    COEUS_TRY(p.gemm_f32_out(l.in, p.x(), p.rows, p.proj()));
    // latents: the visible history out of the ring, then the new rows behind it
    COEUS_TRY(launch_ring_gather(cache, dm.rank, p.batch, hist, p.pos0, p.ws.lat.p, lat_ld, lrows, p.st));
    const LpOut cq_lp{p.ws.mix.p, gemm_ld(mx.q_rank), true};
    COEUS_TRY(launch_latent_norm(p.proj(), dm, l.dq_norm, l.dkv_norm, p.m.stack->cfg.eps, p.batch, p.n,
                                 p.bf16 ? nullptr : (float *)p.ws.mix.p, p.bf16 ? &cq_lp : nullptr, p.ws.lat.p, lat_ld, lrows,
                                 hist, cache, nullptr, p.st));
    COEUS_TRY(launch_ring_append(p.ws.lat.p, lat_ld, lrows, hist, cache, dm.rank, p.batch, p.n, p.pos0, p.st));
    auto expand = [&](const Weight &w, const void *a, uint64_t r, void *dst) {
        Epilogue e;
        if (p.bf16) e.out_lp = LpOut{dst, w.n, true};
        else e.out_f32 = (float *)dst;
        return p.gemm(w, a, r, e);
    };
    COEUS_TRY(expand(l.uq, p.ws.mix.p, p.rows, p.ws.q_lp.p));
    COEUS_TRY(expand(l.ukv, p.ws.lat.p, p.batch * lrows, p.ws.kv_lp.p));
    const LpOut lp{p.ws.b_lp.p, gemm_ld(mx.inner()), true};
    COEUS_TRY(launch_window_attention(p.ws.q_lp.p, l.uq.n, p.ws.kv_lp.p, l.ukv.n, p.bf16, dm.window_shape(), p.batch, p.n, hist,
                                      p.bf16 ? nullptr : p.att(), p.bf16 ? &lp : nullptr, p.st));
    return p.gemm_f32_out(l.o, p.bf16 ? (const void *)p.ws.b_lp.p : (const void *)p.att(), p.rows, p.y());
}

int prefill_memory(const Pass &p, const LayeredLayer &l, const MemoryState &state) {
    COEUS_TRY(p.gemm_f32_out(l.in, p.x(), p.rows, p.proj()));
    const LpOut lp{p.ws.b_lp.p, gemm_ld(l.spec.mixer.inner()), true};
    COEUS_TRY(launch_memory_prompt(p.proj(), l.memory_dims(), l.memory, state, p.batch, p.n, p.bf16 ? nullptr : p.att(),
                                   p.bf16 ? &lp : nullptr, (float *)p.ws.mix.p, p.ws.mix.bytes, p.st));
    return p.gemm_f32_out(l.o, p.bf16 ? (const void *)p.ws.b_lp.p : (const void *)p.att(), p.rows, p.y());
}

int prefill_shared_kv(const Pass &p, const LayeredLayer &l, const RowRing &ring) {
    const MixerSpec &mx = l.spec.mixer;
    const SharedKvDims dm = l.shared_dims();
    const uint64_t hist = visible_history(mx, p.pos0), krows = hist + p.n, rl = dm.row_len();
    COEUS_TRY(p.gemm_f32_out(l.in, p.x(), p.rows, p.proj()));
    // rows of keys: the visible history out of the ring, then the new ones behind it
    COEUS_TRY(launch_ring_gather(ring, rl, p.batch, hist, p.pos0, p.ws.kv_lp.p, rl, krows, p.st));
    COEUS_TRY(launch_shared_kv_prepare(p.proj(), dm, l.wqk, p.m.stack->cfg.eps, p.batch, p.n, p.bf16, p.ws.q_lp.p, p.ws.kv_lp.p, krows, hist, p.st));
    COEUS_TRY(launch_ring_append(p.ws.kv_lp.p, rl, krows, hist, ring, rl, p.batch, p.n, p.pos0, p.st));
    const LpOut lp{p.ws.b_lp.p, gemm_ld(mx.inner()), true};
    COEUS_TRY(launch_window_attention(p.ws.q_lp.p, mx.heads * mx.dim, p.ws.kv_lp.p, rl, p.bf16, dm.window_shape(p.proj() + dm.gate_off()),
                                      p.batch, p.n, hist, p.bf16 ? nullptr : p.att(), p.bf16 ? &lp : nullptr, p.st));
    return p.gemm_f32_out(l.o, p.bf16 ? (const void *)p.ws.b_lp.p : (const void *)p.att(), p.rows, p.y());
}

// The gate between a feed-forward's matrices, as the first one's epilogue.
void gate_epilogue(const LayerSpec &l, Epilogue &e) {
    e.act = l.gate == GateKind::Clamped ? COEUS_EPI_CLAMP_GATE : COEUS_EPI_SILU_GATE;
    e.limit = l.limit;
}

int prefill_ff(const Pass &p, const LayeredLayer &l) {
    Epilogue e;
    gate_epilogue(l.spec, e);
    if (p.bf16) e.out_lp = LpOut{p.ws.b_lp.p, gemm_ld(l.spec.ff), true};
    else e.out_f32 = (float *)p.ws.ff.p;
    COEUS_TRY(p.gemm(l.up, p.x(), p.rows, e));
    return p.gemm_f32_out(l.down, p.bf16 ? (const void *)p.ws.b_lp.p : (const void *)p.ws.ff.p, p.rows, p.y());
}

}  // namespace

int layered_prefill(Model &m, Workspace &ws, LayeredState &state, uint64_t batch, uint64_t n, uint64_t pos0,
                    float *residuals, hipStream_t st) {
    const LayeredStack &stack = *m.stack;
    Pass p{m, ws, batch, n, pos0, batch * n, m.cfg.weight_dtype == COEUS_W_BF16, st};
    const uint64_t W = stack.cfg.width;
    COEUS_TRY(p.begin());
    for (size_t l = 0; l < stack.layers.size(); l++) {
        const LayeredLayer &ly = stack.weights(l);
        const LayeredState::Layer &sl = state.layers[l];
        COEUS_TRY(p.enter(ly.around_mixer));
        switch (ly.spec.mixer.kind) {
            case MixerKind::GatedDelta: COEUS_TRY(prefill_delta(p, ly, sl.delta)); break;
            case MixerKind::LatentAttention: COEUS_TRY(prefill_latent(p, ly, sl.ring)); break;
            case MixerKind::MatrixMemory: COEUS_TRY(prefill_memory(p, ly, sl.memory)); break;
            case MixerKind::SharedKv: COEUS_TRY(prefill_shared_kv(p, ly, sl.ring)); break;
        }
        COEUS_TRY(p.leave(ly.around_mixer));
        if (ly.spec.ff) {
            COEUS_TRY(p.enter(ly.around_ff));
            COEUS_TRY(prefill_ff(p, ly));
            COEUS_TRY(p.leave(ly.around_ff));
        }
        if (residuals) {
            COEUS_TRY(p.settle());
            COEUS_HIP(hipMemcpyAsync(residuals + l * p.rows * W, p.h(), p.rows * W * 4, hipMemcpyDeviceToHost, st));
        }
    }
    return p.settle();
}

// ---------------------------------------------------------------- sessions
int layered_session_init(Session &s) {
    Model &m = *s.m;
    const LayeredStack &stack = *m.stack;
    const uint64_t B = s.batch, W = stack.cfg.width;
    COEUS_TRY(s.state.create(stack, m.cfg.weight_dtype == COEUS_W_BF16, B, s.max_ctx, m.stream));
    uint64_t in = 0, att = 0, ff = 0, q = 0, sc = 0, cnt = 0;
    auto up = [](uint64_t &v, uint64_t x) { if (x > v) v = x; };
    for (size_t l = 0; l < stack.layers.size(); l++) {
        const LayeredLayer &ly = stack.weights(l);
        const MixerSpec &mx = ly.spec.mixer;
        up(in, ly.in.n);
        up(att, mx.inner());
        up(ff, ly.spec.ff);
        if (mx.kind == MixerKind::LatentAttention) {
            up(q, mx.q_rank + mx.heads * mx.dim);
            up(sc, latent_decode_scratch_bytes(ly.latent_dims(), s.state.layers[l].ring, B));
        } else if (mx.kind == MixerKind::SharedKv) {
            up(sc, shared_kv_decode_scratch_bytes(ly.shared_dims(), s.state.layers[l].ring, B));
            up(cnt, shared_kv_decode_counters(ly.shared_dims(), B));
        }
    }
    COEUS_TRY(s.dh.ensure(B * m.streams() * W * 4));
    COEUS_TRY(s.dh2.ensure(B * m.streams() * W * 4));
    if (cnt) {
        COEUS_TRY(s.dcount.ensure(cnt * 4));
        COEUS_HIP(hipMemsetAsync(s.dcount.p, 0, s.dcount.bytes, m.stream));
    }
    COEUS_TRY(s.dx.ensure(B * W * 4));
    COEUS_TRY(s.dqkv.ensure(B * in * 4));
    COEUS_TRY(s.datt.ensure(B * att * 4));
    if (ff) COEUS_TRY(s.dff.ensure(B * ff * 4));
    if (q) COEUS_TRY(s.dmix.ensure(B * q * 4));
    if (sc) COEUS_TRY(s.dscratch.ensure(sc));
    COEUS_TRY(s.dlogits.ensure(B * m.cfg.vocab_size * 4));
    COEUS_TRY(s.dids.ensure(B * 8));
    COEUS_TRY(s.dpos.ensure(64));
    COEUS_TRY(s.dhist.ensure(B * s.max_ctx * 8));
    s.bp = pad_batch(B);
    COEUS_HIP(hipStreamSynchronize(m.stream));
    return COEUS_OK;
}

// One decode step behind the embedding (s.dh holds the residual stream or streams): only enqueues kernels.
// What stands around a sublayer is folded into the matmul that reads the stream next, like the norms in front
// of the transformer's matmuls: `pending` is the sublayer whose output (y) the stream has not taken in yet.  The
// folded form reads the stream and writes the new one, so the two buffers change places.
int layered_decode(Session &s, hipStream_t st, int only, uint64_t *launches, uint64_t *bytes) {
    Model &m = *s.m;
    const LayeredStack &stack = *m.stack;
    const LayeredConfig &cfg = stack.cfg;
    const uint64_t B = s.batch, W = cfg.width;
    const bool matmuls = only != STEP_ATTENTION, mixers = only != STEP_MATMULS, rest = only == STEP_ALL;
    const uint32_t *pos = (const uint32_t *)s.dpos.p;
    float *h = (float *)s.dh.p, *h_other = (float *)s.dh2.p, *y = (float *)s.dx.p, *proj = (float *)s.dqkv.p,
          *att = (float *)s.datt.p, *ff = (float *)s.dff.p;
    const float eps = cfg.eps;
    const Around *pending = nullptr;
    const float *fold = stack.folds;  // the next sublayer's record
    uint64_t n_launch = 0, n_bytes = 0;
    auto count = [&](const Weight &w, bool gated) {
        n_launch++;
        n_bytes += gemv_algorithmic_bytes(w, B, gated, true);
    };
    auto gemv = [&](const Weight &w, const float *x, const Epilogue &e) -> int {
        if (!matmuls) return COEUS_OK;
        count(w, epi_gated(e.act));
        return launch_gemv(w, x, B, e, st);
    };
    auto gemv_to = [&](const Weight &w, const float *x, float *dst) -> int {
        Epilogue e;
        e.out_f32 = dst;
        return gemv(w, x, e);
    };
    // A launch of its own: the pending output into the stream; with hyper-connections also the normalised input
    // of what stands behind `to` (null: the final norm), which takes the pending output's place in y.
    auto settle = [&](const Around *to) -> int {
        if (cfg.streams) {
            HyperStep step = hyper_step(cfg, pending, y, to);
            if (!to) step.norm = m.fin_s;
            if (rest) COEUS_TRY(launch_hyper(h, B, W, step, y, nullptr, st));
        } else if (rest && pending) {
            COEUS_TRY(launch_norm_residual(y, B, W, pending->norm, pending->ls, eps, h, st));
        }
        pending = nullptr;
        return COEUS_OK;
    };
    // a matmul of what a sublayer reads (the same limit on the output rows as for norms in front of it: every
    // workgroup repeats the norm)
    auto stream_gemv = [&](const Weight &w, const Around &to, const Epilogue &e) -> int {
        const float *const this_fold = fold;
        if (fold) fold += kHyperFoldFloats;
        const bool fuse = s.fuse && (cfg.streams || w.n <= 16384) &&
                          (cfg.streams ? gemv_can_fuse_hyper(w, B, cfg.streams) : pending && gemv_can_fuse_post_norm(w, B));
        if (fuse) {
            NormFuse nf;
            nf.h = h; nf.eps = eps; nf.h_out = h_other;
            if (pending) nf.y = y;
            if (cfg.streams) {
                nf.kind = COEUS_NORM_LAYERNORM;
                nf.scale = to.norm; nf.fold = this_fold; nf.streams = (uint32_t)cfg.streams;
            } else {
                nf.kind = COEUS_NORM_RMSNORM;
                nf.scale = pending->norm; nf.ls = pending->ls;
            }
            if (pending) std::swap(h, h_other);
            pending = nullptr;
            if (!matmuls) return COEUS_OK;
            count(w, epi_gated(e.act));
            return launch_gemv(w, nullptr, B, e, st, &nf);
        }
        COEUS_TRY(settle(&to));
        return gemv(w, cfg.streams ? y : h, e);
    };
    for (size_t l = 0; l < stack.layers.size(); l++) {
        const LayeredLayer &ly = stack.weights(l);
        const LayeredState::Layer &sl = s.state.layers[l];
        const MixerSpec &mx = ly.spec.mixer;
        Epilogue ein;
        ein.out_f32 = proj;
        COEUS_TRY(stream_gemv(ly.in, ly.around_mixer, ein));
        auto mixer_bytes = [&](uint64_t nb) {
            if (only != STEP_ATTENTION) return;
            n_launch++;
            n_bytes += nb;
        };
        // positions that a step of attention reads
        const uint64_t nv = sl.ring.cap ? std::min<uint64_t>((uint64_t)s.host_pos[0] + 1, sl.ring.cap) : 0;
        switch (mx.kind) {
            case MixerKind::GatedDelta:
                if (!mixers) break;
                COEUS_TRY(launch_delta_step(proj, ly.delta_dims(), ly.delta, sl.delta, B, pos, att, st));
                // the state in and out, ring, projection, output
                mixer_bytes(B * 4 * (2 * mx.heads * mx.dim * mx.vdim + (mx.conv + 1) * mx.conv_channels() + ly.in.n + mx.inner()));
                break;
            case MixerKind::MatrixMemory:
                if (!mixers) break;
                COEUS_TRY(launch_memory_step(proj, ly.memory_dims(), ly.memory, sl.memory, B, att, st));
                // state and normaliser in and out, projection, output
                mixer_bytes(B * 4 * (2 * mx.heads * mx.dim * (mx.vdim + 1) + ly.in.n + mx.inner()));
                break;
            case MixerKind::SharedKv:
                if (!mixers) break;
                COEUS_TRY(launch_shared_kv_decode(proj, ly.shared_dims(), ly.wqk, eps, sl.ring, B, pos, att, (float *)s.dscratch.p,
                                                  s.dscratch.bytes, (uint32_t *)s.dcount.p, s.dcount.bytes / 4, st));
                // the visible rows, projection, output
                mixer_bytes(B * (nv * ly.shared_dims().row_len() * (sl.ring.bf16 ? 2 : 4) + (ly.in.n + mx.inner()) * 4));
                break;
            case MixerKind::LatentAttention: {
                const LatentDims dm = ly.latent_dims();
                float *cq = (float *)s.dmix.p, *q = cq + B * mx.q_rank;
                const bool fold = s.fuse && gemv_can_fuse_norm_dense(ly.uq, B);
                if (rest && !fold)
                    COEUS_TRY(launch_latent_norm(proj, dm, ly.dq_norm, ly.dkv_norm, eps, B, 1, cq, nullptr, nullptr, 0, 0, 0, sl.ring, pos, st));
                if (fold && matmuls) {  // the query latent's norm rides on its expansion
                    Epilogue e;
                    e.out_f32 = q;
                    NormFuse nf;
                    nf.h = proj; nf.ld = ly.in.n; nf.scale = ly.dq_norm; nf.eps = eps; nf.kind = COEUS_NORM_RMSNORM;
                    count(ly.uq, false);
                    COEUS_TRY(launch_gemv(ly.uq, nullptr, B, e, st, &nf));
                } else if (!fold) {
                    COEUS_TRY(gemv_to(ly.uq, cq, q));
                }
                if (!mixers) break;
                COEUS_TRY(launch_latent_decode(q, ly.ukv.data, dm, LatentNew{proj, ly.dkv_norm, eps}, sl.ring, B, pos, att,
                                               (float *)s.dscratch.p, s.dscratch.bytes, st));
                mixer_bytes(ly.ukv.bytes + B * (nv * mx.kv_rank * (sl.ring.bf16 ? 2 : 4) + (mx.heads * mx.dim + mx.inner()) * 4));
                break;
            }
        }
        COEUS_TRY(gemv_to(ly.o, att, y));
        pending = &ly.around_mixer;
        if (ly.spec.ff) {
            Epilogue eup;
            eup.out_f32 = ff;
            gate_epilogue(ly.spec, eup);
            COEUS_TRY(stream_gemv(ly.up, ly.around_ff, eup));
            COEUS_TRY(gemv_to(ly.down, ff, y));
            pending = &ly.around_ff;
        }
    }
    COEUS_TRY(settle(nullptr));
    if (rest && !cfg.streams)
        COEUS_TRY(launch_norm(COEUS_NORM_RMSNORM, COEUS_SCOPE_TOKEN, h, B, W, m.fin_s, nullptr, eps, y, nullptr, 0, st));
    COEUS_TRY(gemv(m.out, y, m.logits_epilogue((float *)s.dlogits.p)));
    if (launches) *launches = n_launch;
    if (bytes) *bytes = n_bytes;
    return COEUS_OK;
}

}  // namespace coeus
