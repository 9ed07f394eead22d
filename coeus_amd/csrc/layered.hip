// Layered decoder models on the device: construction from a folder (config.json + model.safetensors) or
// from a seed, the state a session carries, and the layers of a prompt pass and of a decode step.
//
// Every design here puts its norms behind the sublayers: a sublayer reads the f32 residual stream
// itself, and norm_residual adds its normalised, scaled output to it.
#include "model.hpp"

#include <cmath>

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

LayeredStack::~LayeredStack() {
    for (LayeredLayer &l : layers)
        for (Weight *w : {&l.in, &l.o, &l.up, &l.down, &l.uq, &l.ukv}) weight_free(*w);
    if (small) (void)hipFree(small);
}

// ---------------------------------------------------------------- state
// Offsets are counted first, then assigned: the recurrent part of every layer, then the rings of cached
// latents.  Those start as zeros and are not cleared again: a position that is not written yet has no weight,
// but its slot may be read, so it has to hold finite values.
int LayeredState::create(const LayeredStack &stack, bool bf16, uint64_t batch_, uint64_t max_ctx, hipStream_t st) {
    batch = batch_;
    layers.assign(stack.layers.size(), Layer{});
    uint64_t off = 0;
    auto take = [&](uint64_t bytes) { const uint64_t o = off; off += round_up(bytes, 256); return o; };
    std::vector<uint64_t> a(layers.size(), 0), r(layers.size(), 0);
    for (size_t l = 0; l < layers.size(); l++) {
        const MixerSpec &m = stack.layers[l].spec.mixer;
        if (m.kind != MixerKind::GatedDelta) continue;
        a[l] = take(batch * m.heads * m.dim * m.vdim * 4);
        r[l] = take(batch * m.conv * m.conv_channels() * 4);
    }
    recurrent_bytes = off;
    for (size_t l = 0; l < layers.size(); l++) {
        const MixerSpec &m = stack.layers[l].spec.mixer;
        if (m.kind != MixerKind::LatentAttention) continue;
        const uint64_t cap = m.window && m.window < max_ctx ? m.window : max_ctx;
        layers[l].latent.cap = (uint32_t)cap;
        layers[l].latent.bf16 = bf16;
        a[l] = take(batch * cap * m.kv_rank * (bf16 ? 2 : 4));
    }
    COEUS_TRY(mem.ensure(off ? off : 256));
    COEUS_HIP(hipMemsetAsync(mem.p, 0, mem.bytes, st));
    for (size_t l = 0; l < layers.size(); l++) {
        char *p = (char *)mem.p;
        if (stack.layers[l].spec.mixer.kind == MixerKind::GatedDelta) layers[l].delta = DeltaState{(float *)(p + a[l]), (float *)(p + r[l])};
        else layers[l].latent.c = p + a[l];
    }
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
    c.norm = COEUS_NORM_RMSNORM;
    c.norm_scope = COEUS_SCOPE_TOKEN;
    c.weight_dtype = wd;
    c.kv_dtype = bf16 ? COEUS_KV_BF16 : COEUS_KV_F32;
    c.max_batch = max_batch;
    m->n_params = total;
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
        const MixerSpec &mx = ly.spec.mixer;
        auto name = [&](const char *s) { return layer_tensor(l, s); };
        // rows behind the last projection pad the row length to a multiple of 4 (16-byte stores); zero weights
        const uint64_t in_rows = round_up(mx.in_rows(), 4);
        COEUS_TRY(weight_alloc(ly.in, wd, cfg.width, in_rows));
        COEUS_HIP(hipMemset(ly.in.data, 0, ly.in.bytes));
        COEUS_TRY(weight_alloc(ly.o, wd, mx.inner(), cfg.width));
        COEUS_TRY(src.rows(name("mix.o"), ly.o, 0, 1, st));
        if (mx.kind == MixerKind::GatedDelta) {
            uint64_t r = 0;
            for (const auto &part : {std::make_pair("mix.q", mx.kv_heads * mx.dim), std::make_pair("mix.k", mx.kv_heads * mx.dim),
                                     std::make_pair("mix.v", mx.inner()), std::make_pair("mix.g", mx.inner()),
                                     std::make_pair("mix.b", mx.heads), std::make_pair("mix.a", mx.heads)}) {
                COEUS_TRY(src.rows(name(part.first), ly.in, r, 1, st));
                r += part.second;
            }
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
        } else {
            COEUS_TRY(src.rows(name("mix.dq"), ly.in, 0, 1, st));
            COEUS_TRY(src.rows(name("mix.dkv"), ly.in, mx.q_rank, 1, st));
            COEUS_TRY(weight_alloc(ly.uq, wd, mx.q_rank, mx.heads * mx.dim));
            COEUS_TRY(src.rows(name("mix.uq"), ly.uq, 0, 1, st));
            COEUS_TRY(weight_alloc(ly.ukv, wd, mx.kv_rank, mx.heads * (mx.dim + mx.vdim)));
            COEUS_TRY(src.rows(name("mix.uk"), ly.ukv, 0, 1, st));
            COEUS_TRY(src.rows(name("mix.uv"), ly.ukv, mx.heads * mx.dim, 1, st));
            COEUS_TRY(put_tensor(&ly.dq_norm, name("mix.dq.norm")));
            COEUS_TRY(put_tensor(&ly.dkv_norm, name("mix.dkv.norm")));
        }
        COEUS_TRY(put_tensor(&ly.norm1, name("norm1")));
        COEUS_TRY(put_tensor(&ly.ls1, name("ls1")));
        if (ly.spec.ff) {
            COEUS_TRY(weight_alloc(ly.up, wd, cfg.width, 2 * ly.spec.ff));  // rows gate_0, up_0, gate_1, ..
            COEUS_TRY(src.rows(name("mlp.gate"), ly.up, 0, 2, st));
            COEUS_TRY(src.rows(name("mlp.up"), ly.up, 1, 2, st));
            COEUS_TRY(weight_alloc(ly.down, wd, ly.spec.ff, cfg.width));
            COEUS_TRY(src.rows(name("mlp.down"), ly.down, 0, 1, st));
            COEUS_TRY(put_tensor(&ly.norm2, name("norm2")));
            COEUS_TRY(put_tensor(&ly.ls2, name("ls2")));
        }
        for (const Weight *w : {&ly.in, &ly.o, &ly.up, &ly.down, &ly.uq, &ly.ukv}) m->weight_bytes += w->bytes;
    }
    COEUS_TRY(put_tensor(&m->fin_s, "final.norm"));
    COEUS_HIP(hipMalloc((void **)&stack.small, small.size() * 4));
    COEUS_HIP(hipMemcpy(stack.small, small.data(), small.size() * 4, hipMemcpyHostToDevice));
    for (auto &f : fix) *f.first = stack.small + f.second;
    m->weight_bytes += small.size() * 4;

    // ---- embedding table = output projection
    COEUS_TRY(weight_alloc(m->out, wd, cfg.width, cfg.vocab));
    m->embed = m->out.data;
    m->embed_bf16 = bf16;
    COEUS_TRY(src.rows("embed", m->out, 0, 1, st));
    m->weight_bytes += m->out.bytes;
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
        up(in, rows * l.in.n * 4);
        up(att, rows * mx.inner() * 4);
        up(lp, rows * gemm_ld(mx.inner()) * 2);
        split(l.in, rows); split(l.o, rows);
        if (mx.kind == MixerKind::GatedDelta) {
            const DeltaDims dm = l.delta_dims();
            const uint64_t qk = round_up(rows * mx.kv_heads * delta_padded_dim(dm.d), 4), g = round_up(rows * mx.heads, 4);
            up(mix, (2 * qk + round_up(rows * mx.inner(), 4) + 2 * g) * 4 + delta_prompt_scratch_bytes(dm, batch, n));
        } else {
            const uint64_t lrows = batch * (visible_history(mx, pos0) + n), es = bf16 ? 2 : 4;
            up(mix, rows * (bf16 ? gemm_ld(mx.q_rank) * 2 : mx.q_rank * 4));
            up(lat, lrows * (bf16 ? gemm_ld(mx.kv_rank) : mx.kv_rank) * es);
            up(q, rows * mx.heads * mx.dim * es);
            up(kv, lrows * mx.heads * (mx.dim + mx.vdim) * es);
            split(l.uq, rows); split(l.ukv, lrows);
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
    if (lat) {
        COEUS_TRY(ws.lat.ensure(lat));
        COEUS_TRY(ws.q_lp.ensure(q));
        COEUS_TRY(ws.kv_lp.ensure(kv));
    }
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

// What the layers of one prompt pass share.  `x` is the residual stream as a matmul operand: 16-bit
// rows next to it (bf16), or the f32 rows themselves.
struct Pass {
    Model &m;
    Workspace &ws;
    uint64_t batch, n, pos0, rows;
    bool bf16;
    hipStream_t st;
    float *h() const { return (float *)ws.h.p; }
    float *y() const { return (float *)ws.x.p; }
    float *proj() const { return (float *)ws.qkv.p; }
    float *att() const { return (float *)ws.att.p; }
    const void *x() const { return bf16 ? (const void *)ws.a_lp.p : (const void *)ws.h.p; }
    LpOut x_lp() const { return LpOut{ws.a_lp.p, gemm_ld(m.stack->cfg.width), true}; }
    int gemm(const Weight &w, const void *a, uint64_t r, const Epilogue &e) const { return launch_gemm(w, a, r, e, ws.gs, st, bf16); }
    int gemm_f32_out(const Weight &w, const void *a, uint64_t r, float *dst) const {
        Epilogue e;
        e.out_f32 = dst;
        return gemm(w, a, r, e);
    }
    // residual += norm(y) * ls, and the next operand
    int add(const float *norm, const float *ls) const {
        const LpOut lp = x_lp();
        return launch_norm_residual(y(), rows, m.stack->cfg.width, norm, ls, m.stack->cfg.eps, h(), st, bf16 ? &lp : nullptr);
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

int prefill_latent(const Pass &p, const LayeredLayer &l, const LatentCache &cache) {
    const MixerSpec &mx = l.spec.mixer;
    const LatentDims dm = l.latent_dims();
    const uint64_t hist = visible_history(mx, p.pos0), lrows = hist + p.n;
    const uint64_t lat_ld = p.bf16 ? gemm_ld(mx.kv_rank) : mx.kv_rank;
    COEUS_TRY(p.gemm_f32_out(l.in, p.x(), p.rows, p.proj()));
    // latents: the visible history out of the ring, then the new rows behind it
    COEUS_TRY(launch_latent_gather(cache, dm.rank, p.batch, hist, p.pos0, p.ws.lat.p, lat_ld, lrows, p.st));
    const LpOut cq_lp{p.ws.mix.p, gemm_ld(mx.q_rank), true};
    COEUS_TRY(launch_latent_norm(p.proj(), dm, l.dq_norm, l.dkv_norm, p.m.stack->cfg.eps, p.batch, p.n,
                                 p.bf16 ? nullptr : (float *)p.ws.mix.p, p.bf16 ? &cq_lp : nullptr, p.ws.lat.p, lat_ld, lrows,
                                 hist, cache, nullptr, p.st));
    COEUS_TRY(launch_latent_append(p.ws.lat.p, lat_ld, lrows, hist, cache, dm.rank, p.batch, p.n, p.pos0, p.st));
    auto expand = [&](const Weight &w, const void *a, uint64_t r, void *dst) {
        Epilogue e;
        if (p.bf16) e.out_lp = LpOut{dst, w.n, true};
        else e.out_f32 = (float *)dst;
        return p.gemm(w, a, r, e);
    };
    COEUS_TRY(expand(l.uq, p.ws.mix.p, p.rows, p.ws.q_lp.p));
    COEUS_TRY(expand(l.ukv, p.ws.lat.p, p.batch * lrows, p.ws.kv_lp.p));
    const LpOut lp{p.ws.b_lp.p, gemm_ld(mx.inner()), true};
    COEUS_TRY(launch_window_attention(p.ws.q_lp.p, l.uq.n, p.ws.kv_lp.p, l.ukv.n, p.bf16, dm, p.batch, p.n, hist,
                                      p.bf16 ? nullptr : p.att(), p.bf16 ? &lp : nullptr, p.st));
    return p.gemm_f32_out(l.o, p.bf16 ? (const void *)p.ws.b_lp.p : (const void *)p.att(), p.rows, p.y());
}

int prefill_ff(const Pass &p, const LayeredLayer &l) {
    Epilogue e;
    e.act = COEUS_EPI_SILU_GATE;
    if (p.bf16) e.out_lp = LpOut{p.ws.b_lp.p, gemm_ld(l.spec.ff), true};
    else e.out_f32 = (float *)p.ws.ff.p;
    COEUS_TRY(p.gemm(l.up, p.x(), p.rows, e));
    return p.gemm_f32_out(l.down, p.bf16 ? (const void *)p.ws.b_lp.p : (const void *)p.ws.ff.p, p.rows, p.y());
}

}  // namespace

int layered_prefill(Model &m, Workspace &ws, LayeredState &state, uint64_t batch, uint64_t n, uint64_t pos0,
                    float *residuals, hipStream_t st) {
    const LayeredStack &stack = *m.stack;
    const Pass p{m, ws, batch, n, pos0, batch * n, m.cfg.weight_dtype == COEUS_W_BF16, st};
    const uint64_t W = stack.cfg.width;
    COEUS_TRY(launch_embed(m.embed, m.embed_bf16, nullptr, (const uint64_t *)ws.ids.p, p.rows, n, pos0, nullptr, W, p.h(),
                           nullptr, st));
    if (p.bf16) COEUS_TRY(launch_f32_to_16(p.h(), ws.a_lp.p, p.rows, W, gemm_ld(W), true, st));
    for (size_t l = 0; l < stack.layers.size(); l++) {
        const LayeredLayer &ly = stack.layers[l];
        if (ly.spec.mixer.kind == MixerKind::GatedDelta) COEUS_TRY(prefill_delta(p, ly, state.layers[l].delta));
        else COEUS_TRY(prefill_latent(p, ly, state.layers[l].latent));
        COEUS_TRY(p.add(ly.norm1, ly.ls1));
        if (ly.spec.ff) {
            COEUS_TRY(prefill_ff(p, ly));
            COEUS_TRY(p.add(ly.norm2, ly.ls2));
        }
        if (residuals)
            COEUS_HIP(hipMemcpyAsync(residuals + l * p.rows * W, p.h(), p.rows * W * 4, hipMemcpyDeviceToHost, st));
    }
    return COEUS_OK;
}

// ---------------------------------------------------------------- sessions
int layered_session_init(Session &s) {
    Model &m = *s.m;
    const LayeredStack &stack = *m.stack;
    const uint64_t B = s.batch, W = stack.cfg.width;
    COEUS_TRY(s.state.create(stack, m.cfg.weight_dtype == COEUS_W_BF16, B, s.max_ctx, m.stream));
    uint64_t in = 0, att = 0, ff = 0, q = 0, sc = 0;
    auto up = [](uint64_t &v, uint64_t x) { if (x > v) v = x; };
    for (size_t l = 0; l < stack.layers.size(); l++) {
        const LayeredLayer &ly = stack.layers[l];
        const MixerSpec &mx = ly.spec.mixer;
        up(in, ly.in.n);
        up(att, mx.inner());
        up(ff, ly.spec.ff);
        if (mx.kind == MixerKind::LatentAttention) {
            up(q, mx.q_rank + mx.heads * mx.dim);
            up(sc, latent_decode_scratch_bytes(ly.latent_dims(), s.state.layers[l].latent, B));
        }
    }
    COEUS_TRY(s.dh.ensure(B * W * 4));
    COEUS_TRY(s.dh2.ensure(B * W * 4));
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

// One decode step behind the embedding (s.dh holds the residual stream): only enqueues kernels.
// The norm behind a sublayer is folded into the matmul that reads the stream next, like the norms in front
// of the transformer's matmuls: `pending` is the sublayer output that the stream has not taken in yet.  The
// folded form reads the stream and writes the new one, so the two buffers change places.
int layered_decode(Session &s, hipStream_t st, int only, uint64_t *launches, uint64_t *bytes) {
    Model &m = *s.m;
    const LayeredStack &stack = *m.stack;
    const uint64_t B = s.batch, W = stack.cfg.width;
    const bool matmuls = only != STEP_ATTENTION, mixers = only != STEP_MATMULS, rest = only == STEP_ALL;
    const uint32_t *pos = (const uint32_t *)s.dpos.p;
    float *h = (float *)s.dh.p, *h_other = (float *)s.dh2.p, *y = (float *)s.dx.p, *proj = (float *)s.dqkv.p,
          *att = (float *)s.datt.p, *ff = (float *)s.dff.p;
    const float eps = stack.cfg.eps;
    struct { const float *norm = nullptr, *ls = nullptr; } pending;
    uint64_t n_launch = 0, n_bytes = 0;
    auto count = [&](const Weight &w, bool gated) {
        n_launch++;
        n_bytes += gemv_algorithmic_bytes(w, B, gated, true);
    };
    auto gemv = [&](const Weight &w, const float *x, float *dst) -> int {
        if (!matmuls) return COEUS_OK;
        Epilogue e;
        e.out_f32 = dst;
        count(w, false);
        return launch_gemv(w, x, B, e, st);
    };
    auto settle = [&]() -> int {  // the pending sublayer output into the stream, as a launch of its own
        if (rest && pending.norm) COEUS_TRY(launch_norm_residual(y, B, W, pending.norm, pending.ls, eps, h, st));
        pending.norm = nullptr;
        return COEUS_OK;
    };
    // a matmul of the residual stream (the same limit on the output rows as for norms in front of it: every
    // workgroup of 16 rows repeats the norm)
    auto stream_gemv = [&](const Weight &w, float *dst, uint32_t act = COEUS_EPI_NONE) -> int {
        Epilogue e;
        e.out_f32 = dst;
        e.act = act;
        if (s.fuse && pending.norm && w.n <= 16384 && gemv_can_fuse_post_norm(w, B)) {
            if (!matmuls) return COEUS_OK;
            NormFuse nf;
            nf.h = h; nf.scale = pending.norm; nf.ls = pending.ls; nf.y = y; nf.h_out = h_other;
            nf.eps = eps; nf.kind = COEUS_NORM_RMSNORM;
            pending.norm = nullptr;
            std::swap(h, h_other);
            count(w, act == COEUS_EPI_SILU_GATE);
            return launch_gemv(w, nullptr, B, e, st, &nf);
        }
        COEUS_TRY(settle());
        if (!matmuls) return COEUS_OK;
        count(w, act == COEUS_EPI_SILU_GATE);
        return launch_gemv(w, h, B, e, st);
    };
    for (size_t l = 0; l < stack.layers.size(); l++) {
        const LayeredLayer &ly = stack.layers[l];
        const LayeredState::Layer &sl = s.state.layers[l];
        const MixerSpec &mx = ly.spec.mixer;
        COEUS_TRY(stream_gemv(ly.in, proj));
        if (mx.kind == MixerKind::GatedDelta) {
            if (mixers) {
                COEUS_TRY(launch_delta_step(proj, ly.delta_dims(), ly.delta, sl.delta, B, pos, att, st));
                if (only == STEP_ATTENTION) {
                    // the state in and out, ring, projection, output
                    n_launch++;
                    n_bytes += B * 4 * (2 * mx.heads * mx.dim * mx.vdim + (mx.conv + 1) * mx.conv_channels() + ly.in.n + mx.inner());
                }
            }
        } else {
            const LatentDims dm = ly.latent_dims();
            float *cq = (float *)s.dmix.p, *q = cq + B * mx.q_rank;
            const bool fold = s.fuse && gemv_can_fuse_norm_dense(ly.uq, B);
            if (rest && !fold)
                COEUS_TRY(launch_latent_norm(proj, dm, ly.dq_norm, ly.dkv_norm, eps, B, 1, cq, nullptr, nullptr, 0, 0, 0, sl.latent, pos, st));
            if (fold && matmuls) {  // the query latent's norm rides on its expansion
                Epilogue e;
                e.out_f32 = q;
                NormFuse nf;
                nf.h = proj; nf.ld = ly.in.n; nf.scale = ly.dq_norm; nf.eps = eps; nf.kind = COEUS_NORM_RMSNORM;
                count(ly.uq, false);
                COEUS_TRY(launch_gemv(ly.uq, nullptr, B, e, st, &nf));
            } else if (!fold) {
                COEUS_TRY(gemv(ly.uq, cq, q));
            }
            if (mixers) {
                COEUS_TRY(launch_latent_decode(q, ly.ukv.data, dm, LatentNew{proj, ly.dkv_norm, eps}, sl.latent, B, pos, att,
                                               (float *)s.dscratch.p, s.dscratch.bytes, st));
                if (only == STEP_ATTENTION) {
                    const uint64_t nv = std::min<uint64_t>((uint64_t)s.host_pos[0] + 1, sl.latent.cap);
                    n_launch++;
                    n_bytes += ly.ukv.bytes + B * (nv * mx.kv_rank * (sl.latent.bf16 ? 2 : 4) + (mx.heads * mx.dim + mx.inner()) * 4);
                }
            }
        }
        COEUS_TRY(gemv(ly.o, att, y));
        pending.norm = ly.norm1;
        pending.ls = ly.ls1;
        if (ly.spec.ff) {
            COEUS_TRY(stream_gemv(ly.up, ff, COEUS_EPI_SILU_GATE));
            COEUS_TRY(gemv(ly.down, ff, y));
            pending.norm = ly.norm2;
            pending.ls = ly.ls2;
        }
    }
    COEUS_TRY(settle());
    if (rest)
        COEUS_TRY(launch_norm(COEUS_NORM_RMSNORM, COEUS_SCOPE_TOKEN, h, B, W, m.fin_s, nullptr, eps, y, nullptr, 0, st));
    COEUS_TRY(gemv(m.out, y, (float *)s.dlogits.p));
    if (launches) *launches = n_launch;
    if (bytes) *bytes = n_bytes;
    return COEUS_OK;
}

}  // namespace coeus
