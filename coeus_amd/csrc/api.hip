// extern "C" surface of libcoeus_mi355x.so (declared in include/coeus.h).  Nothing here throws
// across the boundary: every entry point catches and reports through coeus_last_error().
#include <cmath>
#include <new>

#include "model.hpp"

using namespace coeus;

struct coeus_weight { Weight w; };

extern "C" {

int coeus_device_info(char *name_out, uint64_t name_cap, uint64_t *hbm_bytes, uint32_t *compute_units) {
    COEUS_GUARD_BEGIN
    int n = 0;
    if (hipGetDeviceCount(&n) != hipSuccess || n == 0)
        return fail(COEUS_DEVICE_ERROR, "no HIP device visible");
    hipDeviceProp_t p;
    COEUS_HIP(hipGetDeviceProperties(&p, 0));
    if (name_out && name_cap) snprintf(name_out, name_cap, "%s (%s)", p.name, p.gcnArchName);
    if (hbm_bytes) *hbm_bytes = p.totalGlobalMem;
    if (compute_units) *compute_units = (uint32_t)p.multiProcessorCount;
    return COEUS_OK;
    COEUS_GUARD_END
}

// ---------------------------------------------------------------- device plumbing
int coeus_device_malloc(uint64_t bytes, void **out) {
    if (!out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    *out = nullptr;
    COEUS_HIP(hipMalloc(out, bytes ? bytes : 1));
    return COEUS_OK;
}
int coeus_device_free(void *ptr) {
    if (ptr) COEUS_HIP(hipFree(ptr));
    return COEUS_OK;
}
int coeus_memcpy_h2d(void *dst, const void *src, uint64_t bytes) {
    if (bytes) COEUS_HIP(hipMemcpy(dst, src, bytes, hipMemcpyHostToDevice));
    return COEUS_OK;
}
int coeus_memcpy_d2h(void *dst, const void *src, uint64_t bytes) {
    if (bytes) COEUS_HIP(hipMemcpy(dst, src, bytes, hipMemcpyDeviceToHost));
    return COEUS_OK;
}
int coeus_device_memset(void *dst, int value, uint64_t bytes) {
    if (bytes) COEUS_HIP(hipMemset(dst, value, bytes));
    return COEUS_OK;
}
namespace coeus {
__global__ __launch_bounds__(256) void device_copy_kernel(const uint4 *__restrict__ src, uint4 *__restrict__ dst, uint64_t n16) {
    for (uint64_t i = (uint64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n16; i += (uint64_t)gridDim.x * blockDim.x)
        dst[i] = src[i];
}
}  // namespace coeus
int coeus_device_copy(void *dst, const void *src, uint64_t bytes, void *stream) {
    if (!dst || !src) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (bytes % 16) return fail(COEUS_INVALID_INPUT, "copy size %llu is not a multiple of 16", (unsigned long long)bytes);
    if (bytes == 0) return COEUS_OK;
    const uint64_t n16 = bytes / 16;
    const unsigned grid = (unsigned)(n16 / 256 < 8192 ? (n16 + 255) / 256 : 8192);
    hipLaunchKernelGGL(coeus::device_copy_kernel, dim3(grid), dim3(256), 0, (hipStream_t)stream, (const uint4 *)src, (uint4 *)dst, n16);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}
int coeus_device_synchronize(void) {
    COEUS_HIP(hipDeviceSynchronize());
    return COEUS_OK;
}
int coeus_stream_create(void **out) {
    if (!out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    hipStream_t s = nullptr;
    COEUS_HIP(hipStreamCreateWithFlags(&s, hipStreamNonBlocking));
    *out = s;
    return COEUS_OK;
}
int coeus_stream_synchronize(void *stream) {
    COEUS_HIP(hipStreamSynchronize((hipStream_t)stream));
    return COEUS_OK;
}
int coeus_stream_destroy(void *stream) {
    if (stream) COEUS_HIP(hipStreamDestroy((hipStream_t)stream));
    return COEUS_OK;
}
int coeus_event_create(void **out) {
    if (!out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    hipEvent_t e = nullptr;
    COEUS_HIP(hipEventCreate(&e));
    *out = e;
    return COEUS_OK;
}
int coeus_event_record(void *event, void *stream) {
    COEUS_HIP(hipEventRecord((hipEvent_t)event, (hipStream_t)stream));
    return COEUS_OK;
}
int coeus_event_synchronize(void *event) {
    COEUS_HIP(hipEventSynchronize((hipEvent_t)event));
    return COEUS_OK;
}
int coeus_event_elapsed_ms(void *start, void *stop, float *ms_out) {
    if (!ms_out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    COEUS_HIP(hipEventElapsedTime(ms_out, (hipEvent_t)start, (hipEvent_t)stop));
    return COEUS_OK;
}
int coeus_event_destroy(void *event) {
    if (event) COEUS_HIP(hipEventDestroy((hipEvent_t)event));
    return COEUS_OK;
}

// ---------------------------------------------------------------- model
static int create_common(const coeus_config *cfg, const float *params, uint64_t n, uint64_t seed,
                         coeus_model **out) {
    COEUS_GUARD_BEGIN
    if (!cfg || !out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    *out = nullptr;
    Model *m = nullptr;
    COEUS_TRY(model_create(*cfg, params, n, seed, &m));
    *out = reinterpret_cast<coeus_model *>(m);
    return COEUS_OK;
    COEUS_GUARD_END
}

int coeus_model_create(const coeus_config *cfg, const float *params, uint64_t n_params, coeus_model **out) {
    if (!params) return fail(COEUS_INVALID_INPUT, "null parameter buffer");
    return create_common(cfg, params, n_params, 0, out);
}

int coeus_model_create_seeded(const coeus_config *cfg, uint64_t seed, coeus_model **out) {
    return create_common(cfg, nullptr, 0, seed, out);
}

int coeus_model_load(const char *dir, const coeus_load_options *opt, coeus_model **out) {
    COEUS_GUARD_BEGIN
    if (!dir || !opt || !out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    *out = nullptr;
    Model *m = nullptr;
    COEUS_TRY(layered_load(dir, *opt, &m));
    *out = reinterpret_cast<coeus_model *>(m);
    return COEUS_OK;
    COEUS_GUARD_END
}

int coeus_model_create_layered(const char *json, uint64_t len, const coeus_load_options *opt, uint64_t seed,
                               coeus_model **out) {
    COEUS_GUARD_BEGIN
    if (!json || !opt || !out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    *out = nullptr;
    Model *m = nullptr;
    COEUS_TRY(layered_create_seeded(json, len, *opt, seed, &m));
    *out = reinterpret_cast<coeus_model *>(m);
    return COEUS_OK;
    COEUS_GUARD_END
}

static Model *M(coeus_model *m) { return reinterpret_cast<Model *>(m); }
static const Model *M(const coeus_model *m) { return reinterpret_cast<const Model *>(m); }
static Session *S(coeus_session *s) { return reinterpret_cast<Session *>(s); }

int coeus_model_forward(coeus_model *m, const uint64_t *ids, uint64_t seq_len, float *logits_out) {
    COEUS_GUARD_BEGIN
    if (!m) return fail(COEUS_INVALID_INPUT, "null model");
    return model_forward(*M(m), ids, seq_len, logits_out, false);
    COEUS_GUARD_END
}

int coeus_model_forward_all(coeus_model *m, const uint64_t *ids, uint64_t seq_len, float *logits_out) {
    COEUS_GUARD_BEGIN
    if (!m) return fail(COEUS_INVALID_INPUT, "null model");
    return model_forward(*M(m), ids, seq_len, logits_out, true);
    COEUS_GUARD_END
}

uint64_t coeus_model_num_parameters(const coeus_model *m) { return m ? M(m)->n_params : 0; }
const coeus_config *coeus_model_config(const coeus_model *m) { return m ? &M(m)->cfg : nullptr; }
const char *coeus_model_name(const coeus_model *m) {  // MT:782-784
    return m && M(m)->stack ? M(m)->stack->cfg.architecture.c_str() : "TransformerModel";
}
uint64_t coeus_model_weight_bytes(const coeus_model *m) { return m ? M(m)->weight_bytes : 0; }
uint64_t coeus_model_resident_bytes(const coeus_model *m) {
    if (!m) return 0;
    Model *mm = const_cast<Model *>(M(m));
    std::lock_guard<std::mutex> lock(mm->mu);  // prompt passes charge the budget under this lock
    return mm->weight_bytes + (Model::kExpandBudget - mm->expand_budget);
}
void coeus_model_destroy(coeus_model *m) { delete M(m); }

// ---------------------------------------------------------------- sessions
int coeus_session_create(coeus_model *m, uint64_t batch, uint64_t max_ctx, coeus_session **out) {
    COEUS_GUARD_BEGIN
    if (!m || !out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    *out = nullptr;
    Session *s = nullptr;
    COEUS_TRY(session_create(*M(m), batch, max_ctx, &s));
    *out = reinterpret_cast<coeus_session *>(s);
    return COEUS_OK;
    COEUS_GUARD_END
}

int coeus_session_prefill(coeus_session *s, const uint64_t *ids, uint64_t n, float *logits_out) {
    COEUS_GUARD_BEGIN
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    return session_prefill(*S(s), ids, n, logits_out);
    COEUS_GUARD_END
}

int coeus_session_feed(coeus_session *s, const uint64_t *ids, uint64_t n, const uint64_t *want, uint64_t n_want,
                       float *logits_out, float *residuals_out) {
    COEUS_GUARD_BEGIN
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    return session_feed(*S(s), ids, n, want, n_want, logits_out, residuals_out);
    COEUS_GUARD_END
}

int coeus_session_decode(coeus_session *s, const uint64_t *ids, float *logits_out) {
    COEUS_GUARD_BEGIN
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    return session_decode(*S(s), ids, logits_out);
    COEUS_GUARD_END
}

int coeus_session_decode_greedy(coeus_session *s, const uint64_t *first_ids, uint64_t n_steps,
                                uint64_t *out_ids) {
    COEUS_GUARD_BEGIN
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    return session_decode_greedy(*S(s), first_ids, n_steps, out_ids);
    COEUS_GUARD_END
}

int coeus_session_generate(coeus_session *s, const uint64_t *first_ids, uint64_t n_steps,
                           const coeus_sampling *cfg, uint64_t *out_ids) {
    COEUS_GUARD_BEGIN
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    return session_decode_greedy(*S(s), first_ids, n_steps, out_ids, cfg);
    COEUS_GUARD_END
}

int coeus_op_sample(const float *logits_dev, uint64_t rows, uint64_t vocab, const coeus_sampling *cfg,
                    uint64_t position, uint64_t *out_ids_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!logits_dev || !cfg || !out_ids_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    return launch_sample(logits_dev, rows, vocab, *cfg, position, nullptr, out_ids_dev, nullptr, 0, nullptr,
                         (hipStream_t)stream);
    COEUS_GUARD_END
}

int coeus_session_time_decode_matmuls(coeus_session *s, uint64_t reps, float *ms_out,
                                      uint64_t *launches_out, uint64_t *bytes_out) {
    COEUS_GUARD_BEGIN
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    return session_time_decode_matmuls(*S(s), reps, ms_out, launches_out, bytes_out);
    COEUS_GUARD_END
}

int coeus_session_time_decode_attention(coeus_session *s, uint64_t reps, float *ms_out,
                                        uint64_t *launches_out, uint64_t *bytes_out) {
    COEUS_GUARD_BEGIN
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    return session_time_decode_attention(*S(s), reps, ms_out, launches_out, bytes_out);
    COEUS_GUARD_END
}

int coeus_session_set_graph(coeus_session *s, int enabled) {
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    if (enabled)
        if (const char *why = graph_replay_forbidden())
            return fail(COEUS_INVALID_INPUT, "graph replay refused: %s", why);
    std::lock_guard<std::mutex> lock(S(s)->m->mu);
    S(s)->use_graph = enabled != 0;
    return COEUS_OK;
}

int coeus_session_graph_enabled(const coeus_session *s) {
    if (!s) return 0;
    const Session *ss = reinterpret_cast<const Session *>(s);
    std::lock_guard<std::mutex> lock(ss->m->mu);
    return ss->use_graph ? 1 : 0;
}

uint64_t coeus_session_position(const coeus_session *s) {
    if (!s) return 0;
    const Session *ss = reinterpret_cast<const Session *>(s);
    std::lock_guard<std::mutex> lock(ss->m->mu);
    return ss->pos;
}

int coeus_session_reset(coeus_session *s) {
    if (!s) return fail(COEUS_INVALID_INPUT, "null session");
    COEUS_GUARD_BEGIN
    return session_reset(*S(s));
    COEUS_GUARD_END
}

void coeus_session_destroy(coeus_session *s) { delete S(s); }

// ---------------------------------------------------------------- operators
static int weight_create_common(uint32_t dtype, const float *host_w, uint64_t seed, uint64_t base,
                                uint64_t k, uint64_t n, coeus_weight **out) {
    COEUS_GUARD_BEGIN
    if (!out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    *out = nullptr;
    std::unique_ptr<coeus_weight> w(new coeus_weight());
    int rc = weight_alloc(w->w, dtype, k, n);
    if (rc != COEUS_OK) { weight_free(w->w); return rc; }
    float *dev = nullptr;
    WeightSource src;
    src.seed = seed;
    src.base = base;
    src.n_part = n;
    if (host_w) {
        hipError_t e = hipMalloc((void **)&dev, k * n * 4);
        if (e == hipSuccess) e = hipMemcpy(dev, host_w, k * n * 4, hipMemcpyHostToDevice);
        if (e != hipSuccess) {
            if (dev) (void)hipFree(dev);
            weight_free(w->w);
            return fail(COEUS_DEVICE_ERROR, "weight upload failed: %s", hipGetErrorString(e));
        }
        src.params = dev;
        src.base = 0;
    }
    rc = weight_pack(w->w, src, nullptr);
    hipError_t e = hipDeviceSynchronize();
    if (dev) (void)hipFree(dev);
    if (rc == COEUS_OK && e != hipSuccess) rc = fail(COEUS_DEVICE_ERROR, "weight packing failed: %s", hipGetErrorString(e));
    if (rc == COEUS_OK && dtype >= COEUS_W_Q8_0) {
        e = hipMalloc((void **)&w->w.xq_scratch, w->w.k_pad * 16 * 2);
        if (e != hipSuccess) rc = fail(COEUS_OUT_OF_MEMORY, "hipMalloc(xq scratch) failed");
    }
    if (rc != COEUS_OK) { weight_free(w->w); return rc; }
    *out = w.release();
    return COEUS_OK;
    COEUS_GUARD_END
}

int coeus_weight_create(uint32_t dtype, const float *host_w, uint64_t k_in, uint64_t n_out, coeus_weight **out) {
    if (!host_w) return fail(COEUS_INVALID_INPUT, "null weight matrix");
    return weight_create_common(dtype, host_w, 0, 0, k_in, n_out, out);
}

int coeus_weight_create_seeded(uint32_t dtype, uint64_t seed, uint64_t base_index, uint64_t k_in,
                               uint64_t n_out, coeus_weight **out) {
    return weight_create_common(dtype, nullptr, seed, base_index, k_in, n_out, out);
}

int coeus_weight_dequantize(const coeus_weight *w, float *host_out) {
    COEUS_GUARD_BEGIN
    if (!w || !host_out) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    float *dev = nullptr;
    const uint64_t bytes = w->w.k * w->w.n * 4;
    COEUS_HIP(hipMalloc((void **)&dev, bytes));
    int rc = weight_unpack_to_device(w->w, dev, nullptr);
    hipError_t e = rc == COEUS_OK ? hipMemcpy(host_out, dev, bytes, hipMemcpyDeviceToHost) : hipSuccess;
    (void)hipFree(dev);
    if (rc != COEUS_OK) return rc;
    COEUS_HIP(e);
    return COEUS_OK;
    COEUS_GUARD_END
}

uint64_t coeus_weight_bytes(const coeus_weight *w) { return w ? w->w.bytes : 0; }

void coeus_weight_destroy(coeus_weight *w) {
    if (!w) return;
    weight_free(w->w);
    delete w;
}

static Epilogue make_user_epilogue(const float *bias, const float *residual, uint32_t epilogue, float *y) {
    Epilogue e;
    e.bias = bias;
    e.residual = residual;
    e.act = epilogue;
    e.out_f32 = y;
    return e;
}

int coeus_op_gemv(const coeus_weight *w, const float *x_dev, uint64_t batch, const float *bias_dev,
                  const float *residual_dev, uint32_t epilogue, float *y_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!w || !x_dev || !y_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (epilogue > COEUS_EPI_SILU_GATE) return fail(COEUS_INVALID_INPUT, "unknown epilogue %u", epilogue);
    if (batch == 0 || batch > 16)
        return fail(COEUS_INVALID_INPUT, "decode matmul batch %llu out of range [1, 16]", (unsigned long long)batch);
    hipStream_t st = (hipStream_t)stream;
    const Epilogue e = make_user_epilogue(bias_dev, residual_dev, epilogue, y_dev);
    if (w->w.dtype >= COEUS_W_Q8_0) {
        // f32 activations are rounded to f16 in the kernel's interchange format first
        COEUS_TRY(launch_pack_xq(x_dev, batch, w->w.k, w->w.k_pad, w->w.xq_scratch, st));
        return launch_gemv(w->w, w->w.xq_scratch, batch, e, st);
    }
    return launch_gemv(w->w, x_dev, batch, e, st);
    COEUS_GUARD_END
}

int coeus_op_norm_gemv(const coeus_weight *w, const float *h_dev, uint64_t batch, uint32_t norm_kind,
                       const float *scale_dev, const float *bias_norm_dev, float eps, const float *bias_dev,
                       const float *residual_dev, uint32_t epilogue, float *y_dev, int *fused_out,
                       void *stream) {
    COEUS_GUARD_BEGIN
    if (!w || !h_dev || !y_dev || !scale_dev || (norm_kind == COEUS_NORM_LAYERNORM && !bias_norm_dev))
        return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (norm_kind > COEUS_NORM_RMSNORM) return fail(COEUS_INVALID_INPUT, "unknown norm kind %u", norm_kind);
    if (epilogue > COEUS_EPI_SILU_GATE) return fail(COEUS_INVALID_INPUT, "unknown epilogue %u", epilogue);
    if (batch == 0 || batch > 16)
        return fail(COEUS_INVALID_INPUT, "decode matmul batch %llu out of range [1, 16]", (unsigned long long)batch);
    hipStream_t st = (hipStream_t)stream;
    const Weight &W = w->w;
    const Epilogue e = make_user_epilogue(bias_dev, residual_dev, epilogue, y_dev);
    NormFuse nf;
    nf.h = h_dev; nf.scale = scale_dev; nf.bias = bias_norm_dev; nf.eps = eps; nf.kind = norm_kind;
    const bool quant = W.dtype >= COEUS_W_Q8_0;
    const bool fused = quant ? gemv_can_fuse_norm(W, batch) : gemv_can_fuse_norm_dense(W, batch);
    if (fused_out) *fused_out = fused ? 1 : 0;
    DeviceBuf stats, x;
    int rc = COEUS_OK;
    if (quant && fused) {
        rc = stats.ensure(batch * ceil_div(W.k, 16) * sizeof(float2));
        if (rc == COEUS_OK) rc = launch_row_stats16(h_dev, batch, W.k, (float2 *)stats.p, st);
        nf.stats = (const float2 *)stats.p;
        if (rc == COEUS_OK && norm_kind == COEUS_NORM_RMSNORM) {
            // as a decode step runs it: the rows arrive as h * scale, what the producer of h would have
            // stored next to the records
            rc = x.ensure(batch * W.k * 4);
            if (rc == COEUS_OK) rc = launch_prescale(h_dev, scale_dev, batch, W.k, (float *)x.p, st);
            nf.g = (const float *)x.p;
        }
        if (rc == COEUS_OK) rc = launch_gemv(W, nullptr, batch, e, st, &nf);
    } else if (fused) {
        rc = launch_gemv(W, nullptr, batch, e, st, &nf);
    } else if (quant) {
        // norm as its own launch, straight into the matmul's f16 interchange format (padding rows
        // and columns of the staging buffer are cleared first)
        const uint32_t bp = pad_batch(batch);
        hipError_t me = hipMemsetAsync(W.xq_scratch, 0, W.k_pad * 16 * 2, st);
        if (me != hipSuccess) rc = fail(COEUS_DEVICE_ERROR, "hipMemsetAsync failed: %s", hipGetErrorString(me));
        if (rc == COEUS_OK && (W.k & 7) == 0) {
            // as a decode step does it: row statistics merged from the per-16 records
            rc = stats.ensure(batch * ceil_div(W.k, 16) * sizeof(float2));
            if (rc == COEUS_OK) rc = launch_row_stats16(h_dev, batch, W.k, (float2 *)stats.p, st);
            nf.stats = (const float2 *)stats.p;
            if (rc == COEUS_OK) rc = launch_norm_from_stats(nf, batch, W.k, W.k_pad, W.xq_scratch, st);
        } else if (rc == COEUS_OK) {
            rc = launch_norm(norm_kind, COEUS_SCOPE_TOKEN, h_dev, batch, W.k, scale_dev, bias_norm_dev, eps, nullptr,
                             W.xq_scratch, bp, st);
        }
        if (rc == COEUS_OK) rc = launch_gemv(W, W.xq_scratch, batch, e, st);
    } else {
        rc = x.ensure(batch * W.k * 4);
        if (rc == COEUS_OK)
            rc = launch_norm(norm_kind, COEUS_SCOPE_TOKEN, h_dev, batch, W.k, scale_dev, bias_norm_dev, eps,
                             (float *)x.p, nullptr, 0, st);
        if (rc == COEUS_OK) rc = launch_gemv(W, x.p, batch, e, st);
    }
    if (stats.p || x.p) {  // the buffers die with this call: wait for the kernels that read them
        hipError_t se = hipStreamSynchronize(st);
        stats.release();
        x.release();
        if (rc == COEUS_OK && se != hipSuccess) rc = fail(COEUS_DEVICE_ERROR, "matmul failed: %s", hipGetErrorString(se));
    }
    return rc;
    COEUS_GUARD_END
}

// Staging and split buffers live as long as the call.
static int run_gemm(const Weight &w, const float *a_dev, uint64_t m, const Epilogue &e, hipStream_t st) {
    GemmScratch scr;
    DeviceBuf a_lp, w_lp, part;
    if (w.dtype != COEUS_W_F32) {
        COEUS_TRY(a_lp.ensure(m * gemm_ld(w.k) * 2));
        if (w.dtype >= COEUS_W_Q8_0) {
            int rc = w_lp.ensure(w.n * gemm_ld(w.k) * 2);
            if (rc != COEUS_OK) { a_lp.release(); return rc; }
        }
        scr.a_lp = a_lp.p; scr.a_lp_bytes = a_lp.bytes;
        scr.w_lp = w_lp.p; scr.w_lp_bytes = w_lp.bytes;
    }
    // (a launch of few tiles is split along k when it has room for the partial products; without
    // the room it runs unsplit)
    if (const uint64_t pb = gemm_split_scratch_bytes(w, m))
        if (part.ensure(pb) != COEUS_OK) part.release();
    scr.partials = (float *)part.p; scr.partials_bytes = part.bytes;
    int rc = launch_gemm(w, a_dev, m, e, scr, st);
    if (a_lp.p || w_lp.p || part.p) {
        // the staging buffers die with this call: wait for the kernels that read them
        hipError_t se = hipStreamSynchronize(st);
        a_lp.release();
        w_lp.release();
        part.release();
        if (rc == COEUS_OK && se != hipSuccess) rc = fail(COEUS_DEVICE_ERROR, "matmul failed: %s", hipGetErrorString(se));
    }
    return rc;
}

int coeus_op_gemm(const coeus_weight *w, const float *a_dev, uint64_t m, const float *bias_dev,
                  const float *residual_dev, uint32_t epilogue, float *c_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!w || !a_dev || !c_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (epilogue > COEUS_EPI_SILU_GATE) return fail(COEUS_INVALID_INPUT, "unknown epilogue %u", epilogue);
    return run_gemm(w->w, a_dev, m, make_user_epilogue(bias_dev, residual_dev, epilogue, c_dev), (hipStream_t)stream);
    COEUS_GUARD_END
}

static int limited_epilogue(uint32_t epilogue, float limit, float *y, Epilogue &e) {
    if (epilogue != COEUS_EPI_NONE && epilogue != COEUS_EPI_CLAMP_GATE && epilogue != COEUS_EPI_SOFTCAP)
        return fail(COEUS_INVALID_INPUT, "epilogue %u has no limit", epilogue);
    if (epilogue != COEUS_EPI_NONE && !(limit > 0.f)) return fail(COEUS_INVALID_INPUT, "an epilogue's limit must be positive");
    e = make_user_epilogue(nullptr, nullptr, epilogue, y);
    e.limit = limit;
    return COEUS_OK;
}

int coeus_op_matmul_limited(const coeus_weight *w, const float *x_dev, uint64_t rows, int prompt, uint32_t epilogue, float limit,
                            float *y_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!w || !x_dev || !y_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (w->w.dtype >= COEUS_W_Q8_0) return fail(COEUS_INVALID_INPUT, "an epilogue with a limit takes f32 or bf16 weights");
    Epilogue e;
    COEUS_TRY(limited_epilogue(epilogue, limit, y_dev, e));
    if (prompt) return run_gemm(w->w, x_dev, rows, e, (hipStream_t)stream);
    return launch_gemv(w->w, x_dev, rows, e, (hipStream_t)stream);
    COEUS_GUARD_END
}

int coeus_op_gemm_timed(const coeus_weight *w, const float *a_dev, uint64_t m, uint32_t epilogue,
                        float *c_dev, uint32_t reps, float *ms_out, void *stream) {
    COEUS_GUARD_BEGIN
    if (!w || !a_dev || !c_dev || !ms_out || reps == 0) return fail(COEUS_INVALID_INPUT, "bad timing arguments");
    if (epilogue > COEUS_EPI_SILU_GATE) return fail(COEUS_INVALID_INPUT, "unknown epilogue %u", epilogue);
    hipStream_t st = (hipStream_t)stream;
    const Epilogue e = make_user_epilogue(nullptr, nullptr, epilogue, c_dev);
    GemmScratch scr;
    DeviceBuf a_lp, w_lp, part;
    if (w->w.dtype != COEUS_W_F32) {
        COEUS_TRY(a_lp.ensure(m * gemm_ld(w->w.k) * 2));
        if (w->w.dtype >= COEUS_W_Q8_0) {
            int rc = w_lp.ensure(w->w.n * gemm_ld(w->w.k) * 2);
            if (rc != COEUS_OK) { a_lp.release(); return rc; }
        }
        scr.a_lp = a_lp.p; scr.a_lp_bytes = a_lp.bytes;
        scr.w_lp = w_lp.p; scr.w_lp_bytes = w_lp.bytes;
    }
    if (const uint64_t pb = gemm_split_scratch_bytes(w->w, m))
        if (part.ensure(pb) != COEUS_OK) part.release();
    scr.partials = (float *)part.p; scr.partials_bytes = part.bytes;
    int rc = launch_gemm(w->w, a_dev, m, e, scr, st);  // untimed first run
    hipEvent_t t0 = nullptr, t1 = nullptr;
    (void)hipEventCreate(&t0);
    (void)hipEventCreate(&t1);
    if (rc == COEUS_OK) {
        scr.repeat = reps; scr.ev_begin = t0; scr.ev_end = t1;
        rc = launch_gemm(w->w, a_dev, m, e, scr, st);
    }
    hipError_t se = hipStreamSynchronize(st);
    float ms = 0.f;
    if (rc == COEUS_OK && se == hipSuccess) se = hipEventElapsedTime(&ms, t0, t1);
    (void)hipEventDestroy(t0);
    (void)hipEventDestroy(t1);
    a_lp.release();
    w_lp.release();
    part.release();
    if (rc == COEUS_OK && se != hipSuccess) rc = fail(COEUS_DEVICE_ERROR, "matmul failed: %s", hipGetErrorString(se));
    *ms_out = ms;
    return rc;
    COEUS_GUARD_END
}

int coeus_op_norm(uint32_t kind, uint32_t scope, const float *x_dev, uint64_t rows, uint64_t hidden,
                  const float *scale_dev, const float *bias_dev, float eps, float *y_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!x_dev || !scale_dev || !y_dev || (kind == COEUS_NORM_LAYERNORM && !bias_dev))
        return fail(COEUS_INVALID_INPUT, "null pointer argument");
    // whole-slice statistics over a large slice: many workgroups, through a scratch buffer that
    // lives for this call (the model keeps one in its workspace instead)
    double *part = nullptr;
    if (scope == COEUS_SCOPE_SEQUENCE && rows * hidden >= 32768)
        COEUS_HIP(hipMalloc((void **)&part, norm_sequence_scratch_bytes()));
    const int rc = launch_norm(kind, scope, x_dev, rows, hidden, scale_dev, bias_dev, eps, y_dev, nullptr, 0,
                               (hipStream_t)stream, nullptr, part);
    if (part) {
        (void)hipStreamSynchronize((hipStream_t)stream);
        (void)hipFree(part);
    }
    return rc;
    COEUS_GUARD_END
}

int coeus_op_embed(const float *table_dev, const float *pe_dev, const uint64_t *ids_dev, uint64_t rows,
                   uint64_t pos0, uint64_t hidden, float *x_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!table_dev || !pe_dev || !ids_dev || !x_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    return launch_embed(table_dev, false, pe_dev, ids_dev, rows, rows, pos0, nullptr, hidden, x_dev,
                        nullptr, (hipStream_t)stream);
    COEUS_GUARD_END
}

int coeus_op_attention(const float *qkv_dev, uint64_t rows, uint64_t num_heads, uint64_t head_dim,
                       float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!qkv_dev || !out_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (rows == 0 || num_heads == 0) return fail(COEUS_INVALID_INPUT, "empty attention input");
    hipStream_t st = (hipStream_t)stream;
    DeviceBuf k, v;
    const uint64_t bytes = num_heads * rows * head_dim * 4;
    COEUS_TRY(k.ensure(bytes));
    int rc = v.ensure(bytes);
    if (rc == COEUS_OK)
        rc = launch_kv_append(qkv_dev, k.p, v.p, COEUS_KV_F32, 1, rows, num_heads, head_dim, rows, 0, nullptr, st);
    if (rc == COEUS_OK)
        rc = launch_attention(qkv_dev, k.p, v.p, COEUS_KV_F32, 1, rows, num_heads, head_dim, rows, 0,
                              nullptr, out_dev, nullptr, 0, nullptr, 0, nullptr, st);
    hipError_t se = hipStreamSynchronize(st);
    k.release();
    v.release();
    if (rc == COEUS_OK && se != hipSuccess) rc = fail(COEUS_DEVICE_ERROR, "attention failed: %s", hipGetErrorString(se));
    return rc;
    COEUS_GUARD_END
}

static int check_attention_decode_args(const float *qkv_dev, const void *k, const void *v, uint32_t kv_dtype,
                                       uint64_t batch, uint64_t heads, uint64_t hd, uint64_t max_ctx,
                                       uint64_t ctx, uint32_t *nsplit, uint32_t merge, const float *out_dev) {
    if (!qkv_dev || !k || !v || !out_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (batch == 0 || heads == 0 || batch > 65535 || heads > 65535)
        return fail(COEUS_INVALID_INPUT, "decode attention: batch %llu x heads %llu out of range",
                    (unsigned long long)batch, (unsigned long long)heads);
    if (hd != 64 && hd != 128)
        return fail(COEUS_INVALID_INPUT, "decode attention: head_dim %llu is not 64 or 128", (unsigned long long)hd);
    if (kv_dtype != COEUS_KV_F16 && kv_dtype != COEUS_KV_BF16)
        return fail(COEUS_INVALID_INPUT, "decode attention: the cache must be f16 or bf16");
    // (the kernel indexes positions with 32 bits, like validate_config's bound on max_seq_len)
    if (max_ctx >= (1ull << 31))
        return fail(COEUS_INVALID_INPUT, "decode attention: max_ctx %llu out of range [1, 2^31)",
                    (unsigned long long)max_ctx);
    if (ctx == 0 || ctx > max_ctx)
        return fail(COEUS_INVALID_INPUT, "Sequence length %llu out of range [1, %llu]", (unsigned long long)ctx,
                    (unsigned long long)max_ctx);
    if (merge > COEUS_MERGE_SEPARATE) return fail(COEUS_INVALID_INPUT, "unknown merge mode %u", merge);
    if (*nsplit == 0) *nsplit = attn_decode_splits(batch, heads, max_ctx);
    if (*nsplit > 32) return fail(COEUS_INVALID_INPUT, "decode attention: %u splits out of range [1, 32]", *nsplit);
    return COEUS_OK;
}

int coeus_op_attention_decode(const float *qkv_dev, const void *k_cache_dev, const void *v_cache_dev,
                              uint32_t kv_dtype, uint64_t batch, uint64_t num_heads, uint64_t head_dim,
                              uint64_t max_ctx, uint64_t ctx, uint32_t nsplit, uint32_t merge,
                              float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    COEUS_TRY(check_attention_decode_args(qkv_dev, k_cache_dev, v_cache_dev, kv_dtype, batch, num_heads, head_dim,
                                          max_ctx, ctx, &nsplit, merge, out_dev));
    hipStream_t st = (hipStream_t)stream;
    DeviceBuf part, count;
    COEUS_TRY(part.ensure(batch * num_heads * nsplit * (head_dim + 2) * 4));
    int rc = count.ensure(batch * num_heads * 4);
    hipError_t se = hipSuccess;
    if (rc == COEUS_OK) se = hipMemsetAsync(count.p, 0, count.bytes, st);
    if (rc == COEUS_OK && se == hipSuccess)
        rc = launch_attention(qkv_dev, k_cache_dev, v_cache_dev, kv_dtype, batch, 1, num_heads, head_dim, max_ctx,
                              ctx - 1, nullptr, out_dev, nullptr, 0, (float *)part.p, nsplit,
                              merge == COEUS_MERGE_IN_KERNEL ? (uint32_t *)count.p : nullptr, st);
    const hipError_t se2 = hipStreamSynchronize(st);
    part.release();
    count.release();
    if (rc == COEUS_OK && (se != hipSuccess || se2 != hipSuccess))
        rc = fail(COEUS_DEVICE_ERROR, "decode attention failed: %s", hipGetErrorString(se != hipSuccess ? se : se2));
    return rc;
    COEUS_GUARD_END
}

// ---------------------------------------------------------------- decode attention without allocation
// Device memory for coeus_op_attention_decode_static: the partial (max, sum, output) records of the
// context splits and the arrival counters of the in-kernel merge, in a file-scope array instead of
// a per-call allocation.  Every GPU the library runs on holds its own copy (2.04 MiB) until the
// process ends.  The array's name is only a host-side handle: device code is given the address
// that hipGetSymbolAddress returns for the current device.
constexpr uint64_t kStaticRecords = 4096;  // (sequence, head, split) triples of one call
constexpr uint64_t kStaticPairs = 1024;    // (sequence, head) pairs of one call
constexpr uint64_t kStaticRecordBytes = kStaticRecords * (128 + 2) * sizeof(float);
constexpr uint64_t kStaticScratchBytes = kStaticRecordBytes + kStaticPairs * sizeof(uint32_t);
static __device__ __align__(256) unsigned char scratch[kStaticScratchBytes];

constexpr int kMaxDevices = 64;
static std::mutex g_scratch_mu;
static void *g_scratch_ptr[kMaxDevices];  // per device: the address of its copy of `scratch`

static int static_scratch_for_current_device(unsigned char **out) {
    int dev = 0;
    COEUS_HIP(hipGetDevice(&dev));
    if (dev < 0 || dev >= kMaxDevices) return fail(COEUS_DEVICE_ERROR, "device index %d out of range", dev);
    std::lock_guard<std::mutex> lock(g_scratch_mu);
    if (!g_scratch_ptr[dev]) {
        void *p = nullptr;
        COEUS_HIP(hipGetSymbolAddress(&p, HIP_SYMBOL(scratch)));
        if (!p) return fail(COEUS_DEVICE_ERROR, "hipGetSymbolAddress returned a null address");
        g_scratch_ptr[dev] = p;
    }
    *out = (unsigned char *)g_scratch_ptr[dev];
    return COEUS_OK;
}

__global__ void clear_u32_kernel(uint32_t *p, uint32_t n) {
    const uint32_t i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) p[i] = 0u;
}

int coeus_op_attention_decode_static(const float *qkv_dev, const void *k_cache_dev, const void *v_cache_dev,
                                     uint32_t kv_dtype, uint64_t batch, uint64_t num_heads, uint64_t head_dim,
                                     uint64_t max_ctx, uint64_t ctx, uint32_t nsplit, uint32_t merge,
                                     float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    COEUS_TRY(check_attention_decode_args(qkv_dev, k_cache_dev, v_cache_dev, kv_dtype, batch, num_heads, head_dim,
                                          max_ctx, ctx, &nsplit, merge, out_dev));
    const uint64_t pairs = batch * num_heads, records = pairs * nsplit;
    if (pairs > kStaticPairs || records > kStaticRecords)
        return fail(COEUS_INVALID_INPUT,
                    "decode attention without allocation: batch %llu x heads %llu x splits %u needs %llu partial "
                    "records and %llu counters, the static buffer holds %llu and %llu",
                    (unsigned long long)batch, (unsigned long long)num_heads, nsplit, (unsigned long long)records,
                    (unsigned long long)pairs, (unsigned long long)kStaticRecords, (unsigned long long)kStaticPairs);
    unsigned char *base = nullptr;
    COEUS_TRY(static_scratch_for_current_device(&base));
    float *part = (float *)base;
    uint32_t *counters = (uint32_t *)(base + kStaticRecordBytes);
    hipStream_t st = (hipStream_t)stream;
    if (merge == COEUS_MERGE_IN_KERNEL) {
        // The merging split leaves its counter at zero, but a launch that was cut short would not:
        // clear them with a kernel (a memset node in a captured graph is not reliable here).
        hipLaunchKernelGGL(clear_u32_kernel, dim3((unsigned)ceil_div(pairs, 256)), dim3(256), 0, st, counters,
                           (uint32_t)pairs);
        COEUS_HIP(hipGetLastError());
    }
    return launch_attention(qkv_dev, k_cache_dev, v_cache_dev, kv_dtype, batch, 1, num_heads, head_dim, max_ctx,
                            ctx - 1, nullptr, out_dev, nullptr, 0, part, nsplit,
                            merge == COEUS_MERGE_IN_KERNEL ? counters : nullptr, st);
    COEUS_GUARD_END
}

// ---------------------------------------------------------------- mechanisms of layered models
// Waits for the call's kernels, frees its buffers, and reports whichever failed first.
static int finish_op(int rc, hipStream_t st, std::initializer_list<DeviceBuf *> bufs, const char *what) {
    const hipError_t e = hipStreamSynchronize(st);
    for (DeviceBuf *b : bufs) b->release();
    if (rc == COEUS_OK && e != hipSuccess) rc = fail(COEUS_DEVICE_ERROR, "%s failed: %s", what, hipGetErrorString(e));
    return rc;
}

int coeus_op_norm_residual(const float *y_dev, uint64_t rows, uint64_t hidden, const float *scale_dev, const float *ls_dev,
                           float eps, float *h_dev, void *stream) {
    COEUS_GUARD_BEGIN
    if (!y_dev || !scale_dev || !h_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    hipStream_t st = (hipStream_t)stream;
    return finish_op(launch_norm_residual(y_dev, rows, hidden, scale_dev, ls_dev, eps, h_dev, st), st, {}, "norm");
    COEUS_GUARD_END
}

static bool delta_args(const coeus_delta_shape *s, const coeus_delta_weights *w, DeltaDims &dm, DeltaParams &pr) {
    if (!s || !w || !w->conv_dev || !w->exp_a_dev || !w->dt_bias_dev || !w->norm_dev) return false;
    for (uint64_t v : {s->heads, s->kv_heads, s->dim, s->vdim, s->conv, s->in_ld})
        if (v > 0x7fffffffull) return false;
    dm = DeltaDims{(uint32_t)s->heads, (uint32_t)s->kv_heads, (uint32_t)s->dim, (uint32_t)s->vdim, (uint32_t)s->conv, (uint32_t)s->in_ld};
    pr = DeltaParams{w->conv_dev, w->exp_a_dev, w->dt_bias_dev, w->norm_dev, w->eps};
    return true;
}

int coeus_op_delta_prompt(const coeus_delta_shape *shape, const coeus_delta_weights *w, const float *proj_dev,
                          float *state_dev, float *ring_dev, uint64_t batch, uint64_t n, uint64_t pos0, int chunked,
                          float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    DeltaDims dm;
    DeltaParams pr;
    if (!delta_args(shape, w, dm, pr) || !proj_dev || !state_dev || !ring_dev || !out_dev)
        return fail(COEUS_INVALID_INPUT, "null pointer argument or size out of range");
    if (batch == 0 || n == 0 || batch > 65535 || n > 0x7fffffffull)
        return fail(COEUS_INVALID_INPUT, "delta rule: %llu x %llu rows out of range", (unsigned long long)batch, (unsigned long long)n);
    hipStream_t st = (hipStream_t)stream;
    const uint64_t rows = batch * n, qk = rows * dm.kv_heads * delta_padded_dim(dm.d) * 4;
    DeviceBuf q, k, v, beta, lg, scratch;
    const uint64_t sb = chunked ? delta_prompt_scratch_bytes(dm, batch, n) : 0;
    int rc = q.ensure(qk);
    if (rc == COEUS_OK) rc = k.ensure(qk);
    if (rc == COEUS_OK) rc = v.ensure(rows * dm.heads * dm.e * 4);
    if (rc == COEUS_OK) rc = beta.ensure(rows * dm.heads * 4);
    if (rc == COEUS_OK) rc = lg.ensure(rows * dm.heads * 4);
    if (rc == COEUS_OK && sb) rc = scratch.ensure(sb);
    const DeltaOperands op{(float *)q.p, (float *)k.p, (float *)v.p, (float *)beta.p, (float *)lg.p};
    const DeltaState state{state_dev, ring_dev};
    if (rc == COEUS_OK) rc = launch_delta_prepare(proj_dev, dm, pr, state, batch, n, pos0, op, st);
    if (rc == COEUS_OK) rc = launch_delta_ring(proj_dev, dm, state, batch, n, pos0, st);
    if (rc == COEUS_OK) rc = launch_delta_prompt(dm, op, state, batch, n, out_dev, (float *)scratch.p, scratch.bytes, st);
    if (rc == COEUS_OK) rc = launch_delta_gate(out_dev, proj_dev, dm, pr, rows, out_dev, nullptr, st);
    return finish_op(rc, st, {&q, &k, &v, &beta, &lg, &scratch}, "delta rule");
    COEUS_GUARD_END
}

static int upload_position(uint64_t pos, DeviceBuf &buf, hipStream_t st) {
    if (pos >= 0x7fffffffull) return fail(COEUS_INVALID_INPUT, "position %llu out of range", (unsigned long long)pos);
    const uint32_t p = (uint32_t)pos;
    COEUS_TRY(buf.ensure(4));
    COEUS_HIP(hipMemcpyAsync(buf.p, &p, 4, hipMemcpyHostToDevice, st));
    COEUS_HIP(hipStreamSynchronize(st));
    return COEUS_OK;
}

int coeus_op_delta_step(const coeus_delta_shape *shape, const coeus_delta_weights *w, const float *proj_dev,
                        float *state_dev, float *ring_dev, uint64_t batch, uint64_t pos, float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    DeltaDims dm;
    DeltaParams pr;
    if (!delta_args(shape, w, dm, pr) || !proj_dev || !state_dev || !ring_dev || !out_dev)
        return fail(COEUS_INVALID_INPUT, "null pointer argument or size out of range");
    hipStream_t st = (hipStream_t)stream;
    DeviceBuf p;
    int rc = upload_position(pos, p, st);
    if (rc == COEUS_OK)
        rc = launch_delta_step(proj_dev, dm, pr, DeltaState{state_dev, ring_dev}, batch, (const uint32_t *)p.p, out_dev, st);
    return finish_op(rc, st, {&p}, "delta rule");
    COEUS_GUARD_END
}

static int latent_args(const coeus_latent_shape *s, uint32_t kv_dtype, LatentDims &dm) {
    if (!s) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (kv_dtype != COEUS_KV_BF16 && kv_dtype != COEUS_KV_F32)
        return fail(COEUS_INVALID_INPUT, "latent attention: the tensors must be bf16 or f32");
    for (uint64_t v : {s->heads, s->dim, s->vdim, s->q_rank, s->kv_rank, s->window})
        if (v > 0x3fffffffull) return fail(COEUS_INVALID_INPUT, "latent attention: sizes out of range");
    dm = LatentDims{(uint32_t)s->heads, (uint32_t)s->dim, (uint32_t)s->vdim, (uint32_t)s->q_rank, (uint32_t)s->kv_rank,
                    (uint32_t)s->window, (uint32_t)round_up(s->q_rank + s->kv_rank, 4), s->scale};
    return COEUS_OK;
}

int coeus_op_window_attention(const coeus_latent_shape *shape, uint32_t kv_dtype, const void *q_dev, const void *kv_dev,
                              uint64_t batch, uint64_t n, uint64_t hist, float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    LatentDims dm;
    COEUS_TRY(latent_args(shape, kv_dtype, dm));
    if (!q_dev || !kv_dev || !out_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    hipStream_t st = (hipStream_t)stream;
    const uint64_t q_ld = (uint64_t)dm.heads * dm.d, kv_ld = q_ld + (uint64_t)dm.heads * dm.e;
    return finish_op(launch_window_attention(q_dev, q_ld, kv_dev, kv_ld, kv_dtype == COEUS_KV_BF16, dm.window_shape(), batch, n, hist, out_dev,
                                             nullptr, st), st, {}, "window attention");
    COEUS_GUARD_END
}

int coeus_op_latent_decode(const coeus_latent_shape *shape, uint32_t kv_dtype, const float *q_dev, const float *proj_dev,
                           const float *scale_dev, float eps, const void *ukv_dev, void *cache_dev, uint64_t cap,
                           uint64_t batch, uint64_t pos, float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    LatentDims dm;
    COEUS_TRY(latent_args(shape, kv_dtype, dm));
    if (!q_dev || !proj_dev || !scale_dev || !ukv_dev || !cache_dev || !out_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (cap == 0 || cap > 0x7fffffffull) return fail(COEUS_INVALID_INPUT, "latent attention: cache size out of range");
    hipStream_t st = (hipStream_t)stream;
    const RowRing cache{cache_dev, (uint32_t)cap, kv_dtype == COEUS_KV_BF16};
    DeviceBuf p, scratch;
    int rc = upload_position(pos, p, st);
    const uint64_t sb = latent_decode_scratch_bytes(dm, cache, batch);
    if (rc == COEUS_OK && sb) rc = scratch.ensure(sb);
    if (rc == COEUS_OK)
        rc = launch_latent_decode(q_dev, ukv_dev, dm, LatentNew{proj_dev, scale_dev, eps}, cache, batch, (const uint32_t *)p.p,
                                  out_dev, (float *)scratch.p, scratch.bytes, st);
    return finish_op(rc, st, {&p, &scratch}, "latent attention");
    COEUS_GUARD_END
}

// ---- hyper-connections, matrix memory, attention whose values are its keys
static int hyper_args(const coeus_hyper_step *h, HyperStep &out) {
    if (!h) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (h->streams == 0 || h->streams > kMaxHyperStreams) return fail(COEUS_INVALID_INPUT, "hyper-connections: 1 to %u streams", kMaxHyperStreams);
    if (h->y_dev && (!h->mix_dev || !h->out_dev)) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    out.streams = (uint32_t)h->streams;
    out.y = h->y_dev; out.mix = h->mix_dev; out.out = h->out_dev;
    out.in = h->in_dev; out.norm = h->norm_dev;
    out.mult = h->mult; out.eps = h->eps;
    return COEUS_OK;
}

int coeus_op_hyper(const coeus_hyper_step *step, float *x_dev, uint64_t rows, uint64_t hidden, float *u_dev, void *stream) {
    COEUS_GUARD_BEGIN
    HyperStep h;
    COEUS_TRY(hyper_args(step, h));
    if (!x_dev || !u_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    hipStream_t st = (hipStream_t)stream;
    return finish_op(launch_hyper(x_dev, rows, hidden, h, u_dev, nullptr, st), st, {}, "hyper-connections");
    COEUS_GUARD_END
}

int coeus_op_hyper_gemv(const coeus_weight *w, const coeus_hyper_step *step, const float *x_dev, uint64_t batch, float *x_new_dev,
                        uint32_t epilogue, float limit, float *y_dev, void *stream) {
    COEUS_GUARD_BEGIN
    HyperStep h;
    COEUS_TRY(hyper_args(step, h));
    if (!w || !x_dev || !y_dev || !h.in || !h.norm || (h.y && !x_new_dev)) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (w->w.dtype >= COEUS_W_Q8_0 || !gemv_can_fuse_hyper(w->w, batch, h.streams))
        return fail(COEUS_INVALID_INPUT, "folded hyper-connections: weight type, width, batch or streams out of range");
    Epilogue e;
    COEUS_TRY(limited_epilogue(epilogue, limit, y_dev, e));
    NormFuse nf;
    nf.h = x_dev; nf.h_out = x_new_dev; nf.kind = COEUS_NORM_LAYERNORM; nf.eps = h.eps;
    nf.scale = h.norm; nf.streams = h.streams; nf.y = h.y;
    hipStream_t st = (hipStream_t)stream;
    DeviceBuf fold;
    int rc = fold.ensure(kHyperFoldFloats * 4);
    nf.fold = (const float *)fold.p;
    if (rc == COEUS_OK)
        rc = launch_hyper_fold(h.y ? h.mix : nullptr, h.y ? h.out : nullptr, h.in, h.mult, h.streams, (float *)fold.p, st);
    if (rc == COEUS_OK) rc = launch_gemv(w->w, nullptr, batch, e, st, &nf);
    return finish_op(rc, st, {&fold}, "hyper-connections");
    COEUS_GUARD_END
}

static bool memory_args(const coeus_memory_shape *s, const coeus_memory_weights *w, MemoryDims &dm, MemoryParams &pr) {
    if (!s || !w || !w->in_bias_dev || !w->forget_bias_dev || !w->norm_dev) return false;
    for (uint64_t v : {s->heads, s->dim, s->vdim, s->in_ld})
        if (v > 0x7fffffffull) return false;
    dm = MemoryDims{(uint32_t)s->heads, (uint32_t)s->dim, (uint32_t)s->vdim, (uint32_t)s->in_ld, s->gate_cap};
    pr = MemoryParams{w->in_bias_dev, w->forget_bias_dev, w->norm_dev, w->eps};
    return true;
}

int coeus_op_memory_prompt(const coeus_memory_shape *shape, const coeus_memory_weights *w, const float *proj_dev, float *state_dev,
                           float *norm_state_dev, float *max_dev, uint64_t batch, uint64_t n, int chunked, float *out_dev,
                           void *stream) {
    COEUS_GUARD_BEGIN
    MemoryDims dm;
    MemoryParams pr;
    if (!memory_args(shape, w, dm, pr) || !proj_dev || !state_dev || !norm_state_dev || !max_dev || !out_dev)
        return fail(COEUS_INVALID_INPUT, "null pointer argument or size out of range");
    if (batch == 0 || n == 0 || batch > 65535 || n > 0x7fffffffull)
        return fail(COEUS_INVALID_INPUT, "matrix memory: %llu x %llu rows out of range", (unsigned long long)batch, (unsigned long long)n);
    hipStream_t st = (hipStream_t)stream;
    DeviceBuf scratch;
    int rc = scratch.ensure(memory_prompt_scratch_bytes(dm, batch, n, chunked != 0));
    if (rc == COEUS_OK)
        rc = launch_memory_prompt(proj_dev, dm, pr, MemoryState{state_dev, norm_state_dev, max_dev}, batch, n, out_dev, nullptr,
                                  (float *)scratch.p, scratch.bytes, st, chunked != 0);
    return finish_op(rc, st, {&scratch}, "matrix memory");
    COEUS_GUARD_END
}

int coeus_op_memory_step(const coeus_memory_shape *shape, const coeus_memory_weights *w, const float *proj_dev, float *state_dev,
                         float *norm_state_dev, float *max_dev, uint64_t batch, float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    MemoryDims dm;
    MemoryParams pr;
    if (!memory_args(shape, w, dm, pr) || !proj_dev || !state_dev || !norm_state_dev || !max_dev || !out_dev)
        return fail(COEUS_INVALID_INPUT, "null pointer argument or size out of range");
    hipStream_t st = (hipStream_t)stream;
    return finish_op(launch_memory_step(proj_dev, dm, pr, MemoryState{state_dev, norm_state_dev, max_dev}, batch, out_dev, st), st, {},
                     "matrix memory");
    COEUS_GUARD_END
}

static int shared_kv_args(const coeus_shared_kv_shape *s, uint32_t kv_dtype, SharedKvDims &dm) {
    if (!s) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (kv_dtype != COEUS_KV_BF16 && kv_dtype != COEUS_KV_F32)
        return fail(COEUS_INVALID_INPUT, "shared keys and values: the ring must be bf16 or f32");
    for (uint64_t v : {s->heads, s->kv_heads, s->dim, s->window, s->in_ld})
        if (v > 0x3fffffffull) return fail(COEUS_INVALID_INPUT, "shared keys and values: sizes out of range");
    if (!s->kv_heads || (s->heads + s->kv_heads) * s->dim > (1u << 24))
        return fail(COEUS_INVALID_INPUT, "shared keys and values: sizes out of range");
    dm = SharedKvDims{(uint32_t)s->heads, (uint32_t)s->kv_heads, (uint32_t)s->dim, (uint32_t)s->window, (uint32_t)s->in_ld, s->scale,
                      s->slope_range};
    return COEUS_OK;
}

uint64_t coeus_shared_kv_row_len(uint64_t kv_heads, uint64_t dim) {
    if (kv_heads > (1u << 20) || dim > (1u << 20) || kv_heads * dim > (1u << 24)) return 0;
    SharedKvDims dm{};
    dm.kv_heads = (uint32_t)kv_heads;
    dm.d = (uint32_t)dim;
    return dm.row_len();
}

int coeus_op_shared_kv_prompt(const coeus_shared_kv_shape *shape, uint32_t kv_dtype, const float *proj_dev, const float *wqk_dev,
                              float eps, void *ring_dev, uint64_t cap, uint64_t batch, uint64_t n, uint64_t pos0, float *out_dev,
                              void *stream) {
    COEUS_GUARD_BEGIN
    SharedKvDims dm;
    COEUS_TRY(shared_kv_args(shape, kv_dtype, dm));
    if (!proj_dev || !wqk_dev || !ring_dev || !out_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    const uint64_t hist = dm.window && dm.window - 1 < pos0 ? dm.window - 1 : pos0, krows = hist + n, rl = dm.row_len();
    // (a ring shorter than the window holds the whole context)
    if (cap == 0 || cap > 0x7fffffffull || batch == 0 || batch > 65535 || n == 0 || n > 0x3fffffffull || pos0 > 0x3fffffffull ||
        (dm.window && cap > dm.window) || ((!dm.window || cap < dm.window) && pos0 + n > cap))
        return fail(COEUS_INVALID_INPUT, "shared keys and values: rows or ring out of range");
    hipStream_t st = (hipStream_t)stream;
    const bool bf16 = kv_dtype == COEUS_KV_BF16;
    const uint64_t es = bf16 ? 2 : 4;
    const RowRing ring{ring_dev, (uint32_t)cap, bf16};
    DeviceBuf q, kv;
    int rc = q.ensure(batch * n * dm.heads * dm.d * es);
    if (rc == COEUS_OK) rc = kv.ensure(batch * krows * rl * es);
    if (rc == COEUS_OK) rc = launch_ring_gather(ring, (uint32_t)rl, batch, hist, pos0, kv.p, rl, krows, st);
    if (rc == COEUS_OK) rc = launch_shared_kv_prepare(proj_dev, dm, wqk_dev, eps, batch, n, bf16, q.p, kv.p, krows, hist, st);
    if (rc == COEUS_OK) rc = launch_ring_append(kv.p, rl, krows, hist, ring, (uint32_t)rl, batch, n, pos0, st);
    if (rc == COEUS_OK)
        rc = launch_window_attention(q.p, (uint64_t)dm.heads * dm.d, kv.p, rl, bf16, dm.window_shape(proj_dev + dm.gate_off()), batch, n,
                                     hist, out_dev, nullptr, st);
    return finish_op(rc, st, {&q, &kv}, "shared keys and values");
    COEUS_GUARD_END
}

int coeus_op_shared_kv_decode(const coeus_shared_kv_shape *shape, uint32_t kv_dtype, const float *proj_dev, const float *wqk_dev,
                              float eps, void *ring_dev, uint64_t cap, uint64_t batch, uint64_t pos, float *out_dev, void *stream) {
    COEUS_GUARD_BEGIN
    SharedKvDims dm;
    COEUS_TRY(shared_kv_args(shape, kv_dtype, dm));
    if (!proj_dev || !wqk_dev || !ring_dev || !out_dev) return fail(COEUS_INVALID_INPUT, "null pointer argument");
    if (cap == 0 || cap > 0x7fffffffull || batch == 0 || batch > 65535 || (dm.window && cap > dm.window) ||
        ((!dm.window || cap < dm.window) && pos >= cap))
        return fail(COEUS_INVALID_INPUT, "shared keys and values: batch, position or ring out of range");
    if (dm.heads == 0 || dm.heads % dm.kv_heads || dm.d == 0 || dm.d > 256)
        return fail(COEUS_INVALID_INPUT, "shared keys and values: sizes out of range");
    hipStream_t st = (hipStream_t)stream;
    const RowRing ring{ring_dev, (uint32_t)cap, kv_dtype == COEUS_KV_BF16};
    const uint64_t counters = shared_kv_decode_counters(dm, batch);
    DeviceBuf p, scratch, cnt;
    int rc = upload_position(pos, p, st);
    if (rc == COEUS_OK) rc = scratch.ensure(shared_kv_decode_scratch_bytes(dm, ring, batch));
    if (rc == COEUS_OK) rc = cnt.ensure(counters * 4);
    if (rc == COEUS_OK) {
        hipLaunchKernelGGL(clear_u32_kernel, dim3((unsigned)ceil_div(counters, 256)), dim3(256), 0, st, (uint32_t *)cnt.p,
                           (uint32_t)counters);
        rc = launch_shared_kv_decode(proj_dev, dm, wqk_dev, eps, ring, batch, (const uint32_t *)p.p, out_dev, (float *)scratch.p,
                                     scratch.bytes, (uint32_t *)cnt.p, counters, st);
    }
    return finish_op(rc, st, {&p, &scratch, &cnt}, "shared keys and values");
    COEUS_GUARD_END
}

}  // extern "C"
