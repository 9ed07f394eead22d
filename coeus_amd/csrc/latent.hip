// Attention through low-rank latents with an optional sliding window.
//
//   latent_norm_kernel        RMS norms of the query latent and of the key/value latent
//   latent_gather / append    cached latents in front of a prompt's portion / its own into the ring
//   window_attn_kernel        prompt: one wave per (row, head) on expanded keys and values
//   latent_decode_kernel      decode: the query is taken into latent space (W_uk^T q), scored against the
//                             cached latents, and the weighted latent is expanded by W_uv
#include "device_utils.hpp"
#include "mixers.hpp"

namespace coeus {

template <bool BF16>
__device__ __forceinline__ float lat_load(const void *p, uint64_t i) {
    return BF16 ? bf16_bits_to_f32(((const uint16_t *)p)[i]) : ((const float *)p)[i];
}
template <bool BF16>
__device__ __forceinline__ void lat_store(void *p, uint64_t i, float v) {
    if (BF16) ((uint16_t *)p)[i] = f32_to_bf16_bits(v);
    else ((float *)p)[i] = v;
}

static int check_dims(const LatentDims &dm, const LatentCache &cache) {
    if (dm.heads == 0 || dm.heads > 65535 || dm.d == 0 || dm.d > 256 || dm.e == 0 || dm.e > 256 || dm.q_rank == 0 ||
        dm.rank == 0 || dm.rank > 2048 || dm.in_ld < dm.q_rank + dm.rank)
        return fail(COEUS_INVALID_INPUT, "latent attention: sizes out of range");
    if (cache.cap == 0 || (dm.window && cache.cap > dm.window))
        return fail(COEUS_INVALID_INPUT, "latent attention: cache of %u positions for a window of %u", cache.cap, dm.window);
    return COEUS_OK;
}

// blockIdx.y 0: the query latent, 1: the key/value latent.
template <bool BF16>
__global__ __launch_bounds__(256) void latent_norm_kernel(const float *__restrict__ proj, LatentDims dm,
                                                          const float *__restrict__ q_scale,
                                                          const float *__restrict__ c_scale, float eps, uint64_t n,
                                                          float *cq, uint16_t *cq_lp, uint64_t cq_ld, bool lp_bf16,
                                                          void *lat, uint64_t lat_ld, uint64_t lat_rows,
                                                          uint64_t lat_off, uint32_t cap, const uint32_t *pos_dev) {
    __shared__ float sh[4];
    const uint64_t row = blockIdx.x;
    const bool is_q = blockIdx.y == 0;
    const uint32_t len = is_q ? dm.q_rank : dm.rank, tid = threadIdx.x;
    const float *x = proj + row * dm.in_ld + (is_q ? 0 : dm.q_rank);
    float s2 = 0.f;
    for (uint32_t i = tid; i < len; i += 256) s2 = fmaf(x[i], x[i], s2);
    s2 = wave_sum(s2);
    if ((tid & 63) == 0) sh[tid >> 6] = s2;
    __syncthreads();
    const float rs = 1.0f / sqrtf(((sh[0] + sh[1]) + (sh[2] + sh[3])) / (float)len + eps);
    if (is_q) {
        for (uint32_t i = tid; i < len; i += 256) {
            const float v = x[i] * rs * q_scale[i];
            if (cq) cq[row * len + i] = v;
            if (cq_lp) cq_lp[row * cq_ld + i] = f32_to_lp_bits(v, lp_bf16);
        }
    } else {
        const uint64_t dst = pos_dev ? (row * cap + *pos_dev % cap) * dm.rank
                                     : ((row / n) * lat_rows + lat_off + row % n) * lat_ld;
        for (uint32_t i = tid; i < len; i += 256) lat_store<BF16>(lat, dst + i, x[i] * rs * c_scale[i]);
    }
}

int launch_latent_norm(const float *proj, const LatentDims &dm, const float *q_scale, const float *c_scale, float eps,
                       uint64_t batch, uint64_t n, float *cq, const LpOut *cq_lp, void *lat, uint64_t lat_ld,
                       uint64_t lat_rows, uint64_t lat_off, const LatentCache &cache, const uint32_t *pos_dev,
                       hipStream_t st) {
    COEUS_TRY(check_dims(dm, cache));
    if (batch == 0 || n == 0 || batch * n > 0x7fffffffull || (pos_dev && n != 1))
        return fail(COEUS_INVALID_INPUT, "latent attention: rows out of range");
    const dim3 grid((unsigned)(batch * n), 2);
    uint16_t *lp = cq_lp ? (uint16_t *)cq_lp->p : nullptr;
    const uint64_t ld = cq_lp ? cq_lp->ld : 0;
    const bool lp_bf = cq_lp && cq_lp->bf16;
    void *dst = pos_dev ? cache.c : lat;
    if (cache.bf16)
        hipLaunchKernelGGL(latent_norm_kernel<true>, grid, dim3(256), 0, st, proj, dm, q_scale, c_scale, eps, n, cq, lp, ld,
                           lp_bf, dst, lat_ld, lat_rows, lat_off, cache.cap, pos_dev);
    else
        hipLaunchKernelGGL(latent_norm_kernel<false>, grid, dim3(256), 0, st, proj, dm, q_scale, c_scale, eps, n, cq, lp, ld,
                           lp_bf, dst, lat_ld, lat_rows, lat_off, cache.cap, pos_dev);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// Rows of `rank` elements between the ring and a contiguous buffer: blockIdx.x counts `cnt` positions
// from pos_first, whose buffer row is row_first.
template <typename T, bool TO_RING>
__global__ __launch_bounds__(64) void latent_copy_kernel(T *ring, uint32_t cap, uint32_t rank, T *buf, uint64_t ld,
                                                         uint64_t rows_per_seq, uint64_t pos_first, uint64_t row_first) {
    const uint64_t i = blockIdx.x, b = blockIdx.y;
    T *r = ring + (b * cap + (pos_first + i) % cap) * rank, *l = buf + (b * rows_per_seq + row_first + i) * ld;
    for (uint32_t t = threadIdx.x; t < rank; t += 64) {
        if (TO_RING) r[t] = l[t];
        else l[t] = r[t];
    }
}

template <bool TO_RING>
static int latent_copy(const LatentCache &cache, uint32_t rank, uint64_t batch, uint64_t cnt, uint64_t pos_first, void *buf,
                       uint64_t ld, uint64_t rows_per_seq, uint64_t row_first, hipStream_t st) {
    if (cnt == 0) return COEUS_OK;
    if (cnt > cache.cap || batch == 0 || batch > 65535) return fail(COEUS_INVALID_INPUT, "latent attention: rows out of range");
    const dim3 grid((unsigned)cnt, (unsigned)batch);
    if (cache.bf16)
        hipLaunchKernelGGL((latent_copy_kernel<uint16_t, TO_RING>), grid, dim3(64), 0, st, (uint16_t *)cache.c, cache.cap, rank,
                           (uint16_t *)buf, ld, rows_per_seq, pos_first, row_first);
    else
        hipLaunchKernelGGL((latent_copy_kernel<float, TO_RING>), grid, dim3(64), 0, st, (float *)cache.c, cache.cap, rank,
                           (float *)buf, ld, rows_per_seq, pos_first, row_first);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

int launch_latent_gather(const LatentCache &cache, uint32_t rank, uint64_t batch, uint64_t hist, uint64_t pos0,
                         void *lat, uint64_t lat_ld, uint64_t lat_rows, hipStream_t st) {
    if (hist > pos0) return fail(COEUS_INVALID_INPUT, "latent attention: rows out of range");
    return latent_copy<false>(cache, rank, batch, hist, pos0 - hist, lat, lat_ld, lat_rows, 0, st);
}

int launch_latent_append(const void *lat, uint64_t lat_ld, uint64_t lat_rows, uint64_t hist, const LatentCache &cache,
                         uint32_t rank, uint64_t batch, uint64_t n, uint64_t pos0, hipStream_t st) {
    const uint64_t cnt = n < cache.cap ? n : cache.cap;
    return latent_copy<true>(cache, rank, batch, cnt, pos0 + n - cnt, (void *)lat, lat_ld, lat_rows, hist + n - cnt, st);
}

// ---------------------------------------------------------------- prompt attention, any size and type
// Row i of a sequence is key hist + i and sees keys lo .. hist + i, lo = max(0, hist + i - window + 1).
template <bool BF16>
__global__ __launch_bounds__(256) void window_attn_kernel(const void *__restrict__ q, uint64_t q_ld,
                                                          const void *__restrict__ kv, uint64_t kv_ld, LatentDims dm,
                                                          uint32_t n, uint32_t hist, float *__restrict__ out,
                                                          uint16_t *__restrict__ out_lp, uint64_t lp_ld, bool lp_bf16) {
    extern __shared__ float lds[];  // per wave: q[d] + p[64]
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const uint32_t i = blockIdx.x * 4 + wave, h = blockIdx.y;
    const uint64_t b = blockIdx.z;
    if (i >= n) return;
    float *qs = lds + wave * (dm.d + 64), *ps = qs + dm.d;
    const uint64_t row = b * n + i, k0 = b * (hist + n);
    for (uint32_t t = lane; t < dm.d; t += 64) qs[t] = lat_load<BF16>(q, row * q_ld + h * dm.d + t);
    const uint32_t end = hist + i + 1, lo = dm.window && end > dm.window ? end - dm.window : 0;
    const uint32_t voff = dm.heads * dm.d + h * dm.e;
    float m = -INFINITY, l = 0.f, acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (uint32_t j0 = lo; j0 < end; j0 += 64) {
        const uint32_t j = j0 + lane;
        float s = -INFINITY;
        if (j < end) {
            float dot = 0.f;
            const uint64_t kr = (k0 + j) * kv_ld + h * dm.d;
            for (uint32_t t = 0; t < dm.d; t++) dot = fmaf(qs[t], lat_load<BF16>(kv, kr + t), dot);
            s = dot * dm.scale;
        }
        const float m_new = fmaxf(m, wave_max(s));
        const float p = j < end ? expf(s - m_new) : 0.f, corr = expf(m - m_new);
        l = l * corr + wave_sum(p);
        m = m_new;
        ps[lane] = p;
#pragma unroll
        for (int t = 0; t < 4; t++) acc[t] *= corr;
        const uint32_t cnt = min(64u, end - j0);
        for (uint32_t jj = 0; jj < cnt; jj++) {
            const float pj = ps[jj];
            const uint64_t vr = (k0 + j0 + jj) * kv_ld + voff;
#pragma unroll
            for (int t = 0; t < 4; t++)
                if (lane + 64 * t < dm.e) acc[t] = fmaf(pj, lat_load<BF16>(kv, vr + lane + 64 * t), acc[t]);
        }
    }
    const float inv = 1.0f / l;
#pragma unroll
    for (int t = 0; t < 4; t++) {
        const uint32_t c = lane + 64 * t;
        if (c >= dm.e) continue;
        if (out) out[row * dm.heads * dm.e + h * dm.e + c] = acc[t] * inv;
        if (out_lp) out_lp[row * lp_ld + h * dm.e + c] = f32_to_lp_bits(acc[t] * inv, lp_bf16);
    }
}

int launch_window_attention(const void *q, uint64_t q_ld, const void *kv, uint64_t kv_ld, bool bf16,
                            const LatentDims &dm, uint64_t batch, uint64_t n, uint64_t hist, float *out,
                            const LpOut *out_lp, hipStream_t st) {
    if (batch == 0 || batch > 65535 || n == 0 || hist + n > 0x7fffffffull || dm.heads == 0 || dm.heads > 65535 ||
        dm.d == 0 || dm.d > 256 || dm.e == 0 || dm.e > 256)
        return fail(COEUS_INVALID_INPUT, "window attention: sizes out of range");
    uint16_t *lp = out_lp ? (uint16_t *)out_lp->p : nullptr;
    const uint64_t lp_ld = out_lp ? out_lp->ld : 0;
    const bool lp_bf = out_lp && out_lp->bf16;
    const dim3 grid((unsigned)ceil_div(n, 4), dm.heads, (unsigned)batch);
    const size_t lds = 4 * (dm.d + 64) * sizeof(float);
    if (bf16)
        hipLaunchKernelGGL(window_attn_kernel<true>, grid, dim3(256), lds, st, q, q_ld, kv, kv_ld, dm, (uint32_t)n,
                           (uint32_t)hist, out, lp, lp_ld, lp_bf);
    else
        hipLaunchKernelGGL(window_attn_kernel<false>, grid, dim3(256), lds, st, q, q_ld, kv, kv_ld, dm, (uint32_t)n,
                           (uint32_t)hist, out, lp, lp_ld, lp_bf);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// ---------------------------------------------------------------- decode
// One workgroup per (head, sequence).  The ring never holds more than the visible positions (cap <=
// window), and a softmax does not care about their order: slots 0 .. min(pos + 1, cap) - 1 are the keys.
template <bool BF16>
__global__ __launch_bounds__(256) void latent_decode_kernel(const float *__restrict__ q, const void *__restrict__ ukv,
                                                            LatentDims dm, const void *__restrict__ cache, uint32_t cap,
                                                            const uint32_t *pos_dev, float *__restrict__ out) {
    extern __shared__ float lds[];  // qa[rank], per-wave weighted latents [4][rank]
    __shared__ float sm[4], sl[4];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, R = dm.rank;
    const uint64_t b = blockIdx.y;
    float *qa = lds, *wl = qa + R;
    const float *qh = q + b * dm.heads * dm.d + h * dm.d;
    const uint64_t uk = (uint64_t)h * dm.d * R, uv = ((uint64_t)dm.heads * dm.d + h * dm.e) * R;
    for (uint32_t r = tid; r < R; r += 256) {
        float a = 0.f;
        for (uint32_t t = 0; t < dm.d; t++) a = fmaf(qh[t], lat_load<BF16>(ukv, uk + (uint64_t)t * R + r), a);
        qa[r] = a;
    }
    __syncthreads();
    const uint32_t nv = min(*pos_dev + 1, cap);
    constexpr int U = 32;  // rank <= 2048
    float acc[U], m = -INFINITY, l = 0.f;
#pragma unroll
    for (int u = 0; u < U; u++) acc[u] = 0.f;
    for (uint32_t j = wave; j < nv; j += 4) {
        const uint64_t cr = (b * cap + j) * R;
        float dot = 0.f;
        for (uint32_t r = lane; r < R; r += 64) dot = fmaf(qa[r], lat_load<BF16>(cache, cr + r), dot);
        const float s = wave_sum(dot) * dm.scale;
        const float m_new = fmaxf(m, s), corr = expf(m - m_new), p = expf(s - m_new);
        l = l * corr + p;
        m = m_new;
#pragma unroll
        for (int u = 0; u < U; u++)
            if (lane + 64 * u < R) acc[u] = fmaf(p, lat_load<BF16>(cache, cr + lane + 64 * u), acc[u] * corr);
    }
    if (lane == 0) { sm[wave] = m; sl[wave] = l; }
#pragma unroll
    for (int u = 0; u < U; u++)
        if (lane + 64 * u < R) wl[wave * R + lane + 64 * u] = acc[u];
    __syncthreads();
    const float mm = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
    float cw[4], lt = 0.f;
#pragma unroll
    for (int w = 0; w < 4; w++) { cw[w] = sm[w] == -INFINITY ? 0.f : expf(sm[w] - mm); lt += sl[w] * cw[w]; }
    for (uint32_t r = tid; r < R; r += 256)
        qa[r] = ((wl[r] * cw[0] + wl[R + r] * cw[1]) + (wl[2 * R + r] * cw[2] + wl[3 * R + r] * cw[3])) / lt;
    __syncthreads();
    for (uint32_t c = wave; c < dm.e; c += 4) {
        float a = 0.f;
        for (uint32_t r = lane; r < R; r += 64) a = fmaf(qa[r], lat_load<BF16>(ukv, uv + (uint64_t)c * R + r), a);
        a = wave_sum(a);
        if (lane == 0) out[b * dm.heads * dm.e + h * dm.e + c] = a;
    }
}

uint64_t latent_decode_scratch_bytes(const LatentDims &dm, uint32_t cap, uint64_t batch) {
    (void)dm; (void)cap; (void)batch;
    return 0;
}

int launch_latent_decode(const float *q, const void *ukv, const LatentDims &dm, const LatentCache &cache,
                         uint64_t batch, const uint32_t *pos_dev, float *out, float *scratch, uint64_t scratch_bytes,
                         hipStream_t st) {
    (void)scratch; (void)scratch_bytes;
    COEUS_TRY(check_dims(dm, cache));
    if (batch == 0 || batch > 65535 || !pos_dev) return fail(COEUS_INVALID_INPUT, "latent attention: rows out of range");
    const dim3 grid(dm.heads, (unsigned)batch);
    const size_t lds = 5 * (size_t)dm.rank * 4;
    if (cache.bf16)
        hipLaunchKernelGGL(latent_decode_kernel<true>, grid, dim3(256), lds, st, q, ukv, dm, cache.c, cache.cap, pos_dev, out);
    else
        hipLaunchKernelGGL(latent_decode_kernel<false>, grid, dim3(256), lds, st, q, ukv, dm, cache.c, cache.cap, pos_dev, out);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

}  // namespace coeus
