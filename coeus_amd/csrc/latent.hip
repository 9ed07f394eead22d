// Attention through low-rank latents with an optional sliding window.
//
//   latent_norm_kernel        RMS norms of the query latent and of the key/value latent
//   latent_gather / append    cached latents in front of a prompt's portion / its own into the ring
//   window_prefill_kernel     prompt, bf16: expanded keys and values on the matrix cores
//   window_attn_kernel        prompt: one wave per (row, head), any size and type
// Decode takes the query into latent space (W_uk^T q), scores it against the cached latents, which all
// heads share, and expands the weighted latent by W_uv:
//   latent_absorb_kernel      W_uk^T q of every head; the new token's latent, normalised, into the ring
//   latent_scores_kernel      bf16: 16 heads against a share of the ring on the matrix cores
//   latent_expand_kernel      merge of the shares, W_uv
//   latent_decode_kernel      all of it in one workgroup per head, any size and type
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
    if (dm.heads == 0 || dm.heads > 65534 || dm.d == 0 || dm.d > 256 || dm.e == 0 || dm.e > 256 || dm.q_rank == 0 ||
        dm.rank == 0 || dm.rank > 2048 || dm.in_ld < dm.q_rank + dm.rank)
        return fail(COEUS_INVALID_INPUT, "latent attention: sizes out of range");
    if (cache.cap == 0 || (dm.window && cache.cap > dm.window))
        return fail(COEUS_INVALID_INPUT, "latent attention: cache of %u positions for a window of %u", cache.cap, dm.window);
    return COEUS_OK;
}

// RMS norm of one row by a workgroup of 256 (a decode step's few rows): put(i, value) for every element.
template <typename Put>
__device__ __forceinline__ void norm_row_256(const float *__restrict__ x, uint32_t len, float eps,
                                             const float *__restrict__ scale, float *sh, Put put) {
    const uint32_t tid = threadIdx.x;
    float s2 = 0.f;
    for (uint32_t i = tid; i < len; i += 256) s2 = fmaf(x[i], x[i], s2);
    s2 = wave_sum(s2);
    __syncthreads();  // (sh may still be read for the row before)
    if ((tid & 63) == 0) sh[tid >> 6] = s2;
    __syncthreads();
    const float rs = 1.0f / sqrtf(((sh[0] + sh[1]) + (sh[2] + sh[3])) / (float)len + eps);
    for (uint32_t i = tid; i < len; i += 256) put(i, x[i] * rs * scale[i]);
}

// One wave per (row, latent); part 0: the query latent, 1: the key/value latent, of 2 - part0 a row.  Up to
// 1024 elements stay in registers between the sum and the store.
template <bool BF16>
__global__ __launch_bounds__(256) void latent_norm_kernel(const float *__restrict__ proj, LatentDims dm,
                                                          const float *__restrict__ q_scale,
                                                          const float *__restrict__ c_scale, float eps, uint64_t rows,
                                                          uint64_t n, float *cq, uint16_t *cq_lp, uint64_t cq_ld, bool lp_bf16,
                                                          void *lat, uint64_t lat_ld, uint64_t lat_rows,
                                                          uint64_t lat_off, uint32_t cap, const uint32_t *pos_dev,
                                                          uint32_t part0) {
    const uint32_t lane = threadIdx.x & 63, parts = 2 - part0;
    const uint64_t unit = (uint64_t)blockIdx.x * 4 + (threadIdx.x >> 6), row = unit / parts;
    if (row >= rows) return;
    const bool is_q = unit % parts + part0 == 0;
    const uint32_t len = is_q ? dm.q_rank : dm.rank;
    const float *x = proj + row * dm.in_ld + (is_q ? 0 : dm.q_rank), *scale = is_q ? q_scale : c_scale;
    constexpr int U = 16;
    float v[U], s2 = 0.f;
#pragma unroll
    for (int u = 0; u < U; u++) {
        v[u] = lane + 64 * u < len ? x[lane + 64 * u] : 0.f;
        s2 = fmaf(v[u], v[u], s2);
    }
    for (uint32_t i = lane + 64 * U; i < len; i += 64) s2 = fmaf(x[i], x[i], s2);
    const float rs = 1.0f / sqrtf(wave_sum(s2) / (float)len + eps);
    const uint64_t dst = pos_dev ? (row * cap + *pos_dev % cap) * dm.rank : ((row / n) * lat_rows + lat_off + row % n) * lat_ld;
    auto put = [&](uint32_t i, float y) {
        if (!is_q) lat_store<BF16>(lat, dst + i, y);
        if (is_q && cq) cq[row * dm.q_rank + i] = y;
        if (is_q && cq_lp) cq_lp[row * cq_ld + i] = f32_to_lp_bits(y, lp_bf16);
    };
#pragma unroll
    for (int u = 0; u < U; u++)
        if (lane + 64 * u < len) put(lane + 64 * u, v[u] * rs * scale[lane + 64 * u]);
    for (uint32_t i = lane + 64 * U; i < len; i += 64) put(i, x[i] * rs * scale[i]);
}

int launch_latent_norm(const float *proj, const LatentDims &dm, const float *q_scale, const float *c_scale, float eps,
                       uint64_t batch, uint64_t n, float *cq, const LpOut *cq_lp, void *lat, uint64_t lat_ld,
                       uint64_t lat_rows, uint64_t lat_off, const LatentCache &cache, const uint32_t *pos_dev,
                       hipStream_t st) {
    COEUS_TRY(check_dims(dm, cache));
    if (batch == 0 || n == 0 || batch * n > 0x7fffffffull || (pos_dev && n != 1))
        return fail(COEUS_INVALID_INPUT, "latent attention: rows out of range");
    const uint32_t part0 = cq || cq_lp ? 0 : 1;  // no place for the query latent: its consumer normalises it
    const uint64_t rows = batch * n;
    const dim3 grid((unsigned)ceil_div(rows * (2 - part0), 4));
    uint16_t *lp = cq_lp ? (uint16_t *)cq_lp->p : nullptr;
    const uint64_t ld = cq_lp ? cq_lp->ld : 0;
    const bool lp_bf = cq_lp && cq_lp->bf16;
    void *dst = pos_dev ? cache.c : lat;
    if (cache.bf16)
        hipLaunchKernelGGL(latent_norm_kernel<true>, grid, dim3(256), 0, st, proj, dm, q_scale, c_scale, eps, rows, n, cq, lp, ld,
                           lp_bf, dst, lat_ld, lat_rows, lat_off, cache.cap, pos_dev, part0);
    else
        hipLaunchKernelGGL(latent_norm_kernel<false>, grid, dim3(256), 0, st, proj, dm, q_scale, c_scale, eps, rows, n, cq, lp, ld,
                           lp_bf, dst, lat_ld, lat_rows, lat_off, cache.cap, pos_dev, part0);
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

// ---------------------------------------------------------------- prompt attention on the matrix cores
// The scheme of attn_prefill_kernel (scores and outputs transposed, so that a query stays in its lanes and
// the weights never leave registers) with key and value sizes of their own, rounded up to DK and DV (a
// piece behind the end re-reads the last one: its query dims are zero / its outputs are not stored), and a
// lower edge.  The f32 weights enter the product with V as a sum of two bf16 numbers.
__device__ __forceinline__ void split_bf16(float a, __bf16 &hi, __bf16 &lo) {
    hi = (__bf16)a;
    lo = (__bf16)(a - (float)hi);
}

template <int DK, int DV>
__global__ __launch_bounds__(256) void window_prefill_kernel(const uint16_t *__restrict__ q, uint64_t q_ld,
                                                             const uint16_t *__restrict__ kv, uint64_t kv_ld,
                                                             LatentDims dm, uint32_t n, uint32_t hist,
                                                             float *__restrict__ out, uint16_t *__restrict__ out_lp,
                                                             uint64_t lp_ld, bool lp_bf16) {
    constexpr int KT = 32, KLD = DK + 8, VLD = 36, NKS = DK / 16, NDT = DV / 32, KP = DK / 64, VP = (DV + 127) / 128;
    extern __shared__ __attribute__((aligned(16))) uint16_t lds16[];
    uint16_t *const ks = lds16, *const vt = lds16 + 2 * KT * KLD;  // [2][key][dim], [2][dim][key]
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, qi = lane & 31, hf = lane >> 5;
    uint32_t qt, h;
    prefill_tile_of_block(qt, h);
    const uint64_t b = blockIdx.z;
    const uint32_t r0 = qt * 128 + wave * 32, r = r0 + qi, rc = min(r, n - 1);
    const uint32_t qkey = hist + rc, W = dm.window ? dm.window : 0xffffffffu;  // row rc is key qkey, sees (qkey - W, qkey]
    const float scale2 = 1.4426950408889634f * dm.scale;
    bf16x8_t qf[NKS];
    {
        const uint16_t *qp = q + (b * n + rc) * q_ld + h * dm.d;
#pragma unroll
        for (int s = 0; s < NKS; s++) {
            union { uint4 u; bf16x8_t v; } cv;
            const uint32_t d0 = 16 * s + 8 * hf;
            cv.u = *(const uint4 *)(qp + min(d0, dm.d - 8));
            if (d0 >= dm.d) cv.u = make_uint4(0, 0, 0, 0);
            qf[s] = cv.v;
        }
    }
    const uint16_t *kb = kv + b * (hist + n) * kv_ld + h * dm.d;
    const uint16_t *vb = kv + b * (hist + n) * kv_ld + dm.heads * dm.d + h * dm.e;
    const uint32_t first_q = hist + qt * 128, kmax = hist + min(n, qt * 128 + 128) - 1;
    const uint32_t t_begin = (first_q >= W ? first_q - W + 1 : 0) / KT, t_end = kmax / KT + 1;
    const uint32_t wave_lo = hist + min(r0, n - 1), wave_hi = hist + min(r0 + 31, n - 1);
    const bool wave_live = r0 < n;

    const uint32_t kkey = tid >> 3, kpc = tid & 7, va = tid & 15, vdp = tid >> 4;
    uint4 rk0, rk1, rk2, rk3, rv0, rv1, rv2, rv3;  // (named: arrays captured by the lambdas end up in scratch memory)
    rk0 = rk1 = rk2 = rk3 = rv0 = rv1 = rv2 = rv3 = make_uint4(0, 0, 0, 0);
    auto kload = [&](uint64_t krow, uint32_t u, uint4 &x) { x = *(const uint4 *)(kb + krow + min(8 * (kpc + 8 * u), dm.d - 8)); };
    auto vload = [&](uint32_t t, uint32_t u, uint4 &x, uint4 &y) {
        const uint32_t d0 = min(8 * (vdp + 16 * u), dm.e - 8);
        x = *(const uint4 *)(vb + (uint64_t)min(t * KT + 2 * va, kmax) * kv_ld + d0);
        y = *(const uint4 *)(vb + (uint64_t)min(t * KT + 2 * va + 1, kmax) * kv_ld + d0);
    };
    auto gload = [&](uint32_t t) {
        const uint64_t krow = (uint64_t)min(t * KT + kkey, kmax) * kv_ld;
        kload(krow, 0, rk0);
        if (KP > 1) kload(krow, 1, rk1);
        if (KP > 2) { kload(krow, 2, rk2); kload(krow, 3, rk3); }
        if (DV >= 128 || vdp < DV / 8) vload(t, 0, rv0, rv1);
        if (VP > 1) vload(t, 1, rv2, rv3);
    };
    auto kstore = [&](uint32_t buf, uint32_t u, const uint4 &x) { *(uint4 *)(ks + buf * KT * KLD + kkey * KLD + 8 * (kpc + 8 * u)) = x; };
    auto vstore = [&](uint32_t buf, uint32_t u, const uint4 &x, const uint4 &y) {
        uint32_t *dst = (uint32_t *)(vt + buf * DV * VLD) + (vdp + 16 * u) * (8 * VLD / 2) + va;
        const uint32_t a[4] = {x.x, x.y, x.z, x.w}, c[4] = {y.x, y.y, y.z, y.w};
#pragma unroll
        for (int e = 0; e < 4; e++) {
            dst[e * VLD] = __builtin_amdgcn_perm(c[e], a[e], 0x05040100u);
            dst[e * VLD + VLD / 2] = __builtin_amdgcn_perm(c[e], a[e], 0x07060302u);
        }
    };
    auto lstore = [&](uint32_t buf) {
        kstore(buf, 0, rk0);
        if (KP > 1) kstore(buf, 1, rk1);
        if (KP > 2) { kstore(buf, 2, rk2); kstore(buf, 3, rk3); }
        if (DV >= 128 || vdp < DV / 8) vstore(buf, 0, rv0, rv1);
        if (VP > 1) vstore(buf, 1, rv2, rv3);
    };
    float16_t o[NDT];
#pragma unroll
    for (int d = 0; d < NDT; d++)
#pragma unroll
        for (int i = 0; i < 16; i++) o[d][i] = 0.f;
    float m = -1e30f, l = 0.f;  // (finite: a tile may hold no key that this query sees)

    gload(t_begin);
    lstore(t_begin & 1);
    gload(min(t_begin + 1, t_end - 1));
    for (uint32_t t = t_begin; t < t_end; t++) {
        __syncthreads();
        lstore((t + 1) & 1);
        gload(min(t + 2, t_end - 1));
        const uint32_t k0 = t * KT;
        if (!wave_live || k0 > wave_hi || (wave_lo >= W && k0 + KT - 1 <= wave_lo - W)) continue;  // wave-uniform
        const uint16_t *kt_ = ks + (t & 1) * KT * KLD, *vt_ = vt + (t & 1) * DV * VLD;
        float16_t sc;
#pragma unroll
        for (int i = 0; i < 16; i++) sc[i] = 0.f;
#pragma unroll
        for (int s = 0; s < NKS; s++)
            sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8_t *)(kt_ + qi * KLD + 16 * s + 8 * hf), qf[s], sc, 0, 0, 0);
        float tmax = -INFINITY;
#pragma unroll
        for (int i = 0; i < 16; i++) sc[i] *= scale2;
        if (k0 + KT - 1 > wave_lo || (wave_hi >= W && k0 <= wave_hi - W)) {  // an edge crosses the tile
#pragma unroll
            for (int i = 0; i < 16; i++) {
                const uint32_t key = k0 + 4 * hf + 8 * (i >> 2) + (i & 3);
                sc[i] = key > qkey || qkey - key >= W ? -INFINITY : sc[i];
            }
        }
#pragma unroll
        for (int i = 0; i < 16; i++) tmax = fmaxf(tmax, sc[i]);
        const float m_new = fmaxf(m, both_halves_max(tmax));
        float psum = 0.f, pv[16];
#pragma unroll
        for (int i = 0; i < 16; i++) {
            pv[i] = __builtin_amdgcn_exp2f(sc[i] - m_new);  // 2^(-inf) = 0 for keys that are not seen
            psum += pv[i];
        }
        if (__builtin_amdgcn_ballot_w64(m_new != m) != 0) {
            const float corr = __builtin_amdgcn_exp2f(m - m_new);
            l *= corr;
#pragma unroll
            for (int d = 0; d < NDT; d++)
#pragma unroll
                for (int i = 0; i < 16; i++) o[d][i] *= corr;
        }
        l += psum;
        m = m_new;
        bf16x8_t ph[2], pl[2];
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                __bf16 hi, lo;
                split_bf16(pv[8 * j + e], hi, lo);
                ph[j][e] = hi;
                pl[j][e] = lo;
            }
#pragma unroll
        for (int d = 0; d < NDT; d++)
#pragma unroll
            for (int j = 0; j < 2; j++) {
                const uint16_t *vp = vt_ + (d * 32 + qi) * VLD + 16 * j + 4 * hf;
                const uint2 v0 = *(const uint2 *)vp, v1 = *(const uint2 *)(vp + 8);
                union { uint4 u; bf16x8_t v; } vf;
                vf.u = make_uint4(v0.x, v0.y, v1.x, v1.y);
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf.v, pl[j], o[d], 0, 0, 0);
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf.v, ph[j], o[d], 0, 0, 0);
            }
    }
    if (r >= n) return;
    const float inv = 1.0f / xor32_sum(l);
    const uint64_t row = b * n + r;
#pragma unroll
    for (int d = 0; d < NDT; d++)
#pragma unroll
        for (int gq = 0; gq < 4; gq++) {
            const uint32_t c0 = d * 32 + 8 * gq + 4 * hf;  // e % 8 == 0: four columns are all in or all out
            if (c0 >= dm.e) continue;
            const float v[4] = {o[d][4 * gq] * inv, o[d][4 * gq + 1] * inv, o[d][4 * gq + 2] * inv, o[d][4 * gq + 3] * inv};
            if (out) *(float4 *)(out + row * dm.heads * dm.e + h * dm.e + c0) = make_float4(v[0], v[1], v[2], v[3]);
            if (out_lp) {
                uint2 p;
                p.x = (uint32_t)f32_to_lp_bits(v[0], lp_bf16) | ((uint32_t)f32_to_lp_bits(v[1], lp_bf16) << 16);
                p.y = (uint32_t)f32_to_lp_bits(v[2], lp_bf16) | ((uint32_t)f32_to_lp_bits(v[3], lp_bf16) << 16);
                *(uint2 *)(out_lp + row * lp_ld + h * dm.e + c0) = p;
            }
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
    // the matrix-core kernel moves 8 dims at a time
    if (bf16 && dm.d % 8 == 0 && dm.e % 8 == 0 && q_ld % 8 == 0 && kv_ld % 8 == 0 && lp_ld % 4 == 0) {
        const dim3 pgrid((unsigned)ceil_div(n, 128), dm.heads, (unsigned)batch);
#define COEUS_WP(DKV, DVV)                                                                                           \
    do {                                                                                                             \
        static const bool once = hipFuncSetAttribute((const void *)window_prefill_kernel<DKV, DVV>,                  \
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024) == hipSuccess; \
        (void)once;                                                                                                  \
        hipLaunchKernelGGL((window_prefill_kernel<DKV, DVV>), pgrid, dim3(256), (2 * 32 * (DKV + 8) + 2 * DVV * 36) * 2, st, \
                           (const uint16_t *)q, q_ld, (const uint16_t *)kv, kv_ld, dm, (uint32_t)n, (uint32_t)hist, out, lp, \
                           lp_ld, lp_bf);                                                                            \
    } while (0)
#define COEUS_WPV(DKV) do { if (dm.e <= 64) COEUS_WP(DKV, 64); else if (dm.e <= 128) COEUS_WP(DKV, 128); else COEUS_WP(DKV, 256); } while (0)
        if (dm.d <= 64) COEUS_WPV(64);
        else if (dm.d <= 128) COEUS_WPV(128);
        else COEUS_WPV(256);
#undef COEUS_WPV
#undef COEUS_WP
        COEUS_HIP(hipGetLastError());
        return COEUS_OK;
    }
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

// ---------------------------------------------------------------- decode, 16-bit cache
constexpr uint32_t kKeyTile = 64, kMaxShares = 32;

static bool latent_decode_fast(const LatentDims &dm, bool bf16) {
    return bf16 && dm.rank % 32 == 0 && dm.rank <= 1024 && dm.d % 4 == 0;
}
static uint32_t latent_shares(uint32_t cap) {
    const uint64_t tiles = ceil_div(cap, kKeyTile);
    return (uint32_t)(tiles < kMaxShares ? tiles : kMaxShares);
}

// W_uk^T q as two bf16 numbers per element, [batch][heads][high, low][rank]: one workgroup per (128 columns of the rank, head) and every sequence, so
// that the weights are read once.  Thread (g, r): column pair r, rows g, g + 4, ..  The workgroups behind the
// last head (blockIdx.y == heads) normalise the new tokens' latents into the ring.
template <int BP>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const float *__restrict__ q, const uint16_t *__restrict__ ukv,
                                                            LatentDims dm, uint32_t batch, uint16_t *__restrict__ qa, LatentNew nw,
                                                            uint16_t *__restrict__ cache, uint32_t cap,
                                                            const uint32_t *pos_dev) {
    extern __shared__ float lds[];  // q [BP][d], partial sums [4][BP][128]
    if (blockIdx.y == dm.heads) {
        for (uint32_t b = blockIdx.x; b < batch; b += gridDim.x) {
            __shared__ float sh[4];
            const float *x = nw.proj + (uint64_t)b * dm.in_ld + dm.q_rank;
            uint16_t *dst = cache + ((uint64_t)b * cap + *pos_dev % cap) * dm.rank;
            norm_row_256(x, dm.rank, nw.eps, nw.scale, sh, [&](uint32_t i, float v) { dst[i] = f32_to_bf16_bits(v); });
        }
        return;
    }
    const uint32_t tid = threadIdx.x, g = tid >> 6, rp = tid & 63, h = blockIdx.y, d = dm.d, R = dm.rank;
    const uint32_t r = blockIdx.x * 128 + 2 * rp, rc = min(r, R - 2);
    float *qs = lds, *red = lds + BP * d;
    const uint16_t *w = ukv + (uint64_t)h * d * R + rc;
    for (uint32_t i = tid; i < BP * d; i += 256) {
        const uint32_t b = i / d;
        qs[i] = b < batch ? q[(uint64_t)b * dm.heads * d + h * d + i % d] : 0.f;
    }
    float a0[BP], a1[BP];
#pragma unroll
    for (int b = 0; b < BP; b++) a0[b] = a1[b] = 0.f;
    __syncthreads();
    constexpr int U = BP > 4 ? 8 : 16;  // rows of a thread in flight
    for (uint32_t t0 = g; t0 < d; t0 += 4 * U) {
        uint32_t x[U];
#pragma unroll
        for (int u = 0; u < U; u++) x[u] = *(const uint32_t *)(w + (uint64_t)min(t0 + 4 * u, d - 1) * R);
#pragma unroll
        for (int u = 0; u < U; u++) {
            const uint32_t t = t0 + 4 * u;
            const float lo = __uint_as_float(x[u] << 16), hi = __uint_as_float(x[u] & 0xffff0000u);
#pragma unroll
            for (int b = 0; b < BP; b++) {
                const float qv = t < d ? qs[b * d + t] : 0.f;
                a0[b] = fmaf(qv, lo, a0[b]);
                a1[b] = fmaf(qv, hi, a1[b]);
            }
        }
    }
#pragma unroll
    for (int b = 0; b < BP; b++) *(float2 *)(red + (g * BP + b) * 128 + 2 * rp) = make_float2(a0[b], a1[b]);
    __syncthreads();
    for (uint32_t i = tid; i < batch * 128; i += 256) {
        const uint32_t b = i / 128, cc = i % 128, rr = blockIdx.x * 128 + cc;
        if (rr >= R) continue;
        __bf16 hi, lo;
        split_bf16((red[b * 128 + cc] + red[(BP + b) * 128 + cc]) + (red[(2 * BP + b) * 128 + cc] + red[(3 * BP + b) * 128 + cc]), hi, lo);
        __bf16 *dst = (__bf16 *)qa + ((uint64_t)b * dm.heads + h) * 2 * R + rr;
        dst[0] = hi;
        dst[R] = lo;
    }
}

// One workgroup of four waves per (share of the ring, 16 heads, sequence).  A wave scores 16 of a tile's 64
// latents for 16 heads, the softmax of the tile runs over LDS, then a wave accumulates a quarter of the
// rank.  Absorbed queries and weights enter the products as sums of two bf16 numbers each.
// The share's record: maximum (base 2), sum, weighted latent.
template <int PT>  // 16-wide column tiles of a wave: rank <= 64 PT
__global__ __launch_bounds__(256) void latent_scores_kernel(const uint16_t *__restrict__ qa, LatentDims dm,
                                                            const uint16_t *__restrict__ cache, uint32_t cap,
                                                            const uint32_t *pos_dev, uint32_t keys_per_share,
                                                            float *__restrict__ part) {
    constexpr uint32_t VLD = kKeyTile + 8, PLD = kKeyTile + 8;  // (16-byte rows; row stride 36 dwords)
    extern __shared__ __attribute__((aligned(16))) uint16_t lds16[];
    uint16_t *ct = lds16;                                    // latents of the tile, [rank][VLD]
    uint16_t *ph = ct + dm.rank * VLD, *pl = ph + 16 * PLD;  // weights, high and low parts, [16][PLD]
    float *ss = (float *)(pl + 16 * PLD);                    // scores [16][PLD]
    float *ms = ss + 16 * PLD, *ls = ms + 16, *cs = ls + 16; // running maximum and sum, correction, per head
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4, R = dm.rank;
    const uint32_t share = blockIdx.x, h0 = blockIdx.y * 16, hc = min(h0 + c, dm.heads - 1);
    const uint64_t b = blockIdx.z;
    const uint32_t nv = min(*pos_dev + 1, cap), k_begin = share * keys_per_share, k_end = min(nv, k_begin + keys_per_share);
    // (a share that no position has reached yet leaves an empty record)
    const float scale2 = 1.4426950408889634f * dm.scale;
    if (tid < 16) { ms[tid] = -1e30f; ls[tid] = 0.f; }
    const uint16_t *qp = qa + (b * dm.heads + hc) * 2 * R + 8 * g;
    const uint16_t *cb = cache + b * cap * R;
    constexpr uint32_t RD = PT == 4 ? 256 : 512;  // of the rank in a round
    float4_t acc[PT];
#pragma unroll
    for (int t = 0; t < PT; t++) acc[t] = float4_t{0.f, 0.f, 0.f, 0.f};
    for (uint32_t k0 = k_begin; k0 < k_end; k0 += kKeyTile) {
        // RD of the rank a round.  Everything is requested at once, from addresses that do not depend on the
        // position (slots that are not written yet hold finite values and are masked; a piece behind the end
        // re-reads the last one and is not used): the tile as key pairs for the transposed copy (8 pieces of 8
        // dims x 32 pairs a step), as right operands for keys k0 + 16 wave + c, and the absorbed queries.
        float4_t sc = {0.f, 0.f, 0.f, 0.f}, sc2 = {0.f, 0.f, 0.f, 0.f};
        const uint16_t *kp = cb + (uint64_t)min(k0 + 16 * wave + c, cap - 1) * R + 8 * g;
        const uint32_t a = tid >> 3, steps = R / 32;
        const uint16_t *tx = cb + (uint64_t)min(k0 + 2 * a, cap - 1) * R, *ty = cb + (uint64_t)min(k0 + 2 * a + 1, cap - 1) * R;
        for (uint32_t r0 = 0; r0 < R; r0 += RD) {
            uint4 x[RD / 64], y[RD / 64];
            bf16x8_t kf[RD / 32], qh[RD / 32], ql[RD / 32];
#pragma unroll
            for (int u = 0; u < (int)RD / 64; u++) {
                const uint32_t off = min(r0 + 64 * u + 8 * (tid & 7), R - 8);
                x[u] = *(const uint4 *)(tx + off);
                y[u] = *(const uint4 *)(ty + off);
            }
#pragma unroll
            for (int u = 0; u < (int)RD / 32; u++) {
                const uint32_t off = min(r0 + 32 * u, R - 32);
                kf[u] = *(const bf16x8_t *)(kp + off);
                qh[u] = *(const bf16x8_t *)(qp + off);
                ql[u] = *(const bf16x8_t *)(qp + R + off);
            }
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int u = 0; u < (int)RD / 64; u++) {
                const uint32_t off = min(r0 + 64 * u + 8 * (tid & 7), R - 8);
                const uint32_t xs[4] = {x[u].x, x[u].y, x[u].z, x[u].w}, ys[4] = {y[u].x, y[u].y, y[u].z, y[u].w};
                uint32_t *dst = (uint32_t *)ct + off * (VLD / 2) + a;
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    dst[e * VLD] = __builtin_amdgcn_perm(ys[e], xs[e], 0x05040100u);
                    dst[e * VLD + VLD / 2] = __builtin_amdgcn_perm(ys[e], xs[e], 0x07060302u);
                }
            }
#pragma unroll
            for (int u = 0; u < (int)RD / 32; u++)
                if (r0 / 32 + u < steps) {
                    sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qh[u], kf[u], sc, 0, 0, 0);
                    sc2 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ql[u], kf[u], sc2, 0, 0, 0);
                }
        }
        const uint32_t key = k0 + 16 * wave + c;
#pragma unroll
        for (int i = 0; i < 4; i++) ss[(4 * g + i) * PLD + 16 * wave + c] = key < k_end ? (sc[i] + sc2[i]) * scale2 : -INFINITY;
        __syncthreads();
        // wave w: the softmax of heads 4 w .. 4 w + 3, a key per lane
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t hh = 4 * wave + i;
            const float s = ss[hh * PLD + lane], m_old = ms[hh];
            const float m_new = fmaxf(m_old, wave_max(s)), p = __builtin_amdgcn_exp2f(s - m_new);
            const float sum = wave_sum(p), corr = __builtin_amdgcn_exp2f(m_old - m_new);
            __bf16 hi, lo;
            split_bf16(p, hi, lo);
            ((__bf16 *)ph)[hh * PLD + lane] = hi;
            ((__bf16 *)pl)[hh * PLD + lane] = lo;
            if (lane == 0) { ms[hh] = m_new; ls[hh] = ls[hh] * corr + sum; cs[hh] = corr; }
        }
        __syncthreads();
        float cr[4];
#pragma unroll
        for (int i = 0; i < 4; i++) cr[i] = cs[4 * g + i];
        bf16x8_t pah[2], pal[2];
#pragma unroll
        for (int j = 0; j < 2; j++) {
            pah[j] = *(const bf16x8_t *)(ph + c * PLD + 32 * j + 8 * g);
            pal[j] = *(const bf16x8_t *)(pl + c * PLD + 32 * j + 8 * g);
        }
#pragma unroll
        for (int t = 0; t < PT; t++) {
            const uint32_t tile = wave * PT + t;
            if (16 * tile < R) {  // wave-uniform
#pragma unroll
                for (int i = 0; i < 4; i++) acc[t][i] *= cr[i];
#pragma unroll
                for (int j = 0; j < 2; j++) {
                    const bf16x8_t vf = *(const bf16x8_t *)(ct + (16 * tile + c) * VLD + 32 * j + 8 * g);
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pal[j], vf, acc[t], 0, 0, 0);
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pah[j], vf, acc[t], 0, 0, 0);
                }
            }
        }
        __syncthreads();  // everybody is done with this tile
    }
    if (k_begin >= k_end) __syncthreads();  // an empty share: the initial maxima and sums are its record
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const uint32_t hh = h0 + 4 * g + i;
        if (hh >= dm.heads) continue;
        float *rec = part + ((b * dm.heads + hh) * gridDim.x + share) * (R + 2);
        if (wave == 0 && c == 0) { rec[0] = ms[4 * g + i]; rec[1] = ls[4 * g + i]; }
#pragma unroll
        for (int t = 0; t < PT; t++) {
            const uint32_t r = 16 * (wave * PT + t) + c;
            if (r < R) rec[2 + r] = acc[t][i];
        }
    }
}

// One workgroup per (32 value dims, head, sequence): merges the shares, then W_uv rows against the result.
// A wave's eight rows are requested before the merge, the shares' records sixteen at a time.
template <int RP>  // pieces of 512 of the rank
__global__ __launch_bounds__(256) void latent_expand_kernel(const float *__restrict__ part, const uint16_t *__restrict__ ukv,
                                                            LatentDims dm, uint32_t shares, float *__restrict__ out) {
    extern __shared__ float lds[];  // merged latent [rank]
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.y, R = dm.rank;
    const uint64_t b = blockIdx.z;
    const float *rec = part + (b * dm.heads + h) * shares * (R + 2);
    const uint32_t c0 = blockIdx.x * 32 + wave * 8;
    uint4 w[8][RP];
#pragma unroll
    for (int i = 0; i < 8; i++)
#pragma unroll
        for (int k = 0; k < RP; k++)
            w[i][k] = *(const uint4 *)(ukv + ((uint64_t)dm.heads * dm.d + h * dm.e + min(c0 + i, dm.e - 1)) * R + min(lane * 8 + 512 * k, R - 8));
    // every wave finds the shares' weights for itself
    const uint32_t sl = min(lane, shares - 1);
    const float m = rec[sl * (R + 2)], l = rec[sl * (R + 2) + 1];
    float a[2 * RP];
#pragma unroll
    for (int k = 0; k < 2 * RP; k++) a[k] = 0.f;
    const float mm = wave_max(m), ws = lane < shares ? __builtin_amdgcn_exp2f(m - mm) : 0.f;
    const float inv = 1.0f / wave_sum(l * ws);
    for (uint32_t s0 = 0; s0 < shares; s0 += 16) {
        float x[16][2 * RP];
#pragma unroll
        for (int s = 0; s < 16; s++)
#pragma unroll
            for (int k = 0; k < 2 * RP; k++) x[s][k] = rec[min(s0 + s, shares - 1) * (R + 2) + 2 + min(tid + 256 * k, R - 1)];
#pragma unroll
        for (int s = 0; s < 16; s++) {
            const float wt = __shfl(ws, (int)(s0 + s), 64);  // (0 behind the last share)
#pragma unroll
            for (int k = 0; k < 2 * RP; k++) a[k] = fmaf(wt, x[s][k], a[k]);
        }
    }
#pragma unroll
    for (int k = 0; k < 2 * RP; k++)
        if (tid + 256 * k < R) lds[tid + 256 * k] = a[k] * inv;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 8; i++) {
        float v = 0.f;
#pragma unroll
        for (int k = 0; k < RP; k++) {
            const uint32_t r = lane * 8 + 512 * k;
            if (r >= R) continue;
            const uint32_t xs[4] = {w[i][k].x, w[i][k].y, w[i][k].z, w[i][k].w};
#pragma unroll
            for (int e = 0; e < 4; e++) {
                v = fmaf(__uint_as_float(xs[e] << 16), lds[r + 2 * e], v);
                v = fmaf(__uint_as_float(xs[e] & 0xffff0000u), lds[r + 2 * e + 1], v);
            }
        }
        v = wave_sum(v);
        if (lane == 0 && c0 + i < dm.e) out[b * dm.heads * dm.e + h * dm.e + c0 + i] = v;
    }
}

uint64_t latent_decode_scratch_bytes(const LatentDims &dm, const LatentCache &cache, uint64_t batch) {
    if (!latent_decode_fast(dm, cache.bf16)) return 0;
    // absorbed queries, then a record per (sequence, head, share)
    return batch * dm.heads * (dm.rank + latent_shares(cache.cap) * (dm.rank + 2ull)) * 4;
}

int launch_latent_decode(const float *q, const void *ukv, const LatentDims &dm, const LatentNew &nw,
                         const LatentCache &cache, uint64_t batch, const uint32_t *pos_dev, float *out, float *scratch,
                         uint64_t scratch_bytes, hipStream_t st) {
    COEUS_TRY(check_dims(dm, cache));
    if (batch == 0 || batch > 65535 || !pos_dev) return fail(COEUS_INVALID_INPUT, "latent attention: rows out of range");
    const uint64_t want = latent_decode_scratch_bytes(dm, cache, batch);
    if (want && batch <= 16 && scratch && scratch_bytes >= want) {
        const uint16_t *w = (const uint16_t *)ukv;
        uint16_t *cc = (uint16_t *)cache.c;
        uint16_t *qa = (uint16_t *)scratch;
        float *part = scratch + batch * dm.heads * dm.rank;
        const uint32_t shares = latent_shares(cache.cap), bp = pad_batch(batch), R = dm.rank;
        const uint32_t per_share = (uint32_t)round_up(ceil_div(cache.cap, shares), kKeyTile);
        const dim3 agrid((unsigned)ceil_div(R, 128), dm.heads + 1);
        const size_t alds = (bp * (size_t)dm.d + 4 * bp * 128) * 4;
#define COEUS_LA(BPV) \
    case BPV: hipLaunchKernelGGL(latent_absorb_kernel<BPV>, agrid, dim3(256), alds, st, q, w, dm, (uint32_t)batch, qa, nw, cc, cache.cap, \
                                 pos_dev); break
        switch (bp) { COEUS_LA(1); COEUS_LA(2); COEUS_LA(4); COEUS_LA(8); COEUS_LA(16); }
#undef COEUS_LA
        const size_t slds = ((size_t)R * (kKeyTile + 8) + 2 * 16 * (kKeyTile + 8)) * 2 + (16 * (kKeyTile + 8) + 48) * 4;
        const dim3 sgrid(shares, (unsigned)ceil_div(dm.heads, 16), (unsigned)batch);
#define COEUS_LS(PTV)                                                                                               \
    do {                                                                                                            \
        static const bool once = hipFuncSetAttribute((const void *)latent_scores_kernel<PTV>,                       \
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) == hipSuccess; \
        (void)once;                                                                                                 \
        hipLaunchKernelGGL(latent_scores_kernel<PTV>, sgrid, dim3(256), slds, st, qa, dm, cc, cache.cap, pos_dev, per_share, part); \
    } while (0)
        if (R <= 256) COEUS_LS(4);
        else if (R <= 512) COEUS_LS(8);
        else COEUS_LS(16);
#undef COEUS_LS
        const dim3 egrid((unsigned)ceil_div(dm.e, 32), dm.heads, (unsigned)batch);
        if (R <= 512) hipLaunchKernelGGL(latent_expand_kernel<1>, egrid, dim3(256), (size_t)R * 4, st, part, w, dm, shares, out);
        else hipLaunchKernelGGL(latent_expand_kernel<2>, egrid, dim3(256), (size_t)R * 4, st, part, w, dm, shares, out);
        COEUS_HIP(hipGetLastError());
        return COEUS_OK;
    }
    COEUS_TRY(launch_latent_norm(nw.proj, dm, nullptr, nw.scale, nw.eps, batch, 1, nullptr, nullptr, nullptr, 0, 0, 0, cache, pos_dev, st));
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
