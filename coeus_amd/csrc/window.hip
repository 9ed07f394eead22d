// Windowed attention of a prompt's rows, and the rings of rows that it leaves behind.
//
//   ring_copy_kernel          cached rows in front of a prompt's portion / its own into the ring
//   window_prefill_kernel     prompt, bf16: keys and values on the matrix cores
//   window_attn_kernel        prompt: one wave per (row, head), any size and type
#include "device_utils.hpp"
#include "mixers.hpp"

namespace coeus {

// The f32 value behind a row of keys.
template <bool BF16>
__device__ __forceinline__ float inverse_rms(const void *kv, uint64_t i) {
    return BF16 ? *(const float *)((const uint16_t *)kv + i) : ((const float *)kv)[i];
}

// Rows of `len` elements between the ring and a contiguous buffer: blockIdx.x counts `cnt` positions
// from pos_first, whose buffer row is row_first.
template <typename T, bool TO_RING>
__global__ __launch_bounds__(64) void ring_copy_kernel(T *ring, uint32_t cap, uint32_t len, T *buf, uint64_t ld,
                                                         uint64_t rows_per_seq, uint64_t pos_first, uint64_t row_first) {
    const uint64_t i = blockIdx.x, b = blockIdx.y;
    T *r = ring + (b * cap + (pos_first + i) % cap) * len, *l = buf + (b * rows_per_seq + row_first + i) * ld;
    for (uint32_t t = threadIdx.x; t < len; t += 64) {
        if (TO_RING) r[t] = l[t];
        else l[t] = r[t];
    }
}

template <bool TO_RING>
static int ring_copy(const RowRing &cache, uint32_t len, uint64_t batch, uint64_t cnt, uint64_t pos_first, void *buf,
                       uint64_t ld, uint64_t rows_per_seq, uint64_t row_first, hipStream_t st) {
    if (cnt == 0) return COEUS_OK;
    if (cnt > cache.cap || batch == 0 || batch > 65535) return fail(COEUS_INVALID_INPUT, "window attention: rows out of range");
    const dim3 grid((unsigned)cnt, (unsigned)batch);
    if (cache.bf16)
        hipLaunchKernelGGL((ring_copy_kernel<uint16_t, TO_RING>), grid, dim3(64), 0, st, (uint16_t *)cache.c, cache.cap, len,
                           (uint16_t *)buf, ld, rows_per_seq, pos_first, row_first);
    else
        hipLaunchKernelGGL((ring_copy_kernel<float, TO_RING>), grid, dim3(64), 0, st, (float *)cache.c, cache.cap, len,
                           (float *)buf, ld, rows_per_seq, pos_first, row_first);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

int launch_ring_gather(const RowRing &cache, uint32_t len, uint64_t batch, uint64_t hist, uint64_t pos0,
                         void *buf, uint64_t ld, uint64_t rows_per_seq, hipStream_t st) {
    if (hist > pos0) return fail(COEUS_INVALID_INPUT, "window attention: rows out of range");
    return ring_copy<false>(cache, len, batch, hist, pos0 - hist, buf, ld, rows_per_seq, 0, st);
}

int launch_ring_append(const void *buf, uint64_t ld, uint64_t rows_per_seq, uint64_t hist, const RowRing &cache,
                         uint32_t len, uint64_t batch, uint64_t n, uint64_t pos0, hipStream_t st) {
    const uint64_t cnt = n < cache.cap ? n : cache.cap;
    return ring_copy<true>(cache, len, batch, cnt, pos0 + n - cnt, (void *)buf, ld, rows_per_seq, hist + n - cnt, st);
}

// ---------------------------------------------------------------- prompt attention, any size and type
// Row i of a sequence is key hist + i and sees keys lo .. hist + i, lo = max(0, hist + i - window + 1).
template <bool BF16, bool SHARED>
__global__ __launch_bounds__(256) void window_attn_kernel(const void *__restrict__ q, uint64_t q_ld,
                                                          const void *__restrict__ kv, uint64_t kv_ld, WindowShape dm,
                                                          uint32_t n, uint32_t hist, float *__restrict__ out,
                                                          uint16_t *__restrict__ out_lp, uint64_t lp_ld, bool lp_bf16) {
    extern __shared__ float lds[];  // per wave: q[d] + p[64]
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const uint32_t i = blockIdx.x * 4 + wave, h = blockIdx.y;
    const uint64_t b = blockIdx.z;
    if (i >= n) return;
    float *qs = lds + wave * (dm.d + 64), *ps = qs + dm.d;
    const uint64_t row = b * n + i, k0 = b * (hist + n);
    for (uint32_t t = lane; t < dm.d; t += 64) qs[t] = elem_load<BF16>(q, row * q_ld + h * dm.d + t);
    const uint32_t end = hist + i + 1, lo = dm.window && end > dm.window ? end - dm.window : 0;
    const uint32_t koff = SHARED ? h / (dm.heads / dm.kv_heads) * dm.d : h * dm.d;
    const uint32_t voff = SHARED ? koff : dm.heads * dm.d + h * dm.e;
    const float slope = SHARED ? dm.slope(h) : 0.f;
    float m = -INFINITY, l = 0.f, acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (uint32_t j0 = lo; j0 < end; j0 += 64) {
        const uint32_t j = j0 + lane;
        float s = -INFINITY;
        if (j < end) {
            float dot = 0.f;
            const uint64_t kr = (k0 + j) * kv_ld + koff;
            for (uint32_t t = 0; t < dm.d; t++) dot = fmaf(qs[t], elem_load<BF16>(kv, kr + t), dot);
            s = dot * dm.scale;
            if (SHARED) s = s * inverse_rms<BF16>(kv, (k0 + j) * kv_ld + dm.rms_off) - slope * (float)(end - 1 - j);
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
                if (lane + 64 * t < dm.e) acc[t] = fmaf(pj, elem_load<BF16>(kv, vr + lane + 64 * t), acc[t]);
        }
    }
    const float inv = 1.0f / l;
#pragma unroll
    for (int t = 0; t < 4; t++) {
        const uint32_t c = lane + 64 * t;
        if (c >= dm.e) continue;
        float o = acc[t] * inv;
        if (SHARED) o *= fast_sigmoid(dm.gate[row * dm.gate_ld + h * dm.e + c]);
        if (out) out[row * dm.heads * dm.e + h * dm.e + c] = o;
        if (out_lp) out_lp[row * lp_ld + h * dm.e + c] = f32_to_lp_bits(o, lp_bf16);
    }
}

// ---------------------------------------------------------------- prompt attention on the matrix cores
// The scheme of attn_prefill_kernel (scores and outputs transposed, so that a query stays in its lanes and
// the weights never leave registers) with key and value sizes of their own, rounded up to DK and DV (a
// piece behind the end re-reads the last one: its query dims are zero / its outputs are not stored), and a
// lower edge.  The f32 weights enter the product with V as a sum of two bf16 numbers.
// SHARED (DK == DV): the values are the keys, so that one trip to memory fills both copies in LDS; scores are
// multiplied by the key's inverse root mean square and lose slope * distance, outputs meet their gate.

template <int DK, int DV, bool SHARED>
__global__ __launch_bounds__(256, DK + DV <= 256 ? 2 : 1) void window_prefill_kernel(const uint16_t *__restrict__ q, uint64_t q_ld,
                                                             const uint16_t *__restrict__ kv, uint64_t kv_ld,
                                                             WindowShape dm, uint32_t n, uint32_t hist,
                                                             float *__restrict__ out, uint16_t *__restrict__ out_lp,
                                                             uint64_t lp_ld, bool lp_bf16) {
    constexpr int KT = 32, KLD = DK + 8, VLD = 36, NKS = DK / 16, NDT = DV / 32, KP = DK / 64, VP = (DV + 127) / 128;
    extern __shared__ __attribute__((aligned(16))) uint16_t lds16[];
    uint16_t *const ks = lds16, *const vt = lds16 + 2 * KT * KLD;  // [2][key][dim], [2][dim][key]
    float *const rl = (float *)(vt + 2 * DV * VLD);                // SHARED: [2][key] scale / root mean square
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
    const uint16_t *kv0 = kv + b * (hist + n) * kv_ld;
    const uint16_t *kb = kv0 + (SHARED ? h / (dm.heads / dm.kv_heads) : h) * dm.d;
    const uint16_t *vb = SHARED ? kb : kv0 + dm.heads * dm.d + h * dm.e;
    const float slope2 = SHARED ? 1.4426950408889634f * dm.slope(h) : 0.f;
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
    float rr = 0.f;
    auto gload = [&](uint32_t t) {
        if (SHARED) {
            if (tid < KT) rr = *(const float *)(kv0 + (uint64_t)min(t * KT + tid, kmax) * kv_ld + dm.rms_off);
        } else {
            const uint64_t krow = (uint64_t)min(t * KT + kkey, kmax) * kv_ld;
            kload(krow, 0, rk0);
            if (KP > 1) kload(krow, 1, rk1);
            if (KP > 2) { kload(krow, 2, rk2); kload(krow, 3, rk3); }
        }
        if (DV >= 128 || vdp < DV / 8) vload(t, 0, rv0, rv1);
        if (VP > 1) vload(t, 1, rv2, rv3);
    };
    auto kstore = [&](uint32_t buf, uint32_t u, const uint4 &x) { *(uint4 *)(ks + buf * KT * KLD + kkey * KLD + 8 * (kpc + 8 * u)) = x; };
    auto vstore = [&](uint32_t buf, uint32_t u, const uint4 &x, const uint4 &y) {
        if (SHARED) {
            uint16_t *kd = ks + buf * KT * KLD + 2 * va * KLD + 8 * (vdp + 16 * u);
            *(uint4 *)kd = x;
            *(uint4 *)(kd + KLD) = y;
        }
        uint32_t *dst = (uint32_t *)(vt + buf * DV * VLD) + (vdp + 16 * u) * (8 * VLD / 2) + va;
        const uint32_t a[4] = {x.x, x.y, x.z, x.w}, c[4] = {y.x, y.y, y.z, y.w};
#pragma unroll
        for (int e = 0; e < 4; e++) {
            dst[e * VLD] = __builtin_amdgcn_perm(c[e], a[e], 0x05040100u);
            dst[e * VLD + VLD / 2] = __builtin_amdgcn_perm(c[e], a[e], 0x07060302u);
        }
    };
    auto lstore = [&](uint32_t buf) {
        if (SHARED) {
            if (tid < KT) rl[buf * KT + tid] = scale2 * rr;
        } else {
            kstore(buf, 0, rk0);
            if (KP > 1) kstore(buf, 1, rk1);
            if (KP > 2) { kstore(buf, 2, rk2); kstore(buf, 3, rk3); }
        }
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
        if (SHARED) {
            // register i holds key k0 + 4 hf + 8 (i / 4) + i % 4
            const float near = slope2 * (float)(int)(k0 + 4 * hf - qkey);
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const float4 f = *(const float4 *)(rl + (t & 1) * KT + 4 * hf + 8 * j);
                sc[4 * j] = fmaf(sc[4 * j], f.x, fmaf(slope2, 8.f * j, near));
                sc[4 * j + 1] = fmaf(sc[4 * j + 1], f.y, fmaf(slope2, 8.f * j + 1.f, near));
                sc[4 * j + 2] = fmaf(sc[4 * j + 2], f.z, fmaf(slope2, 8.f * j + 2.f, near));
                sc[4 * j + 3] = fmaf(sc[4 * j + 3], f.w, fmaf(slope2, 8.f * j + 3.f, near));
            }
        } else {
#pragma unroll
            for (int i = 0; i < 16; i++) sc[i] *= scale2;
        }
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
            float v[4] = {o[d][4 * gq] * inv, o[d][4 * gq + 1] * inv, o[d][4 * gq + 2] * inv, o[d][4 * gq + 3] * inv};
            if (SHARED) {
                const float4 gt = *(const float4 *)(dm.gate + row * dm.gate_ld + h * dm.e + c0);
                v[0] *= fast_sigmoid(gt.x); v[1] *= fast_sigmoid(gt.y); v[2] *= fast_sigmoid(gt.z); v[3] *= fast_sigmoid(gt.w);
            }
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
                            const WindowShape &dm, uint64_t batch, uint64_t n, uint64_t hist, float *out,
                            const LpOut *out_lp, hipStream_t st) {
    const bool shared = dm.kv_heads != 0;
    if (batch == 0 || batch > 65535 || n == 0 || hist + n > 0x7fffffffull || dm.heads == 0 || dm.heads > 65535 ||
        dm.d == 0 || dm.d > 256 || dm.e == 0 || dm.e > 256 ||
        (shared && (dm.heads % dm.kv_heads || dm.d != dm.e || !dm.gate || dm.rms_off < dm.kv_heads * dm.d || dm.rms_off % 2 ||
                    kv_ld % 2 || kv_ld < dm.rms_off + 2)))
        return fail(COEUS_INVALID_INPUT, "window attention: sizes out of range");
    uint16_t *lp = out_lp ? (uint16_t *)out_lp->p : nullptr;
    const uint64_t lp_ld = out_lp ? out_lp->ld : 0;
    const bool lp_bf = out_lp && out_lp->bf16;
    // the matrix-core kernel moves 8 dims at a time
    if (bf16 && dm.d % 8 == 0 && dm.e % 8 == 0 && q_ld % 8 == 0 && kv_ld % 8 == 0 && lp_ld % 4 == 0 && (!shared || dm.gate_ld % 4 == 0)) {
        const dim3 pgrid((unsigned)ceil_div(n, 128), dm.heads, (unsigned)batch);
#define COEUS_WP(DKV, DVV, SH)                                                                                       \
    do {                                                                                                             \
        static const bool once = hipFuncSetAttribute((const void *)window_prefill_kernel<DKV, DVV, SH>,              \
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024) == hipSuccess; \
        (void)once;                                                                                                  \
        hipLaunchKernelGGL((window_prefill_kernel<DKV, DVV, SH>), pgrid, dim3(256),                                  \
                           (2 * 32 * (DKV + 8) + 2 * DVV * 36) * 2 + (SH ? 2 * 32 * 4 : 0), st,                      \
                           (const uint16_t *)q, q_ld, (const uint16_t *)kv, kv_ld, dm, (uint32_t)n, (uint32_t)hist, out, lp, \
                           lp_ld, lp_bf);                                                                            \
    } while (0)
#define COEUS_WPV(DKV) \
    do { if (dm.e <= 64) COEUS_WP(DKV, 64, false); else if (dm.e <= 128) COEUS_WP(DKV, 128, false); else COEUS_WP(DKV, 256, false); } while (0)
        if (shared) {
            if (dm.d <= 64) COEUS_WP(64, 64, true);
            else if (dm.d <= 128) COEUS_WP(128, 128, true);
            else COEUS_WP(256, 256, true);
        } else if (dm.d <= 64) COEUS_WPV(64);
        else if (dm.d <= 128) COEUS_WPV(128);
        else COEUS_WPV(256);
#undef COEUS_WPV
#undef COEUS_WP
        COEUS_HIP(hipGetLastError());
        return COEUS_OK;
    }
    const dim3 grid((unsigned)ceil_div(n, 4), dm.heads, (unsigned)batch);
    const size_t lds = 4 * (dm.d + 64) * sizeof(float);
#define COEUS_WA(BFV, SH) \
    hipLaunchKernelGGL((window_attn_kernel<BFV, SH>), grid, dim3(256), lds, st, q, q_ld, kv, kv_ld, dm, (uint32_t)n, (uint32_t)hist, \
                       out, lp, lp_ld, lp_bf)
    if (bf16) { if (shared) COEUS_WA(true, true); else COEUS_WA(true, false); }
    else { if (shared) COEUS_WA(false, true); else COEUS_WA(false, false); }
#undef COEUS_WA
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

}  // namespace coeus
