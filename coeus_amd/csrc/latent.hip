// Attention through low-rank latents with an optional sliding window: the latents' norms and a decode step
// (a prompt's latents are expanded by a matmul and attended to in window.hip).
//
//   latent_norm_kernel        RMS norms of the query latent and of the key/value latent
// Decode takes the query into latent space (W_uk^T q), scores it against the cached latents, which all
// heads share, and expands the weighted latent by W_uv:
//   latent_absorb_kernel      W_uk^T q of every head; the new token's latent, normalised, into the ring
//   latent_scores_kernel      bf16: 16 heads against a share of the ring on the matrix cores
//   latent_expand_kernel      merge of the shares, W_uv
//   latent_decode_kernel      all of it in one workgroup per head, any size and type
#include "device_utils.hpp"
#include "mixers.hpp"

namespace coeus {


static int check_dims(const LatentDims &dm, const RowRing &cache) {
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
        if (!is_q) elem_store<BF16>(lat, dst + i, y);
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
                       uint64_t lat_rows, uint64_t lat_off, const RowRing &cache, const uint32_t *pos_dev,
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
        for (uint32_t t = 0; t < dm.d; t++) a = fmaf(qh[t], elem_load<BF16>(ukv, uk + (uint64_t)t * R + r), a);
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
        for (uint32_t r = lane; r < R; r += 64) dot = fmaf(qa[r], elem_load<BF16>(cache, cr + r), dot);
        const float s = wave_sum(dot) * dm.scale;
        const float m_new = fmaxf(m, s), corr = expf(m - m_new), p = expf(s - m_new);
        l = l * corr + p;
        m = m_new;
#pragma unroll
        for (int u = 0; u < U; u++)
            if (lane + 64 * u < R) acc[u] = fmaf(p, elem_load<BF16>(cache, cr + lane + 64 * u), acc[u] * corr);
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
        for (uint32_t r = lane; r < R; r += 64) a = fmaf(qa[r], elem_load<BF16>(ukv, uv + (uint64_t)c * R + r), a);
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

uint64_t latent_decode_scratch_bytes(const LatentDims &dm, const RowRing &cache, uint64_t batch) {
    if (!latent_decode_fast(dm, cache.bf16)) return 0;
    // absorbed queries, then a record per (sequence, head, share)
    return batch * dm.heads * (dm.rank + latent_shares(cache.cap) * (dm.rank + 2ull)) * 4;
}

int launch_latent_decode(const float *q, const void *ukv, const LatentDims &dm, const LatentNew &nw,
                         const RowRing &cache, uint64_t batch, const uint32_t *pos_dev, float *out, float *scratch,
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
