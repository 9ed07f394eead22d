// Attention whose values are its keys: keys and values cost one trip to memory.  The query and key norms run
// over the whole projections, so a cached row is the keys as projected and one f32, their inverse root mean
// square.
//
//   shared_kv_prepare_kernel  prompt: normalised, weighted queries; the new rows of keys (attention: window.hip)
//   shared_kv_decode_kernel   decode: norms, the new row into the ring, a share of the ring per workgroup for
//                             all query heads of a key head, merge of the shares, gate
#include "device_utils.hpp"
#include "mixers.hpp"

namespace coeus {

static int check_dims(const SharedKvDims &dm) {
    if (dm.heads == 0 || dm.heads > 65535 || dm.kv_heads == 0 || dm.heads % dm.kv_heads || dm.d == 0 || dm.d > 256 ||
        dm.in_ld < dm.gate_off() + dm.heads * dm.d || (uint64_t)dm.heads * dm.d > (1u << 24))
        return fail(COEUS_INVALID_INPUT, "shared keys and values: sizes out of range");
    return COEUS_OK;
}

// Sum over a workgroup of 256; every thread receives it.
__device__ __forceinline__ float2 sum2_256(float a, float b, float2 *sh) {
    a = wave_sum(a);
    b = wave_sum(b);
    if ((threadIdx.x & 63) == 0) sh[threadIdx.x >> 6] = make_float2(a, b);
    __syncthreads();
    const float2 s0 = sh[0], s1 = sh[1], s2 = sh[2], s3 = sh[3];
    return make_float2((s0.x + s1.x) + (s2.x + s3.x), (s0.y + s1.y) + (s2.y + s3.y));
}
// Squares of p[0, len), 256 threads, in pieces of 4 (VEC: len % 4 == 0, p aligned) or single elements.
template <bool VEC>
__device__ __forceinline__ float squares_256(const float *__restrict__ p, uint32_t len) {
    float s = 0.f;
    if (VEC) {
        for (uint32_t i = 4 * threadIdx.x; i < len; i += 1024) {
            const float4 v = *(const float4 *)(p + i);
            s = fmaf(v.x, v.x, s); s = fmaf(v.y, v.y, s); s = fmaf(v.z, v.z, s); s = fmaf(v.w, v.w, s);
        }
    } else {
        for (uint32_t i = threadIdx.x; i < len; i += 256) s = fmaf(p[i], p[i], s);
    }
    return s;
}

// One workgroup per row.
template <bool BF16, bool VEC>
__global__ __launch_bounds__(256) void shared_kv_prepare_kernel(const float *__restrict__ proj, SharedKvDims dm,
                                                                const float *__restrict__ wqk, float eps, uint64_t n,
                                                                void *__restrict__ q, void *__restrict__ kv, uint64_t kv_rows,
                                                                uint64_t kv_off) {
    __shared__ float2 sh[4];
    const uint64_t row = blockIdx.x, dst = ((row / n) * kv_rows + kv_off + row % n) * dm.row_len();
    const uint32_t QL = dm.heads * dm.d, KL = dm.kv_heads * dm.d;
    const float *p = proj + row * dm.in_ld, *pk = p + dm.k_off();
    const float2 s = sum2_256(squares_256<VEC>(p, QL), squares_256<VEC>(pk, KL), sh);
    const float rq = 1.0f / sqrtf(s.x / (float)QL + eps), rk = 1.0f / sqrtf(s.y / (float)KL + eps);
    if (VEC) {
        auto put4 = [&](void *base, uint64_t at, const float4 &v) {
            if (BF16)
                *(uint2 *)((uint16_t *)base + at) = make_uint2((uint32_t)f32_to_bf16_bits(v.x) | (uint32_t)f32_to_bf16_bits(v.y) << 16,
                                                               (uint32_t)f32_to_bf16_bits(v.z) | (uint32_t)f32_to_bf16_bits(v.w) << 16);
            else
                *(float4 *)((float *)base + at) = v;
        };
        for (uint32_t i = 4 * threadIdx.x; i < QL; i += 1024) {
            const float4 v = *(const float4 *)(p + i), w = *(const float4 *)(wqk + i);
            put4(q, row * QL + i, make_float4(v.x * rq * w.x, v.y * rq * w.y, v.z * rq * w.z, v.w * rq * w.w));
        }
        for (uint32_t i = 4 * threadIdx.x; i < KL; i += 1024) put4(kv, dst + i, *(const float4 *)(pk + i));
    } else {
        for (uint32_t i = threadIdx.x; i < QL; i += 256) elem_store<BF16>(q, row * QL + i, p[i] * rq * wqk[i]);
        for (uint32_t i = threadIdx.x; i < KL; i += 256) elem_store<BF16>(kv, dst + i, pk[i]);
    }
    if (threadIdx.x == 0) {
        if (BF16) *(float *)((uint16_t *)kv + dst + dm.rms_off()) = rk;
        else ((float *)kv)[dst + dm.rms_off()] = rk;
    }
}

int launch_shared_kv_prepare(const float *proj, const SharedKvDims &dm, const float *wqk, float eps, uint64_t batch, uint64_t n,
                             bool bf16, void *q, void *kv, uint64_t kv_rows, uint64_t kv_off, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    if (batch == 0 || n == 0 || batch > 65535 || batch * n > 0x7fffffffull)
        return fail(COEUS_INVALID_INPUT, "shared keys and values: rows out of range");
    const bool vec = dm.d % 4 == 0 && dm.in_ld % 4 == 0;
    const dim3 grid((unsigned)(batch * n));
#define COEUS_SP(BFV, VV) \
    hipLaunchKernelGGL((shared_kv_prepare_kernel<BFV, VV>), grid, dim3(256), 0, st, proj, dm, wqk, eps, n, q, kv, kv_rows, kv_off)
    if (bf16) { if (vec) COEUS_SP(true, true); else COEUS_SP(true, false); }
    else { if (vec) COEUS_SP(false, true); else COEUS_SP(false, false); }
#undef COEUS_SP
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// ---------------------------------------------------------------- decode
constexpr uint32_t kKeyTile = 64, kMaxShares = 32;

// A lane owns eight dims of a key, LPK lanes share a key; the same registers are key and value, for HB query
// heads at once.  One workgroup of four waves per (share of the ring, key head and HB of its query heads,
// sequence).  Slots are keys in any order: a slot's distance follows from where the newest token goes.
// VEC: rows and pieces are 16-byte aligned (d % 8 == 0).
template <bool BF16, bool VEC, int LPK, int HB>
__global__ __launch_bounds__(256) void shared_kv_decode_kernel(const float *__restrict__ proj, SharedKvDims dm,
                                                               const float *__restrict__ wqk, float eps, void *ring, uint32_t cap,
                                                               const uint32_t *pos_dev, uint32_t keys_per_share, uint32_t hblocks,
                                                               float *part, uint32_t *counters, float *__restrict__ out) {
    constexpr int KPW = 64 / LPK, U = 4, DP = 8 * LPK;  // keys of a wave-wide load, loads in flight, padded dims
    constexpr float kLog2e = 1.4426950408889634f;
    __shared__ float2 sh[4];
    __shared__ float sm[4][HB], sl[4][HB], sacc[4][HB][DP];
    __shared__ uint32_t is_last;
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, share = blockIdx.x, shares = gridDim.x;
    const uint32_t H = dm.heads, G = dm.kv_heads, d = dm.d, hpg = H / G, kvh = blockIdx.y / hblocks, hb0 = blockIdx.y % hblocks * HB;
    const uint32_t h0 = kvh * hpg + hb0, nh = min((uint32_t)HB, hpg - hb0);
    const uint64_t b = blockIdx.z, RL = dm.row_len();
    const uint32_t piece = lane % LPK, sub = lane / LPK, d0 = 8 * piece, dc = min(d0, d >= 8 ? d - 8 : 0);
    const uint32_t k_begin = share * keys_per_share, k_lim = min(cap, k_begin + keys_per_share);
    const float *p = proj + b * dm.in_ld;
    struct Raw { uint4 a, b; };
    auto request = [&](uint32_t key, Raw &x, float &r) {
        const uint64_t at = (b * cap + min(key, cap - 1)) * RL;
        if (BF16) r = *(const float *)((const uint16_t *)ring + at + dm.rms_off());
        else r = ((const float *)ring)[at + dm.rms_off()];
        if (VEC && BF16) {
            x.a = *(const uint4 *)((const uint16_t *)ring + at + kvh * d + dc);
        } else if (VEC) {
            const uint4 *src = (const uint4 *)((const float *)ring + at + kvh * d + dc);
            x.a = src[0];
            x.b = src[1];
        } else {
            uint32_t v[8];
#pragma unroll
            for (int t = 0; t < 8; t++) v[t] = __float_as_uint(elem_load<BF16>(ring, at + kvh * d + min(d0 + t, d - 1)));
            x.a = make_uint4(v[0], v[1], v[2], v[3]);
            x.b = make_uint4(v[4], v[5], v[6], v[7]);
        }
    };
    auto unpack = [&](const Raw &x, float (&v)[8]) {
        if (VEC && BF16) {
            const uint32_t w[4] = {x.a.x, x.a.y, x.a.z, x.a.w};
#pragma unroll
            for (int t = 0; t < 4; t++) { v[2 * t] = __uint_as_float(w[t] << 16); v[2 * t + 1] = __uint_as_float(w[t] & 0xffff0000u); }
        } else {
            const uint32_t w[8] = {x.a.x, x.a.y, x.a.z, x.a.w, x.b.x, x.b.y, x.b.z, x.b.w};
#pragma unroll
            for (int t = 0; t < 8; t++) v[t] = __uint_as_float(w[t]);
        }
    };
    // eight floats of a row of the projection or of the weights, the lane's dims of one head (zeros behind the end)
    auto dims = [&](const float *row, float (&v)[8]) {
        if (VEC) {
            const float4 v0 = *(const float4 *)(row + dc), v1 = *(const float4 *)(row + dc + 4);
            v[0] = v0.x; v[1] = v0.y; v[2] = v0.z; v[3] = v0.w; v[4] = v1.x; v[5] = v1.y; v[6] = v1.z; v[7] = v1.w;
        } else {
#pragma unroll
            for (int t = 0; t < 8; t++) v[t] = row[min(d0 + t, d - 1)];
        }
    };
    // The projection is requested first (loads return in order and it is at hand), then the first tile, before the
    // position is known (slots not written yet hold finite values).
    const float sq_q = squares_256<VEC>(p, H * d), sq_k = squares_256<VEC>(p + dm.k_off(), G * d);
    float q[HB][8], wq[HB][8], slope[HB];
#pragma unroll
    for (int j = 0; j < HB; j++) {
        const uint32_t h = h0 + min((uint32_t)j, nh - 1);
        slope[j] = dm.slope_range == 0.f ? 0.f : kLog2e * exp2f(-dm.slope_range * (float)(h + 1) / (float)H);
        dims(p + h * d, q[j]);
        dims(wqk + h * d, wq[j]);
    }
    uint32_t base = k_begin + wave * U * KPW;
    Raw x[U];
    float r[U];
#pragma unroll
    for (int u = 0; u < U; u++) request(base + u * KPW + sub, x[u], r[u]);
    const uint32_t pos = *pos_dev, fresh = pos % cap, nv = min(pos < 0xffffffffu ? pos + 1 : pos, cap), k_end = min(nv, k_lim);
    // norms over the whole projections
    const float2 sq = sum2_256(sq_q, sq_k, sh);
    const float rq = kLog2e * dm.scale / sqrtf(sq.x / (float)(H * d) + eps), rk = 1.0f / sqrtf(sq.y / (float)(G * d) + eps);
#pragma unroll
    for (int j = 0; j < HB; j++)
#pragma unroll
        for (int t = 0; t < 8; t++) q[j][t] = d0 + t < d ? q[j][t] * rq * wq[j][t] : 0.f;  // (base 2 scores)
    float m[HB], l[HB], acc[HB][8];
#pragma unroll
    for (int j = 0; j < HB; j++) {
        m[j] = -1e30f;  // (finite: a tile may hold no key)
        l[j] = 0.f;
#pragma unroll
        for (int t = 0; t < 8; t++) acc[j][t] = 0.f;
    }
    for (; base < k_end; base += 4 * U * KPW) {  // wave-uniform
        if (fresh >= base && fresh < base + U * KPW) {  // wave-uniform: the new token's row comes from the projection
#pragma unroll
            for (int u = 0; u < U; u++) {
                const uint32_t key = base + u * KPW + sub;
                if (key != fresh) continue;
                const uint64_t at = (b * cap + key) * RL;
                float nk[8];
                uint32_t w[8];
                dims(p + dm.k_off() + kvh * d, nk);
#pragma unroll
                for (int t = 0; t < 8; t++) {
                    w[t] = BF16 ? (uint32_t)f32_to_bf16_bits(nk[t]) : __float_as_uint(nk[t]);
                    if (hb0 == 0 && d0 + t < d) {
                        if (BF16) ((uint16_t *)ring)[at + kvh * d + d0 + t] = (uint16_t)w[t];
                        else ((float *)ring)[at + kvh * d + d0 + t] = nk[t];
                    }
                }
                if (VEC && BF16) {
                    x[u].a = make_uint4(w[0] | w[1] << 16, w[2] | w[3] << 16, w[4] | w[5] << 16, w[6] | w[7] << 16);
                } else {
                    const uint32_t sft = BF16 ? 16 : 0;
                    x[u].a = make_uint4(w[0] << sft, w[1] << sft, w[2] << sft, w[3] << sft);
                    x[u].b = make_uint4(w[4] << sft, w[5] << sft, w[6] << sft, w[7] << sft);
                }
                r[u] = rk;
                if (blockIdx.y == 0 && piece == 0) {
                    if (BF16) *(float *)((uint16_t *)ring + at + dm.rms_off()) = rk;
                    else ((float *)ring)[at + dm.rms_off()] = rk;
                }
            }
        }
        float v[U][8], s[HB][U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            unpack(x[u], v[u]);
            const uint32_t key = base + u * KPW + sub;
            const float dist = (float)(fresh >= key ? fresh - key : fresh + cap - key);
#pragma unroll
            for (int j = 0; j < HB; j++) {
                float dot = 0.f;
#pragma unroll
                for (int t = 0; t < 8; t++) dot = fmaf(q[j][t], v[u][t], dot);
                if (LPK == 8) dot = group_sum<8>(dot);
                else dot = group_sum<16>(dot);
                if (LPK == 32) dot = xor16_sum(dot);
                s[j][u] = key < k_end ? fmaf(dot, r[u], -slope[j] * dist) : -INFINITY;
            }
        }
        const uint32_t next = base + 4 * U * KPW;
        if (next < k_end)
#pragma unroll
            for (int u = 0; u < U; u++) request(next + u * KPW + sub, x[u], r[u]);
#pragma unroll
        for (int j = 0; j < HB; j++) {
            float top = s[j][0];
#pragma unroll
            for (int u = 1; u < U; u++) top = fmaxf(top, s[j][u]);
            const float m_new = fmaxf(m[j], wave_max(top)), corr = __builtin_amdgcn_exp2f(m[j] - m_new);
            l[j] *= corr;
#pragma unroll
            for (int t = 0; t < 8; t++) acc[j][t] *= corr;
#pragma unroll
            for (int u = 0; u < U; u++) {
                const float w = __builtin_amdgcn_exp2f(s[j][u] - m_new);
                l[j] += w;
#pragma unroll
                for (int t = 0; t < 8; t++) acc[j][t] = fmaf(w, v[u][t], acc[j][t]);
            }
            m[j] = m_new;
        }
    }
    // keys of a wave, then its waves
#pragma unroll
    for (int j = 0; j < HB; j++) {
        const float lw = wave_sum(l[j]) * (1.0f / LPK);
        if (lane == 0) { sm[wave][j] = m[j]; sl[wave][j] = lw; }
#pragma unroll
        for (int t = 0; t < 8; t++) {
            float a = acc[j][t];
            if (LPK == 8) a += dpp_f32<DPP_ROW_ROR8>(a);
            if (LPK <= 16) a = xor16_sum(a);
            a = xor32_sum(a);
            if (lane < LPK) sacc[wave][j][d0 + t] = a;
        }
    }
    __syncthreads();
    auto gated = [&](uint32_t h, uint32_t c, float v) {
        out[(b * H + h) * d + c] = v * fast_sigmoid(p[dm.gate_off() + h * d + c]);
    };
    for (uint32_t it = tid; it < nh * d; it += 256) {
        const uint32_t j = it / d, c = it % d;
        const float mm = fmaxf(fmaxf(sm[0][j], sm[1][j]), fmaxf(sm[2][j], sm[3][j]));
        float lt = 0.f, a = 0.f;
#pragma unroll
        for (int w = 0; w < 4; w++) {
            const float f = __builtin_amdgcn_exp2f(sm[w][j] - mm);
            lt = fmaf(sl[w][j], f, lt);
            a = fmaf(sacc[w][j][c], f, a);
        }
        if (shares == 1) {
            gated(h0 + j, c, a / lt);
        } else {
            float *rec = part + ((b * H + h0 + j) * shares + share) * (d + 2);
            if (c == 0) {
                __hip_atomic_store(rec, mm, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                __hip_atomic_store(rec + 1, lt, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
            }
            __hip_atomic_store(rec + 2 + c, a, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        }
    }
    if (shares == 1) return;
    // The share that arrives last merges all of them (attn_decode_kernel's protocol: device-scope stores that
    // have completed before the barrier, then a relaxed counter).
    __builtin_amdgcn_s_waitcnt(0);
    __syncthreads();
    if (tid == 0) {
        uint32_t *cnt = counters + b * gridDim.y + blockIdx.y;
        is_last = __hip_atomic_fetch_add(cnt, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == shares - 1;
        if (is_last) __hip_atomic_store(cnt, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    __syncthreads();
    if (!is_last) return;
    const float *rec = part + (b * H + h0) * shares * (d + 2);
    for (uint32_t it = tid; it < nh * d; it += 256) {
        const uint32_t j = it / d, c = it % d;
        const float *q0 = rec + (uint64_t)j * shares * (d + 2);
        float mm = -INFINITY, lt = 0.f, a = 0.f;
        for (uint32_t s0 = 0; s0 < shares; s0 += 16) {  // sixteen records in one trip
            float ym[16], yl[16], y[16];
#pragma unroll
            for (uint32_t s = 0; s < 16; s++) {
                const float *qs = q0 + (uint64_t)min(s0 + s, shares - 1) * (d + 2);
                ym[s] = __hip_atomic_load(qs, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                yl[s] = __hip_atomic_load(qs + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                y[s] = __hip_atomic_load(qs + 2 + c, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
            }
            float top = mm;
#pragma unroll
            for (uint32_t s = 0; s < 16; s++) top = fmaxf(top, ym[s]);
            const float corr = __builtin_amdgcn_exp2f(mm - top);
            lt *= corr;
            a *= corr;
            mm = top;
#pragma unroll
            for (uint32_t s = 0; s < 16; s++) {
                if (s0 + s >= shares) break;
                const float f = __builtin_amdgcn_exp2f(ym[s] - mm);
                lt = fmaf(yl[s], f, lt);
                a = fmaf(y[s], f, a);
            }
        }
        gated(h0 + j, c, a / lt);
    }
}

struct DecodePlan {
    uint32_t hb, hblocks, shares, per_share;
    bool vec;
};
static DecodePlan decode_plan(const SharedKvDims &dm, const RowRing &ring, uint64_t batch) {
    DecodePlan p;
    const uint32_t hpg = dm.heads / dm.kv_heads;
    p.vec = dm.d % 8 == 0 && dm.in_ld % 4 == 0;
    p.hb = !p.vec || hpg == 2 ? 2 : hpg == 1 ? 1 : hpg <= 4 ? 4 : 8;
    p.hblocks = (uint32_t)ceil_div(hpg, p.hb);
    // enough workgroups to fill the chip, at least a tile of keys each
    const uint64_t tiles = ceil_div(ring.cap, kKeyTile), wgs = (uint64_t)dm.kv_heads * p.hblocks * batch;
    uint64_t s = std::max<uint64_t>(1, 1024 / wgs);
    s = std::min<uint64_t>(s, std::min<uint64_t>(tiles, kMaxShares));
    p.per_share = (uint32_t)round_up(ceil_div(ring.cap, s), kKeyTile);
    p.shares = (uint32_t)ceil_div(ring.cap, p.per_share);
    return p;
}

uint64_t shared_kv_decode_scratch_bytes(const SharedKvDims &dm, const RowRing &ring, uint64_t batch) {
    return batch * dm.heads * decode_plan(dm, ring, batch).shares * (dm.d + 2ull) * 4;
}
uint64_t shared_kv_decode_counters(const SharedKvDims &dm, uint64_t batch) { return batch * dm.heads; }

int launch_shared_kv_decode(const float *proj, const SharedKvDims &dm, const float *wqk, float eps, const RowRing &ring,
                            uint64_t batch, const uint32_t *pos_dev, float *out, float *scratch, uint64_t scratch_bytes,
                            uint32_t *counters, uint64_t n_counters, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    if (batch == 0 || batch > 65535 || !pos_dev || ring.cap == 0 || (dm.window && ring.cap > dm.window) ||
        !scratch || scratch_bytes < shared_kv_decode_scratch_bytes(dm, ring, batch) || !counters ||
        n_counters < shared_kv_decode_counters(dm, batch))
        return fail(COEUS_INVALID_INPUT, "shared keys and values: bad ring, batch or scratch");
    const DecodePlan pl = decode_plan(dm, ring, batch);
    const dim3 grid(pl.shares, dm.kv_heads * pl.hblocks, (unsigned)batch);
#define COEUS_SD(BFV, VV, LV, HV)                                                                                           \
    hipLaunchKernelGGL((shared_kv_decode_kernel<BFV, VV, LV, HV>), grid, dim3(256), 0, st, proj, dm, wqk, eps, ring.c, ring.cap, \
                       pos_dev, pl.per_share, pl.hblocks, scratch, counters, out)
#define COEUS_SDL(BFV, VV, HV) \
    do { if (dm.d <= 64) COEUS_SD(BFV, VV, 8, HV); else if (dm.d <= 128) COEUS_SD(BFV, VV, 16, HV); else COEUS_SD(BFV, VV, 32, HV); } while (0)
#define COEUS_SDH(BFV)                                                                                             \
    do {                                                                                                           \
        if (!pl.vec) COEUS_SDL(BFV, false, 2);                                                                     \
        else if (pl.hb == 1) COEUS_SDL(BFV, true, 1);                                                              \
        else if (pl.hb == 2) COEUS_SDL(BFV, true, 2);                                                              \
        else if (pl.hb == 4) COEUS_SDL(BFV, true, 4);                                                              \
        else COEUS_SDL(BFV, true, 8);                                                                              \
    } while (0)
    if (ring.bf16) COEUS_SDH(true);
    else COEUS_SDH(false);
#undef COEUS_SDH
#undef COEUS_SDL
#undef COEUS_SD
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

}  // namespace coeus
