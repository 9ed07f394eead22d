// Gated delta rule: a linear recurrence with a matrix state per head, its short convolutions and its
// gated output norm.
//
//   delta_prepare_kernel  prompt: convolution + SiLU of q, k, v, unit norms, step sizes and decays
//   delta_ring_kernel     prompt: the last projections of every sequence into the convolution ring
//   delta_scan_kernel     short prompts: the recurrence token by token, state in registers
//   delta_chunk_kernel    prompt: everything of a chunk of 64 tokens that does not need the state
//   delta_carry_kernel    prompt: the state through the chunks, on the matrix cores
//   delta_gate_kernel     prompt: per-head RMS norm of the read-out times silu(gate)
//   delta_step_kernel     decode: all of it for one token per sequence
//
// Everything behind the projections is f32: convolutions, norms, gates, state and products.
#include "device_utils.hpp"
#include "mixers.hpp"

namespace coeus {

constexpr float kUnitEps = 1e-6f;  // under the root of the unit norms of q and k
constexpr uint32_t kMaxTaps = 16;

uint32_t delta_padded_dim(uint32_t d) { return (uint32_t)round_up(d, 16); }

__device__ __forceinline__ float softplus(float x) { return x > 20.0f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
// log of the decay: -exp(A_log) softplus(a + dt_bias)
__device__ __forceinline__ float log_decay(float a, float exp_a, float dt_bias) { return -exp_a * softplus(a + dt_bias); }

// Input of the convolution `back` positions before row i of sequence b (position pos0 + i): a row of this
// prompt, a slot of the ring, or zero in front of the sequence.
__device__ __forceinline__ float conv_input(const float *__restrict__ proj, const float *__restrict__ ring, uint32_t taps,
                                            uint32_t channels, uint64_t in_ld, uint64_t b, uint64_t n, uint64_t i,
                                            uint64_t pos0, uint32_t back, uint32_t c) {
    if (back <= i) return proj[(b * n + i - back) * in_ld + c];
    if (back <= pos0 + i) return ring[(b * taps + (pos0 + i - back) % taps) * channels + c];
    return 0.f;
}

// One wave per (strip of rows, unit).  A unit is a head of q or k, 256 channels of v, or the gates of all heads;
// lane l owns channels l, l + 64, .. of it.  T taps (1 .. 4) slide through registers, so that every input is
// read once; four rows are requested at a time.
constexpr uint32_t kStrip = 16;
template <int T>
__global__ __launch_bounds__(256) void delta_prepare_kernel(const float *__restrict__ proj, DeltaDims dm, DeltaParams pr,
                                                            const float *__restrict__ ring, uint64_t n, uint64_t pos0,
                                                            uint32_t dp, DeltaOperands op) {
    const uint32_t lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6);
    const uint64_t b = blockIdx.z, i0 = (uint64_t)blockIdx.x * kStrip, i1 = min(i0 + kStrip, n);
    const uint32_t KH = dm.kv_heads, H = dm.heads, C = dm.channels(), V = H * dm.e, vunits = (V + 255) / 256;
    if (unit > 2 * KH + vunits) return;
    if (unit == 2 * KH + vunits) {
        for (uint64_t t = lane; t < (i1 - i0) * H; t += 64) {
            const uint64_t row = b * n + i0 + t / H;
            const uint32_t h = (uint32_t)(t % H);
            const float *p = proj + row * dm.in_ld;
            op.beta[row * H + h] = sigmoid(p[dm.beta_off() + h]);
            op.lg[row * H + h] = log_decay(p[dm.decay_off() + h], pr.exp_a[h], pr.dt_bias[h]);
        }
        return;
    }
    const bool is_v = unit >= 2 * KH;
    const uint32_t vu = unit - 2 * KH, c0 = is_v ? 2 * KH * dm.d + 256 * vu : unit * dm.d;
    const uint32_t len = is_v ? min(256u, V - 256 * vu) : dm.d;  // d <= 256
    float *dst = is_v ? op.v + 256 * vu : (unit < KH ? op.q + unit * dp : op.k + (unit - KH) * dp);
    const uint64_t dst_ld = is_v ? V : (uint64_t)KH * dp;
    const uint32_t dst_len = is_v ? len : dp;  // (q and k: zeros behind d)
    const float post = unit < KH ? 1.0f / sqrtf((float)dm.d) : 1.0f;
    constexpr int TT = T ? T : 1;
    float w[TT][4], x[TT][4];
#pragma unroll
    for (int j = 0; j < T; j++)
#pragma unroll
        for (int s = 0; s < 4; s++) {
            const uint32_t c = lane + 64 * s;
            w[j][s] = c < len ? pr.conv[(uint64_t)j * C + c0 + c] : 0.f;
            x[j][s] = j + 1 < T && c < len ? conv_input(proj, ring, dm.taps, C, dm.in_ld, b, n, i0, pos0, T - 1 - j, c0 + c) : 0.f;
        }
    for (uint64_t ib = i0; ib < i1; ib += 4) {
        float in[4][4];
#pragma unroll
        for (int u = 0; u < 4; u++)
#pragma unroll
            for (int s = 0; s < 4; s++) {
                const uint32_t c = lane + 64 * s;
                in[u][s] = c < len && ib + u < i1 ? proj[(b * n + ib + u) * dm.in_ld + c0 + c] : 0.f;
            }
#pragma unroll
        for (int u = 0; u < 4; u++) {
            if (ib + u >= i1) break;
            float y[4], s2 = 0.f;
#pragma unroll
            for (int s = 0; s < 4; s++) {
                float acc = 0.f;
                if (T) {
                    x[TT - 1][s] = in[u][s];
#pragma unroll
                    for (int j = 0; j < T; j++) acc = fmaf(w[j][s], x[j][s], acc);
#pragma unroll
                    for (int j = 0; j + 1 < T; j++) x[j][s] = x[j + 1][s];
                } else if (lane + 64 * s < len) {  // any number of taps
                    for (uint32_t j = 0; j < dm.taps; j++)
                        acc = fmaf(pr.conv[(uint64_t)j * C + c0 + lane + 64 * s],
                                   conv_input(proj, ring, dm.taps, C, dm.in_ld, b, n, ib + u, pos0, dm.taps - 1 - j, c0 + lane + 64 * s), acc);
                }
                y[s] = fast_silu(acc);
                s2 = fmaf(y[s], y[s], s2);
            }
            const float r = is_v ? 1.0f : post / sqrtf(wave_sum(s2) + kUnitEps);
            float *o = dst + (b * n + ib + u) * dst_ld;
#pragma unroll
            for (int s = 0; s < 4; s++)
                if (lane + 64 * s < dst_len) o[lane + 64 * s] = y[s] * r;
        }
    }
}

static int check_dims(const DeltaDims &dm) {
    if (dm.heads == 0 || dm.kv_heads == 0 || dm.heads % dm.kv_heads || dm.d == 0 || dm.d > 256 || dm.e == 0 || dm.e > 1024 ||
        dm.taps == 0 || dm.taps > kMaxTaps || dm.in_ld < dm.decay_off() + dm.heads)
        return fail(COEUS_INVALID_INPUT, "delta rule: sizes out of range");
    return COEUS_OK;
}

static int check_rows(uint64_t batch, uint64_t n) {
    if (batch == 0 || n == 0 || batch > 65535 || batch * n > 0x7fffffffull)
        return fail(COEUS_INVALID_INPUT, "delta rule: %llu x %llu rows out of range", (unsigned long long)batch, (unsigned long long)n);
    return COEUS_OK;
}

int launch_delta_prepare(const float *proj, const DeltaDims &dm, const DeltaParams &pr, const DeltaState &state,
                         uint64_t batch, uint64_t n, uint64_t pos0, const DeltaOperands &op, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    COEUS_TRY(check_rows(batch, n));
    const dim3 grid((unsigned)ceil_div(n, kStrip), (unsigned)ceil_div(2 * dm.kv_heads + ceil_div((uint64_t)dm.heads * dm.e, 256) + 1, 4),
                    (unsigned)batch);
#define COEUS_DP(TV) \
    hipLaunchKernelGGL(delta_prepare_kernel<TV>, grid, dim3(256), 0, st, proj, dm, pr, state.ring, n, pos0, delta_padded_dim(dm.d), op)
    switch (dm.taps) {
        case 1: COEUS_DP(1); break;
        case 2: COEUS_DP(2); break;
        case 3: COEUS_DP(3); break;
        case 4: COEUS_DP(4); break;
        default: COEUS_DP(0); break;
    }
#undef COEUS_DP
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

__global__ __launch_bounds__(256) void delta_ring_kernel(const float *__restrict__ proj, DeltaDims dm, float *ring,
                                                         uint64_t n, uint64_t pos0) {
    const uint32_t c = blockIdx.x * 256 + threadIdx.x, C = dm.channels();
    const uint64_t b = blockIdx.y;
    if (c >= C) return;
    const uint64_t m = n < dm.taps ? n : dm.taps;
    for (uint64_t i = n - m; i < n; i++)
        ring[(b * dm.taps + (pos0 + i) % dm.taps) * C + c] = proj[(b * n + i) * dm.in_ld + c];
}

int launch_delta_ring(const float *proj, const DeltaDims &dm, const DeltaState &state, uint64_t batch, uint64_t n,
                      uint64_t pos0, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    COEUS_TRY(check_rows(batch, n));
    hipLaunchKernelGGL(delta_ring_kernel, dim3((unsigned)ceil_div(dm.channels(), 256), (unsigned)batch), dim3(256), 0, st,
                       proj, dm, state.ring, n, pos0);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// ---------------------------------------------------------------- the recurrence, token by token
// 16 lanes share a column of S (lane s of 16 holds rows R s .. R s + R - 1), 4 columns per wave, 16 per
// workgroup.  Columns never meet, so the heads' columns spread over the chip; the operands of token
// t + 1 are requested before token t is computed.
template <int R>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaDims dm, DeltaOperands op, float *state, uint64_t n,
                                                         float *__restrict__ o) {
    constexpr uint32_t dp = 16 * R;
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, sub = lane & 15;
    const uint32_t col = blockIdx.x * 16 + wave * 4 + (lane >> 4), colc = min(col, dm.e - 1);
    const uint32_t h = blockIdx.y, H = dm.heads, KH = dm.kv_heads, hk = h / (H / KH);
    const uint64_t b = blockIdx.z;
    float *sp = state + ((b * H + h) * dm.d) * dm.e + colc;
    float s[R];
#pragma unroll
    for (int r = 0; r < R; r++) s[r] = sub * R + r < dm.d ? sp[(uint64_t)(sub * R + r) * dm.e] : 0.f;
    const float *kp = op.k + ((b * n) * KH + hk) * dp + sub * R, *qp = op.q + ((b * n) * KH + hk) * dp + sub * R;
    const float *vp = op.v + ((b * n) * H + h) * dm.e + colc, *bp = op.beta + b * n * H + h, *gp = op.lg + b * n * H + h;
    float k[R], q[R], v, be, lg;
    auto fetch = [&](uint64_t t) {
#pragma unroll
        for (int r = 0; r < R; r++) { k[r] = kp[t * KH * dp + r]; q[r] = qp[t * KH * dp + r]; }
        v = vp[t * H * dm.e]; be = bp[t * H]; lg = gp[t * H];
    };
    fetch(0);
    for (uint64_t t = 0; t < n; t++) {
        float kc[R], qc[R];
#pragma unroll
        for (int r = 0; r < R; r++) { kc[r] = k[r]; qc[r] = q[r]; }
        const float vc = v, bc = be, g = expf(lg);
        fetch(t + 1 < n ? t + 1 : t);
        float dot = 0.f;
#pragma unroll
        for (int r = 0; r < R; r++) { s[r] *= g; dot = fmaf(s[r], kc[r], dot); }
        const float u = bc * (vc - group_sum<16>(dot));
        float out = 0.f;
#pragma unroll
        for (int r = 0; r < R; r++) { s[r] = fmaf(kc[r], u, s[r]); out = fmaf(s[r], qc[r], out); }
        out = group_sum<16>(out);
        if (sub == 0 && col < dm.e) o[((b * n + t) * H + h) * dm.e + col] = out;
    }
    if (col < dm.e)
#pragma unroll
        for (int r = 0; r < R; r++)
            if (sub * R + r < dm.d) sp[(uint64_t)(sub * R + r) * dm.e] = s[r];
}

// ---------------------------------------------------------------- the recurrence, chunk by chunk
// With G_i the sum of the log decays of a chunk's tokens up to i and S0 the state in front of it:
//   (I + A) U = beta (V - e^G K S0),   A_ij = beta_i e^(G_i - G_j) (k_i . k_j) for j < i
//   O   = e^G Q S0 + P U,              P_ij = e^(G_i - G_j) (q_i . k_j) for j <= i
//   S_C = e^(G_C) S0 + K^T (e^(G_C - G) U)
// U = V' - W S0 where (I + A) [W | V'] = beta [e^G K | V] is solved by forward substitution: every exponent
// is of a sum of log decays that lie between two tokens, so nothing overflows however fast the state decays.
// delta_chunk_kernel does everything that does not need S0, for all chunks at once; delta_carry_kernel
// then walks the chunks with one workgroup per head and 16 columns of S.  All products are f32
// (v_mfma_f32_16x16x4_f32, or fused multiply-adds in the substitution).
//
// A reduction index of a matrix instruction is only a label: instruction i of a 16-wide step sums over
// {4 g + i : g = lane / 16}, so a lane's operand pieces are 16 consecutive bytes, and an accumulator
// tile (rows 4 g + i) is the next product's right operand as it stands.
// The chunk operands lie in memory in that order, [16-row tile][16-wide step][lane][4]: a wave's load is
// 1 KiB in a row (operand_index); V' as accumulator tiles, [16-row tile][16 columns][lane][4].
constexpr uint32_t kChunk = 64;
constexpr uint64_t kSegment = 4096;  // tokens whose chunk operands are in memory at once

__device__ __forceinline__ uint32_t operand_index(uint32_t row, uint32_t k, uint32_t steps) {
    return (((row >> 4) * steps + (k >> 4)) * 64 + ((k >> 2) & 3) * 16 + (row & 15)) * 4 + (k & 3);
}

struct ChunkBuf {
    float *w, *vp, *p, *eg, *ed, *kt, *q;
    uint32_t chunks;  // per sequence
};
static uint32_t chunk_dim(uint32_t d) { return (uint32_t)round_up(d, 64); }
static uint64_t chunk_floats(const DeltaDims &dm, uint64_t batch, uint64_t chunks) {
    const uint64_t dq = chunk_dim(dm.d);
    return batch * chunks * (dm.heads * (kChunk * (dq + round_up(dm.e, 16) + kChunk) + 2 * kChunk) + 2ull * dm.kv_heads * dq * kChunk);
}

// One workgroup of 256 per (chunk, head, sequence).  dp: row length of the prepared q and k.
template <int NT>  // 16-wide steps of the padded query/key size
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaDims dm, DeltaOperands op, uint32_t dp, uint64_t n,
                                                          uint64_t t0, uint64_t seg, ChunkBuf cb) {
    constexpr uint32_t DQ = 16 * NT, KLD = DQ + 4, ALD = kChunk + 4, TLD = 20;
    extern __shared__ float lds[];
    float *kl = lds, *al = kl + kChunk * KLD, *tl = al + kChunk * ALD;  // K [64][KLD], A [64][ALD], -T [64][TLD]
    __shared__ float gs[kChunk], es[kChunk], bs[kChunk];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const uint32_t chunk = blockIdx.x, h = blockIdx.y, H = dm.heads, KH = dm.kv_heads, hk = h / (H / KH);
    const uint64_t b = blockIdx.z, tok0 = t0 + (uint64_t)chunk * kChunk, left = seg - (uint64_t)chunk * kChunk;
    const uint32_t live = left < kChunk ? (uint32_t)left : kChunk;  // tokens behind the end: beta = 0, k = q = v = 0
    const uint64_t row0 = b * n + tok0, ci = ((b * H + h) * cb.chunks + chunk);
    // Q and K^T in operand order are written once per query/key head, by the first of the heads that share it
    const bool first = h % (H / KH) == 0;
    const uint64_t ki = ((b * KH + hk) * cb.chunks + chunk) * DQ * kChunk;
    if (wave == 0) {
        float lg = lane < live ? op.lg[(row0 + lane) * H + h] : 0.f;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float o = __shfl_up(lg, off, 64);
            if ((int)lane >= off) lg += o;
        }
        const float be = lane < live ? op.beta[(row0 + lane) * H + h] : 0.f;
        gs[lane] = lg;
        es[lane] = expf(lg);
        bs[lane] = be;
        cb.eg[ci * kChunk + lane] = es[lane];
        cb.ed[ci * kChunk + lane] = expf(__shfl(lg, 63, 64) - lg);
    }
    for (uint32_t i = tid; i < kChunk * (DQ / 4); i += 256) {
        const uint32_t r = i / (DQ / 4), q4 = 4 * (i % (DQ / 4));
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (r < live && q4 < dp) v = *(const float4 *)(op.k + ((row0 + r) * KH + hk) * dp + q4);
        *(float4 *)(kl + r * KLD + q4) = v;
    }
    __syncthreads();
    // 16 x 16 tiles of K K^T and Q K^T up to the diagonal, rows block by block, five tiles a wave: (K, rows
    // 3) + (Q, 0), (Q, 3) + (K, 0), (K, 2) + (Q, 1), (Q, 2) + (K, 1)
#pragma unroll
    for (int part = 0; part < 2; part++) {
        const uint32_t blk = part == 0 ? 3 - (wave >> 1) : wave >> 1;
        const bool is_q = ((wave & 1) ^ part) != 0;
        const uint32_t r = 16 * blk + c;
        float4 ra[NT];
#pragma unroll
        for (int m = 0; m < NT; m++) {
            const uint32_t q4 = 16 * m + 4 * g;
            if (!is_q) {
                ra[m] = *(const float4 *)(kl + r * KLD + q4);
            } else {
                ra[m] = make_float4(0.f, 0.f, 0.f, 0.f);
                if (r < live && q4 < dp) ra[m] = *(const float4 *)(op.q + ((row0 + r) * KH + hk) * dp + q4);
                if (first) *(float4 *)(cb.q + ki + ((blk * NT + m) * 64 + lane) * 4) = ra[m];
            }
        }
        for (uint32_t t = 0; t < 4; t++) {
            float4_t acc = {0.f, 0.f, 0.f, 0.f};
            if (t <= blk) {
#pragma unroll
                for (int m = 0; m < NT; m++) acc = mfma4(ra[m], *(const float4_t *)(kl + (16 * t + c) * KLD + 16 * m + 4 * g), acc);
            }
            const uint32_t j = 16 * t + c;
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const uint32_t ri = 16 * blk + 4 * g + i;
                const float e = j <= ri ? expf(gs[ri] - gs[j]) * acc[i] : 0.f;
                if (is_q) cb.p[ci * kChunk * kChunk + operand_index(ri, j, 4)] = e;
                else al[ri * ALD + j] = j < ri ? bs[ri] * e : 0.f;
            }
        }
    }
    __syncthreads();
    // Forward substitution by blocks of 16 tokens: X_I = T_I (R_I - sum_J<I A_IJ X_J) with T_I the inverse of the
    // diagonal block I + A_II, which wave I finds column by column.  -T is kept: the products accumulate A X - R.
    {
        float t[16];
#pragma unroll
        for (int i = 0; i < 16; i++) {
            float x = i == (int)c ? 1.f : 0.f;
#pragma unroll
            for (int k = 0; k < i; k++) x = fmaf(-al[(16 * wave + i) * ALD + 16 * wave + k], t[k], x);
            t[i] = x;
        }
        if (lane < 16)
#pragma unroll
            for (int i = 0; i < 16; i++) tl[(16 * wave + i) * TLD + lane] = -t[i];
    }
    __syncthreads();
    float4 ta[4], aa[6];
#pragma unroll
    for (int i = 0; i < 4; i++) ta[i] = *(const float4 *)(tl + (16 * i + c) * TLD + 4 * g);
#pragma unroll
    for (int i = 1, k = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < i; j++, k++) aa[k] = *(const float4 *)(al + (16 * i + c) * ALD + 16 * j + 4 * g);
    const uint32_t tiles = NT + (dm.e + 15) / 16;
    for (uint32_t t = wave; t < tiles; t += 4) {
        const bool is_w = t < NT;
        const uint32_t col = 16 * (is_w ? t : t - NT) + c;
        float4_t x[4];
#pragma unroll
        for (int i = 0; i < 4; i++)
#pragma unroll
            for (int k = 0; k < 4; k++) {
                const uint32_t r = 16 * i + 4 * g + k;
                float v = 0.f;
                if (is_w) v = es[r] * kl[r * KLD + col];
                else if (r < live && col < dm.e) v = op.v[((row0 + r) * H + h) * dm.e + col];
                x[i][k] = -bs[r] * v;
            }
#pragma unroll
        for (int i = 0, k = 0; i < 4; i++) {
#pragma unroll
            for (int j = 0; j < i; j++, k++) x[i] = mfma4(aa[k], x[j], x[i]);
            x[i] = mfma4(ta[i], x[i], float4_t{0.f, 0.f, 0.f, 0.f});
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            if (is_w) {
#pragma unroll
                for (int k = 0; k < 4; k++) cb.w[ci * kChunk * DQ + operand_index(16 * i + 4 * g + k, col, NT)] = x[i][k];
            } else {
                *(float4_t *)(cb.vp + ci * kChunk * 16 * (tiles - NT) + ((i * (tiles - NT) + t - NT) * 64 + lane) * 4) = x[i];
            }
        }
    }
    if (first)
        for (uint32_t i = tid; i < DQ * kChunk; i += 256) {
            const uint32_t dim = i % DQ, tk = i / DQ;
            cb.kt[ki + operand_index(dim, tk, 4)] = kl[tk * KLD + dim];
        }
}

// One workgroup of eight waves per (16 columns of S, head, sequence).  Waves 0-3 carry the state: wave w keeps
// rows 16 QW w .. of it in accumulators, computes tokens 16 w .. of U, and hands both to the others through
// LDS.  Waves 4-7, one on each SIMD beside them, compute the outputs, which nobody waits for: they fill the
// matrix cores while the state's waves exchange their pieces.
template <int QW>
__global__ __launch_bounds__(512) void delta_carry_kernel(DeltaDims dm, uint64_t n, uint64_t t0, uint64_t seg,
                                                          ChunkBuf cb, float *state, float *__restrict__ o,
                                                          uint32_t blocks, uint32_t units) {
    constexpr uint32_t NT = 4 * QW, DQ = 16 * NT;
    __shared__ float4_t sl[2][NT][64], ul[2][4][64];
    const uint32_t lane = threadIdx.x & 63, wave = (threadIdx.x >> 6) & 3, c = lane & 15, g = lane >> 4;
    const bool carries = threadIdx.x < 256;
    const uint32_t H = dm.heads, KH = dm.kv_heads;
    // all column blocks of a head on one XCD (consecutive workgroups go round the 8 XCDs): its chunk
    // operands are fetched into one L2
    uint32_t blk = blockIdx.x % blocks, unit = blockIdx.x / blocks;
    if ((units & 7) == 0) {
        const uint32_t idx = blockIdx.x >> 3;
        blk = idx % blocks;
        unit = (blockIdx.x & 7) + 8 * (idx / blocks);
    }
    const uint32_t h = unit % H, hk = h / (H / KH);
    const uint64_t b = unit / H;
    const uint32_t col = blk * 16 + c, colc = min(col, dm.e - 1);
    const uint32_t chunks = (uint32_t)((seg + kChunk - 1) / kChunk);
    const uint64_t ci0 = (b * H + h) * cb.chunks, ki0 = (b * KH + hk) * cb.chunks;
    // A chunk's operands are requested as soon as the registers of the chunk before are free.
    if (carries) {
        __builtin_amdgcn_s_setprio(2);  // the next chunk waits for these waves
        float *sp = state + ((b * H + h) * (uint64_t)dm.d) * dm.e + colc;
        float4_t s[QW];
#pragma unroll
        for (int t = 0; t < QW; t++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const uint32_t r = 16 * (QW * wave + t) + 4 * g + i;
                s[t][i] = r < dm.d ? sp[(uint64_t)r * dm.e] : 0.f;
            }
        float4 wa[NT], ka[QW][4], ed4[4];
        float4_t v4;
        float egc;
        auto fetch_w = [&](uint32_t ch) {
            const float4 *wp = (const float4 *)(cb.w + (ci0 + ch) * kChunk * DQ) + wave * NT * 64 + lane;
#pragma unroll
            for (uint32_t m = 0; m < NT; m++) wa[m] = wp[64 * m];
            v4 = *(const float4_t *)(cb.vp + (ci0 + ch) * kChunk * 16 * blocks + ((wave * blocks + blk) * 64 + lane) * 4);
        };
        auto fetch_k = [&](uint32_t ch) {
            const float4 *kp = (const float4 *)(cb.kt + (ki0 + ch) * kChunk * DQ) + QW * wave * 4 * 64 + lane;
#pragma unroll
            for (int t = 0; t < 4; t++) {
#pragma unroll
                for (int u = 0; u < QW; u++) ka[u][t] = kp[(4 * u + t) * 64];
                ed4[t] = *(const float4 *)(cb.ed + (ci0 + ch) * kChunk + 16 * t + 4 * g);
            }
            egc = cb.eg[(ci0 + ch) * kChunk + kChunk - 1];
        };
        fetch_w(0);
        fetch_k(0);
        for (uint32_t ch = 0; ch < chunks; ch++) {
            const uint32_t buf = ch & 1, next = ch + 1 < chunks ? ch + 1 : ch;
#pragma unroll
            for (int t = 0; t < QW; t++) sl[buf][QW * wave + t][lane] = s[t];
            lds_barrier();
            float4_t a0 = {0.f, 0.f, 0.f, 0.f}, a1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (uint32_t m = 0; m < NT; m += 2) {
                a0 = mfma4(wa[m], sl[buf][m][lane], a0);
                a1 = mfma4(wa[m + 1], sl[buf][m + 1][lane], a1);
            }
            ul[buf][wave][lane] = v4 - (a0 + a1);
            __builtin_amdgcn_sched_barrier(0);
            fetch_w(next);
            __builtin_amdgcn_sched_barrier(0);
            lds_barrier();
#pragma unroll
            for (int w = 0; w < QW; w++) s[w] *= egc;
#pragma unroll
            for (int t = 0; t < 4; t++) {
                float4_t ub = ul[buf][t][lane];
                ub[0] *= ed4[t].x; ub[1] *= ed4[t].y; ub[2] *= ed4[t].z; ub[3] *= ed4[t].w;
#pragma unroll
                for (int w = 0; w < QW; w++) s[w] = mfma4(ka[w][t], ub, s[w]);
            }
            __builtin_amdgcn_sched_barrier(0);
            fetch_k(next);
            __builtin_amdgcn_sched_barrier(0);
        }
        if (col < dm.e)
#pragma unroll
            for (int t = 0; t < QW; t++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const uint32_t r = 16 * (QW * wave + t) + 4 * g + i;
                    if (r < dm.d) sp[(uint64_t)r * dm.e] = s[t][i];
                }
    } else {
        constexpr uint32_t SPLIT = (3 * NT / 4) & ~1u;  // (even and below NT: every wave meets two barriers a chunk)
        float4 qa[NT], pa[4], eg4;
        auto fetch = [&](uint32_t ch) {
            const float4 *qp = (const float4 *)(cb.q + (ki0 + ch) * kChunk * DQ) + wave * NT * 64 + lane;
            const float4 *pp = (const float4 *)(cb.p + (ci0 + ch) * kChunk * kChunk) + wave * 4 * 64 + lane;
#pragma unroll
            for (uint32_t m = 0; m < NT; m++) qa[m] = qp[64 * m];
#pragma unroll
            for (int t = 0; t < 4; t++) pa[t] = pp[64 * t];
            eg4 = *(const float4 *)(cb.eg + (ci0 + ch) * kChunk + 16 * wave + 4 * g);
        };
        fetch(0);
        for (uint32_t ch = 0; ch < chunks; ch++) {
            const uint32_t buf = ch & 1;
            lds_barrier();  // S is there; it stays until the state's waves have passed this chunk's successor
            float4_t a0 = {0.f, 0.f, 0.f, 0.f}, a1 = {0.f, 0.f, 0.f, 0.f}, ap = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (uint32_t m = 0; m < NT; m += 2) {
                if (m == SPLIT) lds_barrier();  // U is there
                a0 = mfma4(qa[m], sl[buf][m][lane], a0);
                a1 = mfma4(qa[m + 1], sl[buf][m + 1][lane], a1);
            }
#pragma unroll
            for (int t = 0; t < 4; t++)
                if (t <= (int)wave) ap = mfma4(pa[t], ul[buf][t][lane], ap);
            a0 += a1;
            const float r[4] = {fmaf(eg4.x, a0[0], ap[0]), fmaf(eg4.y, a0[1], ap[1]), fmaf(eg4.z, a0[2], ap[2]), fmaf(eg4.w, a0[3], ap[3])};
            __builtin_amdgcn_sched_barrier(0);
            fetch(ch + 1 < chunks ? ch + 1 : ch);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const uint64_t row = (uint64_t)ch * kChunk + 16 * wave + 4 * g + i;
                if (row < seg && col < dm.e) o[((b * n + t0 + row) * H + h) * dm.e + col] = r[i];
            }
        }
    }
}

// A few dozen tokens are quicker one by one than through two launches of chunks.
constexpr uint64_t kChunkedFrom = 48;

uint64_t delta_prompt_scratch_bytes(const DeltaDims &dm, uint64_t batch, uint64_t n) {
    if (n < kChunkedFrom) return 0;
    return chunk_floats(dm, batch, ceil_div(n < kSegment ? n : kSegment, kChunk)) * 4;
}

template <int QW>
static int launch_chunks(const DeltaDims &dm, const DeltaOperands &op, const DeltaState &state, uint64_t batch, uint64_t n,
                         float *o, float *scratch, hipStream_t st) {
    constexpr uint32_t DQ = 64 * QW;
    const uint32_t dp = delta_padded_dim(dm.d);
    const size_t lds = (kChunk * (DQ + 4) + kChunk * (kChunk + 4) + kChunk * 20) * 4;
    static const bool once = [] {
        (void)hipFuncSetAttribute((const void *)delta_chunk_kernel<4 * QW>, hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
        return true;
    }();
    (void)once;
    for (uint64_t t0 = 0; t0 < n; t0 += kSegment) {
        const uint64_t seg = n - t0 < kSegment ? n - t0 : kSegment;
        ChunkBuf cb;
        cb.chunks = (uint32_t)ceil_div(seg, kChunk);
        float *p = scratch;
        const uint64_t hc = batch * cb.chunks * dm.heads;
        auto take = [&](uint64_t k) { float *r = p; p += k; return r; };
        cb.w = take(hc * kChunk * DQ);
        cb.p = take(hc * kChunk * kChunk);
        cb.eg = take(hc * kChunk);
        cb.ed = take(hc * kChunk);
        cb.vp = take(hc * kChunk * round_up(dm.e, 16));
        cb.kt = take(batch * cb.chunks * dm.kv_heads * DQ * kChunk);
        cb.q = take(batch * cb.chunks * dm.kv_heads * DQ * kChunk);
        hipLaunchKernelGGL((delta_chunk_kernel<4 * QW>), dim3(cb.chunks, dm.heads, (unsigned)batch), dim3(256), lds, st, dm,
                           op, dp, n, t0, seg, cb);
        const uint32_t blocks = (uint32_t)ceil_div(dm.e, 16), units = (uint32_t)(dm.heads * batch);
        hipLaunchKernelGGL((delta_carry_kernel<QW>), dim3(blocks * units), dim3(512), 0, st, dm, n, t0, seg, cb,
                           state.s, o, blocks, units);
    }
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

int launch_delta_prompt(const DeltaDims &dm, const DeltaOperands &op, const DeltaState &state, uint64_t batch,
                        uint64_t n, float *o, float *scratch, uint64_t scratch_bytes, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    COEUS_TRY(check_rows(batch, n));
    if (dm.heads > 65535 || (uint64_t)dm.heads * batch * ceil_div(dm.e, 16) > 0x7fffffffull)
        return fail(COEUS_INVALID_INPUT, "delta rule: too many heads");
    const uint64_t want = delta_prompt_scratch_bytes(dm, batch, n);
    if (want && scratch && scratch_bytes >= want) {
        switch (chunk_dim(dm.d) / 64) {
            case 1: return launch_chunks<1>(dm, op, state, batch, n, o, scratch, st);
            case 2: return launch_chunks<2>(dm, op, state, batch, n, o, scratch, st);
            case 3: return launch_chunks<3>(dm, op, state, batch, n, o, scratch, st);
            default: return launch_chunks<4>(dm, op, state, batch, n, o, scratch, st);
        }
    }
    const dim3 grid((unsigned)ceil_div(dm.e, 16), dm.heads, (unsigned)batch);
#define COEUS_DS(RV) \
    case RV: hipLaunchKernelGGL(delta_scan_kernel<RV>, grid, dim3(256), 0, st, dm, op, state.s, n, o); break
    switch (delta_padded_dim(dm.d) / 16) {
        COEUS_DS(1); COEUS_DS(2); COEUS_DS(3); COEUS_DS(4); COEUS_DS(5); COEUS_DS(6); COEUS_DS(7); COEUS_DS(8);
        COEUS_DS(9); COEUS_DS(10); COEUS_DS(11); COEUS_DS(12); COEUS_DS(13); COEUS_DS(14); COEUS_DS(15); COEUS_DS(16);
    }
#undef COEUS_DS
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// One wave per (row, head); out may be o itself.  With LG lanes a head (e = 4 LG), 64 / LG heads per wave in
// 16-byte pieces instead.
template <int LG>
__global__ __launch_bounds__(256) void delta_gate_kernel(const float *o, const float *__restrict__ proj,
                                                         DeltaDims dm, const float *__restrict__ norm, float eps,
                                                         uint64_t units, float *out, uint16_t *__restrict__ out_lp,
                                                         uint64_t lp_ld, bool lp_bf16) {
    const uint32_t lane = threadIdx.x & 63, H = dm.heads;
    const uint64_t wave = (uint64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (LG) {
        constexpr uint32_t PER = LG ? 64 / LG : 1, GL = LG ? LG : 1;
        const uint64_t unit = wave * PER + lane / GL, uc = unit < units ? unit : units - 1, row = uc / H;
        const uint32_t h = (uint32_t)(uc % H), c = 4 * (lane % GL);
        const float4 v = *(const float4 *)(o + uc * dm.e + c);
        const float4 gt = *(const float4 *)(proj + row * dm.in_ld + dm.gate_off() + h * dm.e + c);
        const float4 nw = *(const float4 *)(norm + c);
        float s2 = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, v.w * v.w)));
#pragma unroll
        for (uint32_t off = 1; off < GL; off <<= 1) s2 += __shfl_xor(s2, (int)off, 64);
        const float rs = 1.0f / sqrtf(s2 / (float)dm.e + eps);
        if (unit >= units) return;
        const float4 r = make_float4(v.x * rs * nw.x * fast_silu(gt.x), v.y * rs * nw.y * fast_silu(gt.y),
                                     v.z * rs * nw.z * fast_silu(gt.z), v.w * rs * nw.w * fast_silu(gt.w));
        if (out) *(float4 *)(out + unit * dm.e + c) = r;
        if (out_lp) {
            uint2 p;
            p.x = (uint32_t)f32_to_lp_bits(r.x, lp_bf16) | ((uint32_t)f32_to_lp_bits(r.y, lp_bf16) << 16);
            p.y = (uint32_t)f32_to_lp_bits(r.z, lp_bf16) | ((uint32_t)f32_to_lp_bits(r.w, lp_bf16) << 16);
            *(uint2 *)(out_lp + row * lp_ld + h * dm.e + c) = p;
        }
        return;
    }
    if (wave >= units) return;
    const uint64_t row = wave / H;
    const uint32_t h = (uint32_t)(wave % H);
    const float *op = o + wave * dm.e, *gp = proj + row * dm.in_ld + dm.gate_off() + h * dm.e;
    float s2 = 0.f;
    for (uint32_t c = lane; c < dm.e; c += 64) s2 = fmaf(op[c], op[c], s2);
    const float rs = 1.0f / sqrtf(wave_sum(s2) / (float)dm.e + eps);
    for (uint32_t c = lane; c < dm.e; c += 64) {
        const float v = op[c] * rs * norm[c] * fast_silu(gp[c]);
        if (out) out[wave * dm.e + c] = v;
        if (out_lp) out_lp[row * lp_ld + h * dm.e + c] = f32_to_lp_bits(v, lp_bf16);
    }
}

int launch_delta_gate(const float *o, const float *proj, const DeltaDims &dm, const DeltaParams &pr, uint64_t rows,
                      float *out, const LpOut *out_lp, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    COEUS_TRY(check_rows(1, rows));
    const uint64_t units = rows * dm.heads;
    uint16_t *lp = out_lp ? (uint16_t *)out_lp->p : nullptr;
    const uint64_t ld = out_lp ? out_lp->ld : 0;
    const bool lp_bf = out_lp && out_lp->bf16;
    // 16-byte pieces: heads of 16, 32, .. 256 values behind a gate that starts on a boundary
    const bool vec = dm.in_ld % 4 == 0 && dm.gate_off() % 4 == 0 && ld % 4 == 0;
#define COEUS_DG(LGV, PERV) \
    hipLaunchKernelGGL(delta_gate_kernel<LGV>, dim3((unsigned)ceil_div(units, 4 * PERV)), dim3(256), 0, st, o, proj, dm, pr.norm, \
                       pr.eps, units, out, lp, ld, lp_bf)
    if (vec && dm.e == 32) COEUS_DG(8, 8);
    else if (vec && dm.e == 64) COEUS_DG(16, 4);
    else if (vec && dm.e == 128) COEUS_DG(32, 2);
    else if (vec && dm.e == 256) COEUS_DG(64, 1);
    else COEUS_DG(0, 1);
#undef COEUS_DG
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// ---------------------------------------------------------------- decode step
// One workgroup of 512 per (head, sequence).  Both products with the state are taken of the old state in
// one pass (o = exp(lg) S^T q + (k . q) u), thread (g, c) of the pass owning columns VW c .. of rows
// g, g + DG, ..: up to RM of them stay in registers between the products and the update.
template <int VW, int RM, int T>  // T taps (1 .. 4), 0: any number
__global__ __launch_bounds__(512) void delta_step_kernel(const float *__restrict__ proj, DeltaDims dm, DeltaParams pr,
                                                         float *state, float *ring, const uint32_t *pos_dev,
                                                         float *__restrict__ out) {
    extern __shared__ float lds[];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const uint32_t h = blockIdx.x, H = dm.heads, KH = dm.kv_heads, hk = h / (H / KH), d = dm.d, e = dm.e, C = dm.channels();
    const uint64_t b = blockIdx.y;
    const uint32_t cg = e / VW, DG = 512 / cg;           // column groups, row groups
    float *qs = lds, *ks = qs + d, *vs = ks + d, *us = vs + e, *pk = us + e, *pq = pk + DG * e;
    __shared__ float red[8], kq_s;
    float *S = state + (b * H + h) * (uint64_t)d * e;
    const float *p = proj + b * dm.in_ld;
    const uint32_t pos = *pos_dev;
    const uint32_t g0 = tid / cg, c0 = (tid % cg) * VW;
    const bool live = g0 < DG;
    // the state's first rows are requested before anything else
    float sr[RM][VW];
    auto load_row = [&](uint32_t r, float (&x)[VW]) {
        const float *sp = S + (uint64_t)r * e + c0;
        if (VW == 4) { const float4 t = *(const float4 *)sp; x[0] = t.x; x[1] = t.y; x[2] = t.z; x[3] = t.w; }
        else x[0] = *sp;
    };
#pragma unroll
    for (int i = 0; i < RM; i++) {
        const uint32_t r = g0 + i * DG;
#pragma unroll
        for (int t = 0; t < VW; t++) sr[i][t] = 0.f;
        if (live && r < d) load_row(r, sr[i]);
    }
    // Convolution ring: every workgroup that shares a channel writes the same value.  All slots are requested
    // without knowing the position (one trip to memory); the position then says which tap each slot meets.
    // Slots in front of the sequence hold the zeros that a cleared state starts with.
    auto channel = [&](uint32_t c) -> float {
        const float x = p[c];
        float acc;
        if (T) {
            constexpr uint32_t TT = T ? T : 1;
            float r[TT], w[TT];
#pragma unroll
            for (uint32_t j = 0; j < TT; j++) {
                r[j] = ring[(b * TT + j) * C + c];
                w[j] = pr.conv[(uint64_t)j * C + c];
            }
            acc = w[TT - 1] * x;
            const uint32_t slot = pos % TT;
#pragma unroll
            for (uint32_t k = 0; k < TT; k++)  // slot k is uniform: one of these runs
                if (slot == k)
#pragma unroll
                    for (uint32_t back = 1; back < TT; back++) acc = fmaf(w[TT - 1 - back], r[(k + TT - back) % TT], acc);
        } else {
            acc = pr.conv[(uint64_t)(dm.taps - 1) * C + c] * x;
            for (uint32_t back = 1; back < dm.taps && back <= pos; back++)
                acc = fmaf(pr.conv[(uint64_t)(dm.taps - 1 - back) * C + c], ring[(b * dm.taps + (pos - back) % dm.taps) * C + c], acc);
        }
        ring[(b * dm.taps + pos % dm.taps) * C + c] = x;
        return fast_silu(acc);
    };
    if (wave < 2) {  // wave 0: q, wave 1: k
        const uint32_t base = (wave * KH + hk) * d;
        float v[4], s2 = 0.f;
#pragma unroll
        for (int t = 0; t < 4; t++) {
            const uint32_t c = lane + 64 * t;
            v[t] = c < d ? channel(base + c) : 0.f;
            s2 = fmaf(v[t], v[t], s2);
        }
        const float r = (wave == 0 ? 1.0f / sqrtf((float)d) : 1.0f) / sqrtf(wave_sum(s2) + kUnitEps);
#pragma unroll
        for (int t = 0; t < 4; t++)
            if (lane + 64 * t < d) (wave == 0 ? qs : ks)[lane + 64 * t] = v[t] * r;
    } else {
        for (uint32_t c = tid - 128; c < e; c += 384) vs[c] = channel(2 * KH * d + h * e + c);
    }
    const float beta = sigmoid(p[dm.beta_off() + h]);
    const float g = expf(log_decay(p[dm.decay_off() + h], pr.exp_a[h], pr.dt_bias[h]));
    __syncthreads();
    if (wave == 7) {
        float t = 0.f;
        for (uint32_t c = lane; c < d; c += 64) t = fmaf(qs[c], ks[c], t);
        t = wave_sum(t);
        if (lane == 0) kq_s = t;
    }
    float ak[VW], aq[VW];
#pragma unroll
    for (int t = 0; t < VW; t++) ak[t] = aq[t] = 0.f;
    if (live) {
#pragma unroll
        for (int i = 0; i < RM; i++) {
            const uint32_t r = g0 + i * DG;
            if (r >= d) break;
            const float kr = ks[r], qr = qs[r];
#pragma unroll
            for (int t = 0; t < VW; t++) { ak[t] = fmaf(sr[i][t], kr, ak[t]); aq[t] = fmaf(sr[i][t], qr, aq[t]); }
        }
        for (uint32_t r = g0 + RM * DG; r < d; r += DG) {
            float x[VW];
            load_row(r, x);
            const float kr = ks[r], qr = qs[r];
#pragma unroll
            for (int t = 0; t < VW; t++) { ak[t] = fmaf(x[t], kr, ak[t]); aq[t] = fmaf(x[t], qr, aq[t]); }
        }
#pragma unroll
        for (int t = 0; t < VW; t++) { pk[g0 * e + c0 + t] = ak[t]; pq[g0 * e + c0 + t] = aq[t]; }
    }
    __syncthreads();
    float s2 = 0.f;
    for (uint32_t c = tid; c < e; c += 512) {
        float sk = 0.f, sq = 0.f;
#pragma unroll 8
        for (uint32_t i = 0; i < DG; i++) { sk += pk[i * e + c]; sq += pq[i * e + c]; }
        const float u = beta * (vs[c] - g * sk);
        us[c] = u;
        const float o = fmaf(kq_s, u, g * sq);
        vs[c] = o;
        s2 = fmaf(o, o, s2);
    }
    s2 = wave_sum(s2);
    if (lane == 0) red[wave] = s2;
    __syncthreads();
    if (live) {
        float u[VW];
#pragma unroll
        for (int t = 0; t < VW; t++) u[t] = us[c0 + t];
        auto store_row = [&](uint32_t r, const float (&x)[VW]) {
            const float kr = ks[r];
            float *sp = S + (uint64_t)r * e + c0;
            if (VW == 4)
                *(float4 *)sp = make_float4(fmaf(kr, u[0], g * x[0]), fmaf(kr, u[1 % VW], g * x[1 % VW]),
                                            fmaf(kr, u[2 % VW], g * x[2 % VW]), fmaf(kr, u[3 % VW], g * x[3 % VW]));
            else *sp = fmaf(kr, u[0], g * x[0]);
        };
#pragma unroll
        for (int i = 0; i < RM; i++) {
            const uint32_t r = g0 + i * DG;
            if (r >= d) break;
            store_row(r, sr[i]);
        }
        for (uint32_t r = g0 + RM * DG; r < d; r += DG) {
            float x[VW];
            load_row(r, x);
            store_row(r, x);
        }
    }
    float tot = 0.f;
#pragma unroll
    for (int w = 0; w < 8; w++) tot += red[w];
    const float rs = 1.0f / sqrtf(tot / (float)e + pr.eps);
    for (uint32_t c = tid; c < e; c += 512)
        out[(b * H + h) * e + c] = vs[c] * rs * pr.norm[c] * fast_silu(p[dm.gate_off() + h * e + c]);
}

int launch_delta_step(const float *proj, const DeltaDims &dm, const DeltaParams &pr, const DeltaState &state,
                      uint64_t batch, const uint32_t *pos_dev, float *out, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    COEUS_TRY(check_rows(batch, 1));
    const bool vec = dm.e % 4 == 0;
    const uint32_t cg = vec ? dm.e / 4 : dm.e;
    if (cg > 512) return fail(COEUS_INVALID_INPUT, "delta rule: a value size above 512 must be a multiple of 4");
    const uint32_t DG = 512 / cg, per = (uint32_t)ceil_div(dm.d, DG);
    const size_t lds = (2 * dm.d + 2 * dm.e + 2 * (size_t)DG * dm.e) * 4;
    const dim3 grid(dm.heads, (unsigned)batch);
#define COEUS_DST2(VWV, RMV, TV) \
    hipLaunchKernelGGL((delta_step_kernel<VWV, RMV, TV>), grid, dim3(512), lds, st, proj, dm, pr, state.s, state.ring, pos_dev, out)
#define COEUS_DST(VWV, RMV)                            \
    do {                                               \
        switch (dm.taps) {                             \
            case 1: COEUS_DST2(VWV, RMV, 1); break;    \
            case 2: COEUS_DST2(VWV, RMV, 2); break;    \
            case 3: COEUS_DST2(VWV, RMV, 3); break;    \
            case 4: COEUS_DST2(VWV, RMV, 4); break;    \
            default: COEUS_DST2(VWV, RMV, 0); break;   \
        }                                              \
    } while (0)
    if (vec) { if (per <= 8) COEUS_DST(4, 8); else COEUS_DST(4, 16); }
    else { if (per <= 8) COEUS_DST(1, 8); else COEUS_DST(1, 32); }
#undef COEUS_DST
#undef COEUS_DST2
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

}  // namespace coeus
