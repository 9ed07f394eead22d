// Gated delta rule: a linear recurrence with a matrix state per head, its short convolutions and its
// gated output norm.
//
//   delta_prepare_kernel  prompt: convolution + SiLU of q, k, v, unit norms, step sizes and decays
//   delta_ring_kernel     prompt: the last projections of every sequence into the convolution ring
//   delta_scan_kernel     prompt: the recurrence token by token, state in registers
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

// Convolution + SiLU of channel c at row i of sequence b (position pos0 + i).
__device__ __forceinline__ float conv_silu(const float *__restrict__ proj, const float *__restrict__ ring,
                                           const float *__restrict__ taps_w, uint32_t taps, uint32_t channels,
                                           uint64_t in_ld, uint64_t b, uint64_t n, uint64_t i, uint64_t pos0, uint32_t c) {
    float acc = 0.f;
    for (uint32_t j = 0; j < taps; j++) {
        const uint32_t back = taps - 1 - j;  // this tap looks `back` positions behind
        float x = 0.f;
        if (back <= i) x = proj[(b * n + i - back) * in_ld + c];
        else if (back <= pos0 + i) x = ring[(b * taps + (pos0 + i - back) % taps) * channels + c];
        acc = fmaf(taps_w[(uint64_t)j * channels + c], x, acc);
    }
    return silu(acc);
}

// One wave per (row, unit); a unit is one head of q, k or v, or the gates of all heads.
__global__ __launch_bounds__(256) void delta_prepare_kernel(const float *__restrict__ proj, DeltaDims dm, DeltaParams pr,
                                                            const float *__restrict__ ring, uint64_t n, uint64_t pos0,
                                                            uint32_t dp, DeltaOperands op) {
    const uint32_t lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6);
    const uint64_t row = blockIdx.x, b = row / n, i = row % n;
    const uint32_t KH = dm.kv_heads, H = dm.heads, C = dm.channels();
    if (unit < 2 * KH) {
        const bool is_q = unit < KH;
        const uint32_t c0 = unit * dm.d;  // q heads, then k heads
        float v[4], s2 = 0.f;             // d <= 256
#pragma unroll
        for (int t = 0; t < 4; t++) {
            const uint32_t c = lane + 64 * t;
            v[t] = c < dm.d ? conv_silu(proj, ring, pr.conv, dm.taps, C, dm.in_ld, b, n, i, pos0, c0 + c) : 0.f;
            s2 = fmaf(v[t], v[t], s2);
        }
        const float r = (is_q ? 1.0f / sqrtf((float)dm.d) : 1.0f) / sqrtf(wave_sum(s2) + kUnitEps);
        float *dst = (is_q ? op.q : op.k) + (row * KH + (is_q ? unit : unit - KH)) * dp;
#pragma unroll
        for (int t = 0; t < 4; t++)
            if (lane + 64 * t < dp) dst[lane + 64 * t] = v[t] * r;  // (zeros behind d)
    } else if (unit < 2 * KH + H) {
        const uint32_t h = unit - 2 * KH, c0 = 2 * KH * dm.d + h * dm.e;
        for (uint32_t c = lane; c < dm.e; c += 64)
            op.v[(row * H + h) * dm.e + c] = conv_silu(proj, ring, pr.conv, dm.taps, C, dm.in_ld, b, n, i, pos0, c0 + c);
    } else if (unit == 2 * KH + H) {
        const float *p = proj + row * dm.in_ld;
        for (uint32_t h = lane; h < H; h += 64) {
            op.beta[row * H + h] = sigmoid(p[dm.beta_off() + h]);
            op.lg[row * H + h] = log_decay(p[dm.decay_off() + h], pr.exp_a[h], pr.dt_bias[h]);
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
    const dim3 grid((unsigned)(batch * n), (unsigned)ceil_div(2 * dm.kv_heads + dm.heads + 1, 4));
    hipLaunchKernelGGL(delta_prepare_kernel, grid, dim3(256), 0, st, proj, dm, pr, state.ring, n, pos0,
                       delta_padded_dim(dm.d), op);
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

uint64_t delta_prompt_scratch_bytes(const DeltaDims &dm, uint64_t batch, uint64_t n) {
    (void)dm; (void)batch; (void)n;
    return 0;
}

int launch_delta_prompt(const DeltaDims &dm, const DeltaOperands &op, const DeltaState &state, uint64_t batch,
                        uint64_t n, float *o, float *scratch, uint64_t scratch_bytes, hipStream_t st) {
    (void)scratch; (void)scratch_bytes;
    COEUS_TRY(check_dims(dm));
    COEUS_TRY(check_rows(batch, n));
    if (dm.heads > 65535) return fail(COEUS_INVALID_INPUT, "delta rule: too many heads");
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

// One wave per (row, head); out may be o itself.
__global__ __launch_bounds__(256) void delta_gate_kernel(const float *o, const float *__restrict__ proj,
                                                         DeltaDims dm, const float *__restrict__ norm, float eps,
                                                         uint64_t units, float *out,
                                                         uint16_t *__restrict__ out_lp, uint64_t lp_ld, bool lp_bf16) {
    const uint32_t lane = threadIdx.x & 63, H = dm.heads;
    const uint64_t unit = (uint64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (unit >= units) return;
    const uint64_t row = unit / H;
    const uint32_t h = (uint32_t)(unit % H);
    const float *op = o + unit * dm.e, *gp = proj + row * dm.in_ld + dm.gate_off() + h * dm.e;
    float s2 = 0.f;
    for (uint32_t c = lane; c < dm.e; c += 64) s2 = fmaf(op[c], op[c], s2);
    const float rs = 1.0f / sqrtf(wave_sum(s2) / (float)dm.e + eps);
    for (uint32_t c = lane; c < dm.e; c += 64) {
        const float v = op[c] * rs * norm[c] * silu(gp[c]);
        if (out) out[unit * dm.e + c] = v;
        if (out_lp) out_lp[row * lp_ld + h * dm.e + c] = f32_to_lp_bits(v, lp_bf16);
    }
}

int launch_delta_gate(const float *o, const float *proj, const DeltaDims &dm, const DeltaParams &pr, uint64_t rows,
                      float *out, const LpOut *out_lp, hipStream_t st) {
    COEUS_TRY(check_dims(dm));
    COEUS_TRY(check_rows(1, rows));
    const uint64_t units = rows * dm.heads;
    hipLaunchKernelGGL(delta_gate_kernel, dim3((unsigned)ceil_div(units, 4)), dim3(256), 0, st, o, proj, dm, pr.norm, pr.eps,
                       units, out, out_lp ? (uint16_t *)out_lp->p : nullptr, out_lp ? out_lp->ld : 0, out_lp && out_lp->bf16);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// ---------------------------------------------------------------- decode step
// One workgroup of 512 per (head, sequence).  Both products with the state are taken of the old state in
// one pass (o = exp(lg) S^T q + (k . q) u), thread (g, c) of the pass owning columns VW c .. of rows
// g, g + DG, ..: up to RM of them stay in registers between the products and the update.
template <int VW, int RM>
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
    // convolution ring: every workgroup that shares a channel writes the same value
    auto channel = [&](uint32_t c) -> float {
        const float x = p[c];
        float acc = pr.conv[(uint64_t)(dm.taps - 1) * C + c] * x;
        for (uint32_t back = 1; back < dm.taps; back++) {
            if (back > pos) break;
            acc = fmaf(pr.conv[(uint64_t)(dm.taps - 1 - back) * C + c], ring[(b * dm.taps + (pos - back) % dm.taps) * C + c], acc);
        }
        ring[(b * dm.taps + pos % dm.taps) * C + c] = x;
        return silu(acc);
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
        out[(b * H + h) * e + c] = vs[c] * rs * pr.norm[c] * silu(p[dm.gate_off() + h * e + c]);
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
#define COEUS_DST(VWV, RMV) \
    hipLaunchKernelGGL((delta_step_kernel<VWV, RMV>), grid, dim3(512), lds, st, proj, dm, pr, state.s, state.ring, pos_dev, out)
    if (vec) { if (per <= 8) COEUS_DST(4, 8); else COEUS_DST(4, 16); }
    else { if (per <= 8) COEUS_DST(1, 8); else COEUS_DST(1, 32); }
#undef COEUS_DST
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

}  // namespace coeus
