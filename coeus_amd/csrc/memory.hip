// Matrix memory: a linear recurrence with a matrix state and a normaliser per head under exponential gates,
// which are kept in range by a running maximum, and its gated output norm.
//
//   memory_local_kernel   prompt: what each chunk of 64 tokens adds to the state, all chunks at once
//   memory_carry_kernel   prompt: the state in front of every chunk (element by element over the chunks)
//   memory_read_kernel    prompt: the outputs of every chunk, normalised and gated, all chunks at once
//   memory_scan_kernel    short prompts and odd sizes: token by token, state in registers
//   memory_finish_kernel  its outputs: normaliser, RMS norm, gate
//   memory_step_kernel    decode: all of it for one token per sequence
//
// Everything behind the projections is f32: gates, state, normaliser, products and norms.
#include "device_utils.hpp"
#include "mixers.hpp"

namespace coeus {

constexpr float kFloor = 1e-6f;  // added to the normaliser
constexpr uint32_t kMaxDim = 512, kMaxChunkDim = 256;

__device__ __forceinline__ float log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }
// Logarithms of the input and forget gates of one token, p its row of the projection.
__device__ __forceinline__ void log_gates(const float *__restrict__ p, const MemoryDims &dm, const MemoryParams &pr, uint32_t h,
                                          float &in, float &forget) {
    in = dm.cap * tanhf((p[dm.in_off() + h] + pr.in_bias[h]) / dm.cap);
    forget = log_sigmoid(dm.cap * tanhf((p[dm.forget_off() + h] + pr.forget_bias[h]) / dm.cap));
}
__device__ __forceinline__ float sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float normaliser(float nq, float m) { return fmaxf(fabsf(nq), expf(-m)) + kFloor; }

static int check_args(const MemoryDims &dm, uint64_t batch, uint64_t n) {
    if (dm.heads == 0 || dm.heads > 65535 || dm.d == 0 || dm.d > kMaxDim || dm.e == 0 || dm.e > 1024 ||
        dm.in_ld < dm.forget_off() + dm.heads || !(dm.cap > 0.f))
        return fail(COEUS_INVALID_INPUT, "matrix memory: sizes out of range");
    if (batch == 0 || n == 0 || batch > 65535 || batch * n > 0x7fffffffull)
        return fail(COEUS_INVALID_INPUT, "matrix memory: %llu x %llu rows out of range", (unsigned long long)batch, (unsigned long long)n);
    return COEUS_OK;
}

// ---------------------------------------------------------------- chunk by chunk
// With F_t the sum of the log forget gates of a chunk's tokens up to t, a_s = i_s - F_s, and (S0, n0, m0) the
// state in front of it, all of it divided by e^m0:
//   m_t = F_t + max(m0, max_{s <= t} a_s)
//   o_t = e^(F_t + m0 - m_t) S0^T q_t + sum_{s <= t} e^(F_t + a_s - m_t) (k_s . q_t) v_s      (n alike with v = 1)
//   S_C = e^(F_C + m0 - m_C) S0 + sum_s e^(F_C + a_s - m_C) k_s v_s^T
// so no exponent is positive.  The state's two terms do not meet before the end: each chunk's own sum
// (relative to its own maximum) is found for all chunks at once, a carry pass over the chunks turns the sums
// into the states in front of them, and then all outputs follow at once.  F and a are f64: sums of many
// strong gates cancel in their differences.
//
// Chunk states lie as accumulator tiles of the f32 matrix instructions, [16 dims][16 columns][lane][4]: lane
// 16 g + c holds dims 4 g .. 4 g + 3 of column c, which is at once the right operand of the next product.
constexpr uint32_t kChunk = 64, kColBlock = 128;
constexpr uint64_t kSegment = 4096;  // tokens whose chunk states are in memory at once

struct MemoryChunks {
    float *s;   // [unit][chunks][dtiles][etiles][64][4]
    float *n;   // [unit][chunks][d]
    float *f;   // [unit][chunks]: F_C
    float *mc;  // [unit][chunks]: F_C + the largest a
    float *m0;  // [unit][chunks + 1]: the state's maximum in front of each chunk, and behind the last
    uint32_t chunks, dtiles, etiles;
};
static uint64_t chunk_floats(const MemoryDims &dm, uint64_t units, uint64_t chunks) {
    return units * (chunks * (ceil_div(dm.d, 16) * ceil_div(dm.e, 16) * 256 + dm.d + 2) + chunks + 1) + 64;
}
static bool chunked(const MemoryDims &dm, uint64_t n) {
    // (a few dozen tokens are quicker one by one than through three launches)
    return n >= 48 && dm.d % 4 == 0 && dm.e % 4 == 0 && dm.in_ld % 4 == 0 && dm.d <= kMaxChunkDim && dm.e <= kMaxChunkDim;
}

struct ChunkGates {
    double F, a, top;  // running sum of the log forget gates, log input gate - F, running maximum of that
};
// Lane t: token t of a chunk; tokens behind the end keep everything and add nothing.
__device__ __forceinline__ ChunkGates chunk_gates(const float *__restrict__ p, const MemoryDims &dm, const MemoryParams &pr, uint32_t h,
                                                  uint32_t lane, uint32_t live) {
    float in = 0.f, forget = 0.f;
    if (lane < live) log_gates(p + (uint64_t)lane * dm.in_ld, dm, pr, h, in, forget);
    ChunkGates g;
    g.F = (double)forget;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double o = __shfl_up(g.F, off, 64);
        if ((int)lane >= off) g.F += o;
    }
    g.a = lane < live ? (double)in - g.F : -INFINITY;
    g.top = g.a;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double o = __shfl_up(g.top, off, 64);
        if ((int)lane >= off) g.top = fmax(g.top, o);
    }
    return g;
}

// One workgroup per (chunk, head and up to 128 columns, sequence): K^T diag(w) V.  Wave w owns the 16-dim tiles
// w, w + 4, ..
template <int NDT>
__global__ __launch_bounds__(256) void memory_local_kernel(const float *__restrict__ proj, MemoryDims dm, MemoryParams pr, uint64_t n,
                                                           uint64_t t0, uint64_t seg, uint32_t cblocks, MemoryChunks cb) {
    constexpr uint32_t VLD = kColBlock + 4;
    __shared__ __attribute__((aligned(16))) float vl[kChunk * VLD];
    __shared__ float ws[kChunk];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const uint32_t chunk = blockIdx.x, h = blockIdx.y / cblocks, cblk = blockIdx.y % cblocks, H = dm.heads, d = dm.d, e = dm.e;
    const uint64_t b = blockIdx.z, left = seg - (uint64_t)chunk * kChunk, row0 = b * n + t0 + (uint64_t)chunk * kChunk;
    const uint32_t live = left < kChunk ? (uint32_t)left : kChunk, c0 = cblk * kColBlock;
    const uint64_t ci = (b * H + h) * cb.chunks + chunk;
    const float *p = proj + row0 * dm.in_ld;
    float4_t k[NDT][4];
#pragma unroll
    for (int t = 0; t < NDT; t++) {
        const uint32_t dim = 16 * (wave + 4 * t) + c, dimc = min(dim, d - 1);
#pragma unroll
        for (int m = 0; m < 4; m++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const float v = p[(uint64_t)min(16u * m + 4 * g + i, live - 1) * dm.in_ld + dm.k_off() + h * d + dimc];
                k[t][m][i] = dim < d ? v : 0.f;
            }
    }
    for (uint32_t i = tid; i < kChunk * (kColBlock / 4); i += 256) {
        const uint32_t r = i / (kColBlock / 4), q4 = 4 * (i % (kColBlock / 4));
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (r < live && c0 + q4 < e) v = *(const float4 *)(p + (uint64_t)r * dm.in_ld + dm.v_off() + h * e + c0 + q4);
        *(float4 *)(vl + r * VLD + q4) = v;
    }
    if (wave == 0) {
        const ChunkGates cg = chunk_gates(p, dm, pr, h, lane, live);
        const double top = __shfl(cg.top, 63, 64);
        ws[lane] = expf((float)(cg.a - top));
        if (lane == 63 && cblk == 0) {
            cb.f[ci] = (float)cg.F;
            cb.mc[ci] = (float)(cg.F + top);
        }
    }
    __syncthreads();
#pragma unroll
    for (int m = 0; m < 4; m++) {
        const float4_t w = *(const float4_t *)(ws + 16 * m + 4 * g);
#pragma unroll
        for (int t = 0; t < NDT; t++) k[t][m] *= w;
    }
    const uint32_t ct = min(kColBlock / 16, cb.etiles - c0 / 16);
    for (uint32_t u = 0; u < ct; u++) {
        float4_t acc[NDT];
#pragma unroll
        for (int t = 0; t < NDT; t++) acc[t] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int m = 0; m < 4; m++) {
            float4_t v;
#pragma unroll
            for (int i = 0; i < 4; i++) v[i] = vl[(16 * m + 4 * g + i) * VLD + 16 * u + c];
#pragma unroll
            for (int t = 0; t < NDT; t++) acc[t] = mfma4(k[t][m], v, acc[t]);
        }
#pragma unroll
        for (int t = 0; t < NDT; t++)
            if (wave + 4 * t < cb.dtiles)
                *(float4_t *)(cb.s + ((ci * cb.dtiles + wave + 4 * t) * cb.etiles + c0 / 16 + u) * 256 + lane * 4) = acc[t];
    }
    if (cblk == 0)
#pragma unroll
        for (int t = 0; t < NDT; t++) {
            float s = 0.f;
#pragma unroll
            for (int m = 0; m < 4; m++) s += (k[t][m][0] + k[t][m][1]) + (k[t][m][2] + k[t][m][3]);
            s = xor32_sum(xor16_sum(s));
            const uint32_t dim = 16 * (wave + 4 * t) + c;
            if (lane < 16 && dim < d) cb.n[ci * d + dim] = s;
        }
}

// A thread owns four dims of one column of the state (or one element of the normaliser, or the maximum) and
// walks the chunks: the chunk's sum is read, the state in front of the chunk takes its place.
__global__ __launch_bounds__(256) void memory_carry_kernel(MemoryDims dm, MemoryState st, MemoryChunks cb) {
    const uint32_t H = dm.heads, d = dm.d, e = dm.e, NU = cb.dtiles * cb.etiles * 64, u = blockIdx.x * 256 + threadIdx.x;
    const uint64_t unit = (uint64_t)blockIdx.z * H + blockIdx.y;
    if (u > NU + d) return;
    const float *f = cb.f + unit * cb.chunks, *mc = cb.mc + unit * cb.chunks;
    float m = st.m[unit];
    // factors of the old state and of chunk ch's sum; m moves on
    auto factors = [&](uint32_t ch, float &keep, float &add) {
        const float fm = f[ch] + m, top = fmaxf(fm, mc[ch]);
        keep = expf(fm - top);
        add = expf(mc[ch] - top);
        m = top;
    };
    float keep, add;
    if (u < NU) {
        const uint32_t tile = u >> 6, lane = u & 63, col = 16 * (tile % cb.etiles) + (lane & 15), r0 = 16 * (tile / cb.etiles) + 4 * (lane >> 4);
        float *sp = st.s + unit * d * e;
        float4_t s;
#pragma unroll
        for (int i = 0; i < 4; i++) s[i] = r0 + i < d && col < e ? sp[(uint64_t)(r0 + i) * e + col] : 0.f;
        float4_t *x = (float4_t *)cb.s + unit * cb.chunks * NU + u;
        constexpr uint32_t A = 8;  // chunks in flight
        float4_t nx[A];
#pragma unroll
        for (uint32_t j = 0; j < A; j++) nx[j] = x[(uint64_t)min(j, cb.chunks - 1) * NU];
        for (uint32_t ch0 = 0; ch0 < cb.chunks; ch0 += A) {
            float4_t cur[A];
#pragma unroll
            for (uint32_t j = 0; j < A; j++) cur[j] = nx[j];
            if (ch0 + A < cb.chunks)
#pragma unroll
                for (uint32_t j = 0; j < A; j++) nx[j] = x[(uint64_t)min(ch0 + A + j, cb.chunks - 1) * NU];
#pragma unroll
            for (uint32_t j = 0; j < A; j++) {
                if (ch0 + j >= cb.chunks) break;
                factors(ch0 + j, keep, add);
                x[(uint64_t)(ch0 + j) * NU] = s;
                s = keep * s + add * cur[j];
            }
        }
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (r0 + i < d && col < e) sp[(uint64_t)(r0 + i) * e + col] = s[i];
    } else if (u < NU + d) {
        float *np = st.n + unit * d + (u - NU), s = *np;
        float *x = cb.n + unit * cb.chunks * d + (u - NU);
        for (uint32_t ch = 0; ch < cb.chunks; ch++) {
            factors(ch, keep, add);
            const float v = x[(uint64_t)ch * d];
            x[(uint64_t)ch * d] = s;
            s = keep * s + add * v;
        }
        *np = s;
    } else {
        // (the session's maximum itself is moved on by the next launch: other threads of this one read it)
        float *x = cb.m0 + unit * (cb.chunks + 1);
        for (uint32_t ch = 0; ch < cb.chunks; ch++) {
            x[ch] = m;
            factors(ch, keep, add);
        }
        x[cb.chunks] = m;
    }
}

// One workgroup of eight waves per (chunk, head, sequence); wave w owns the 16-column tiles w, w + 8, .. of all 64
// rows, so that a chunk's state is read once and the values once.  Queries and keys are in LDS (rows of an odd
// number of quads); the weighted scores take the keys' place.
static uint32_t read_ld(const MemoryDims &dm) { return 16 * (uint32_t)ceil_div(dm.d, 16) + 4; }
constexpr uint32_t kScoreLd = kChunk + 4;
static size_t read_lds_bytes(const MemoryDims &dm) { return kChunk * (size_t)(read_ld(dm) + std::max(read_ld(dm), kScoreLd)) * 4; }

template <int NCT>
__global__ __launch_bounds__(512) void memory_read_kernel(const float *__restrict__ proj, MemoryDims dm, MemoryParams pr, MemoryState st,
                                                          uint64_t n, uint64_t t0, uint64_t seg, MemoryChunks cb,
                                                          float *__restrict__ out, uint16_t *__restrict__ out_lp, uint64_t lp_ld,
                                                          bool lp_bf16) {
    constexpr uint32_t PLD = kScoreLd, W = 8;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ double rs[kChunk], as[kChunk];  // F - m of a row, a of a column
    __shared__ __attribute__((aligned(16))) float carry[kChunk], floor_[kChunk], psum[4][kChunk], qn[kChunk], dinv[kChunk], rsum[W][kChunk];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const uint32_t chunk = blockIdx.x, h = blockIdx.y, H = dm.heads, d = dm.d, e = dm.e, LD = 16 * cb.dtiles + 4;
    const uint64_t b = blockIdx.z, left = seg - (uint64_t)chunk * kChunk, row0 = b * n + t0 + (uint64_t)chunk * kChunk;
    const uint32_t live = left < kChunk ? (uint32_t)left : kChunk;
    const uint64_t unit = b * H + h, ci = unit * cb.chunks + chunk;
    const float *p = proj + row0 * dm.in_ld, *qp = p + h * d, *kp = p + dm.k_off() + h * d, *vp = p + dm.v_off() + h * e;
    float *const ql = lds, *const kl = ql + kChunk * LD, *const pl = kl;
    const float qs = 1.0f / sqrtf((float)d);
    // the first tiles of the state and the values are requested before anything else
    const float *sp = cb.s + ci * cb.dtiles * cb.etiles * 256 + lane * 4;
    auto sload = [&](uint32_t m, float4_t (&x)[NCT]) {
#pragma unroll
        for (int t = 0; t < NCT; t++) x[t] = *(const float4_t *)(sp + (min(m, cb.dtiles - 1) * cb.etiles + min(wave + W * t, cb.etiles - 1)) * 256);
    };
    float4_t s[4][NCT], v[4][NCT];
#pragma unroll
    for (int q = 0; q < 4; q++) sload(q, s[q]);
#pragma unroll
    for (int m = 0; m < 4; m++)
#pragma unroll
        for (int t = 0; t < NCT; t++)
#pragma unroll
            for (int i = 0; i < 4; i++) v[m][t][i] = vp[(uint64_t)min(16u * m + 4 * g + i, live - 1) * dm.in_ld + min(16 * (wave + W * t) + c, e - 1)];
    // queries and keys, half a wave per row: rows behind the end repeat the last one, dims behind the end are zero
    for (uint32_t x = 4 * (tid & 31); x < 16 * cb.dtiles; x += 128)
#pragma unroll
        for (uint32_t r = tid >> 5; r < kChunk; r += 16) {
            const uint64_t at = (uint64_t)min(r, live - 1) * dm.in_ld + min(x, d - 4);
            float4_t qv = *(const float4_t *)(qp + at), kv = *(const float4_t *)(kp + at);
            if (x >= d) qv = kv = float4_t{0.f, 0.f, 0.f, 0.f};
            *(float4_t *)(ql + r * LD + x) = qv;
            *(float4_t *)(kl + r * LD + x) = kv;
        }
    if (wave == W - 1) {
        const ChunkGates cg = chunk_gates(p, dm, pr, h, lane, live);
        const double m0 = (double)cb.m0[unit * (cb.chunks + 1) + chunk], top = fmax(m0, cg.top);
        rs[lane] = -top;  // F - m
        as[lane] = cg.a;
        carry[lane] = qs * expf((float)(m0 - top));
        floor_[lane] = expf((float)-(cg.F + top));
        if (chunk == cb.chunks - 1 && lane == 0) st.m[unit] = cb.m0[unit * (cb.chunks + 1) + cb.chunks];
    }
    __syncthreads();
    auto operand = [&](const float *rows, uint32_t tile, uint32_t m) { return *(const float4_t *)(rows + (16 * tile + c) * LD + 16 * m + 4 * g); };
    // ---- Q S0
    float4_t acc[4][NCT];
#pragma unroll
    for (int r = 0; r < 4; r++)
#pragma unroll
        for (int t = 0; t < NCT; t++) acc[r][t] = float4_t{0.f, 0.f, 0.f, 0.f};
    for (uint32_t m0 = 0; m0 < cb.dtiles; m0 += 4)
#pragma unroll
        for (int q = 0; q < 4; q++) {
            const uint32_t m = m0 + q;
            if (m >= cb.dtiles) break;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const float4_t a = operand(ql, r, m);
#pragma unroll
                for (int t = 0; t < NCT; t++) acc[r][t] = mfma4(a, s[q][t], acc[r][t]);
            }
            if (m + 4 < cb.dtiles) sload(m + 4, s[q]);
        }
    // ---- q . n0, eight threads a row
    {
        const float *n0 = cb.n + ci * d;
        float dot = 0.f;
        for (uint32_t dim = 4 * (tid & 7); dim < d; dim += 32) {
            const float4_t q = *(const float4_t *)(ql + (tid >> 3) * LD + dim), x = *(const float4_t *)(n0 + dim);
            dot = fmaf(q[0], x[0], dot); dot = fmaf(q[1], x[1], dot); dot = fmaf(q[2], x[2], dot); dot = fmaf(q[3], x[3], dot);
        }
        dot = group_sum<8>(dot);
        if ((tid & 7) == 0) qn[tid >> 3] = dot;
    }
    // ---- scores up to the diagonal: ten 16 x 16 tiles over the eight waves, then weighted
    auto tile_of = [](uint32_t idx, uint32_t &r, uint32_t &t) {
        r = idx < 1 ? 0 : idx < 3 ? 1 : idx < 6 ? 2 : 3;
        t = idx - r * (r + 1) / 2;
    };
    float4_t sc[2];
#pragma unroll
    for (int u = 0; u < 2; u++) {
        sc[u] = float4_t{0.f, 0.f, 0.f, 0.f};
        if (wave + W * u >= 10) continue;
        uint32_t r, t;
        tile_of(wave + W * u, r, t);
        for (uint32_t m = 0; m < cb.dtiles; m++) sc[u] = mfma4(operand(ql, r, m), operand(kl, t, m), sc[u]);
    }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 2; u++) {
        if (wave + W * u >= 10) continue;
        uint32_t r, t;
        tile_of(wave + W * u, r, t);
        const uint32_t j = 16 * t + c;
        const double aj = as[j];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t ri = 16 * r + 4 * g + i;
            const float w = j <= ri ? qs * expf((float)(rs[ri] + aj)) * sc[u][i] : 0.f;
            pl[ri * PLD + j] = w;
            const float sum = group_sum<16>(w);
            if (c == 0) psum[t][ri] = sum;
        }
    }
#pragma unroll
    for (int r = 0; r < 4; r++) {
        const float4_t f = *(const float4_t *)(carry + 16 * r + 4 * g);
#pragma unroll
        for (int t = 0; t < NCT; t++) acc[r][t] *= f;
    }
    float4_t gate[4][NCT];
#pragma unroll
    for (int r = 0; r < 4; r++)
#pragma unroll
        for (int t = 0; t < NCT; t++)
#pragma unroll
            for (int i = 0; i < 4; i++)
                gate[r][t][i] = p[(uint64_t)min(16u * r + 4 * g + i, live - 1) * dm.in_ld + dm.gate_off() + h * e + min(16 * (wave + W * t) + c, e - 1)];
    __syncthreads();
    if (tid < kChunk) {
        float nq = qn[tid] * carry[tid];
        for (uint32_t t = 0; t <= tid / 16; t++) nq += psum[t][tid];
        dinv[tid] = 1.0f / (fmaxf(fabsf(nq), floor_[tid]) + kFloor);
    }
    // ---- P V
#pragma unroll
    for (int m = 0; m < 4; m++)
#pragma unroll
        for (int r = m; r < 4; r++) {
            const float4_t a = *(const float4_t *)(pl + (16 * r + c) * PLD + 16 * m + 4 * g);
#pragma unroll
            for (int t = 0; t < NCT; t++) acc[r][t] = mfma4(a, v[m][t], acc[r][t]);
        }
    __syncthreads();
    // ---- normaliser, norm, gate
#pragma unroll
    for (int r = 0; r < 4; r++) {
        const float4_t f = *(const float4_t *)(dinv + 16 * r + 4 * g);
        float4_t s2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < NCT; t++) {
            acc[r][t] *= f;
            if (16 * (wave + W * t) + c < e) s2 += acc[r][t] * acc[r][t];
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float x = group_sum<16>(s2[i]);
            if (c == 0) rsum[wave][16 * r + 4 * g + i] = x;
        }
    }
    __syncthreads();
    if (tid < kChunk) {  // (dinv has been used: the root mean square's inverse takes its place)
        float x = 0.f;
#pragma unroll
        for (uint32_t w = 0; w < W; w++) x += rsum[w][tid];
        dinv[tid] = 1.0f / sqrtf(x / (float)e + pr.eps);
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < NCT; t++) {
        const uint32_t col = 16 * (wave + W * t) + c;
        if (col >= e) continue;
        const float w = pr.norm[h * e + col];
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float4_t f = *(const float4_t *)(dinv + 16 * r + 4 * g);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const uint32_t ri = 16 * r + 4 * g + i;
                if (ri >= live) continue;
                const float o = acc[r][t][i] * f[i] * w * fast_sigmoid(gate[r][t][i]);
                if (out) out[((row0 + ri) * H + h) * e + col] = o;
                if (out_lp) out_lp[(row0 + ri) * lp_ld + h * e + col] = f32_to_lp_bits(o, lp_bf16);
            }
        }
    }
}

// ---------------------------------------------------------------- token by token
// 16 lanes share a column of S (lane s of 16 holds rows R s .. R s + R - 1), 4 columns per wave, 16 per
// workgroup; column e is the normaliser, whose value is 1.  raw: [rows][heads][e] read-outs; nq, mt: [rows][heads].
template <int R>
__global__ __launch_bounds__(256) void memory_scan_kernel(const float *__restrict__ proj, MemoryDims dm, MemoryParams pr, MemoryState st,
                                                          uint64_t n, float *__restrict__ raw, float *__restrict__ nq, float *__restrict__ mt) {
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, sub = lane & 15, d = dm.d, e = dm.e, H = dm.heads, h = blockIdx.y;
    const uint32_t col = blockIdx.x * 16 + wave * 4 + (lane >> 4);
    const bool is_n = col == e, is_s = col < e;
    const uint64_t b = blockIdx.z, unit = b * H + h;
    float *sp = is_s ? st.s + unit * d * e + col : st.n + unit * d;
    const uint64_t ld = is_s ? e : 1;
    float s[R], k[R], q[R], v, in, forget, m = st.m[unit];
#pragma unroll
    for (int r = 0; r < R; r++) s[r] = sub * R + r < d ? sp[(sub * R + r) * ld] : 0.f;
    const float qs = 1.0f / sqrtf((float)d);
    auto fetch = [&](uint64_t t) {
        const float *p = proj + (b * n + t) * dm.in_ld;
#pragma unroll
        for (int r = 0; r < R; r++) {
            const uint32_t dim = min(sub * R + r, d - 1);
            const bool real = sub * R + r < d;
            q[r] = real ? p[h * d + dim] * qs : 0.f;
            k[r] = real ? p[dm.k_off() + h * d + dim] : 0.f;
        }
        v = is_s ? p[dm.v_off() + h * e + col] : 1.0f;
        log_gates(p, dm, pr, h, in, forget);
    };
    fetch(0);
    for (uint64_t t = 0; t < n; t++) {
        float kc[R], qc[R];
#pragma unroll
        for (int r = 0; r < R; r++) { kc[r] = k[r]; qc[r] = q[r]; }
        const float fm = forget + m, top = fmaxf(fm, in), keep = expf(fm - top), av = expf(in - top) * v;
        m = top;
        fetch(t + 1 < n ? t + 1 : t);
        float o = 0.f;
#pragma unroll
        for (int r = 0; r < R; r++) {
            s[r] = fmaf(kc[r], av, keep * s[r]);
            o = fmaf(s[r], qc[r], o);
        }
        o = group_sum<16>(o);
        const uint64_t row = b * n + t;
        if (sub == 0 && is_s) raw[(row * H + h) * e + col] = o;
        if (sub == 0 && is_n) { nq[row * H + h] = o; mt[row * H + h] = m; }
    }
    if (is_s || is_n)
#pragma unroll
        for (int r = 0; r < R; r++)
            if (sub * R + r < d) sp[(sub * R + r) * ld] = s[r];
}

// One wave per (row, head).
__global__ __launch_bounds__(256) void memory_finish_kernel(const float *__restrict__ proj, MemoryDims dm, MemoryParams pr, float *m_state,
                                                            uint64_t n, uint64_t units, const float *__restrict__ raw,
                                                            const float *__restrict__ nq, const float *__restrict__ mt,
                                                            float *__restrict__ out, uint16_t *__restrict__ out_lp, uint64_t lp_ld, bool lp_bf16) {
    const uint32_t lane = threadIdx.x & 63, H = dm.heads, e = dm.e;
    const uint64_t u = (uint64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (u >= units) return;
    const uint64_t row = u / H;
    const uint32_t h = (uint32_t)(u % H);
    const float m = mt[u], inv = 1.0f / normaliser(nq[u], m);
    if (lane == 0 && row % n == n - 1) m_state[row / n * H + h] = m;
    float s2 = 0.f;
    for (uint32_t i = lane; i < e; i += 64) s2 = fmaf(raw[u * e + i] * inv, raw[u * e + i] * inv, s2);
    const float f = inv / sqrtf(wave_sum(s2) / (float)e + pr.eps);
    for (uint32_t i = lane; i < e; i += 64) {
        const float o = raw[u * e + i] * f * pr.norm[h * e + i] * fast_sigmoid(proj[row * dm.in_ld + dm.gate_off() + h * e + i]);
        if (out) out[u * e + i] = o;
        if (out_lp) out_lp[row * lp_ld + h * e + i] = f32_to_lp_bits(o, lp_bf16);
    }
}

uint64_t memory_prompt_scratch_bytes(const MemoryDims &dm, uint64_t batch, uint64_t n, bool may_chunk) {
    if (may_chunk && chunked(dm, n)) return chunk_floats(dm, batch * dm.heads, ceil_div(n < kSegment ? n : kSegment, kChunk)) * 4;
    return batch * n * dm.heads * (dm.e + 2ull) * 4;
}

int launch_memory_prompt(const float *proj, const MemoryDims &dm, const MemoryParams &pr, const MemoryState &state, uint64_t batch,
                         uint64_t n, float *out, const LpOut *out_lp, float *scratch, uint64_t scratch_bytes, hipStream_t st,
                         bool may_chunk) {
    COEUS_TRY(check_args(dm, batch, n));
    if (!scratch || scratch_bytes < memory_prompt_scratch_bytes(dm, batch, n, may_chunk))
        return fail(COEUS_INVALID_INPUT, "matrix memory: scratch too small");
    uint16_t *lp = out_lp ? (uint16_t *)out_lp->p : nullptr;
    const uint64_t lp_ld = out_lp ? out_lp->ld : 0;
    const bool lp_bf = out_lp && out_lp->bf16;
    if (may_chunk && chunked(dm, n)) {
        const uint64_t units = batch * dm.heads;
        for (uint64_t t0 = 0; t0 < n; t0 += kSegment) {
            const uint64_t seg = n - t0 < kSegment ? n - t0 : kSegment;
            MemoryChunks cb;
            cb.chunks = (uint32_t)ceil_div(seg, kChunk);
            cb.dtiles = (uint32_t)ceil_div(dm.d, 16);
            cb.etiles = (uint32_t)ceil_div(dm.e, 16);
            float *p = scratch;
            auto take = [&](uint64_t k) { float *r = p; p += round_up(k, 4); return r; };
            const uint64_t cu = units * cb.chunks;
            cb.s = take(cu * cb.dtiles * cb.etiles * 256);
            cb.n = take(cu * dm.d);
            cb.f = take(cu);
            cb.mc = take(cu);
            cb.m0 = take(cu + units);
            const uint32_t cblocks = (uint32_t)ceil_div(dm.e, kColBlock);
            if ((uint64_t)dm.heads * cblocks > 65535) return fail(COEUS_INVALID_INPUT, "matrix memory: too many heads");
            const dim3 lgrid(cb.chunks, dm.heads * cblocks, (unsigned)batch);
#define COEUS_ML(NV) hipLaunchKernelGGL(memory_local_kernel<NV>, lgrid, dim3(256), 0, st, proj, dm, pr, n, t0, seg, cblocks, cb)
            switch (ceil_div(cb.dtiles, 4)) {
                case 1: COEUS_ML(1); break;
                case 2: COEUS_ML(2); break;
                case 3: COEUS_ML(3); break;
                default: COEUS_ML(4); break;
            }
#undef COEUS_ML
            const dim3 cgrid((unsigned)ceil_div(cb.dtiles * cb.etiles * 64 + dm.d + 1, 256), dm.heads, (unsigned)batch);
            hipLaunchKernelGGL(memory_carry_kernel, cgrid, dim3(256), 0, st, dm, state, cb);
            const dim3 rgrid(cb.chunks, dm.heads, (unsigned)batch);
#define COEUS_MR(NV)                                                                                                              \
    do {                                                                                                                          \
        static const bool once = hipFuncSetAttribute((const void *)memory_read_kernel<NV>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                                     136 * 1024) == hipSuccess;                                                   \
        (void)once;                                                                                                               \
        hipLaunchKernelGGL(memory_read_kernel<NV>, rgrid, dim3(512), read_lds_bytes(dm), st, proj, dm, pr, state, n, t0, seg, cb, out, lp, \
                           lp_ld, lp_bf);                                                                                         \
    } while (0)
            if (cb.etiles <= 8) COEUS_MR(1);
            else COEUS_MR(2);
#undef COEUS_MR
        }
        COEUS_HIP(hipGetLastError());
        return COEUS_OK;
    }
    float *raw = scratch, *nq = raw + batch * n * dm.heads * dm.e, *mt = nq + batch * n * dm.heads;
    const dim3 grid((unsigned)ceil_div(dm.e + 1, 16), dm.heads, (unsigned)batch);
#define COEUS_MS(RV) hipLaunchKernelGGL(memory_scan_kernel<RV>, grid, dim3(256), 0, st, proj, dm, pr, state, n, raw, nq, mt)
    if (dm.d <= 16) COEUS_MS(1);
    else if (dm.d <= 32) COEUS_MS(2);
    else if (dm.d <= 64) COEUS_MS(4);
    else if (dm.d <= 128) COEUS_MS(8);
    else if (dm.d <= 256) COEUS_MS(16);
    else COEUS_MS(32);
#undef COEUS_MS
    const uint64_t units = batch * n * dm.heads;
    hipLaunchKernelGGL(memory_finish_kernel, dim3((unsigned)ceil_div(units, 4)), dim3(256), 0, st, proj, dm, pr, state.m, n, units, raw, nq,
                       mt, out, lp, lp_ld, lp_bf);
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

// ---------------------------------------------------------------- decode step
// One workgroup of 512 per (head, sequence), one pass over the state: S^T q of the old state while the new one
// is stored (o = keep S^T q + add (k . q) v).  Thread (g, c) owns columns VW c .. of rows g, g + DG, ..; the
// first RM of them are requested before anything else.
template <int VW, int RM>
__global__ __launch_bounds__(512) void memory_step_kernel(const float *__restrict__ proj, MemoryDims dm, MemoryParams pr, MemoryState st,
                                                          float *__restrict__ out) {
    extern __shared__ float lds[];
    __shared__ float red[8], kq_s, nq_s;
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, H = dm.heads, d = dm.d, e = dm.e;
    const uint64_t b = blockIdx.y, unit = b * H + h;
    const uint32_t cg = (e + VW - 1) / VW, DG = 512 / cg, g0 = tid / cg, c0 = (tid % cg) * VW;  // (VW = 4: e % 4 == 0)
    float *qs = lds, *ks = qs + d, *vs = ks + d, *pq = vs + e;  // pq [DG][e]
    float *S = st.s + unit * d * e, *N = st.n + unit * d;
    const float *p = proj + b * dm.in_ld;
    const bool live = g0 < DG;
    float sr[RM][VW];
    auto load_row = [&](uint32_t r, float (&x)[VW]) {
        const float *sp = S + (uint64_t)r * e + c0;
        if (VW == 4) { const float4 t = *(const float4 *)sp; x[0] = t.x; x[1 % VW] = t.y; x[2 % VW] = t.z; x[3 % VW] = t.w; }
        else x[0] = *sp;
    };
#pragma unroll
    for (int i = 0; i < RM; i++)
        if (live && g0 + i * DG < d) load_row(g0 + i * DG, sr[i]);
        else
#pragma unroll
            for (int t = 0; t < VW; t++) sr[i][t] = 0.f;
    const float qsc = 1.0f / sqrtf((float)d);
    for (uint32_t i = tid; i < d; i += 512) { qs[i] = p[h * d + i] * qsc; ks[i] = p[dm.k_off() + h * d + i]; }
    for (uint32_t i = tid; i < e; i += 512) vs[i] = p[dm.v_off() + h * e + i];
    const float m0 = st.m[unit];
    float in, forget;
    log_gates(p, dm, pr, h, in, forget);
    const float fm = forget + m0, top = fmaxf(fm, in), keep = expf(fm - top), add = expf(in - top);
    __syncthreads();  // (everybody has read the old maximum as well)
    if (wave == 7) {
        float nq = 0.f, kq = 0.f;
        for (uint32_t i = lane; i < d; i += 64) {
            const float nv = N[i];
            nq = fmaf(nv, qs[i], nq);
            kq = fmaf(ks[i], qs[i], kq);
            N[i] = fmaf(add, ks[i], keep * nv);
        }
        nq = wave_sum(nq);
        kq = wave_sum(kq);
        if (lane == 0) { nq_s = nq; kq_s = kq; st.m[unit] = top; }
    }
    if (live) {
        float a[VW], av[VW];
#pragma unroll
        for (int t = 0; t < VW; t++) { a[t] = 0.f; av[t] = add * vs[c0 + t]; }
        auto take = [&](uint32_t r, const float (&x)[VW]) {
            const float kr = ks[r], qr = qs[r];
            float *sp = S + (uint64_t)r * e + c0;
            float y[VW];
#pragma unroll
            for (int t = 0; t < VW; t++) {
                a[t] = fmaf(x[t], qr, a[t]);
                y[t] = fmaf(kr, av[t], keep * x[t]);
            }
            if (VW == 4) *(float4 *)sp = make_float4(y[0], y[1 % VW], y[2 % VW], y[3 % VW]);
            else *sp = y[0];
        };
#pragma unroll
        for (int i = 0; i < RM; i++)
            if (g0 + i * DG < d) take(g0 + i * DG, sr[i]);
        for (uint32_t r = g0 + RM * DG; r < d; r += DG) {
            float x[VW];
            load_row(r, x);
            take(r, x);
        }
#pragma unroll
        for (int t = 0; t < VW; t++) pq[g0 * e + c0 + t] = a[t];
    }
    __syncthreads();
    const float kq = kq_s, inv = 1.0f / normaliser(fmaf(add, kq, keep * nq_s), top);
    float s2 = 0.f;
    for (uint32_t i = tid; i < e; i += 512) {
        float sq = 0.f;
#pragma unroll 8
        for (uint32_t j = 0; j < DG; j++) sq += pq[j * e + i];
        const float o = fmaf(add * kq, vs[i], keep * sq) * inv;
        vs[i] = o;  // (only this thread's own element is read from here on)
        s2 = fmaf(o, o, s2);
    }
    s2 = wave_sum(s2);
    if (lane == 0) red[wave] = s2;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int w = 0; w < 8; w++) tot += red[w];
    const float f = 1.0f / sqrtf(tot / (float)e + pr.eps);
    for (uint32_t i = tid; i < e; i += 512)
        out[unit * e + i] = vs[i] * f * pr.norm[h * e + i] * sigmoid(p[dm.gate_off() + h * e + i]);
}

int launch_memory_step(const float *proj, const MemoryDims &dm, const MemoryParams &pr, const MemoryState &state, uint64_t batch,
                       float *out, hipStream_t st) {
    COEUS_TRY(check_args(dm, batch, 1));
    const bool vec = dm.e % 4 == 0;
    const uint32_t cg = vec ? dm.e / 4 : dm.e;
    if (cg > 512) return fail(COEUS_INVALID_INPUT, "matrix memory: a value size above 512 must be a multiple of 4");
    const uint32_t DG = 512 / cg, per = (uint32_t)ceil_div(dm.d, DG);
    const size_t lds = (2 * (size_t)dm.d + dm.e + (size_t)DG * dm.e) * 4;
    const dim3 grid(dm.heads, (unsigned)batch);
#define COEUS_MT(VWV, RMV) hipLaunchKernelGGL((memory_step_kernel<VWV, RMV>), grid, dim3(512), lds, st, proj, dm, pr, state, out)
    if (vec) { if (per <= 8) COEUS_MT(4, 8); else COEUS_MT(4, 16); }
    else { if (per <= 8) COEUS_MT(1, 8); else COEUS_MT(1, 32); }
#undef COEUS_MT
    COEUS_HIP(hipGetLastError());
    return COEUS_OK;
}

}  // namespace coeus
