// Launchers of the token mixers of layered models: the gated delta rule (delta.hip), the matrix memory
// (memory.hip), and windowed attention (window.hip) through latents (latent.hip) or on keys that are also the
// values (shared_kv.hip).  Rows are batch * n, sequence-major, unless stated.
#pragma once

#include "common.hpp"

namespace coeus {

// ---------------------------------------------------------------- gated delta rule
// Per head, with a state S [d, e] in f32:
//   S <- exp(lg) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// q and k (unit vectors, q also / sqrt(d)) are shared by heads / kv_heads heads; q, k, v have passed a
// causal convolution of `taps` taps per channel and a SiLU.
struct DeltaDims {
    uint32_t heads, kv_heads, d, e, taps;
    uint32_t in_ld;  // row stride of the fused projection: q | k | v | gate | step size | decay (| padding)
    __host__ __device__ uint32_t channels() const { return 2 * kv_heads * d + heads * e; }
    __host__ __device__ uint32_t gate_off() const { return channels(); }
    __host__ __device__ uint32_t beta_off() const { return channels() + heads * e; }
    __host__ __device__ uint32_t decay_off() const { return beta_off() + heads; }
};
struct DeltaParams {
    const float *conv;     // [taps][channels], tap taps - 1 meets the newest input
    const float *exp_a;    // [heads] exp(A_log)
    const float *dt_bias;  // [heads]
    const float *norm;     // [e]
    float eps;
};
// Per-sequence state: S [batch][heads][d][e]; ring [batch][taps][channels]: the projection of position p
// lives in slot p % taps, so the step that writes position p overwrites the one slot it does not read.
struct DeltaState {
    float *s;
    float *ring;
};
uint32_t delta_padded_dim(uint32_t d);  // row length of prepared q and k: d rounded up, zeros behind
// Prepared operands of a prompt: q, k [rows][kv_heads][dp], v [rows][heads * e], beta, log decay [rows][heads]
struct DeltaOperands {
    float *q, *k, *v, *beta, *lg;
};
int launch_delta_prepare(const float *proj, const DeltaDims &dm, const DeltaParams &pr, const DeltaState &state,
                         uint64_t batch, uint64_t n, uint64_t pos0, const DeltaOperands &op, hipStream_t st);
// The recurrence over the n new tokens of every sequence: o [rows][heads * e], state updated.
int launch_delta_prompt(const DeltaDims &dm, const DeltaOperands &op, const DeltaState &state, uint64_t batch,
                        uint64_t n, float *o, float *scratch, uint64_t scratch_bytes, hipStream_t st);
uint64_t delta_prompt_scratch_bytes(const DeltaDims &dm, uint64_t batch, uint64_t n);
// out = RMSNorm(o per head) * silu(gate), f32 rows (out) and / or 16-bit rows (out_lp)
int launch_delta_gate(const float *o, const float *proj, const DeltaDims &dm, const DeltaParams &pr, uint64_t rows,
                      float *out, const LpOut *out_lp, hipStream_t st);
// One new token per sequence, all of the above in one launch; position from *pos_dev.
int launch_delta_step(const float *proj, const DeltaDims &dm, const DeltaParams &pr, const DeltaState &state,
                      uint64_t batch, const uint32_t *pos_dev, float *out, hipStream_t st);
// Ring slots of the last min(n, taps) of n rows at positions pos0 ..
int launch_delta_ring(const float *proj, const DeltaDims &dm, const DeltaState &state, uint64_t batch, uint64_t n,
                      uint64_t pos0, hipStream_t st);

// ---------------------------------------------------------------- matrix memory
// Per head, with a state S [d, e], a normaliser n [d] and a running maximum m, all f32 and zero at the start,
// log gates i = cap tanh((x_i + in_bias) / cap), f = logsigmoid(cap tanh((x_f + forget_bias) / cap)):
//   m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n alike with v = 1;  m <- m'
//   o = S^T q / (max(|n . q|, e^-m) + 1e-6),  q scaled by 1 / sqrt(d)
// then per head o / rms(o), times norm, times sigmoid(gate).
struct MemoryDims {
    uint32_t heads, d, e;
    uint32_t in_ld;  // row stride of the fused projection: q | k | v | gate | input gate | forget gate (| padding)
    float cap;
    __host__ __device__ uint32_t k_off() const { return heads * d; }
    __host__ __device__ uint32_t v_off() const { return 2 * heads * d; }
    __host__ __device__ uint32_t gate_off() const { return 2 * heads * d + heads * e; }
    __host__ __device__ uint32_t in_off() const { return 2 * heads * (d + e); }
    __host__ __device__ uint32_t forget_off() const { return in_off() + heads; }
};
struct MemoryParams {
    const float *in_bias, *forget_bias;  // [heads]
    const float *norm;                   // [heads * e]
    float eps;
};
struct MemoryState {
    float *s, *n, *m;  // [batch][heads][d][e], [batch][heads][d], [batch][heads]
};
// n new tokens per sequence: f32 rows (out) and / or 16-bit rows (out_lp), state moved on.  may_chunk false:
// token by token whatever the length.
int launch_memory_prompt(const float *proj, const MemoryDims &dm, const MemoryParams &pr, const MemoryState &state, uint64_t batch,
                         uint64_t n, float *out, const LpOut *out_lp, float *scratch, uint64_t scratch_bytes, hipStream_t st,
                         bool may_chunk = true);
uint64_t memory_prompt_scratch_bytes(const MemoryDims &dm, uint64_t batch, uint64_t n, bool may_chunk = true);
int launch_memory_step(const float *proj, const MemoryDims &dm, const MemoryParams &pr, const MemoryState &state, uint64_t batch,
                       float *out, hipStream_t st);

// ---------------------------------------------------------------- rings and windowed attention
// Rows of a fixed length per sequence, [batch][cap]: position p in slot p % cap (cap = window, or the context).
struct RowRing {
    void *c;
    uint32_t cap;
    bool bf16;  // else f32
};
// buffer rows [0, hist) of every sequence <- ring positions pos0 - hist .. pos0 - 1; buffer row (b, i) lies at
// (b * rows_per_seq + i) * ld elements, ring rows are len elements
int launch_ring_gather(const RowRing &ring, uint32_t len, uint64_t batch, uint64_t hist, uint64_t pos0, void *buf, uint64_t ld,
                       uint64_t rows_per_seq, hipStream_t st);
// ring <- the last min(n, cap) of the n rows behind `hist` of every sequence (positions pos0 ..)
int launch_ring_append(const void *buf, uint64_t ld, uint64_t rows_per_seq, uint64_t hist, const RowRing &ring, uint32_t len,
                       uint64_t batch, uint64_t n, uint64_t pos0, hipStream_t st);
struct WindowShape {
    uint32_t heads, d, e, window;  // window 0: all earlier positions
    float scale;
    // kv_heads 0: rows of kv hold heads * d keys, then heads * e values.  Else they hold kv_heads * d keys, each
    // head's shared by heads / kv_heads query heads, which are the values too (e = d), and at element rms_off
    // an f32 that scores with this row are multiplied by; then from the score slope(h) * distance is taken off,
    // and outputs are multiplied by sigmoid(gate).
    uint32_t kv_heads = 0, rms_off = 0;
    float slope_range = 0.f;  // slope(h) = 2^(-slope_range (h + 1) / heads); 0: no slopes
    const float *gate = nullptr;  // rows of gate_ld floats, heads * e used
    uint64_t gate_ld = 0;
    __device__ float slope(uint32_t h) const { return slope_range == 0.f ? 0.f : exp2f(-slope_range * (float)(h + 1) / (float)heads); }
};
// Attention of n rows per sequence over hist + n rows of keys and values, all bf16 or all f32; q [batch * n]
// rows of q_ld elements (heads * d); kv [batch * (hist + n)] rows of kv_ld elements, the last n of a sequence
// being the queries' own.  out f32 [rows, heads * e] or 16-bit rows.
int launch_window_attention(const void *q, uint64_t q_ld, const void *kv, uint64_t kv_ld, bool bf16,
                            const WindowShape &dm, uint64_t batch, uint64_t n, uint64_t hist, float *out,
                            const LpOut *out_lp, hipStream_t st);

// ---------------------------------------------------------------- attention whose values are its keys
// The projection's rows are q | k | gate (| padding).  q and k are normalised over all heads at once, so a
// cached row is the keys as projected, which the values are, and one f32, their inverse root mean square; the
// norms' weights meet in the query: wqk [heads * d] = q weight * k weight of the key head it looks at.
struct SharedKvDims {
    uint32_t heads, kv_heads, d, window;
    uint32_t in_ld;
    float scale, slope_range;
    __host__ __device__ uint32_t k_off() const { return heads * d; }
    __host__ __device__ uint32_t gate_off() const { return (heads + kv_heads) * d; }
    __host__ __device__ uint32_t rms_off() const { return (kv_heads * d + 7) / 8 * 8; }
    __host__ __device__ uint32_t row_len() const { return rms_off() + 8; }
    WindowShape window_shape(const float *gate) const {
        WindowShape s{heads, d, d, window, scale};
        s.kv_heads = kv_heads; s.rms_off = rms_off(); s.slope_range = slope_range; s.gate = gate; s.gate_ld = in_ld;
        return s;
    }
};
// Queries of every row, normalised and weighted, f32 or bf16 rows of heads * d (q); its cached row goes to
// kv row (b, i) at (b * kv_rows + kv_off + i) * row_len elements.
int launch_shared_kv_prepare(const float *proj, const SharedKvDims &dm, const float *wqk, float eps, uint64_t batch, uint64_t n,
                             bool bf16, void *q, void *kv, uint64_t kv_rows, uint64_t kv_off, hipStream_t st);
// One new token per sequence, from its projection to the gated output [batch, heads * d] f32; its row goes into
// the ring.  counters: zeros, left as zeros.
int launch_shared_kv_decode(const float *proj, const SharedKvDims &dm, const float *wqk, float eps, const RowRing &ring,
                            uint64_t batch, const uint32_t *pos_dev, float *out, float *scratch, uint64_t scratch_bytes,
                            uint32_t *counters, uint64_t n_counters, hipStream_t st);
uint64_t shared_kv_decode_scratch_bytes(const SharedKvDims &dm, const RowRing &ring, uint64_t batch);
uint64_t shared_kv_decode_counters(const SharedKvDims &dm, uint64_t batch);

// ---------------------------------------------------------------- latent attention
// Queries and keys / values go through low-rank latents; only the normalised key/value latent c is
// cached, in a ring of rows of `rank` elements.
struct LatentDims {
    uint32_t heads, d, e, q_rank, rank, window;  // window 0: all earlier positions
    uint32_t in_ld;                              // row stride of the fused projection: query latent | key/value latent
    float scale;
    WindowShape window_shape() const { return WindowShape{heads, d, e, window, scale}; }
};
// Normalises both latents of every row.  cq: f32 rows (cq) and / or 16-bit rows (cq_lp); neither: only c.  c goes to
// `lat`, rows of lat_ld elements in the cache's type, row (b, i) at b * lat_rows + lat_off + i; with
// `pos_dev` (one row per sequence) it goes to the cache slot of position *pos_dev instead.
int launch_latent_norm(const float *proj, const LatentDims &dm, const float *q_scale, const float *c_scale, float eps,
                       uint64_t batch, uint64_t n, float *cq, const LpOut *cq_lp, void *lat, uint64_t lat_ld,
                       uint64_t lat_rows, uint64_t lat_off, const RowRing &cache, const uint32_t *pos_dev,
                       hipStream_t st);
// One new token per sequence: its latent, normalised, goes into the ring, and its query is scored against
// the cached latents (its own included).  q [batch, heads * d] f32, ukv [heads * d keys | heads * e
// values][rank] in the cache's type, out [batch, heads * e] f32.
struct LatentNew {
    const float *proj;   // fused projection of the new tokens
    const float *scale;  // [rank]
    float eps;
};
int launch_latent_decode(const float *q, const void *ukv, const LatentDims &dm, const LatentNew &nw,
                         const RowRing &cache, uint64_t batch, const uint32_t *pos_dev, float *out, float *scratch,
                         uint64_t scratch_bytes, hipStream_t st);
uint64_t latent_decode_scratch_bytes(const LatentDims &dm, const RowRing &cache, uint64_t batch);

}  // namespace coeus
