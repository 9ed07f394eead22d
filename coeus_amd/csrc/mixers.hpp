// Launchers of the token mixers of layered models: the gated delta rule (delta.hip) and windowed
// latent attention (latent.hip).  Rows are batch * n, sequence-major, unless stated.
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

// ---------------------------------------------------------------- latent attention
// Queries and keys / values go through low-rank latents; only the normalised key/value latent c is
// cached, [batch][cap][rank] as a ring (position p in slot p % cap; cap = window, or the context).
struct LatentDims {
    uint32_t heads, d, e, q_rank, rank, window;  // window 0: all earlier positions
    uint32_t in_ld;                              // row stride of the fused projection: query latent | key/value latent
    float scale;
};
struct LatentCache {
    void *c;
    uint32_t cap;
    bool bf16;  // else f32
};
// Normalises both latents of every row.  cq: f32 rows (cq) and / or 16-bit rows (cq_lp); neither: only c.  c goes to
// `lat`, rows of lat_ld elements in the cache's type, row (b, i) at b * lat_rows + lat_off + i; with
// `pos_dev` (one row per sequence) it goes to the cache slot of position *pos_dev instead.
int launch_latent_norm(const float *proj, const LatentDims &dm, const float *q_scale, const float *c_scale, float eps,
                       uint64_t batch, uint64_t n, float *cq, const LpOut *cq_lp, void *lat, uint64_t lat_ld,
                       uint64_t lat_rows, uint64_t lat_off, const LatentCache &cache, const uint32_t *pos_dev,
                       hipStream_t st);
// lat rows [0, hist) of every sequence <- cache positions pos0 - hist .. pos0 - 1
int launch_latent_gather(const LatentCache &cache, uint32_t rank, uint64_t batch, uint64_t hist, uint64_t pos0,
                         void *lat, uint64_t lat_ld, uint64_t lat_rows, hipStream_t st);
// cache <- the last min(n, cap) of the n rows behind `hist` of every sequence (positions pos0 ..)
int launch_latent_append(const void *lat, uint64_t lat_ld, uint64_t lat_rows, uint64_t hist, const LatentCache &cache,
                         uint32_t rank, uint64_t batch, uint64_t n, uint64_t pos0, hipStream_t st);
// Attention of n rows per sequence over hist + n expanded keys / values.  q [batch * n] rows of q_ld
// elements (heads * d); kv [batch * (hist + n)] rows of kv_ld elements (heads * d keys, heads * e values),
// both bf16 or both f32; out f32 [rows, heads * e] or 16-bit rows.
int launch_window_attention(const void *q, uint64_t q_ld, const void *kv, uint64_t kv_ld, bool bf16,
                            const LatentDims &dm, uint64_t batch, uint64_t n, uint64_t hist, float *out,
                            const LpOut *out_lp, hipStream_t st);
// One new token per sequence: its latent, normalised, goes into the ring, and its query is scored against
// the cached latents (its own included).  q [batch, heads * d] f32, ukv [heads * d keys | heads * e
// values][rank] in the cache's type, out [batch, heads * e] f32.
struct LatentNew {
    const float *proj;   // fused projection of the new tokens
    const float *scale;  // [rank]
    float eps;
};
int launch_latent_decode(const float *q, const void *ukv, const LatentDims &dm, const LatentNew &nw,
                         const LatentCache &cache, uint64_t batch, const uint32_t *pos_dev, float *out, float *scratch,
                         uint64_t scratch_bytes, hipStream_t st);
uint64_t latent_decode_scratch_bytes(const LatentDims &dm, const LatentCache &cache, uint64_t batch);

}  // namespace coeus
