// Model / session objects behind the C ABI.
#pragma once

#include <memory>

#include "common.hpp"
#include "layered.hpp"
#include "mixers.hpp"

namespace coeus {

const char *last_error();
int validate_config(const coeus_config &c);
void positional_encoding_host(uint64_t max_seq_len, uint64_t hidden, float *table);
bool profiler_attached();
const char *graph_replay_forbidden();

struct DeviceBuf {
    void *p = nullptr;
    uint64_t bytes = 0;
    int ensure(uint64_t want);  // grows (contents are not preserved)
    void release();
};

struct LayerWeights {
    Weight qkv, o, up, down;  // up holds interleaved (gate, up) rows for a gated FFN
    const float *ln1_s = nullptr, *ln1_b = nullptr, *ln2_s = nullptr, *ln2_b = nullptr;
    const float *b_qkv = nullptr, *b_o = nullptr, *b_up = nullptr, *b_down = nullptr;
};

// What stands around one sublayer of a layered model: its norm, then either the per-channel scale of a norm
// behind it, or the hyper-connections' weights.
struct Around {
    const float *norm = nullptr, *ls = nullptr;
    const float *in = nullptr, *out = nullptr, *mix = nullptr;
};
// One layer of a layered model on the device (one that uses another's tensors holds none).
struct LayeredLayer {
    LayerSpec spec;
    Weight in, o, up, down;  // fused input projection, output projection; up: interleaved (gate, up) rows
    Weight uq, ukv;          // latent attention: query expansion; key and value expansions, one behind the other
    DeltaParams delta{};
    const float *dq_norm = nullptr, *dkv_norm = nullptr;
    MemoryParams memory{};
    const float *wqk = nullptr;  // shared keys and values: query norm weight * key norm weight
    Around around_mixer, around_ff;
    DeltaDims delta_dims() const;
    LatentDims latent_dims() const;
    MemoryDims memory_dims() const;
    SharedKvDims shared_dims() const;
};
struct LayeredStack {
    LayeredConfig cfg;
    std::vector<LayeredLayer> layers;
    float *small = nullptr;  // every f32 vector of every layer
    float *folds = nullptr;  // kHyperFoldFloats per sublayer, in their order (hyper-connections that can be folded)
    ~LayeredStack();
    const LayeredLayer &weights(size_t l) const { return layers[cfg.layers[l].source]; }
};
// What the sequences of a session carry from token to token, layer by layer: matrix states and
// convolution rings of recurrent layers, rings of cached rows of attention layers.
struct LayeredState {
    struct Layer {
        DeltaState delta{};
        MemoryState memory{};
        RowRing ring{};  // latents, or keys that are also the values
    };
    std::vector<Layer> layers;
    DeviceBuf mem;
    uint64_t batch = 0, recurrent_bytes = 0;  // the recurrent part comes first in `mem` and starts at zero
    int create(const LayeredStack &stack, bool bf16, uint64_t batch, uint64_t max_ctx, hipStream_t st);
    int clear(hipStream_t st);  // start of another sequence
    void release() { mem.release(); layers.clear(); }
};

struct Model;

// Activation buffers of the matrix-core (prefill) path, grown on demand.
struct Workspace {
    uint64_t rows = 0;
    DeviceBuf h, x, qkv, att, ff, ids, a_lp, b_lp, w_lp, logits, xq, norm_part, gemm_part;
    DeviceBuf mix, lat, q_lp, kv_lp;  // layered models: mixer operands, cached and new rows, queries / keys and values
    DeviceBuf streams;                // hyper-connections: [rows][streams][hidden]
    GemmScratch gs;
    int ensure(const Model &m, uint64_t rows_needed, uint64_t logit_rows);
    void release();
};

struct Cache {
    void *k, *v;
    uint64_t max_ctx;
    uint64_t layer_bytes;
    bool per_layer;  // false: one layer's worth of storage reused by every layer
};

struct Model {
    coeus_config cfg{};
    Layout L{};
    uint64_t n_params = 0, weight_bytes = 0;
    std::vector<LayerWeights> layers;
    Weight out;
    void *embed = nullptr;
    bool embed_bf16 = false;
    float *pe = nullptr, *small = nullptr;
    const float *fin_s = nullptr, *fin_b = nullptr;
    hipStream_t stream = nullptr;
    std::mutex mu;  // serialises every call that touches the stream or the workspaces
    Workspace ws;
    DeviceBuf tmp_k, tmp_v;
    // HBM that resident f16 copies of quantised weights may still take (prefill matmul operands)
    static constexpr uint64_t kExpandBudget = 64ull << 30;
    uint64_t expand_budget = kExpandBudget;
    float embed_scale = 1.f, logit_softcap = 0.f;
    std::unique_ptr<LayeredStack> stack;  // set: the blocks are the stack's layers, not `layers`
    ~Model();
    uint32_t streams() const { return stack && stack->cfg.streams ? (uint32_t)stack->cfg.streams : 1; }
    Epilogue logits_epilogue(float *dst) const {
        Epilogue e;
        e.out_f32 = dst;
        if (logit_softcap > 0.f) { e.act = COEUS_EPI_SOFTCAP; e.limit = logit_softcap; }
        return e;
    }
};

struct Session {
    Model *m = nullptr;
    uint64_t batch = 0, max_ctx = 0, pos = 0, layer_bytes = 0;
    uint32_t bp = 1, nsplit = 1;
    bool use_graph = true;
    bool fuse = true;  // fold norms into the decode matmuls where possible
    uint32_t host_pos[2] = {0, 0};
    DeviceBuf kc, vc;
    LayeredState state;  // layered models (instead of kc / vc)
    Workspace ws;  // prefill
    DeviceBuf dh, dx, dqkv, datt, dff, dlogits, dids, dpos, dhist, dpart, dcount, dstats, xq_h, xq_inner, xq_ff, xq_g;
    DeviceBuf drows, dwant;    // rows whose logits session_feed was asked for
    DeviceBuf dh2;             // layered models: the residual stream changes buffers at every folded norm
    DeviceBuf dmix, dscratch;  // layered models: latent queries of a decode step, attention partials
    hipGraph_t graph = nullptr;
    hipGraphExec_t graph_exec = nullptr;
    ~Session();
};

int model_create(const coeus_config &cfg, const float *params, uint64_t n_params, uint64_t seed,
                 Model **out);
int model_forward(Model &m, const uint64_t *ids, uint64_t seq_len, float *logits_out, bool all_rows);
int session_create(Model &m, uint64_t batch, uint64_t max_ctx, Session **out);
int session_prefill(Session &s, const uint64_t *ids, uint64_t n, float *logits_out);
int session_feed(Session &s, const uint64_t *ids, uint64_t n, const uint64_t *want, uint64_t n_want,
                 float *logits_out, float *residuals_out);
int session_reset(Session &s);
int session_decode(Session &s, const uint64_t *ids, float *logits_out);
int session_decode_greedy(Session &s, const uint64_t *first_ids, uint64_t n_steps, uint64_t *out_ids,
                          const coeus_sampling *sampling = nullptr);

int session_time_decode_matmuls(Session &s, uint64_t reps, float *ms_out, uint64_t *launches_out,
                                uint64_t *bytes_out);
int session_time_decode_attention(Session &s, uint64_t reps, float *ms_out, uint64_t *launches_out,
                                  uint64_t *bytes_out);

// ---------------------------------------------------------------- layered models (layered.hip)
int layered_load(const char *dir, const coeus_load_options &opt, Model **out);
int layered_create_seeded(const char *json, uint64_t len, const coeus_load_options &opt, uint64_t seed, Model **out);
int layered_workspace(const Model &m, Workspace &ws, uint64_t batch, uint64_t n, uint64_t pos0);
// All layers over n new rows per sequence; the residual stream is in ws.h.  residuals (nullable, host):
// [layer][batch * n][width] after every layer.
int layered_prefill(Model &m, Workspace &ws, LayeredState &state, uint64_t batch, uint64_t n, uint64_t pos0,
                    float *residuals, hipStream_t st);
int layered_session_init(Session &s);
// Parts of a decode step: everything, only the matmuls, or only the mixers.
enum { STEP_ALL = 0, STEP_MATMULS = 1, STEP_ATTENTION = 2 };
int layered_decode(Session &s, hipStream_t st, int only, uint64_t *launches, uint64_t *bytes);
uint64_t gemv_algorithmic_bytes(const Weight &w, uint64_t batch, bool gated, bool normed);
int check_device();

}  // namespace coeus
