// Layered decoder models: a stack whose layers name their own token mixer (a recurrence or a kind of
// attention), its sizes, and an optional feed-forward.  Configuration, tensor names and the weight
// file are host code (layered_config.hip, safetensors.hip); the layers run in layered.hip.
#pragma once

#include <memory>

#include "common.hpp"

namespace coeus {

// ---------------------------------------------------------------- JSON (layered_config.hip)
struct Json {
    enum Type { Null, Bool, Number, String, Array, Object } type = Null;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<Json> items;                           // Array
    std::vector<std::pair<std::string, Json>> fields;  // Object, in file order
    const Json *get(const char *key) const;            // Object member or nullptr
};
// Parses one JSON value that fills the text; nesting is limited.  False leaves a message in `err`.
bool json_parse(const char *text, uint64_t len, Json &out, std::string &err);

// ---------------------------------------------------------------- configuration (layered_config.hip)
enum class MixerKind : uint32_t { GatedDelta, LatentAttention, MatrixMemory, SharedKv };

struct MixerSpec {
    MixerKind kind = MixerKind::GatedDelta;
    uint64_t heads = 0, dim = 0, vdim = 0;  // query/key size and value size per head
    // GatedDelta: q/k heads (each shared by heads / kv_heads value heads) and taps of the short convolution
    // SharedKv: heads of keys, which are also the values (vdim = dim)
    uint64_t kv_heads = 0, conv = 0;
    // LatentAttention: sizes of the query and key/value latents
    uint64_t q_rank = 0, kv_rank = 0;
    // attention: score scale, window (0: every earlier position; else position i sees the `window` positions
    // that end at i)
    uint64_t window = 0;
    float scale = 0.f;
    float gate_cap = 0.f;  // MatrixMemory: the gates' logarithms are cap * tanh(x / cap)
    uint64_t conv_channels() const { return 2 * kv_heads * dim + heads * vdim; }
    uint64_t inner() const { return heads * vdim; }
    // rows of the fused input projection: q | k | v | gate | step size | decay, query latent | key/value latent,
    // q | k | v | gate | input gate | forget gate, or q | k | gate
    uint64_t in_rows() const {
        switch (kind) {
            case MixerKind::GatedDelta: return conv_channels() + inner() + 2 * heads;
            case MixerKind::LatentAttention: return q_rank + kv_rank;
            case MixerKind::MatrixMemory: return 2 * heads * dim + 2 * inner() + 2 * heads;
            default: return heads * dim + kv_heads * dim + inner();
        }
    }
    bool operator==(const MixerSpec &o) const {
        return kind == o.kind && heads == o.heads && dim == o.dim && vdim == o.vdim && kv_heads == o.kv_heads && conv == o.conv &&
               q_rank == o.q_rank && kv_rank == o.kv_rank && window == o.window && scale == o.scale && gate_cap == o.gate_cap;
    }
};

// What stands between a feed-forward's two matrices: silu(gate) * up, or with both halves clamped
// g = min(gate, limit), u = clamp(up, -limit, limit): g * sigmoid(1.702 g) * (u + 1).
enum class GateKind : uint32_t { Silu, Clamped };

struct LayerSpec {
    MixerSpec mixer;
    uint64_t ff = 0;  // width of the gated feed-forward, 0: none
    GateKind gate = GateKind::Silu;
    float limit = 0.f;
    uint64_t source = 0;  // the layer whose tensors this one uses (its own number: it has its own)
};

struct LayeredConfig {
    std::string architecture;
    uint64_t width = 0, vocab = 0;
    float eps = 0.f;
    float embed_scale = 1.f;
    float logit_softcap = 0.f;  // 0: none
    bool tied = true;           // the embedding table is the output projection
    // 0: one residual stream; each sublayer reads it and its RMS-normalised, scaled output is added.  Else
    // hyper-connections: that many streams; a sublayer reads the layer norm of their weighted sum, then
    // stream t becomes sum_s mix[s][t] x_s + residual_mult out[t] y.
    uint64_t streams = 0;
    float residual_mult = 1.f;
    std::vector<LayerSpec> layers;
};

// What a weight holds when no file provides it (synthetic models): mean + spread * z.
struct TensorSpec {
    std::string name;
    uint64_t rows = 0, cols = 0;  // cols 0: a vector of `rows`
    float mean = 0.f;
    uint64_t elems() const { return rows * (cols ? cols : 1); }
};

// Reads a config.json text; "architecture" selects the reader from the registry.
int layered_config_parse(const char *text, uint64_t len, LayeredConfig &out);
// Every tensor of a configuration with its shape, in a fixed order.
std::vector<TensorSpec> layered_tensors(const LayeredConfig &c);
std::string layer_tensor(uint64_t layer, const char *suffix);  // "l<layer>.<suffix>"

// ---------------------------------------------------------------- weight files (safetensors.hip)
struct SafeTensor {
    std::string dtype;  // "BF16", "F32", ...
    std::vector<uint64_t> shape;
    const uint8_t *data = nullptr;
    uint64_t bytes = 0;
};
// A safetensors file mapped read-only: 8-byte little-endian header length, JSON header, data.
class SafeTensors {
public:
    SafeTensors() = default;
    ~SafeTensors();
    SafeTensors(const SafeTensors &) = delete;
    SafeTensors &operator=(const SafeTensors &) = delete;
    int open(const std::string &path);
    const SafeTensor *find(const std::string &name) const;
    uint64_t count() const { return tensors_.size(); }

private:
    void *map_ = nullptr;
    uint64_t size_ = 0;
    std::vector<std::pair<std::string, SafeTensor>> tensors_;  // sorted by name
};
int read_text_file(const std::string &path, std::string &out);
// Checks that the file holds exactly the shapes of `want`, in a type that can be converted.
int check_tensors(const SafeTensors &file, const std::vector<TensorSpec> &want);

}  // namespace coeus
