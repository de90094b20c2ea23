// Configuration of layered models: decoders whose config.json lists their layers one by one, each with a mixer (a kind of
// attention or a recurrence) and a feed-forward of its own.  An architecture names how its config.json is read and how a layer
// joins its branches to the residual stream; the mixers are shared between architectures.
#pragma once

#include <string>
#include <vector>

namespace esp {

// Rotary positions: pairs of the first `dims` dimensions of a head turn by position * frequency_i.
struct RotarySpec {
    int dims = 0;
    double base = 0;
    bool interleaved = false;        // pairs (2i, 2i + 1); otherwise (i, i + dims / 2)
    // linear: every frequency over the factor.  yarn: frequencies between the `fast` and `slow` turn counts blend towards 1 / factor
    enum class Scaling { none, linear, yarn } scaling = Scaling::none;
    double factor = 1, original = 0, fast = 0, slow = 0;
    // frequency of every pair, and the factor on cosine and sine
    void frequencies(std::vector<double> *f, double *amplitude) const;
    bool operator==(const RotarySpec &o) const;
};

enum class MixerKind { retention, latent_attention, attention, mamba2 };
inline bool has_cache(MixerKind m) { return m == MixerKind::latent_attention || m == MixerKind::attention; }
enum class Activation { silu, gelu_tanh };   // of a gated feed-forward's gate

struct LayerSpec {
    MixerKind mixer = MixerKind::retention;
    int heads = 0, dim = 0, vdim = 0;
    RotarySpec rot;
    std::vector<double> decay;       // retention: one per head
    int kv_rank = 0, rot_dim = 0;    // latent attention: latent size, size of the shared rotated key part
    int kv_heads = 0;                // attention: query head h reads key and value head h / (heads / kv_heads)
    int kv_from = -1;                // either attention: the layer whose cache this layer reads (-1: its own)
    int window = 0;                  // either attention: a token sees itself and the window - 1 tokens before it
    double scale = 0;
    int state = 0, groups = 0;       // mamba2: state size; groups of heads that share B and C
    int conv = 0, norm_groups = 0;   // mamba2: taps of the causal convolution; parts of the output norm
    int ff = 0;                      // width of the gated feed-forward, 0 = none
    Activation activation = Activation::silu;
};

// How a layer's branches join the residual stream.
enum class BlockKind {
    parallel_two_norms,              // x + m * (mixer(norm1 x) + ff(norm2 x))
    sequential_post_norms,           // x + norm1(mixer(x)), then x + norm2(ff(x))
};

struct LayeredConfig {
    std::string architecture;
    BlockKind block = BlockKind::parallel_two_norms;
    int vocab = 0, width = 0;
    bool embed_norm = true;          // the embedding is normed ("embed.norm")
    bool tied_head = false;          // the head is the embedding table (no "head")
    double norm_eps = 0, residual_mult = 1, logit_softcap = 0;   // softcap 0 = none
    std::vector<LayerSpec> layers;
    // [(name, rows, cols)] of every tensor a model of this configuration has (cols 0: a vector)
    struct TensorSpec { std::string name; int rows, cols; };
    std::vector<TensorSpec> tensors() const;
};

struct LayeredArchitecture {
    const char *name;                                            // config.json "architecture"
    bool (*parse)(const struct JsonNode &root, LayeredConfig *out, std::string *error);
};
// Registered architectures; find returns nullptr for an unknown name.
const std::vector<LayeredArchitecture> &layered_architectures();
const LayeredArchitecture *find_layered_architecture(const std::string &name);

bool parse_layered_config(const std::string &json_text, LayeredConfig *out, std::string *error);
// config.json of a model directory
bool load_layered_config(const std::string &model_dir, LayeredConfig *out, std::string *error);
// True when the directory holds a config.json that names a registered architecture.
bool is_layered_model_dir(const std::string &model_dir);

}  // namespace esp
