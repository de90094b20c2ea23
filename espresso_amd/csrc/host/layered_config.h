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
    bool scaled = false;             // YaRN: frequencies between the `fast` and `slow` turn counts blend towards 1 / factor
    double factor = 1, original = 0, fast = 0, slow = 0;
    // frequency of every pair, and the factor on cosine and sine
    void frequencies(std::vector<double> *f, double *amplitude) const;
    bool operator==(const RotarySpec &o) const;
};

enum class MixerKind { retention, latent_attention };

struct LayerSpec {
    MixerKind mixer = MixerKind::retention;
    int heads = 0, dim = 0, vdim = 0;
    RotarySpec rot;
    std::vector<double> decay;       // retention: one per head
    int kv_rank = 0, rot_dim = 0;    // latent attention: latent size, size of the shared rotated key part
    int kv_from = -1;                // latent attention: the layer whose cached latents this layer reads (-1: its own)
    int window = 0;                  // latent attention: a token sees itself and the window - 1 tokens before it
    double scale = 0;
    int ff = 0;                      // width of the gated feed-forward, 0 = none
};

// How a layer's branches join the residual stream.
enum class BlockKind {
    parallel_two_norms,              // x + m * (mixer(norm1 x) + ff(norm2 x))
};

struct LayeredConfig {
    std::string architecture;
    BlockKind block = BlockKind::parallel_two_norms;
    int vocab = 0, width = 0;
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
