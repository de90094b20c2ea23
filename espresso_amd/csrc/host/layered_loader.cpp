#include "layered_loader.h"

#include <cmath>
#include <cstring>

#include "../generation.h"
#include "runtime_registry.h"
#include "safetensors.h"

namespace esp {
namespace {

uint16_t float_to_bf16(float v) {
    uint32_t b;
    std::memcpy(&b, &v, 4);
    return (uint16_t)((b + 0x7FFFu + ((b >> 16) & 1u)) >> 16);
}

class SafetensorsWeights : public LayeredWeights {
  public:
    explicit SafetensorsWeights(const SafetensorsFile &f) : f_(f) {}
    int matrix(const std::string &name, int rows, int cols, std::vector<uint16_t> *out) override {
        const TensorView *t = nullptr;
        const int rc = tensor(name, {rows, cols}, &t);
        if (rc != ESP_OK) return rc;
        if (t->dtype != "BF16") return fail(ESP_ERR_UNSUPPORTED, "tensor %s: matrices are BF16, not %s", name.c_str(), t->dtype.c_str());
        out->resize(t->elements());
        std::memcpy(out->data(), t->data, t->bytes);
        return ESP_OK;
    }
    int vector(const std::string &name, int count, std::vector<float> *out) override {
        const TensorView *t = nullptr;
        const int rc = tensor(name, {count}, &t);
        if (rc != ESP_OK) return rc;
        out->resize(count);
        if (t->dtype == "F32") { std::memcpy(out->data(), t->data, t->bytes); return ESP_OK; }
        if (t->dtype != "BF16" && t->dtype != "F16") return fail(ESP_ERR_UNSUPPORTED, "tensor %s: vectors are BF16, F16 or F32, not %s", name.c_str(), t->dtype.c_str());
        for (int i = 0; i < count; i++) {
            uint16_t b;
            std::memcpy(&b, t->data + 2 * (size_t)i, 2);
            const uint32_t wide = (uint32_t)b << 16;
            if (t->dtype == "BF16") std::memcpy(out->data() + i, &wide, 4);
            else (*out)[i] = half_to_float(b);
        }
        return ESP_OK;
    }

  private:
    int tensor(const std::string &name, const std::vector<int64_t> &shape, const TensorView **out) {
        const TensorView *t = f_.find(name);
        if (!t) return fail(ESP_ERR_IO, "missing tensor %s", name.c_str());
        if (t->shape != shape) {
            std::string want, got;
            for (int64_t d : shape) want += " " + std::to_string(d);
            for (int64_t d : t->shape) got += " " + std::to_string(d);
            return fail(ESP_ERR_INVALID_ARGUMENT, "tensor %s has shape%s, the configuration wants%s", name.c_str(), got.c_str(), want.c_str());
        }
        *out = t;
        return ESP_OK;
    }
    const SafetensorsFile &f_;
};

// Every tensor is a stretch of one table of seeded values, from a start that its name picks.
class SyntheticWeights : public LayeredWeights {
  public:
    SyntheticWeights(uint64_t seed, float std_dev) : seed_(seed), table_(kTable) {
        SplitMix64 g{seed};
        const double span = std_dev * std::sqrt(12.0);
        for (uint16_t &v : table_) v = float_to_bf16((float)((g.unit() - 0.5) * span));
    }
    int matrix(const std::string &name, int rows, int cols, std::vector<uint16_t> *out) override {
        const size_t n = (size_t)rows * cols;
        out->resize(n);
        size_t at = start(name);
        for (size_t i = 0; i < n;) {
            const size_t take = std::min(n - i, kTable - at);
            std::memcpy(out->data() + i, table_.data() + at, take * 2);
            i += take;
            at = 0;
        }
        return ESP_OK;
    }
    int vector(const std::string &name, int count, std::vector<float> *out) override {
        SplitMix64 g{seed_ ^ start(name)};
        auto is = [&](const char *end) { const size_t n = std::strlen(end); return name.size() >= n && name.compare(name.size() - n, n, end) == 0; };
        out->resize(count);
        for (float &v : *out) {
            const double u = g.unit();
            if (is("sink")) v = (float)(u - 0.5);
            else if (is("A_log")) v = (float)std::log(1.0 + 15.0 * u);   // decays and step sizes of a trained model's range
            else if (is("dt_bias")) v = (float)(-6.9 + 4.6 * u);
            else if (is("conv.b")) v = (float)(0.1 * (u - 0.5));
            else v = (float)(0.9 + 0.2 * u);
        }
        return ESP_OK;
    }

  private:
    static constexpr size_t kTable = 4000037;   // a prime: rows of a matrix do not line up with it
    size_t start(const std::string &name) const {
        uint64_t h = 1469598103934665603ull ^ seed_;
        for (unsigned char c : name) h = (h ^ c) * 1099511628211ull;
        return (size_t)(h % kTable);
    }
    uint64_t seed_;
    std::vector<uint16_t> table_;
};

int create(const LayeredConfig &config, const LayeredOptions &options, LayeredWeights &weights, std::unique_ptr<LayeredRuntime> *out) {
    LayeredRuntime *raw = nullptr;
    const int rc = LayeredRuntime::create(config, options, weights, &raw);
    if (rc == ESP_OK) out->reset(raw);
    return rc;
}

}  // namespace

int layered_model_config(const std::string &model_dir, int max_seq, MultiModelConfig *out) {
    LayeredConfig c;
    std::string error;
    if (!load_layered_config(model_dir, &c, &error)) return fail(ESP_ERR_INVALID_ARGUMENT, "%s", error.c_str());
    if (max_seq < 1) return fail(ESP_ERR_INVALID_ARGUMENT, "the context length must be positive");
    MultiModelConfig m;
    m.name = c.architecture;
    m.architecture = MultiModelConfig::Architecture::layered;
    m.nLayer = (int)c.layers.size(); m.dModel = c.width; m.vocab = c.vocab; m.maxSeq = max_seq; m.normEps = (float)c.norm_eps;
    m.nHead = m.nKVHead = c.layers[0].heads; m.headDim = c.layers[0].dim ? c.layers[0].dim : c.layers[0].vdim;   // layers differ: the first one's, for reports
    for (const LayerSpec &L : c.layers) m.hiddenDim = std::max(m.hiddenDim, L.ff);
    *out = m;
    return ESP_OK;
}

int load_layered_model(const std::string &model_dir, const LayeredOptions &options, std::unique_ptr<LayeredRuntime> *out) {
    LayeredConfig c;
    std::string error;
    if (!load_layered_config(model_dir, &c, &error)) return fail(ESP_ERR_INVALID_ARGUMENT, "%s", error.c_str());
    std::unique_ptr<SafetensorsFile> file;
    if (!SafetensorsFile::open(joinPath(model_dir, "model.safetensors"), &file, &error)) return fail(ESP_ERR_IO, "%s", error.c_str());
    SafetensorsWeights weights(*file);
    return create(c, options, weights, out);
}

int make_synthetic_layered_model(const LayeredConfig &config, const LayeredOptions &options, uint64_t seed, float std_dev, std::unique_ptr<LayeredRuntime> *out) {
    SyntheticWeights weights(seed, std_dev);
    return create(config, options, weights, out);
}

namespace {
// The engine's loader: ESPRESSO_HIP_PRECISION = bf16 | f32, ESPRESSO_HIP_MAX_SEQUENCES = sequence slots.
int load_layered(const MultiModelConfig &config, const std::string &modelDir, const Environment &env, std::unique_ptr<DecoderRuntime> *out) {
    LayeredOptions o;
    o.max_seq = config.maxSeq;
    o.eos_token = config.hasEosToken ? (int)config.eosToken : -1;
    auto get = [&](const char *k) { auto it = env.find(k); return it == env.end() ? std::string() : it->second; };
    const std::string precision = get("ESPRESSO_HIP_PRECISION"), sequences = get("ESPRESSO_HIP_MAX_SEQUENCES");
    if (!precision.empty() && precision != "bf16" && precision != "f32") return fail(ESP_ERR_INVALID_ARGUMENT, "ESPRESSO_HIP_PRECISION must be bf16 or f32, not %s", precision.c_str());
    if (precision == "f32") o.precision = Precision::f32;
    if (!sequences.empty()) o.max_sequences = std::atoi(sequences.c_str());
    std::unique_ptr<LayeredRuntime> rt;
    const int rc = load_layered_model(modelDir, o, &rt);
    if (rc != ESP_OK) return rc;
    if (rt->shape().vocab != config.vocab || rt->shape().d_model != config.dModel || (int)rt->config().layers.size() != config.nLayer)
        return fail(ESP_ERR_INVALID_ARGUMENT, "config.json of %s does not match the given configuration", modelDir.c_str());
    *out = std::move(rt);
    return ESP_OK;
}

const RuntimeFamilyRegistration registration(MultiModelConfig::Architecture::layered, load_layered);
}  // namespace

}  // namespace esp
