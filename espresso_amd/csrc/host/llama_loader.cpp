// Weight directories of llama models (LayerWeightPaths, sidecars, metadata.json) into the GPU-resident runtime.
#include "../llama_runtime.h"
#include "runtime_registry.h"

namespace esp {
namespace {

const int kPackedFormats[] = {FMT_Q4_K, FMT_Q8_0, FMT_Q4_0};

LlamaConfig to_runtime_config(const MultiModelConfig &c, const Environment &env) {
    LlamaConfig r;
    r.n_layer = c.nLayer; r.n_head = c.nHead; r.n_kv_head = c.nKVHead; r.d_model = c.dModel; r.head_dim = c.headDim;
    r.hidden_dim = c.hiddenDim; r.vocab = c.vocab; r.max_seq = c.maxSeq; r.norm_eps = c.normEps; r.rope_theta = c.ropeTheta;
    r.eos_token = c.hasEosToken ? (int)c.eosToken : -1;
    auto it = env.find("ESPRESSO_HIP_KV_CACHE");   // "f16" halves KV traffic; default keeps the reference's fp32 caches
    r.kv_format = (it != env.end() && it->second == "f16") ? FMT_F16 : FMT_F32;
    r.max_sequences = 1;
    return r;
}

// One tensor: packed GGUF blocks if a packed sidecar exists, else the exact float32 sidecar
// (loadWeightTablePreferringFloat32Sidecar, :7830-7879), else the fp16 BLOBFILE payload.
int load_tensor(LlamaRuntime &rt, int layer, int slot, const std::string &path, size_t elements, bool matrix, bool optional,
                bool *present) {
    if (present) *present = false;
    std::vector<uint8_t> raw;
    if (matrix) {
        for (int fmt : kPackedFormats) {
            const std::string p = packedSidecarPath(path, fmt);
            if (!fileExists(p)) continue;
            if (!readFile(p, &raw)) return fail(ESP_ERR_IO, "Failed to read %s", p.c_str());
            if (present) *present = true;
            return rt.set_weight(layer, slot, fmt, raw.data(), raw.size());
        }
    }
    const std::string sidecar = exactFloat32SidecarPath(path);
    if (fileExists(sidecar)) {
        if (!readFile(sidecar, &raw)) return fail(ESP_ERR_IO, "Failed to read float32 sidecar %s", sidecar.c_str());
        if (raw.size() != elements * 4)
            return fail(ESP_ERR_INVALID_ARGUMENT, "invalid weight count in %s: expected %zu, got %zu", sidecar.c_str(), elements, raw.size() / 4);
        if (present) *present = true;
        return rt.set_weight(layer, slot, FMT_F32, raw.data(), raw.size());
    }
    if (!fileExists(path)) {
        if (optional) return ESP_OK;
        return fail(ESP_ERR_IO, "missing weight file %s", path.c_str());
    }
    std::vector<uint16_t> half;
    BlobWeightLoaderError e = BlobWeightLoader::loadFP16(path, &half);
    if (e != BlobWeightLoaderError::none) return fail(ESP_ERR_IO, "BlobWeightLoader error %d for %s", (int)e, path.c_str());
    if (half.size() != elements)
        return fail(ESP_ERR_INVALID_ARGUMENT, "invalid weight count in %s: expected %zu, got %zu", path.c_str(), elements, half.size());
    if (present) *present = true;
    return rt.set_weight(layer, slot, FMT_F16, half.data(), half.size() * 2);
}

int load_llama(const MultiModelConfig &config, const std::string &weightDir, const Environment &env, std::unique_ptr<DecoderRuntime> *out) {
    const std::string bad = validateRuntimeConfig(config);
    if (!bad.empty()) return fail(ESP_ERR_INVALID_ARGUMENT, "%s", bad.c_str());
    if (!directoryExists(weightDir)) return fail(ESP_ERR_IO, "missing path: %s", weightDir.c_str());
    const std::string meta = validateMetadataIfPresent(config, weightDir);
    if (!meta.empty()) return fail(ESP_ERR_INVALID_ARGUMENT, "%s", meta.c_str());
    LlamaTopLevelWeightPaths top;
    std::string err;
    if (!resolveLlamaTopLevelWeightPaths(weightDir, &top, &err)) return fail(ESP_ERR_IO, "%s", err.c_str());

    LlamaRuntime *raw = nullptr;
    int rc = LlamaRuntime::create(to_runtime_config(config, env), &raw);
    if (rc != ESP_OK) return rc;
    std::unique_ptr<LlamaRuntime> rt(raw);
    const size_t d = config.dModel, ad = config.attentionDim(), kd = config.kvDim(), hd = config.hiddenDim, v = config.vocab;
    if ((rc = load_tensor(*rt, 0, SLOT_TOKEN_EMBEDDING, top.tokenEmbedding, v * d, false, false, nullptr)) != ESP_OK) return rc;
    if ((rc = load_tensor(*rt, 0, SLOT_FINAL_NORM, top.finalNormGamma, d, false, false, nullptr)) != ESP_OK) return rc;
    if ((rc = load_tensor(*rt, 0, SLOT_LM_HEAD, top.lmHead, v * d, true, false, nullptr)) != ESP_OK) return rc;
    for (int l = 0; l < config.nLayer; l++) {
        const LayerWeightPaths p = LayerWeightPaths::forLayer(l, config, weightDir);
        struct Item { int slot; const std::string *path; size_t n; bool matrix; };
        const Item items[] = {{SLOT_RMS_ATT, &p.rmsAtt, d, false}, {SLOT_WQ, &p.wq, ad * d, true}, {SLOT_WK, &p.wk, kd * d, true},
                              {SLOT_WV, &p.wv, kd * d, true}, {SLOT_WO, &p.wo, d * ad, true}, {SLOT_RMS_FFN, &p.rmsFfn, d, false},
                              {SLOT_W1, &p.w1, hd * d, true}, {SLOT_W2, &p.w2, d * hd, true}, {SLOT_W3, &p.w3, hd * d, true}};
        for (const Item &it : items)
            if ((rc = load_tensor(*rt, l, it.slot, *it.path, it.n, it.matrix, false, nullptr)) != ESP_OK) return rc;
        // q_norm / k_norm are used only when both files exist (:6585-6607)
        if (fileExists(p.qNorm) && fileExists(p.kNorm)) {
            if ((rc = load_tensor(*rt, l, SLOT_Q_NORM, p.qNorm, config.headDim, false, false, nullptr)) != ESP_OK) return rc;
            if ((rc = load_tensor(*rt, l, SLOT_K_NORM, p.kNorm, config.headDim, false, false, nullptr)) != ESP_OK) return rc;
        }
    }
    if ((rc = rt->finalize()) != ESP_OK) return rc;
    *out = std::move(rt);
    return ESP_OK;
}

const RuntimeFamilyRegistration registration(MultiModelConfig::Architecture::llama, load_llama);

}  // namespace
}  // namespace esp
