// C ABI: model configurations (metadata.json, config.json, the registries) and the inference engine.
#include "capi_common.h"
#include "host/layered_loader.h"

using namespace esp;
using namespace esp::capi;

extern "C" {

int esp_model_config_load_metadata(const char *path, ESPModelConfig *out) {
    if (!path || !out) return fail(ESP_ERR_INVALID_ARGUMENT, "null pointer");
    MultiModelConfig m;
    std::string err;
    if (!loadConfigFromMetadataFile(path, &m, &err)) return fail(ESP_ERR_IO, "%s", err.c_str());
    to_c(m, out);
    return ESP_OK;
}

int esp_model_config_write_metadata(const ESPModelConfig *config, const char *path) {
    if (!path || !config) return fail(ESP_ERR_INVALID_ARGUMENT, "null pointer");
    const std::string j = metadataJSON(from_c(*config));
    return writeFile(path, j.data(), j.size()) ? ESP_OK : fail(ESP_ERR_IO, "cannot write %s", path);
}

int esp_model_config_load_dir(const char *model_dir, int max_seq, ESPModelConfig *out) {
    if (!model_dir || !out) return fail(ESP_ERR_INVALID_ARGUMENT, "null argument");
    MultiModelConfig m;
    if (is_layered_model_dir(model_dir) || !fileExists(joinPath(model_dir, "metadata.json"))) {
        const int rc = layered_model_config(model_dir, max_seq, &m);
        if (rc != ESP_OK) return rc;
    } else {
        std::string err;
        if (!loadConfigFromMetadataFile(joinPath(model_dir, "metadata.json"), &m, &err)) return fail(ESP_ERR_INVALID_ARGUMENT, "%s", err.c_str());
    }
    to_c(m, out);
    return ESP_OK;
}

int esp_layered_architecture_count(void) { return (int)layered_architectures().size(); }
const char *esp_layered_architecture_at(int index) {
    return index >= 0 && index < (int)layered_architectures().size() ? layered_architectures()[index].name : nullptr;
}

int esp_model_registry_count(void) { return (int)ModelRegistry::all().size(); }
int esp_model_registry_at(int index, ESPModelConfig *out) {
    if (!out || index < 0 || index >= (int)ModelRegistry::all().size()) return fail(ESP_ERR_INVALID_ARGUMENT, "model registry: index %d", index);
    to_c(ModelRegistry::all()[(size_t)index], out);
    return ESP_OK;
}
int esp_model_registry_config(const char *name, ESPModelConfig *out) {
    if (!name || !out) return fail(ESP_ERR_INVALID_ARGUMENT, "model registry: null argument");
    const MultiModelConfig *c = ModelRegistry::config(name);
    if (!c) return fail(ESP_ERR_INVALID_ARGUMENT, "model registry: no configuration named %s", name);
    to_c(*c, out);
    return ESP_OK;
}
int esp_classifier_strategy_select(const ESPModelConfig *config, int has_exact_float32_lm_head, char *out_label, size_t label_bytes) {
    if (!config) return fail(ESP_ERR_INVALID_ARGUMENT, "classifier strategy: null config");
    const ClassifierStrategy s = selectClassifierStrategy(from_c(*config), has_exact_float32_lm_head != 0);
    if (out_label && label_bytes) { std::strncpy(out_label, exactHeadBackendLabel(s), label_bytes - 1); out_label[label_bytes - 1] = 0; }
    return (int)s;
}

ESPEngine *esp_engine_build(const ESPModelConfig *config, const char *weight_dir, const char *tokenizer_dir,
                            const char *const *env_keys, const char *const *env_values, int env_count) {
    if (!config || !weight_dir) { fail(ESP_ERR_INVALID_ARGUMENT, "null config or weight directory"); return nullptr; }
    std::unique_ptr<RealModelInferenceEngine> e;
    if (RealModelInferenceEngine::build(from_c(*config), weight_dir, tokenizer_dir ? tokenizer_dir : "",
                                        env_from(env_keys, env_values, env_count), &e) != ESP_OK)
        return nullptr;
    ESPEngine *h = new ESPEngine();
    h->engine = std::move(e);
    h->runtime_handle.rt = &h->engine->runtime();
    return h;
}

void esp_engine_free(ESPEngine *engine) { delete engine; }

ESPLlamaRuntime *esp_engine_runtime(ESPEngine *engine) { return engine ? &engine->runtime_handle : nullptr; }

int esp_engine_generate(ESPEngine *engine, const uint32_t *prompt_tokens, int prompt_count, int max_tokens, float temperature,
                        const char *const *env_keys, const char *const *env_values, int env_count, uint32_t *out_tokens,
                        ESPGenerationResult *result) {
    if (!engine) return fail(ESP_ERR_INVALID_ARGUMENT, "null engine");
    std::vector<TokenID> prompt;
    if (prompt_tokens && prompt_count > 0) prompt.assign(prompt_tokens, prompt_tokens + prompt_count);
    GenerationResult r;
    int rc = engine->engine->generate(prompt, max_tokens, temperature, env_from(env_keys, env_values, env_count), &r);
    if (rc != ESP_OK) return rc;
    if (out_tokens) for (size_t i = 0; i < r.tokens.size(); i++) out_tokens[i] = r.tokens[i];
    if (result) fill_result(r, result);
    return ESP_OK;
}

int esp_engine_generate_text(ESPEngine *engine, const char *prompt_utf8, size_t prompt_bytes, int max_tokens, float temperature,
                             const char *const *env_keys, const char *const *env_values, int env_count, uint32_t *out_tokens,
                             char *out_text, size_t text_capacity, size_t *out_text_bytes, ESPGenerationResult *result) {
    if (!engine || (!prompt_utf8 && prompt_bytes)) return fail(ESP_ERR_INVALID_ARGUMENT, "null engine or prompt");
    GenerationResult r;
    int rc = engine->engine->generateText(std::string(prompt_utf8 ? prompt_utf8 : "", prompt_bytes), max_tokens, temperature,
                                          env_from(env_keys, env_values, env_count), &r);
    if (rc != ESP_OK) return rc;
    if (out_tokens) for (size_t i = 0; i < r.tokens.size(); i++) out_tokens[i] = r.tokens[i];
    if (out_text_bytes) *out_text_bytes = r.text.size();
    if (out_text && text_capacity) std::memcpy(out_text, r.text.data(), std::min(text_capacity, r.text.size()));
    if (result) fill_result(r, result);
    return ESP_OK;
}

}  // extern "C"
