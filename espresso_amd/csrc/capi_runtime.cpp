// C ABI: runtimes of every family (ESPLlamaRuntime is the handle's historical name) and the generation loops they share.
#include "capi_common.h"

using namespace esp;
using namespace esp::capi;

extern "C" {

void esp_llama_free(ESPLlamaRuntime *runtime) {
    if (!runtime) return;
    delete runtime->rt;
    delete runtime;
}
size_t esp_llama_weight_bytes(const ESPLlamaRuntime *runtime) { return runtime ? runtime->rt->weight_bytes_per_token() : 0; }
size_t esp_llama_resident_weight_bytes(const ESPLlamaRuntime *runtime) { return runtime ? runtime->rt->resident_weight_bytes() : 0; }
int esp_llama_reset(ESPLlamaRuntime *runtime) { return runtime ? runtime->rt->reset() : bad_handle(); }
int esp_llama_prefill(ESPLlamaRuntime *runtime, int sequence, const uint32_t *tokens, int count) {
    if (!runtime) return bad_handle();
    if (!runtime->rt->finalized()) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    return runtime->rt->prefill(sequence, tokens, count);
}
int esp_llama_advance(ESPLlamaRuntime *runtime, int sequence, uint32_t token) {
    if (!runtime) return bad_handle();
    if (!runtime->rt->finalized()) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    return runtime->rt->advance(sequence, token);
}
int esp_llama_select_greedy_token(ESPLlamaRuntime *runtime, int sequence, uint32_t *token) {
    return runtime ? runtime->rt->select_greedy(sequence, token) : bad_handle();
}
int esp_llama_visible_token_count(const ESPLlamaRuntime *runtime, int sequence) {
    return runtime ? runtime->rt->visible(sequence) : -1;
}
int esp_llama_set_visible_token_count(ESPLlamaRuntime *runtime, int sequence, int count) {
    return runtime ? runtime->rt->set_visible(sequence, count) : bad_handle();
}
int esp_llama_read_last_hidden(ESPLlamaRuntime *runtime, int sequence, float *out) {
    return runtime ? runtime->rt->read_last_hidden(sequence, out) : bad_handle();
}
int esp_llama_read_logits(ESPLlamaRuntime *runtime, int sequence, float *out) {
    return runtime ? runtime->rt->read_logits(sequence, out) : bad_handle();
}

int esp_llama_append(ESPLlamaRuntime *runtime, int sequence, const uint32_t *tokens, int count, const int *want, int want_count, float *logits) {
    if (!runtime) return bad_handle();
    return runtime->rt->append(sequence, tokens, count, want, want_count, logits);
}
int esp_llama_acquire_sequence(ESPLlamaRuntime *runtime, int *sequence) { return runtime ? runtime->rt->acquire_sequence(sequence) : bad_handle(); }
int esp_llama_release_sequence(ESPLlamaRuntime *runtime, int sequence) { return runtime ? runtime->rt->release_sequence(sequence) : bad_handle(); }

int esp_llama_generate_sampled(ESPLlamaRuntime *runtime, const uint32_t *prompt, int prompt_count, int max_tokens, float temperature,
                               uint64_t seed, uint32_t *out_tokens, int *out_count, ESPGenerationStats *stats) {
    if (!runtime) return bad_handle();
    if (!runtime->rt->finalized()) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    if (out_count) *out_count = 0;
    std::vector<uint32_t> toks;
    GenerationTiming timing;
    const int rc = generate_sampled(*runtime->rt, prompt, prompt_count, max_tokens, temperature, seed, &toks, &timing);
    if (rc != ESP_OK) return rc;
    for (size_t i = 0; i < toks.size(); i++) if (out_tokens) out_tokens[i] = toks[i];
    if (out_count) *out_count = (int)toks.size();
    fill_stats(stats, timing, toks.size());
    return ESP_OK;
}

int esp_llama_generate(ESPLlamaRuntime *runtime, const uint32_t *prompt, int prompt_count, int max_tokens,
                       uint32_t *out_tokens, int *out_count, ESPGenerationStats *stats, double *token_latencies_ms) {
    if (!runtime) return bad_handle();
    if (!runtime->rt->finalized()) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    if (out_count) *out_count = 0;
    std::vector<uint32_t> toks;
    GenerationTiming timing;
    int rc = generate_greedy(*runtime->rt, prompt, prompt_count, max_tokens, &toks, &timing);
    if (rc != ESP_OK) return rc;
    for (size_t i = 0; i < toks.size(); i++) {
        if (out_tokens) out_tokens[i] = toks[i];
        if (token_latencies_ms) token_latencies_ms[i] = timing.token_latencies_ms[i];
    }
    if (out_count) *out_count = (int)toks.size();
    fill_stats(stats, timing, toks.size());
    return ESP_OK;
}

int esp_llama_continue_greedy(ESPLlamaRuntime *runtime, int sequence, int steps, uint32_t *out_tokens) {
    if (!runtime) return bad_handle();
    if (!runtime->rt->finalized()) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    return runtime->rt->continue_greedy(sequence, steps, out_tokens);
}

int esp_llama_set_graph_replay(ESPLlamaRuntime *runtime, int enabled) {
    if (!runtime) return bad_handle();
    runtime->rt->set_use_graph(enabled != 0);
    return ESP_OK;
}

int esp_llama_set_matrix_prefill(ESPLlamaRuntime *runtime, int enabled) {
    if (!runtime || !runtime->rt) return bad_handle();
    runtime->rt->set_matrix_prefill(enabled != 0);
    return ESP_OK;
}

}  // extern "C"
