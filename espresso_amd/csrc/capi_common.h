// Helpers of the C ABI's translation units: handles, configurations, environments and results across the boundary.
#pragma once

#include <algorithm>
#include <cstring>

#include "generation.h"
#include "host/engine.h"

namespace esp {
namespace capi {

inline int bad_handle() { return fail(ESP_ERR_INVALID_ARGUMENT, "null runtime handle"); }
inline void fill_stats(ESPGenerationStats *stats, const GenerationTiming &t, size_t generated) {
    if (!stats) return;
    stats->generated = (int32_t)generated;
    stats->prefill_ms = t.prefill_ms;
    stats->decode_ms = t.decode_ms;
    stats->first_token_latency_ms = t.first_token_latency_ms;
    stats->tokens_per_second = generated ? (double)generated / (t.decode_ms > 1e-9 ? t.decode_ms / 1e3 : 1e-9) : 0.0;
}

inline MultiModelConfig from_c(const ESPModelConfig &c) {
    MultiModelConfig m;
    m.name = std::string(c.name, strnlen(c.name, sizeof(c.name)));
    m.nLayer = c.n_layer; m.nHead = c.n_head; m.nKVHead = c.n_kv_head; m.dModel = c.d_model; m.headDim = c.head_dim;
    m.hiddenDim = c.hidden_dim; m.vocab = c.vocab; m.maxSeq = c.max_seq; m.normEps = c.norm_eps; m.ropeTheta = c.rope_theta;
    m.hasEosToken = c.eos_token >= 0;
    m.eosToken = c.eos_token >= 0 ? (TokenID)c.eos_token : 0;
    m.architecture = c.architecture == 0 ? MultiModelConfig::Architecture::gpt2
                     : c.architecture == 2 ? MultiModelConfig::Architecture::layered : MultiModelConfig::Architecture::llama;
    return m;
}

inline void to_c(const MultiModelConfig &m, ESPModelConfig *c) {
    std::memset(c, 0, sizeof(*c));
    std::strncpy(c->name, m.name.c_str(), sizeof(c->name) - 1);
    c->n_layer = m.nLayer; c->n_head = m.nHead; c->n_kv_head = m.nKVHead; c->d_model = m.dModel; c->head_dim = m.headDim;
    c->hidden_dim = m.hiddenDim; c->vocab = m.vocab; c->max_seq = m.maxSeq; c->norm_eps = m.normEps; c->rope_theta = m.ropeTheta;
    c->eos_token = m.hasEosToken ? (int32_t)m.eosToken : -1;
    c->architecture = m.architecture == MultiModelConfig::Architecture::gpt2 ? 0 : m.architecture == MultiModelConfig::Architecture::layered ? 2 : 1;
}

inline Environment env_from(const char *const *keys, const char *const *values, int count) {
    Environment e;
    for (int i = 0; i < count; i++) if (keys && values && keys[i] && values[i]) e[keys[i]] = values[i];
    return e;
}

inline void fill_result(const GenerationResult &r, ESPGenerationResult *result) {
    std::memset(result, 0, sizeof(*result));
    result->token_count = (int32_t)r.tokens.size();
    result->tokens_per_second = r.tokensPerSecond;
    result->compile_time_ms = r.compileTimeMs;
    result->first_token_latency_ms = r.firstTokenLatencyMs;
    result->has_two_token_stats = r.hasTwoTokenStats ? 1 : 0;
    result->committed_exact_tokens_per_pass = r.committedExactTokensPerPass;
    result->accepted_future_tokens_per_pass = r.acceptedFutureTokensPerPass;
    std::strncpy(result->exact_head_backend, r.exactHeadBackend.c_str(), sizeof(result->exact_head_backend) - 1);
}
}  // namespace capi
}  // namespace esp

struct ESPEngine {
    std::unique_ptr<esp::RealModelInferenceEngine> engine;
    ESPLlamaRuntime runtime_handle{nullptr};
};
