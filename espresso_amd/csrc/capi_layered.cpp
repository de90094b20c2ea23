// C ABI: what only layered runtimes have (measurement and test aids; the generation entry points are those of every runtime).
#include <algorithm>

#include "host/layered_loader.h"

using namespace esp;

namespace {
int layered_of(const ESPLlamaRuntime *h, LayeredRuntime **out) {
    if (!h || !h->rt) return fail(ESP_ERR_INVALID_ARGUMENT, "null runtime handle");
    *out = h->rt->as_layered();
    return *out ? ESP_OK : fail(ESP_ERR_UNSUPPORTED, "this call needs a layered runtime");
}
}  // namespace

extern "C" {

ESPLlamaRuntime *esp_layered_create_synthetic(const char *config_json, int float32, int max_seq, int max_sequences, uint64_t seed, float std_dev) {
    if (!config_json) { fail(ESP_ERR_INVALID_ARGUMENT, "null configuration"); return nullptr; }
    LayeredConfig c;
    std::string error;
    if (!parse_layered_config(config_json, &c, &error)) { fail(ESP_ERR_INVALID_ARGUMENT, "%s", error.c_str()); return nullptr; }
    LayeredOptions o;
    o.precision = float32 ? Precision::f32 : Precision::bf16;
    o.max_seq = max_seq; o.max_sequences = max_sequences;
    std::unique_ptr<LayeredRuntime> rt;
    if (make_synthetic_layered_model(c, o, seed, std_dev, &rt) != ESP_OK) return nullptr;
    return new ESPLlamaRuntime{rt.release()};
}

int esp_layered_set_min_block_rows(ESPLlamaRuntime *runtime, int rows) {
    LayeredRuntime *rt = nullptr;
    const int rc = layered_of(runtime, &rt);
    if (rc == ESP_OK) rt->set_min_block_rows(rows);
    return rc;
}

int esp_layered_trace_layers(ESPLlamaRuntime *runtime, int sequence, const uint32_t *tokens, int count, float *out) {
    LayeredRuntime *rt = nullptr;
    int rc = layered_of(runtime, &rt);
    if (rc != ESP_OK) return rc;
    if (!out || count < 1 || count > kPrefillBlockRows) return fail(ESP_ERR_INVALID_ARGUMENT, "trace_layers: 1..%d tokens", kPrefillBlockRows);
    int status = ESP_OK;
    rt->set_min_block_rows(1);
    rt->set_layer_observer([&](int layer) {
        const int r = rt->read_hidden_rows(count, out + (size_t)layer * count * rt->shape().d_model);
        if (r != ESP_OK) status = r;
    });
    rc = rt->append(sequence, tokens, count);
    rt->set_layer_observer(nullptr);
    rt->set_min_block_rows(LayeredRuntime::kMinBlockRows);
    return rc != ESP_OK ? rc : status;
}

long long esp_layered_sequence_bytes(const ESPLlamaRuntime *runtime) {
    LayeredRuntime *rt = nullptr;
    const int rc = layered_of(runtime, &rt);
    return rc == ESP_OK ? (long long)rt->sequence_bytes() : rc;
}

int esp_layered_set_kernel_timing(ESPLlamaRuntime *runtime, int enabled) {
    LayeredRuntime *rt = nullptr;
    const int rc = layered_of(runtime, &rt);
    if (rc == ESP_OK) rt->set_kernel_timing(enabled != 0);
    return rc;
}

int esp_layered_kernel_times(ESPLlamaRuntime *runtime, double *total_us, int64_t *launches, uint64_t *bytes, int reset) {
    LayeredRuntime *rt = nullptr;
    int rc = layered_of(runtime, &rt);
    if (rc != ESP_OK) return rc;
    double t[LayeredRuntime::K_CLASS_COUNT];
    long n[LayeredRuntime::K_CLASS_COUNT];
    if ((rc = rt->collect_kernel_times(t, n, LayeredRuntime::K_CLASS_COUNT, reset != 0)) != ESP_OK) return rc;
    for (int k = 0; k < LayeredRuntime::K_CLASS_COUNT; k++) {
        if (total_us) total_us[k] = t[k];
        if (launches) launches[k] = n[k];
        if (bytes) bytes[k] = rt->kernel_bytes(k);
    }
    return ESP_OK;
}

}  // extern "C"
