#include "generation.h"

#include <cmath>

#include "generation_loop.h"

namespace esp {

using namespace loop;

int generate_greedy(DecoderRuntime &rt, const uint32_t *prompt, int prompt_count, int max_tokens,
                    std::vector<uint32_t> *out, GenerationTiming *timing) {
    out->clear();
    const DecoderShape &c = rt.shape();
    if (prompt_count <= 0 || !prompt) return fail(ESP_ERR_INVALID_ARGUMENT, "Prompt tokens must not be empty");       // (:6200-6202)
    if (max_tokens < 0) return fail(ESP_ERR_INVALID_ARGUMENT, "maxTokens must be >= 0");                               // (:1411-1413)
    if (prompt_count >= c.max_seq) return fail(ESP_ERR_OUT_OF_RANGE, "prompt of %d tokens does not fit context %d", prompt_count, c.max_seq);
    const int eff = max_tokens < c.max_seq - prompt_count ? max_tokens : c.max_seq - prompt_count;
    auto t_prefill = Clock::now();
    int rc = rt.prefill(0, prompt, prompt_count);
    if (rc != ESP_OK) return rc;
    if (timing) timing->prefill_ms = ms_since(t_prefill);

    auto t_start = Clock::now(), t_emit = t_start;
    int all = prompt_count;
    if (eff > 1) {
        // The first eff-1 tokens need no host decision (the step graph notices a stop token by itself), so they run as graph
        // replays with a synchronisation at the end or every 32 tokens; the last token is selected but not advanced, as in the
        // loop below.
        out->resize(eff - 1);
        int produced = eff - 1;
        if (c.eos_token < 0) rc = rt.continue_greedy(0, eff - 1, out->data());
        else rc = rt.continue_greedy_until_stop(0, eff - 1, out->data(), &produced);
        if (rc != ESP_OK) return rc;
        out->resize(produced);
        all += produced;
        if (timing && produced > 0) {
            const double per_token = ms_since(t_start) / produced;
            timing->first_token_latency_ms = per_token;
            timing->token_latencies_ms.assign(produced, per_token);   // one measurement for the whole run
        }
        t_emit = Clock::now();
        if (produced > 0 && c.eos_token >= 0 && out->back() == (uint32_t)c.eos_token) {   // EOS is appended, then the loop ends (:6385-6388)
            if (timing) timing->decode_ms = ms_since(t_start);
            return ESP_OK;
        }
    }
    while ((int)out->size() < eff) {
        uint32_t next = 0;
        if ((rc = rt.select_greedy(0, &next)) != ESP_OK) return rc;
        auto now = Clock::now();
        if (timing) {
            if (out->empty()) timing->first_token_latency_ms = std::chrono::duration<double, std::milli>(now - t_start).count();
            timing->token_latencies_ms.push_back(std::chrono::duration<double, std::milli>(now - t_emit).count());
        }
        out->push_back(next);
        if (c.eos_token >= 0 && next == (uint32_t)c.eos_token) break;   // EOS is appended, then the loop ends (:6385-6388)
        all++;
        if ((int)out->size() >= eff || all >= c.max_seq) break;         // (:6407)
        if ((rc = rt.advance(0, next)) != ESP_OK) return rc;            // position all - 1 (:6411)
        t_emit = now;
    }
    if (timing) timing->decode_ms = ms_since(t_start);
    return ESP_OK;
}

int sample_token(const float *logits, int count, float temperature, double unit) {
    if (count <= 0) return 0;
    auto first_max = [&]() { int b = 0; for (int i = 1; i < count; i++) if (logits[b] < logits[i]) b = i; return b; };
    if (temperature <= 0.0f) return first_max();
    float max_logit = logits[0];
    for (int i = 1; i < count; i++) if (logits[i] > max_logit) max_logit = logits[i];
    std::vector<double> scaled(count);
    double total = 0.0;
    for (int i = 0; i < count; i++) {
        scaled[i] = std::exp((double)((logits[i] - max_logit) / temperature));
        total += scaled[i];
    }
    if (!std::isfinite(total) || total <= 0.0) return first_max();
    double threshold = unit * total;
    for (int i = 0; i < count; i++) {
        threshold -= scaled[i];
        if (threshold <= 0.0) return i;
    }
    return count - 1;
}

int generate_sampled(DecoderRuntime &rt, const uint32_t *prompt, int prompt_count, int max_tokens, float temperature,
                     uint64_t seed, std::vector<uint32_t> *out, GenerationTiming *timing) {
    out->clear();
    const DecoderShape &c = rt.shape();
    if (prompt_count <= 0 || !prompt) return fail(ESP_ERR_INVALID_ARGUMENT, "Prompt tokens must not be empty");
    if (max_tokens < 0) return fail(ESP_ERR_INVALID_ARGUMENT, "maxTokens must be >= 0");
    if (prompt_count >= c.max_seq) return fail(ESP_ERR_OUT_OF_RANGE, "prompt of %d tokens does not fit the context", prompt_count);
    const int eff = max_tokens < c.max_seq - prompt_count ? max_tokens : c.max_seq - prompt_count;
    auto t_prefill = Clock::now();
    int rc = rt.prefill(0, prompt, prompt_count);
    if (rc != ESP_OK) return rc;
    if (timing) timing->prefill_ms = ms_since(t_prefill);
    auto t_start = Clock::now(), t_emit = t_start;
    SplitMix64 rng{seed};
    std::vector<float> logits(c.vocab);
    int all = prompt_count;
    while ((int)out->size() < eff && all < c.max_seq) {
        if ((rc = rt.read_logits(0, logits.data())) != ESP_OK) return rc;
        const uint32_t tok = (uint32_t)sample_token(logits.data(), c.vocab, temperature, rng.unit());
        auto now = Clock::now();
        if (timing) {
            if (out->empty()) timing->first_token_latency_ms = std::chrono::duration<double, std::milli>(now - t_start).count();
            timing->token_latencies_ms.push_back(std::chrono::duration<double, std::milli>(now - t_emit).count());
        }
        t_emit = now;
        out->push_back(tok);
        all++;
        if (c.eos_token >= 0 && tok == (uint32_t)c.eos_token) break;        // appended, then stop (:6385-6388)
        if ((int)out->size() >= eff || all >= c.max_seq) break;
        if ((rc = rt.advance(0, tok)) != ESP_OK) return rc;
    }
    if (timing) timing->decode_ms = ms_since(t_start);
    return ESP_OK;
}

// ---- lock-step batches of independent sequences ---------------------------------------------------
namespace loop {
int batch_budget(const DecoderRuntime &a, const DecoderRuntime *b, const int *prompt_counts, int n_seq, int max_tokens, int *eff) {
    if (n_seq < 1 || n_seq > a.shape().max_sequences || (b && n_seq > b->shape().max_sequences) || 2 * n_seq > kMaxStepRows)
        return fail(ESP_ERR_INVALID_ARGUMENT, "batch of %d sequences does not fit the runtime", n_seq);
    int max_seq = a.shape().max_seq;
    if (b && b->shape().max_seq < max_seq) max_seq = b->shape().max_seq;
    int budget = max_tokens;
    for (int s = 0; s < n_seq; s++) {
        if (prompt_counts[s] <= 0) return fail(ESP_ERR_INVALID_ARGUMENT, "Prompt tokens must not be empty");
        if (prompt_counts[s] >= max_seq) return fail(ESP_ERR_OUT_OF_RANGE, "prompt of %d tokens does not fit the context", prompt_counts[s]);
        if (max_seq - prompt_counts[s] < budget) budget = max_seq - prompt_counts[s];
    }
    *eff = budget < 0 ? 0 : budget;
    return ESP_OK;
}
}  // namespace loop

int generate_greedy_batch(DecoderRuntime &rt, const uint32_t *const *prompts, const int *prompt_counts, int n_seq, int max_tokens,
                          std::vector<std::vector<uint32_t>> *out, double *decode_ms) {
    out->assign(n_seq, {});
    int eff = 0, rc = batch_budget(rt, nullptr, prompt_counts, n_seq, max_tokens, &eff);
    if (rc != ESP_OK) return rc;
    for (int s = 0; s < n_seq; s++)
        if ((rc = rt.prefill(s, prompts[s], prompt_counts[s])) != ESP_OK) return rc;
    auto t0 = Clock::now();
    if (eff > 0) {
        std::vector<uint32_t> current(n_seq);
        for (int s = 0; s < n_seq; s++) {
            if ((rc = rt.select_greedy(s, &current[s])) != ESP_OK) return rc;
            (*out)[s].push_back(current[s]);
        }
        int first_host_step = 1;
        if (rt.graph_replay_enabled() && eff > 2) {
            // every step but none of the decisions needs the host: rows feed themselves on the device, one graph per step
            hipStream_t st = context().stream;
            const int steps = eff - 1;
            DeviceArray<int> d_log, d_step;
            if ((rc = d_log.alloc((size_t)steps * n_seq)) != ESP_OK || (rc = d_step.alloc(1)) != ESP_OK) return rc;
            StepRows rows{};
            rows.count = n_seq;
            for (int s = 0; s < n_seq; s++) { rows.token[s] = (int)current[s]; rows.pos[s] = rt.visible(s); rows.seq[s] = s; }
            if ((rc = hip_ok(launch_set_rows(rows, rt.device_row_tokens(), rt.device_row_positions(), rt.device_row_sequences(), st), "rows")) != ESP_OK) return rc;
            if ((rc = hip_ok(launch_set_ints(d_step.p, 0, nullptr, 0, st), "step")) != ESP_OK) return rc;
            auto pass = [&]() {
                int r = rt.enqueue_device_rows(n_seq);
                if (r == ESP_OK) r = rt.enqueue_device_head(n_seq);
                if (r == ESP_OK) r = hip_ok(launch_batch_greedy_feed(rt.device_head_tokens(), n_seq, rt.device_row_tokens(), rt.device_row_positions(), d_log.p,
                                                                     d_step.p, steps, st), "feed");
                return r;
            };
            PassGraph graph;
            if ((rc = pass()) != ESP_OK) return rc;
            if ((rc = graph.capture(pass)) != ESP_OK) return rc;
            if ((rc = graph.launch(steps - 1)) != ESP_OK) return rc;
            std::vector<int> log((size_t)steps * n_seq);
            if ((rc = hip_ok(hipMemcpyAsync(log.data(), d_log.p, sizeof(int) * log.size(), hipMemcpyDeviceToHost, st), "log")) != ESP_OK) return rc;
            if ((rc = hip_ok(hipStreamSynchronize(st), "greedy batch")) != ESP_OK) return rc;
            for (int s = 0; s < n_seq; s++) {
                for (int i = 0; i < steps; i++) (*out)[s].push_back((uint32_t)log[(size_t)i * n_seq + s]);
                rt.set_visible(s, rt.visible(s) + steps);
            }
            first_host_step = eff;
        }
        for (int step = first_host_step; step < eff; step++) {
            StepRows rows{};
            rows.count = n_seq;
            for (int s = 0; s < n_seq; s++) { rows.token[s] = (int)current[s]; rows.pos[s] = rt.visible(s); rows.seq[s] = s; }
            uint32_t next[kMaxStepRows];
            if ((rc = rt.forward_rows(rows)) != ESP_OK) return rc;
            if ((rc = rt.head_rows(n_seq, next)) != ESP_OK) return rc;
            for (int s = 0; s < n_seq; s++) {
                rt.set_visible(s, rows.pos[s] + 1);
                current[s] = next[s];
                (*out)[s].push_back(next[s]);
            }
        }
    }
    if (decode_ms) *decode_ms = ms_since(t0);
    return ESP_OK;
}

}  // namespace esp
