#include "decoder_runtime.h"

#include <algorithm>
#include <atomic>

namespace esp {

DecoderRuntime::DecoderRuntime() {
    static std::atomic<unsigned long long> next_id{1};
    id_ = next_id.fetch_add(1);
}

DecoderRuntime::~DecoderRuntime() {
    free_device(hidden_); free_device(logits_); free_device(last_hidden_); free_device(want_rows_);
    free_device(d_tokens_); free_device(d_pos_); free_device(d_seq_); free_device(d_out_tokens_);
    free_device(d_visible_); free_device(d_log_); free_device(d_log_count_);
    free_device(argmax_scratch_.part_value); free_device(argmax_scratch_.part_index);
    for (hipGraphExec_t g : step_graphs_) if (g) (void)hipGraphExecDestroy(g);
    for (hipGraphExec_t g : multi_graphs_) if (g) (void)hipGraphExecDestroy(g);
    for (TimedLaunch &t : timed_) { (void)hipEventDestroy(t.start); (void)hipEventDestroy(t.stop); }
    for (hipEvent_t e : event_pool_) (void)hipEventDestroy(e);
}

int DecoderRuntime::allocate_common(int block_rows, int hidden_stride) {
    const DecoderShape &c = shape();
    block_rows_ = block_rows;
    hidden_stride_ = hidden_stride;
    const size_t R = block_rows > kMaxStepRows ? block_rows : kMaxStepRows, RS = kMaxStepRows, d = hidden_stride;
    int rc;
    if ((rc = device_alloc(&hidden_, R * d)) != ESP_OK) return rc;
    if ((rc = device_alloc(&logits_, RS * c.vocab)) != ESP_OK) return rc;
    if ((rc = device_alloc(&last_hidden_, (size_t)c.max_sequences * d)) != ESP_OK) return rc;
    if ((rc = device_alloc(&want_rows_, RS * d)) != ESP_OK) return rc;
    if ((rc = device_alloc(&d_tokens_, R)) != ESP_OK) return rc;
    if ((rc = device_alloc(&d_pos_, R)) != ESP_OK) return rc;
    if ((rc = device_alloc(&d_seq_, R)) != ESP_OK) return rc;
    if ((rc = device_alloc(&d_out_tokens_, R)) != ESP_OK) return rc;
    if ((rc = device_alloc(&d_visible_, (size_t)c.max_sequences)) != ESP_OK) return rc;
    if ((rc = device_alloc(&d_log_, (size_t)c.max_seq)) != ESP_OK) return rc;
    if ((rc = device_alloc(&d_log_count_, 3)) != ESP_OK) return rc;   // tokens logged, stopped, stop enabled (greedy_tail_kernel)
    step_graphs_.assign(c.max_sequences, nullptr);
    multi_graphs_.assign(c.max_sequences, nullptr);
    // one (value, index) pair per workgroup of the head GEMV and row: a workgroup owns eight rows, or the grid is persistent
    head_partial_capacity_ = (c.vocab + 7) / 8 > 4096 ? (c.vocab + 7) / 8 : 4096;
    const size_t argmax_slots = (size_t)2 * head_partial_capacity_ > (size_t)kArgmaxScratchSlots ? (size_t)2 * head_partial_capacity_ : (size_t)kArgmaxScratchSlots;
    if ((rc = device_alloc(&argmax_scratch_.part_value, argmax_slots)) != ESP_OK) return rc;
    if ((rc = device_alloc(&argmax_scratch_.part_index, argmax_slots)) != ESP_OK) return rc;
    visible_.assign(c.max_sequences, 0);
    taken_.assign(c.max_sequences, 0);
    return ESP_OK;
}

hipEvent_t DecoderRuntime::take_event() {
    if (!event_pool_.empty()) {
        hipEvent_t e = event_pool_.back();
        event_pool_.pop_back();
        return e;
    }
    hipEvent_t e = nullptr;
    if (hipEventCreate(&e) != hipSuccess) return nullptr;
    return e;
}

int DecoderRuntime::time_begin(int kernel_class) {
    if (!timing_enabled_) return ESP_OK;
    TimedLaunch t{kernel_class, take_event(), take_event()};
    if (!t.start || !t.stop) return fail(ESP_ERR_OUT_OF_MEMORY, "hipEventCreate failed");
    ESP_HIP_TRY(hipEventRecord(t.start, context().stream));
    timed_.push_back(t);
    return ESP_OK;
}

int DecoderRuntime::time_end() {
    if (!timing_enabled_) return ESP_OK;
    ESP_HIP_TRY(hipEventRecord(timed_.back().stop, context().stream));
    return ESP_OK;
}

int DecoderRuntime::collect_kernel_times(double *total_us, long *launches, int classes, bool reset) {
    ESP_HIP_TRY(hipStreamSynchronize(context().stream));
    for (TimedLaunch &t : timed_) {
        float ms = 0.0f;
        ESP_HIP_TRY(hipEventElapsedTime(&ms, t.start, t.stop));
        time_total_us_[t.kernel_class] += (double)ms * 1e3;
        time_launches_[t.kernel_class] += 1;
        event_pool_.push_back(t.start);
        event_pool_.push_back(t.stop);
    }
    timed_.clear();
    for (int k = 0; k < classes && k < kMaxKernelClasses; k++) {
        if (total_us) total_us[k] = time_total_us_[k];
        if (launches) launches[k] = time_launches_[k];
        if (reset) { time_total_us_[k] = 0; time_launches_[k] = 0; }
    }
    return ESP_OK;
}

int DecoderRuntime::check_sequence(int seq) const {
    if (seq < 0 || seq >= shape().max_sequences) return fail(ESP_ERR_OUT_OF_RANGE, "sequence %d of %d", seq, shape().max_sequences);
    return ESP_OK;
}

int DecoderRuntime::reset() {
    if (!finalized_) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    int rc = clear_state();
    if (rc != ESP_OK) return rc;
    ESP_HIP_TRY(hipMemsetAsync(last_hidden_, 0, (size_t)shape().max_sequences * hidden_stride_ * 4, context().stream));
    ESP_HIP_TRY(hipStreamSynchronize(context().stream));
    std::fill(visible_.begin(), visible_.end(), 0);
    std::fill(taken_.begin(), taken_.end(), 0);
    return ESP_OK;
}

int DecoderRuntime::visible(int seq) const {
    return seq >= 0 && seq < (int)visible_.size() ? visible_[seq] : -1;
}

int DecoderRuntime::set_visible(int seq, int count) {
    if (seq < 0 || seq >= (int)visible_.size() || count < 0 || count > shape().max_seq)
        return fail(ESP_ERR_OUT_OF_RANGE, "set_visible(seq %d, count %d) out of range", seq, count);
    if (!can_roll_back() && count != 0 && count != visible_[seq])
        return fail(ESP_ERR_UNSUPPORTED, "set_visible: recurrent state of sequence %d cannot go from token %d to %d", seq, visible_[seq], count);
    visible_[seq] = count;
    return ESP_OK;
}

int DecoderRuntime::acquire_sequence(int *seq) {
    if (!finalized_ || !seq) return fail(ESP_ERR_INVALID_ARGUMENT, "acquire_sequence: runtime is not finalized");
    for (size_t i = 0; i < taken_.size(); i++) {
        if (taken_[i]) continue;
        taken_[i] = 1;
        visible_[i] = 0;
        *seq = (int)i;
        return ESP_OK;
    }
    return fail(ESP_ERR_OUT_OF_RANGE, "all %zu sequence slots are taken", taken_.size());
}

int DecoderRuntime::release_sequence(int seq) {
    int rc = check_sequence(seq);
    if (rc != ESP_OK) return rc;
    taken_[seq] = 0;
    visible_[seq] = 0;
    return ESP_OK;
}

int DecoderRuntime::forward_rows(const StepRows &rows) {
    if (!finalized_) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    if (rows.count < 1 || rows.count > kMaxStepRows) return fail(ESP_ERR_INVALID_ARGUMENT, "forward_rows: %d rows", rows.count);
    for (int i = 0; i < rows.count; i++) {
        if (rows.token[i] < 0 || rows.token[i] >= shape().vocab)
            return fail(ESP_ERR_OUT_OF_RANGE, "token %d is outside vocab %d", rows.token[i], shape().vocab);   // (:687-689)
        if (rows.pos[i] < 0 || rows.pos[i] >= shape().max_seq)
            return fail(ESP_ERR_OUT_OF_RANGE, "position %d exceeds context %d", rows.pos[i], shape().max_seq);  // (:673-677)
        if (rows.seq[i] < 0 || rows.seq[i] >= shape().max_sequences)
            return fail(ESP_ERR_OUT_OF_RANGE, "sequence %d of %d", rows.seq[i], shape().max_sequences);
    }
    if (!takes_rows_of_one_sequence())
        for (int i = 1; i < rows.count; i++)
            for (int j = 0; j < i; j++)
                if (rows.seq[i] == rows.seq[j]) return fail(ESP_ERR_UNSUPPORTED, "this model takes one row of a sequence per step");
    ESP_HIP_TRY(launch_set_rows(rows, d_tokens_, d_pos_, d_seq_, context().stream));
    return enqueue_trunk(rows.count);
}

void DecoderRuntime::drop_captured_graphs() {
    for (auto &g : step_graphs_) if (g) { (void)hipGraphExecDestroy(g); g = nullptr; }
    for (auto &g : multi_graphs_) if (g) { (void)hipGraphExecDestroy(g); g = nullptr; }
    graph_epoch_++;
}

// esp_set_tuning changes which kernels a step launches: graphs captured before it would keep replaying the old ones.
void DecoderRuntime::sync_tuning() {
    const unsigned e = tuning_epoch();
    if (e == tuning_epoch_) return;
    tuning_epoch_ = e;
    drop_captured_graphs();
}

int DecoderRuntime::keep_row(int row, int seq) {
    if (row < 0 || row >= block_rows_ || seq < 0 || seq >= shape().max_sequences)
        return fail(ESP_ERR_OUT_OF_RANGE, "keep_row(%d, %d)", row, seq);
    ESP_HIP_TRY(launch_copy_rows(hidden_ + (size_t)row * hidden_stride_, last_hidden_ + (size_t)seq * hidden_stride_, 1, hidden_stride_,
                                 context().stream));
    return ESP_OK;
}

int DecoderRuntime::advance(int seq, uint32_t token) {
    if (seq < 0 || seq >= shape().max_sequences) return fail(ESP_ERR_OUT_OF_RANGE, "sequence %d of %d", seq, shape().max_sequences);
    if (visible_[seq] >= shape().max_seq)
        return fail(ESP_ERR_OUT_OF_RANGE, "runtime position %d exceeds context %d", visible_[seq], shape().max_seq);
    if (token >= (uint32_t)shape().vocab) return fail(ESP_ERR_OUT_OF_RANGE, "token %u is outside vocab %d", token, shape().vocab);
    StepRows rows{};
    rows.count = 1; rows.token[0] = (int)token; rows.pos[0] = visible_[seq]; rows.seq[0] = seq;
    int rc = forward_rows(rows);
    if (rc != ESP_OK) return rc;
    if ((rc = keep_row(0, seq)) != ESP_OK) return rc;
    visible_[seq] += 1;
    return ESP_OK;
}

int DecoderRuntime::prefill(int seq, const uint32_t *tokens, int count) {
    if (count <= 0 || !tokens) return fail(ESP_ERR_INVALID_ARGUMENT, "Prompt tokens must not be empty");
    int rc = check_sequence(seq);
    if (rc != ESP_OK) return rc;
    visible_[seq] = 0;
    return append(seq, tokens, count);
}

int DecoderRuntime::append(int seq, const uint32_t *tokens, int count, const int *want, int want_count, float *logits) {
    if (!finalized_) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    if (count <= 0 || !tokens) return fail(ESP_ERR_INVALID_ARGUMENT, "Prompt tokens must not be empty");
    int rc = check_sequence(seq);
    if (rc != ESP_OK) return rc;
    const int vocab = shape().vocab, max_seq = shape().max_seq;
    if (want_count < 0 || (want_count > 0 && (!want || !logits))) return fail(ESP_ERR_INVALID_ARGUMENT, "append: no place for the wanted logits");
    for (int i = 0; i < want_count; i++)
        if (want[i] < 0 || want[i] >= count || (i > 0 && want[i] <= want[i - 1]))
            return fail(ESP_ERR_OUT_OF_RANGE, "append: wanted places must ascend within 0..%d", count - 1);
    const int start = visible_[seq];   // every token is checked before the first one changes any state
    if (start + count > max_seq) return fail(ESP_ERR_OUT_OF_RANGE, "runtime position %d exceeds context %d", max_seq, max_seq);
    for (int i = 0; i < count; i++)
        if (tokens[i] >= (uint32_t)vocab) return fail(ESP_ERR_OUT_OF_RANGE, "token %u is outside vocab %d", tokens[i], vocab);
    hipStream_t s = context().stream;
    int given = 0;   // wanted rows delivered so far
    auto deliver = [&](const float *rows, int n) -> int {
        int r = run_head(rows, n, true);
        if (r != ESP_OK) return r;
        ESP_HIP_TRY(hipMemcpyAsync(logits + (size_t)given * vocab, logits_, (size_t)n * vocab * 4, hipMemcpyDeviceToHost, s));
        ESP_HIP_TRY(hipStreamSynchronize(s));
        given += n;
        return ESP_OK;
    };
    if (matrix_prefill_ && count >= matrix_prefill_min_tokens() && matrix_prefill_supported()) {
        // blocks of rows through the MFMA kernels (one pass over the weights per block)
        for (int off = 0; off < count; off += block_rows_) {
            const int rows = count - off < block_rows_ ? count - off : block_rows_;
            if ((rc = prefill_block(seq, tokens + off, rows, start + off)) != ESP_OK) return rc;
            if (off + rows == count && (rc = keep_row(rows - 1, seq)) != ESP_OK) return rc;
            while (given < want_count && want[given] < off + rows) {
                int n = 0;
                while (n < kMaxStepRows && given + n < want_count && want[given + n] < off + rows) {
                    int run = 1;   // rows that follow each other are copied together
                    while (n + run < kMaxStepRows && given + n + run < want_count && want[given + n + run] < off + rows && want[given + n + run] == want[given + n] + run) run++;
                    ESP_HIP_TRY(launch_copy_rows(hidden_ + (size_t)(want[given + n] - off) * hidden_stride_, want_rows_ + (size_t)n * hidden_stride_, run, hidden_stride_, s));
                    n += run;
                }
                if ((rc = deliver(want_rows_, n)) != ESP_OK) return rc;
            }
        }
        ESP_HIP_TRY(hipStreamSynchronize(s));
        visible_[seq] = start + count;
        return ESP_OK;
    }
    for (int i = 0; i < count; i++) {
        if ((rc = advance(seq, tokens[i])) != ESP_OK) return rc;
        if (given < want_count && want[given] == i && (rc = deliver(device_last_hidden(seq), 1)) != ESP_OK) return rc;
    }
    return ESP_OK;
}

// Token, position and sequence of a block's rows into the device arrays.
int DecoderRuntime::upload_block_rows(int seq, const uint32_t *tokens, int rows, int base) {
    hipStream_t s = context().stream;
    std::vector<int> h_tok(rows), h_pos(rows), h_seq(rows, seq);
    for (int i = 0; i < rows; i++) { h_tok[i] = (int)tokens[i]; h_pos[i] = base + i; }
    ESP_HIP_TRY(hipMemcpyAsync(d_tokens_, h_tok.data(), sizeof(int) * rows, hipMemcpyHostToDevice, s));
    ESP_HIP_TRY(hipMemcpyAsync(d_pos_, h_pos.data(), sizeof(int) * rows, hipMemcpyHostToDevice, s));
    ESP_HIP_TRY(hipMemcpyAsync(d_seq_, h_seq.data(), sizeof(int) * rows, hipMemcpyHostToDevice, s));
    ESP_HIP_TRY(hipStreamSynchronize(s));   // the host vectors go out of scope
    return ESP_OK;
}

int DecoderRuntime::select_greedy(int seq, uint32_t *token) {
    if (!finalized_) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    if (seq < 0 || seq >= shape().max_sequences || !token) return fail(ESP_ERR_OUT_OF_RANGE, "select_greedy(seq %d)", seq);
    int rc = run_head(last_hidden_ + (size_t)seq * hidden_stride_, 1);
    if (rc != ESP_OK) return rc;
    int t = 0;
    ESP_HIP_TRY(hipMemcpyAsync(&t, d_out_tokens_, sizeof(int), hipMemcpyDeviceToHost, context().stream));
    ESP_HIP_TRY(hipStreamSynchronize(context().stream));
    *token = (uint32_t)t;
    return ESP_OK;
}

int DecoderRuntime::head_rows(int count, uint32_t *tokens) {
    if (!finalized_) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    if (count < 1 || count > kMaxStepRows || !tokens) return fail(ESP_ERR_INVALID_ARGUMENT, "head_rows(%d)", count);
    int rc = run_head(hidden_, count);
    if (rc != ESP_OK) return rc;
    int t[kMaxStepRows];
    ESP_HIP_TRY(hipMemcpyAsync(t, d_out_tokens_, sizeof(int) * count, hipMemcpyDeviceToHost, context().stream));
    ESP_HIP_TRY(hipStreamSynchronize(context().stream));
    for (int i = 0; i < count; i++) tokens[i] = (uint32_t)t[i];
    return ESP_OK;
}

// Both step graphs of a sequence, at its first replayed step (a one-off of a few milliseconds per runtime, outside any later call).
int DecoderRuntime::capture_step_graph(int seq) {
    const int rc = capture_steps(seq, 1, &step_graphs_[seq]);
    return rc != ESP_OK ? rc : capture_steps(seq, kStepsPerGraph, &multi_graphs_[seq]);
}

// Replays `steps` greedy steps: graphs of kStepsPerGraph steps while that many are left, single steps for the rest.  Every boundary between two graph launches costs about 3.5 us on the device, whatever the graphs hold
// (6-layer model: 8.1 k tok/s with one step per graph, 8.35 k with four, 8.45 k with sixteen; 8B: 736 / 738.5 / 738.5).
int DecoderRuntime::replay_steps(int seq, int steps) {
    hipStream_t s = context().stream;
    int i = 0;
    if (multi_graphs_[seq])
        for (; i + kStepsPerGraph <= steps; i += kStepsPerGraph) ESP_HIP_TRY(hipGraphLaunch(multi_graphs_[seq], s));
    for (; i < steps; i++) ESP_HIP_TRY(hipGraphLaunch(step_graphs_[seq], s));
    return ESP_OK;
}

// head(last hidden of seq) -> arg-max -> feed row 0 -> trunk, whose last layer writes where the next step's head reads; `count` steps.
int DecoderRuntime::capture_steps(int seq, int count, hipGraphExec_t *out) {
    hipStream_t s = context().stream;
    hipGraph_t graph = nullptr;
    ESP_HIP_TRY(hipStreamSynchronize(s));
    ESP_HIP_TRY(hipStreamBeginCapture(s, hipStreamCaptureModeThreadLocal));
    int rc = ESP_OK;
    capturing_ = true;
    for (int step = 0; step < count && rc == ESP_OK; step++) {
        rc = enqueue_greedy_token(seq);
        if (rc == ESP_OK) rc = enqueue_trunk(1, true, device_last_hidden(seq));
    }
    capturing_ = false;
    hipError_t e = hipStreamEndCapture(s, &graph);
    if (rc != ESP_OK) { if (graph) (void)hipGraphDestroy(graph); return rc; }
    if (e != hipSuccess) return fail_hip(e, "hipStreamEndCapture");
    hipGraphExec_t exec = nullptr;
    e = hipGraphInstantiate(&exec, graph, nullptr, nullptr, 0);
    (void)hipGraphDestroy(graph);
    if (e != hipSuccess) return fail_hip(e, "hipGraphInstantiate");
    *out = exec;
    return ESP_OK;
}

int DecoderRuntime::continue_greedy(int seq, int steps, uint32_t *out_tokens) {
    if (!finalized_) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    sync_tuning();
    if (seq < 0 || seq >= shape().max_sequences) return fail(ESP_ERR_OUT_OF_RANGE, "sequence %d of %d", seq, shape().max_sequences);
    if (steps < 0) return fail(ESP_ERR_INVALID_ARGUMENT, "steps must be >= 0");
    if (visible_[seq] + steps > shape().max_seq)
        return fail(ESP_ERR_OUT_OF_RANGE, "runtime position %d + %d steps exceeds context %d", visible_[seq], steps, shape().max_seq);
    if (steps == 0) return ESP_OK;
    hipStream_t s = context().stream;
    int rc;
    if (!use_graph_ || timing_enabled_) {
        for (int i = 0; i < steps; i++) {
            uint32_t t = 0;
            if ((rc = select_greedy(seq, &t)) != ESP_OK) return rc;
            if (out_tokens) out_tokens[i] = t;
            if ((rc = advance(seq, t)) != ESP_OK) return rc;
        }
        return ESP_OK;
    }
    if (!step_graphs_[seq]) {
        // one eager step first: it configures every kernel's LDS limit outside the capture
        uint32_t t = 0;
        if ((rc = select_greedy(seq, &t)) != ESP_OK) return rc;
        if (out_tokens) out_tokens[0] = t;
        if ((rc = advance(seq, t)) != ESP_OK) return rc;
        if ((rc = capture_step_graph(seq)) != ESP_OK) return rc;
        if (out_tokens) out_tokens += 1;
        steps -= 1;
        if (steps == 0) return ESP_OK;
    }
    ESP_HIP_TRY(launch_set_ints(d_visible_ + seq, visible_[seq], d_log_count_, 0, s));
    ESP_HIP_TRY(launch_set_ints(d_log_count_ + 1, 0, d_log_count_ + 2, 0, s));   // not stopped, and no stop at the stop token
    if ((rc = replay_steps(seq, steps)) != ESP_OK) return rc;
    std::vector<int> log(steps);
    ESP_HIP_TRY(hipMemcpyAsync(log.data(), d_log_, sizeof(int) * steps, hipMemcpyDeviceToHost, s));
    ESP_HIP_TRY(hipStreamSynchronize(s));
    visible_[seq] += steps;
    if (out_tokens) for (int i = 0; i < steps; i++) out_tokens[i] = (uint32_t)log[i];
    return ESP_OK;
}

// continue_greedy that ends with the stop token: the token is emitted and not consumed, as in the reference loop (:6385-6388).  The
// replays run in chunks; the step graph itself notices the stop token, and replays after it change nothing.
int DecoderRuntime::continue_greedy_until_stop(int seq, int steps, uint32_t *out_tokens, int *produced) {
    if (!finalized_) return fail(ESP_ERR_INVALID_ARGUMENT, "runtime is not finalized");
    if (seq < 0 || seq >= shape().max_sequences || !out_tokens || !produced) return fail(ESP_ERR_OUT_OF_RANGE, "continue_greedy_until_stop(seq %d)", seq);
    *produced = 0;
    sync_tuning();
    if (steps < 0) return fail(ESP_ERR_INVALID_ARGUMENT, "steps must be >= 0");
    if (visible_[seq] + steps > shape().max_seq)
        return fail(ESP_ERR_OUT_OF_RANGE, "runtime position %d + %d steps exceeds context %d", visible_[seq], steps, shape().max_seq);
    const int eos = shape().eos_token;
    hipStream_t s = context().stream;
    int rc;
    auto eager_step = [&](bool *stopped) {
        uint32_t t = 0;
        int r = select_greedy(seq, &t);
        if (r != ESP_OK) return r;
        out_tokens[(*produced)++] = t;
        *stopped = eos >= 0 && t == (uint32_t)eos;
        return *stopped ? ESP_OK : advance(seq, t);
    };
    bool stopped = false;
    if (!use_graph_ || timing_enabled_) {
        while (*produced < steps && !stopped)
            if ((rc = eager_step(&stopped)) != ESP_OK) return rc;
        return ESP_OK;
    }
    if (steps > 0) {
        // The first step always runs from the host.  A replay that finds the stop token re-embeds the row that sits in
        // d_tokens_/d_pos_/d_seq_[0] and lets the trunk recompute it, which changes nothing only when that row is the one this
        // sequence consumed last; after a prompt block or another sequence's pass those arrays hold something else.  advance()
        // leaves exactly that row there (and the eager step configures every kernel's LDS limit outside a capture).
        if ((rc = eager_step(&stopped)) != ESP_OK) return rc;
        if (stopped) return ESP_OK;
        if (!step_graphs_[seq] && (rc = capture_step_graph(seq)) != ESP_OK) return rc;
    }
    if (*produced >= steps) return ESP_OK;
    const int first = *produced, want = steps - first;
    ESP_HIP_TRY(launch_set_ints(d_visible_ + seq, visible_[seq], d_log_count_, 0, s));
    ESP_HIP_TRY(launch_set_ints(d_log_count_ + 1, 0, d_log_count_ + 2, 1, s));
    int state[2] = {0, 0};   // tokens logged, stopped
    for (int launched = 0; launched < want && !state[1];) {
        const int chunk = want - launched < 32 ? want - launched : 32;
        if ((rc = replay_steps(seq, chunk)) != ESP_OK) return rc;
        launched += chunk;
        ESP_HIP_TRY(hipMemcpyAsync(state, d_log_count_, sizeof(state), hipMemcpyDeviceToHost, s));
        ESP_HIP_TRY(hipStreamSynchronize(s));
    }
    const int logged = state[0] < want ? state[0] : want;
    std::vector<int> log(logged > 0 ? logged : 1);
    if (logged > 0) {
        ESP_HIP_TRY(hipMemcpyAsync(log.data(), d_log_, sizeof(int) * logged, hipMemcpyDeviceToHost, s));
        ESP_HIP_TRY(hipStreamSynchronize(s));
    }
    for (int i = 0; i < logged; i++) out_tokens[first + i] = (uint32_t)log[i];
    *produced = first + logged;
    visible_[seq] += logged - (state[1] ? 1 : 0);   // every logged token was consumed, except a stop token
    return ESP_OK;
}

int DecoderRuntime::read_last_hidden(int seq, float *out) {
    if (!finalized_ || seq < 0 || seq >= shape().max_sequences || !out) return fail(ESP_ERR_INVALID_ARGUMENT, "read_last_hidden");
    ESP_HIP_TRY(hipMemcpyAsync(out, last_hidden_ + (size_t)seq * hidden_stride_, (size_t)shape().d_model * 4, hipMemcpyDeviceToHost,
                               context().stream));
    ESP_HIP_TRY(hipStreamSynchronize(context().stream));
    return ESP_OK;
}

int DecoderRuntime::read_hidden_rows(int rows, float *out) {
    if (!finalized_ || rows < 1 || rows > block_rows_ || !out) return fail(ESP_ERR_INVALID_ARGUMENT, "read_hidden_rows");
    const size_t d = shape().d_model;
    ESP_HIP_TRY(hipMemcpy2DAsync(out, d * 4, hidden_, (size_t)hidden_stride_ * 4, d * 4, rows, hipMemcpyDeviceToHost, context().stream));
    ESP_HIP_TRY(hipStreamSynchronize(context().stream));
    return ESP_OK;
}

int DecoderRuntime::read_logits(int seq, float *out) {
    if (!finalized_ || seq < 0 || seq >= shape().max_sequences || !out) return fail(ESP_ERR_INVALID_ARGUMENT, "read_logits");
    int rc = run_head(last_hidden_ + (size_t)seq * hidden_stride_, 1, true);
    if (rc != ESP_OK) return rc;
    ESP_HIP_TRY(hipMemcpyAsync(out, logits_, (size_t)shape().vocab * 4, hipMemcpyDeviceToHost, context().stream));
    ESP_HIP_TRY(hipStreamSynchronize(context().stream));
    return ESP_OK;
}

}  // namespace esp
