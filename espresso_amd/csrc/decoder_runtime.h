// What every device-resident decoder shares, whatever its layers are: sequence slots and their visible lengths, the rows of a
// step, kept hidden states, the output head's token selection, prompts in blocks and portions, greedy steps as captured graphs.
// LlamaRuntime (llama_runtime.h) and LayeredRuntime (layered_runtime.h) supply the layers; the generation loops (generation.h),
// the engine (host/engine.h) and the C ABI drive this class.
#pragma once

#include <string>
#include <vector>

#include "context.h"
#include "kernels/decode_ops.h"

namespace esp {

class LlamaRuntime;
class LayeredRuntime;

constexpr int kPrefillBlockRows = 512;        // rows per MFMA prefill block
constexpr int kStepsPerGraph = 8;             // greedy steps in the longer of the two captured step graphs
constexpr int kMatrixPrefillMinTokens = 32;   // shorter prompts take the exact per-token path
constexpr size_t kGemmWorkspaceFloats = (size_t)8 << 20;

struct DecoderShape {
    int d_model = 0, vocab = 0, max_seq = 0;
    int eos_token = -1;
    int max_sequences = 1;    // independent sequence slots (KV caches, recurrent states)
};

class DecoderRuntime {
  public:
    virtual ~DecoderRuntime();
    virtual const DecoderShape &shape() const = 0;
    virtual LlamaRuntime *as_llama() { return nullptr; }
    virtual LayeredRuntime *as_layered() { return nullptr; }

    bool finalized() const { return finalized_; }
    int reset();                                  // all sequences (RealModelInferenceEngine.swift:616-635)
    int visible(int seq) const;
    // Rollback = lower the visible length.  Runtimes with recurrent state (can_roll_back() false) take only 0 and the length
    // the sequence has.
    int set_visible(int seq, int count);
    virtual bool can_roll_back() const { return true; }
    // whether one step may hold several rows of one sequence (draft verification)
    virtual bool takes_rows_of_one_sequence() const { return true; }
    // Sequence slots for callers with requests that come and go: the lowest free slot, and its return.  A slot that is taken
    // again starts as an empty sequence.
    int acquire_sequence(int *seq);
    int release_sequence(int seq);

    // Runs the trunk over `rows` (token, position, sequence); positions are written into the caches.
    // Does not change the visible counts.
    int forward_rows(const StepRows &rows);
    // forward one token at the sequence's visible position and keep its hidden state (:672-680)
    int advance(int seq, uint32_t token);
    int prefill(int seq, const uint32_t *tokens, int count);   // from an empty sequence (:637-645)
    // The next `count` tokens of a sequence, from the caches and state that its earlier tokens left.  `want` lists (ascending)
    // the places among them whose logits go to `logits` ([want_count][vocab]).
    int append(int seq, const uint32_t *tokens, int count, const int *want = nullptr, int want_count = 0, float *logits = nullptr);
    // Final norm + LM head + first-max argmax of kept hidden states (:663-670, :825-849).
    int select_greedy(int seq, uint32_t *token);
    // Head over rows of the most recent forward_rows(); tokens[i] for row i.
    int head_rows(int count, uint32_t *tokens);
    // Keep row `row` of the most recent forward_rows() as sequence `seq`'s last hidden state.
    int keep_row(int row, int seq);
    // `steps` greedy tokens from the sequence's current state (select, then advance, per token) as
    // replays of captured HIP graphs (eight steps per graph while that many are left, then one); the host synchronises once at the end.
    int continue_greedy(int seq, int steps, uint32_t *out_tokens);
    // The same, ending early at the configuration's stop token: the stop token is emitted (it is the last of *produced tokens) and not
    // consumed.  The step graph notices it on the device; the host looks once per 32 replays.
    int continue_greedy_until_stop(int seq, int steps, uint32_t *out_tokens, int *produced);
    void set_use_graph(bool enabled) { use_graph_ = enabled; }
    // Prompts of matrix_prefill_min_tokens() or more run in blocks through the MFMA kernels (default on).
    void set_matrix_prefill(bool enabled) { matrix_prefill_ = enabled; }
    int read_last_hidden(int seq, float *out);
    int read_logits(int seq, float *out);         // runs the head on the kept hidden state
    // the residual stream of rows of the most recent block or step (measurement and tests)
    int read_hidden_rows(int rows, float *out);

    virtual size_t weight_bytes_per_token() const = 0;
    // what the weights hold in HBM: the packed matrices, the tiled copies the matrix-core GEMVs read beside them, the embedding table
    virtual size_t resident_weight_bytes() const = 0;

    // Steps whose rows (token, position, sequence) already sit in the device arrays below: generation loops that keep
    // their decisions on the device enqueue these, also under stream capture.  Nothing here synchronises.
    int *device_row_tokens() { return d_tokens_; }
    int *device_row_positions() { return d_pos_; }
    int *device_row_sequences() { return d_seq_; }
    const int *device_head_tokens() const { return d_out_tokens_; }
    const float *device_hidden_rows() const { return hidden_; }
    float *device_last_hidden(int seq) { return last_hidden_ + (size_t)seq * hidden_stride_; }
    int enqueue_device_rows(int rows, bool embedded = false) { return enqueue_trunk(rows, embedded); }   // embedding (unless the rows hold it already), then every layer
    int enqueue_device_head(int rows) { return run_head(hidden_, rows); }         // final norm, head, first-max arg-max per row
    bool graph_replay_enabled() const { return use_graph_ && !timing_enabled_; }
    unsigned long long id() const { return id_; }
    // changes whenever the kernels a captured graph would hold have changed (switches of this runtime, esp_set_tuning): holders
    // of captured passes compare it before they replay
    unsigned long long graph_epoch() { sync_tuning(); return graph_epoch_; }

    // Per-kernel timing with HIP events on the library stream.  While enabled, every launch of the
    // kernels of a class is bracketed by an event pair; collect_kernel_times() synchronises and adds the
    // elapsed times to the totals.  The classes are the runtime's own.
    static constexpr int kMaxKernelClasses = 16;
    void set_kernel_timing(bool enabled) { timing_enabled_ = enabled; }
    int collect_kernel_times(double *total_us, long *launches, int classes, bool reset);

  protected:
    DecoderRuntime();
    // ---- what the layers supply ----
    // embedded: hidden_ already holds the rows' embeddings; final_out: where the last layer writes (default hidden_)
    virtual int enqueue_trunk(int rows, bool embedded = false, float *final_out = nullptr) = 0;
    // want_logits: the full-vocabulary logits are needed in logits_ (otherwise the head may store none)
    virtual int run_head(const float *hidden_rows, int count, bool want_logits = false) = 0;
    // One greedy choice under capture: head over the sequence's kept state, the token into row 0 and the log, and what
    // enqueue_trunk(1, true) needs of its embedding.
    virtual int enqueue_greedy_token(int seq) = 0;
    // `rows` tokens at positions base.. of one sequence as one block; their rows end in hidden_.
    virtual int prefill_block(int seq, const uint32_t *tokens, int rows, int base) = 0;
    virtual bool matrix_prefill_supported() const = 0;
    virtual int matrix_prefill_min_tokens() const { return kMatrixPrefillMinTokens; }
    virtual int clear_state() = 0;                       // every cache and state of every sequence, enqueued on the stream
    virtual unsigned tuning_epoch() const { return 0; }

    // The buffers this class owns, for `block_rows` rows per block and hidden rows of `hidden_stride` floats.
    int allocate_common(int block_rows, int hidden_stride);
    int finish_finalize() { finalized_ = true; return reset(); }
    void drop_captured_graphs();
    void sync_tuning();
    int capture_step_graph(int seq);
    int capture_steps(int seq, int count, hipGraphExec_t *out);
    int replay_steps(int seq, int steps);
    int upload_block_rows(int seq, const uint32_t *tokens, int rows, int base);
    int check_sequence(int seq) const;

    bool finalized_ = false;
    int hidden_stride_ = 0, block_rows_ = 0;
    float *hidden_ = nullptr, *logits_ = nullptr, *last_hidden_ = nullptr, *want_rows_ = nullptr;
    int *d_tokens_ = nullptr, *d_pos_ = nullptr, *d_seq_ = nullptr, *d_out_tokens_ = nullptr;
    std::vector<int> visible_;
    std::vector<char> taken_;
    // captured greedy step per sequence (head -> feed -> trunk -> keep), and its device-side state
    bool use_graph_ = true;
    std::vector<hipGraphExec_t> step_graphs_, multi_graphs_;   // one step, kStepsPerGraph steps
    unsigned long long id_ = 0, graph_epoch_ = 1;
    unsigned tuning_epoch_ = 0;   // the kernel-selection epoch this runtime's captured graphs were made under
    int *d_visible_ = nullptr, *d_log_ = nullptr, *d_log_count_ = nullptr;
    ArgmaxScratch argmax_scratch_;
    int head_partial_capacity_ = 0;      // (value, index) slots per row for the head's per-workgroup candidates
    bool matrix_prefill_ = true;
    bool capturing_ = false;             // enqueue_trunk is being captured into a sequence's step graph (replays may follow its stop token)

    struct TimedLaunch { int kernel_class; hipEvent_t start, stop; };
    bool timing_enabled_ = false;
    std::vector<TimedLaunch> timed_;        // pending pairs
    std::vector<hipEvent_t> event_pool_;
    double time_total_us_[kMaxKernelClasses] = {};
    long time_launches_[kMaxKernelClasses] = {};
    hipEvent_t take_event();
    int time_begin(int kernel_class);
    int time_end();
};

template <typename T>
void free_device(T *&p) {
    if (p) (void)hipFree(p);
    p = nullptr;
}

}  // namespace esp

// handle behind the runtime entry points of the C ABI, whatever the architecture
struct ESPLlamaRuntime {
    esp::DecoderRuntime *rt;
};
