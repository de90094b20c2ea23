// Device-resident llama decoder state: the MI355X counterpart of the reference's
// CPUExactLlamaRuntime (Sources/RealModelInference/RealModelInferenceEngine.swift:548-850).
#pragma once

#include <string>
#include <vector>

#include "decoder_runtime.h"

namespace esp {

// weight slots; names follow LayerWeightPaths (Sources/ModelSupport/LayerWeightPaths.swift:22-84)
enum WeightSlot : int {
    SLOT_TOKEN_EMBEDDING = 0, SLOT_FINAL_NORM = 1, SLOT_LM_HEAD = 2,
    SLOT_RMS_ATT = 10, SLOT_WQ = 11, SLOT_WK = 12, SLOT_WV = 13, SLOT_WO = 14,
    SLOT_RMS_FFN = 15, SLOT_W1 = 16, SLOT_W2 = 17, SLOT_W3 = 18, SLOT_Q_NORM = 19, SLOT_K_NORM = 20,
};

struct LlamaConfig : DecoderShape {
    int n_layer = 0, n_head = 0, n_kv_head = 0, head_dim = 0, hidden_dim = 0;
    float norm_eps = 1e-5f, rope_theta = 10000.0f;
    int kv_format = FMT_F32;  // FMT_F32 or FMT_F16
    int attention_dim() const { return n_head * head_dim; }
    int kv_dim() const { return n_kv_head * head_dim; }
};

// What a device-resident generation loop over two runtimes (target + draft) keeps between calls, owned by the target: its state
// and token log in device memory and the captured graphs of its passes.  The graphs hold pointers into both runtimes, so the
// session names the partner by an identifier no later runtime can have, and both runtimes' graph epochs (which change whenever a
// runtime's kernels for a step change): a session that does not match is rebuilt, never replayed.
struct DeviceLoopSession {
    unsigned long long partner_id = 0, epoch = 0, partner_epoch = 0;
    void *state = nullptr;
    int *log = nullptr;
    int log_capacity = 0;
    hipGraphExec_t one = nullptr, many = nullptr;   // one pass; several passes in a row
};

class LlamaRuntime : public DecoderRuntime {
  public:
    static int create(const LlamaConfig &config, LlamaRuntime **out);
    ~LlamaRuntime() override;

    const LlamaConfig &config() const { return c_; }
    const DecoderShape &shape() const override { return c_; }
    LlamaRuntime *as_llama() override { return this; }

    // Copies the bytes.  Matrices: GGUF block layout, row-major [rows, cols]; norms: f32 or f16 vectors;
    // embedding: f32 or f16 table.
    int set_weight(int layer, int slot, int format, const void *data, size_t bytes);
    // Fuses wq|wk|wv and w1|w3, uploads everything, builds the RoPE table.
    int finalize();

    // Decode steps of one or two rows: attention as one launch that leaves partial states, merged by the wo GEMV
    // (on by default where the shapes allow); off = the split kernel plus the merge kernel.
    void set_merged_attention(bool enabled);
    // Decode steps of one or two rows feed every layer GEMV that has the form (matrix-core Q4_K) hi / lo fp16 pairs of the fp32
    // activations instead of their fp16 roundings (default on; ESPRESSO_HIP_SPLIT_ACTIVATIONS=0 at creation switches it off).
    void set_split_activations(bool enabled);
    bool split_activations() const { return split_activations_; }
    bool merged_attention_in_use() const { return !layers_.empty() && wo_merges_attention(layers_[0], 1); }

    size_t weight_bytes_per_token() const override { return weight_bytes_; }
    size_t resident_weight_bytes() const override { return resident_weight_bytes_; }

    EmbedTarget device_embed_target() { EmbedTarget e; e.table = embedding_; e.table_is_f16 = embedding_f16_ ? 1 : 0; e.d = c_.d_model; e.hidden = hidden_; return e; }
    DeviceLoopSession &loop_session() { return loop_session_; }
    void release_loop_session();   // destroys the session's graphs and frees its buffers

    enum KernelClass { K_QKV = 0, K_WO, K_GATE_UP, K_DOWN, K_HEAD, K_ATTENTION, K_EVENT_PAIR, K_CLASS_COUNT };
    size_t kernel_bytes(int kernel_class) const;   // algorithmic bytes of one batch-1 launch
    // mean_us: launches back to back between two events; kernel_only_us (optional): the same launches with events
    // of their own per launch (the kernels' own durations, as a kernel trace reports them)
    int time_kernel_class(int kernel_class, int iters, double *mean_us, double *kernel_only_us = nullptr);

  private:
    LlamaRuntime() = default;
    struct HostTensor { int format = -1; std::vector<uint8_t> bytes; };
    struct HostLayer { HostTensor rms_att, wq, wk, wv, wo, rms_ffn, w1, w2, w3, q_norm, k_norm; };
    struct Layer {
        float *rms_att = nullptr, *rms_ffn = nullptr, *q_norm = nullptr, *k_norm = nullptr;
        DeviceMatrix wqkv, wo, w13, w2;
        void *k_cache = nullptr, *v_cache = nullptr;
    };
    int upload_vector(const HostTensor &t, size_t count, float **out, const char *what);
    // without want_logits one or two rows take the head whose epilogue is the arg-max and store none
    int run_head(const float *hidden_rows, int count, bool want_logits = false) override;
    bool head_fuses_argmax() const { return fused_head_argmax_ && gemv_supports_argmax(lm_head_); }
    int enqueue_trunk(int rows, bool embedded = false, float *final_out = nullptr) override;
    int enqueue_greedy_token(int seq) override;
    int prefill_block(int seq, const uint32_t *tokens, int rows, int base) override;
    int clear_state() override;
    unsigned tuning_epoch() const override { return gemv_tuning_epoch(); }
    int enqueue_layers_matrix(int rows, bool one_sequence_consecutive = false);
    bool matrix_prefill_supported() const override;
    bool wo_merges_attention(const Layer &L, int rows) const;
    HostTensor *host_slot(int layer, int slot);

    LlamaConfig c_;
    HostTensor h_embedding_, h_final_norm_, h_lm_head_;
    std::vector<HostLayer> h_layers_;

    void *embedding_ = nullptr;
    bool embedding_f16_ = true;
    float *final_norm_ = nullptr;
    DeviceMatrix lm_head_;
    std::vector<Layer> layers_;
    float *rope_cos_ = nullptr, *rope_sin_ = nullptr;
    // activations for up to kMaxStepRows rows
    float *qkv_ = nullptr, *q_ = nullptr, *gu_ = nullptr;
    uint16_t *xn_ = nullptr, *ctx_ = nullptr, *act_ = nullptr;
    // prompt blocks with split activations: the lo planes and sub-block sums beside xn_, ctx_ and act_ (SplitRowsView)
    uint16_t *xn_lo_ = nullptr, *ctx_lo_ = nullptr, *act_lo_ = nullptr, *xn_sums_ = nullptr, *ctx_sums_ = nullptr, *act_sums_ = nullptr;
    bool split_blocks_supported() const;
    int enqueue_layers_split(int rows);
    size_t weight_bytes_ = 0, resident_weight_bytes_ = 0;
    DeviceLoopSession loop_session_;
    bool fused_head_argmax_ = true;      // ESPRESSO_HIP_FUSED_HEAD_ARGMAX=0: head GEMV stores logits, separate arg-max launches
    float *attn_scratch_ = nullptr;
    bool merged_attention_ = true;
    bool split_activations_ = true;
    bool prompt_attention_ = false;   // prompt blocks run attention on the matrix cores
    float *gemm_workspace_ = nullptr;
    GemmSplitSharedK gemm_shared_k_;   // the device's pool for launch_gemm_split's hand-over between workgroups (not owned)
};

}  // namespace esp
