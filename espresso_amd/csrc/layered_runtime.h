// Device-resident runtime of layered models (host/layered_config.h): bf16 weights, an fp32 residual stream, per-sequence recurrent
// states and rings of cached latents or keys and values.  Decode steps of one row run on the dense GEMV kernels with fp32 activations;
// blocks of rows on the matrix cores in bf16 (or fp32, Precision::f32, which also keeps the caches in fp32).
//
// How branches join the stream (BlockKind) and what a mixer computes (MixerKind) are independent: layered_runtime.cpp walks the layers,
// layered_mixers.cpp holds each mixer's weights, state and cache, its step and its block.
#pragma once

#include <functional>
#include <string>
#include <vector>

#include "decoder_runtime.h"
#include "host/layered_config.h"
#include "kernels/layer_ops.h"

namespace esp {

struct LayeredOptions {
    Precision precision = Precision::bf16;
    int max_seq = 0;
    int max_sequences = 1;
    int eos_token = -1;
};

// Where a layered model's tensors come from: fills `out` ([rows][cols] bf16 bits for matrices, fp32 values for vectors).
// Returns ESP_OK or an error with its text set.
class LayeredWeights {
  public:
    virtual ~LayeredWeights() = default;
    virtual int matrix(const std::string &name, int rows, int cols, std::vector<uint16_t> *out) = 0;
    virtual int vector(const std::string &name, int count, std::vector<float> *out) = 0;
};

class LayeredRuntime : public DecoderRuntime {
  public:
    static int create(const LayeredConfig &config, const LayeredOptions &options, LayeredWeights &weights, LayeredRuntime **out);
    ~LayeredRuntime() override;

    const LayeredConfig &config() const { return c_; }
    const DecoderShape &shape() const override { return shape_; }
    LayeredRuntime *as_layered() override { return this; }
    Precision precision() const { return precision_; }
    // Recurrent states cannot be taken back; a model of attention layers alone can.
    bool can_roll_back() const override { return !recurrent_; }
    bool takes_rows_of_one_sequence() const override { return false; }
    size_t weight_bytes_per_token() const override { return weight_bytes_; }
    size_t resident_weight_bytes() const override { return weight_bytes_ + (size_t)c_.vocab * c_.width * 2; }
    // what one sequence holds in states and caches
    size_t sequence_bytes() const { return sequence_bytes_; }
    static constexpr int kMinBlockRows = 3;
    // Blocks shorter than this run token by token (tests and measurements move it; default kMinBlockRows).
    void set_min_block_rows(int rows) { min_block_rows_ = rows < 1 ? 1 : rows; }
    // Residual stream after every layer of a block, one call per layer (tests).
    void set_layer_observer(std::function<void(int layer)> f) { layer_observer_ = std::move(f); }

    enum KernelClass { K_IN = 0, K_RETENTION, K_LATENT, K_OUT, K_HEAD, K_NORM, K_ATTENTION, K_MAMBA2, K_CLASS_COUNT };
    size_t kernel_bytes(int kernel_class) const;   // algorithmic bytes of the class's launches in one decode step

  private:
    LayeredRuntime() = default;
    struct Layer {
        MixerKind mixer = MixerKind::retention;
        GateFunction gate_function = GateFunction::silu;
        float *norm1 = nullptr, *norm2 = nullptr;
        // Parallel branches: the feed-forward's rows follow the mixer's in `in`, its columns in `out`.  Sequential ones: up and down.
        DenseMatrix in, out, up, down, uk, uv;
        int mix_rows = 0, mix_cols = 0;        // rows of `in` and columns of `out` that belong to the mixer
        std::vector<float *> vectors;          // the mixer's parameters (named by its shape)
        std::vector<int *> tables;
        float *state = nullptr, *inputs = nullptr;   // recurrent states and convolution inputs of every sequence
        size_t state_floats = 0, input_floats = 0;   // of one sequence
        void *cache = nullptr;                 // latents, or keys and values, of every sequence (layers with a cache of their own)
        size_t cache_row_bytes = 0;
        int ring = 0, splits = 0;
        float *cos = nullptr, *sin = nullptr;  // shared between layers of equal rotation
        RetentionShape retention{};
        LatentShape latent{};
        AttentionShape attention{};
        Mamba2Shape mamba2{};
    };
    int build(LayeredWeights &weights);
    int build_layer(size_t index, LayeredWeights &weights);
    int upload_matrix(const std::vector<uint16_t> &host, int rows, int ld, DenseMatrix *out);
    int upload_floats(const std::vector<float> &host, float **out);
    int padded_vector(LayeredWeights &weights, const std::string &name, int count, int padded, float **out);
    int head_vector(LayeredWeights &weights, const std::string &name, int heads, int size, int padded, float **out);   // heads padded
    int rotary_table(const RotarySpec &spec, float **cos, float **sin);
    int allocate_scratch();

    int enqueue_trunk(int rows, bool embedded = false, float *final_out = nullptr) override;
    int run_head(const float *hidden_rows, int count, bool want_logits = false) override;
    int enqueue_greedy_token(int seq) override;
    int prefill_block(int seq, const uint32_t *tokens, int rows, int base) override;
    bool matrix_prefill_supported() const override { return true; }
    int matrix_prefill_min_tokens() const override { return min_block_rows_; }
    int clear_state() override;
    int enqueue_step(float *final_out);
    int enqueue_step_sequential(float *final_out);
    // Layers over `rows` rows: one sequence at positions base.. (seq >= 0), or one row each of several sequences (seq < 0).
    int enqueue_block(int rows, int seq, int base, float *final_out);
    int enqueue_block_sequential(int rows, int seq, int base, float *final_out);
    int enqueue_planes(const DenseMatrix &w, int rows, int *splits);   // the product of act_ with w, into planes of the workspace

    // ---- mixers (layered_mixers.cpp) ----
    static int mixer_rows(const LayerSpec &spec);             // rows of the mixer's projections, heads padded
    int place_mixer_rows(size_t index, LayeredWeights &weights, std::vector<uint16_t> *in);
    int build_mixer(size_t index, LayeredWeights &weights);   // parameters, state and cache
    int build_retention(size_t index, LayeredWeights &weights);
    int build_latent(size_t index, LayeredWeights &weights);
    int build_attention(size_t index, LayeredWeights &weights);
    int build_mamba2(size_t index, LayeredWeights &weights);
    int allocate_cache(size_t index, size_t row_elements);
    int allocate_mixer_scratch();
    // One row from mixed_: enqueues the mixer and says what the output product stages.
    int mixer_step(Layer &L, DenseGemvOut *out);
    // Rows from mixed_ to act_ (rows of L.out.ld elements).
    int mixer_block(Layer &L, int rows, int seq, int base);
    struct KeyRange { int first, keys, keys_p; };
    static KeyRange visible_keys(int window, int rows, int base);

    LayeredConfig c_;
    DecoderShape shape_;
    Precision precision_ = Precision::bf16;
    bool recurrent_ = false;
    int min_block_rows_ = kMinBlockRows;
    int width_p_ = 0, mix_max_ = 0, out_cols_max_ = 0;
    size_t weight_bytes_ = 0, sequence_bytes_ = 0;
    uint16_t *embedding_ = nullptr;            // the head's matrix where the two are tied
    int embedding_ld_ = 0;
    float *embed_norm_ = nullptr, *final_norm_ = nullptr;
    DenseMatrix head_;
    std::vector<Layer> layers_;
    struct RotaryTable { RotarySpec spec; float *cos, *sin; };
    std::vector<RotaryTable> rotary_;
    std::function<void(int)> layer_observer_;

    // rows of a block or step
    float *stream_ = nullptr, *branch_ = nullptr;   // a step's second copy of the stream, and the branch about to join it
    float *mixed_ = nullptr, *act32_ = nullptr, *mix32_ = nullptr, *squares_ = nullptr, *absorbed_ = nullptr, *partial_ = nullptr, *partial_ml_ = nullptr;
    void *n1_ = nullptr, *n2_ = nullptr, *act_ = nullptr;
    float *workspace_ = nullptr;
    size_t workspace_floats_ = 0;
    void *r_q_ = nullptr, *r_k_ = nullptr, *r_kt_hi_ = nullptr, *r_kt_lo_ = nullptr, *r_vt_ = nullptr, *r_states_hi_ = nullptr, *r_states_lo_ = nullptr;
    void *r_vs_hi_ = nullptr, *r_vs_lo_ = nullptr;
    float *r_log_hi_ = nullptr, *r_log_lo_ = nullptr, *r_step_ = nullptr;
    void *l_q_ = nullptr, *l_latents_ = nullptr, *l_key_rot_ = nullptr, *l_k_ = nullptr, *l_vt_ = nullptr;
};

}  // namespace esp
