// Argument blocks and launchers of the layered models' kernels: dense products with bf16 weights (dense_gemv.hip, dense_gemm.hip),
// norms and embeddings (layer_ops.hip), retention (retention.hip), Mamba-2 (mamba2.hip), latent attention (latent_attention.hip), grouped
// attention in a window (window_attention.hip) and the block form that both attentions use (block_attention.hip).
//
// Sizes with a _p are padded at upload (heads to multiples of 32 dimensions, products to multiples of 64) with zero weights, so
// padded places hold zeros throughout; means divide by the true sizes.
// Every launcher returns hipErrorInvalidValue for shapes its kernel does not take.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace esp {

// What the operands of prompt kernels and the latent caches are held in.  Weights are bf16 in both.
enum class Precision : int { bf16 = 0, f32 = 1 };
inline size_t precision_bytes(Precision p) { return p == Precision::bf16 ? 2 : 4; }

// The function on the gate of a gated feed-forward.
enum class GateFunction : int { silu = 0, gelu_tanh = 1 };

// A bf16 matrix [rows][ld], ld a multiple of 64.
struct DenseMatrix {
    uint16_t *w = nullptr;
    int rows = 0, ld = 0;
};

// ---- one row, fp32 activations (dense_gemv.hip) -------------------------------------------------------
// The input side of a layer: y[0 .. mix_rows) = W norm1(x), and after them pairs of rows (gate_i, up_i) over norm2(x):
// act[i] = f(gate_i) * up_i.  mix_rows is a multiple of 32.  Without norm1 and norm2 the product reads x itself.  With `branch`, what is
// read is x + branch over its root mean square times branch_norm (a branch that is normed as it joins the stream), and that sum goes
// to x_out, which is not x.
struct DenseGemvIn {
    DenseMatrix w;
    int mix_rows = 0;
    const float *x = nullptr, *norm1 = nullptr, *norm2 = nullptr;   // [ld]
    const float *branch = nullptr, *branch_norm = nullptr;          // [ld]
    float *x_out = nullptr;
    int width = 0;
    float eps = 0;
    float *y = nullptr, *act = nullptr;
    GateFunction gate_function = GateFunction::silu;
};
hipError_t launch_dense_gemv_in(const DenseGemvIn &p, hipStream_t s);

// The output side: out[r] = residual[r] + mult * (W [mix | act])[r] (residual null: the product alone).  mix: values as they are; or the
// retention output o whose heads are first divided by their root mean square (from `squares`, [heads][parts] partial sums) and multiplied
// by silu(gate); or values whose parts are divided by their root mean squares and multiplied by part_norm.
struct DenseGemvOut {
    DenseMatrix w;
    int mix_cols = 0, act_at = 0, act_cols = 0;   // the feed-forward's values start at column act_at
    const float *mix = nullptr, *act = nullptr;
    const float *squares = nullptr, *gate = nullptr;   // retention only
    int parts = 0, vdim = 0, vdim_p = 0;
    const int *part_of = nullptr, *part_starts = nullptr;   // part of a column [mix_cols]; first column of a part [part_count + 1]
    const float *part_norm = nullptr;                       // [mix_cols]
    int part_count = 0;
    float part_size = 0;                                    // values per part (columns without a value are zero)
    bool part_by_eight = false;                             // every part starts at a multiple of eight columns
    float eps = 0, mult = 1;
    const float *residual = nullptr;
    float *out = nullptr;
    int rows = 0;
};
hipError_t launch_dense_gemv_out(const DenseGemvOut &p, hipStream_t s);

// Output head: logits[r] = cap * tanh((W norm(x))[r] / cap), cap 0 = none.
struct DenseGemvHead {
    DenseMatrix w;
    const float *x = nullptr, *norm = nullptr;
    int width = 0, vocab = 0;
    float eps = 0, cap = 0;
    float *logits = nullptr;            // [vocab], or null
    // optional: every workgroup's largest logit and the lowest row that has it, dense_gemv_head_workgroups of them
    float *best_value = nullptr;
    int *best_index = nullptr;
};
int dense_gemv_head_workgroups(const DenseMatrix &w);
hipError_t launch_dense_gemv_head(const DenseGemvHead &p, hipStream_t s);

// ---- blocks of rows on the matrix cores (dense_gemm.hip) -----------------------------------------------
// y[m][n] = sum_k a[m][k] b[n][k].  Either operand bf16 or fp32; the product runs in bf16 when both are bf16, else in fp32.
enum class GemmOut : int {
    planes,       // fp32 partial sums [splits][M][N] (gemm_planes_splits says how many)
    mix_gated,    // columns < mix_cols: fp32 y[m][n]; after them (gate, up) pairs: act[m][i] = f(gate) * up in the operands' type
    elems,        // y in the operands' type
    logits,       // fp32, capped, columns < n_store
};
struct DenseGemm {
    const void *a = nullptr, *a2 = nullptr;   // a2: the rows of columns >= mix_cols (mix_gated)
    const void *b = nullptr;
    Precision a_type = Precision::bf16, b_type = Precision::bf16;
    int lda = 0, ldb = 0;
    int m = 0, n = 0, k = 0;                  // k a multiple of 64
    GemmOut out = GemmOut::planes;
    void *y = nullptr;
    int ldy = 0;
    int mix_cols = 0;                         // a multiple of 128
    void *act = nullptr;
    int ld_act = 0;
    GateFunction gate_function = GateFunction::silu;
    int n_store = 0;
    float cap = 0;
    int splits = 1;
};
int gemm_planes_splits(int m, int n, int k, size_t workspace_floats);
hipError_t launch_dense_gemm(const DenseGemm &p, hipStream_t s);

// ---- embedding, residual stream and norms (layer_ops.hip) -------------------------------------------------
// x[m][..] = RMS norm of embedding row tokens[m] times weight (weight null: the row itself); table bf16 [vocab][ld_table], x rows of ld
// floats, zero past width
hipError_t launch_embed_norm(const uint16_t *table, int ld_table, const int *tokens, const float *weight, float eps, int rows, int width, int ld, float *x, hipStream_t s);
// x += mult * (sum of `splits` planes), then up to two normed copies in `type` (null: none)
struct ResidualNorm {
    float *x = nullptr;
    int rows = 0, width = 0, ld = 0;
    const float *planes = nullptr;
    int splits = 0;
    size_t plane = 0;
    float mult = 1, eps = 0;
    const float *norm1 = nullptr, *norm2 = nullptr;
    void *out1 = nullptr, *out2 = nullptr;
    float *final_x = nullptr;   // when set, the new rows go here instead of x
};
hipError_t launch_residual_norm(const ResidualNorm &p, Precision type, hipStream_t s);
// x += branch over its root mean square, times norm; the branch is the sum of `splits` planes (0: x stays), then a copy in `type` (null: none)
struct BranchNorm {
    float *x = nullptr;
    int rows = 0, width = 0, ld = 0;
    const float *planes = nullptr;
    int splits = 0;
    size_t plane = 0;
    float eps = 0;
    const float *norm = nullptr;
    void *out = nullptr;
    float *final_x = nullptr;   // when set, the new rows go here instead of x
};
hipError_t launch_branch_norm(const BranchNorm &p, Precision type, hipStream_t s);

// tokens per chunk of a recurrence's block form (chunk_recurrence.h)
constexpr int kRecurrenceChunk = 64;

// ---- retention (retention.hip) --------------------------------------------------------------------------
struct RetentionShape {
    int heads, dim, vdim, dim_p, vdim_p;
    int rot_dims, ld_mix;                    // columns of the mixed rows: q | k | v | gate, heads padded
    int max_seq;
    const float *cos, *sin;                  // [max_seq][rot_dims / 2], pair i = (i, i + rot_dims / 2)
    const float *decay, *powers;             // [heads]; [heads][kRecurrenceChunk + 1] powers 0..64
    float *state;                            // [sequence][heads][vdim_p][dim_p] (transposed), fp32
};
int retention_step_parts(int vdim_p);        // partial sums of squares per head a step leaves
// One step per row (rows of different sequences): updates the state at position pos[row] (a position of 0 starts from zero), leaves
// o [rows][heads * vdim_p] and partial sums of squares [rows][heads][parts].  halt: when *halt is not 0 the states stay as they are
// (they hold the row's token already) and only the outputs are computed again.
struct RetentionStep {
    const float *mixed;
    const int *pos, *seq;
    const int *halt;
    float *o, *squares;
    int rows;
};
hipError_t launch_retention_step(const RetentionShape &r, const RetentionStep &p, hipStream_t s);
// A block of rows of one sequence at positions base..: chunked form.  Scratch for R = rows rounded up to 64 in `type`:
struct RetentionBlock {
    const float *mixed;                      // [rows][ld_mix]
    int rows, base, seq;
    void *q, *k;                             // [heads][R][dim_p]
    void *kt_hi, *kt_lo;                     // [heads][dim_p][R], times the decay to the end of the chunk (fp32: kt_lo unused)
    void *vt;                                // [heads][vdim_p][R]
    void *states_hi, *states_lo;             // [R / 64][heads][vdim_p][dim_p], the state before each chunk
    float *o;                                // [rows][heads * vdim_p]
};
hipError_t launch_retention_block(const RetentionShape &r, const RetentionBlock &p, Precision type, hipStream_t s);
// act[m][h * vdim_p + j] = o / rms(o of the head) * silu(gate) in `type`
hipError_t launch_retention_gate(const RetentionShape &r, const float *o, const float *mixed, int rows, float eps, void *act, int ld_act, Precision type, hipStream_t s);

// ---- Mamba-2 (mamba2.hip) -----------------------------------------------------------------------------------
constexpr int kMamba2MaxTaps = 256, kMamba2MaxState = 4096, kMamba2MaxNormGroups = 4096;
struct Mamba2Shape {
    int heads, vdim, state, groups, taps, norm_groups;
    int vdim_p, state_p;
    int ld_mix;                              // columns of the mixed rows: z | x | B | C | dt, heads and groups padded
    int max_seq;
    const float *conv, *conv_bias;           // [taps][channels], last row the current token's; [channels], channels x | B | C
    const float *dt_bias, *rate, *skip;      // [heads]; rate: a token's decay is exp(-rate dt)
    const float *norm;                       // [heads * vdim_p]
    const int *norm_part, *norm_starts;      // part of a value [heads * vdim_p]; first value of a part [norm_groups + 1]
    bool norm_by_eight;                      // every part starts at a multiple of eight values
    float *state_of;                         // [sequence][heads][vdim_p][state_p] (transposed), fp32
    float *inputs;                           // [sequence][taps][channels]: the convolution's input of position p at row p % taps
};
// One step per row (rows of different sequences): updates state and inputs at position pos[row] (a position of 0 starts from zero) and
// leaves y [rows][heads * vdim_p], gated and not yet normed.  halt: as for a retention step.
struct Mamba2Step {
    const float *mixed;
    const int *pos, *seq;
    const int *halt;
    float *y;
    int rows;
};
hipError_t launch_mamba2_step(const Mamba2Shape &r, const Mamba2Step &p, hipStream_t s);
// A block of rows of one sequence at positions base..: the same y in chunked form; the inputs are kept by the norm.  Scratch for R = rows
// rounded up to 64 in `type`:
struct Mamba2Block {
    const float *mixed;                      // [rows][ld_mix]
    int rows, base, seq;
    void *q, *k;                             // C and B, [groups][R][state_p]
    void *kt;                                // [groups][state_p][R]
    void *vt;                                // x, [heads][vdim_p][R]
    void *vs_hi, *vs_lo;                     // x times dt and the decay to the end of its chunk (fp32: vs_lo unused)
    float *log_hi, *log_lo, *step;           // [heads][R]: the decay's logarithm summed from the chunk's start, dt
    void *states_hi, *states_lo;             // [R / 64][heads][vdim_p][state_p], the state before each chunk
    float *y;
};
hipError_t launch_mamba2_block(const Mamba2Shape &r, const Mamba2Block &p, Precision type, hipStream_t s);
// act = parts of y over their root mean squares, times the norm's weights; after a block of one sequence (block_rows) also its last
// inputs into the sequence's ring
struct Mamba2Norm {
    const float *y;
    void *act;
    int ld_act;
    float eps;
    int block_rows, base, seq;
    const float *mixed;
    int pieces;                              // set by the launcher
};
hipError_t launch_mamba2_norm(const Mamba2Shape &r, const Mamba2Norm &p, int rows, Precision type, hipStream_t s);

// ---- attention of a block over gathered keys (block_attention.hip) ------------------------------------------
struct BlockAttention {
    int heads = 0, kv_heads = 0;             // query head h reads key and value head h / (heads / kv_heads)
    int dim_p = 0, rot_p = 0, vdim_p = 0, window = 0;
    float scale = 1;
    int rows = 0, before = 0, keys_p = 0;    // row m is key before + m; keys_p a multiple of 64
    const void *q = nullptr;                 // [heads][rows rounded up to 32][dim_p + rot_p]
    const void *k = nullptr;                 // [keys_p][kv_heads * dim_p]
    const void *key_rot = nullptr;           // [keys_p][rot_p], shared by all heads (rot_p > 0)
    const void *vt = nullptr;                // [kv_heads * vdim_p][keys_p]
    const float *sink = nullptr;             // [heads], or null
    const float *gate = nullptr;             // [rows][ld_gate]: the output of head h times sigmoid(gate[h]), or null
    int ld_gate = 0;
    void *act = nullptr;                     // [rows][ld_act]
    int ld_act = 0;
};
hipError_t launch_block_attention(const BlockAttention &p, Precision type, hipStream_t s);

// ---- grouped attention in a window (window_attention.hip) ------------------------------------------------------
constexpr int kAttentionMaxHead = 1024;
struct AttentionShape {
    int heads, kv_heads, dim, vdim;
    int dim_p, vdim_p;                       // a cached row is kv_heads * (dim_p + vdim_p) elements: keys, then values
    int rot_dims, window;
    int ld_mix, k_at;                        // columns of the mixed rows: q | k | v (k_at < 0: q alone)
    int max_seq, ring;                       // the cache holds position p at row p % ring
    float scale, eps;
    const float *cos, *sin;                  // [max_seq][rot_dims / 2], pair i = (i, i + rot_dims / 2)
    const float *q_norm, *k_norm;            // [heads * dim_p], [kv_heads * dim_p]
    void *cache;                             // [sequence][ring][kv_heads * (dim_p + vdim_p)]
};
// One query per row (rows of different sequences): the row's own key and value into the cache where the layer has them, then attention.
int attention_step_splits(const AttentionShape &l);
struct AttentionStep {
    const float *mixed;
    const int *pos, *seq;
    float *partial, *partial_ml;             // [rows][splits][heads][vdim_p], [rows][splits][heads][2]
    int splits, rows;
    float *mix;                              // fp32 out [rows][heads * vdim_p], or
    void *act;                               // `type` out, rows of ld_act
    int ld_act;
};
hipError_t launch_attention_step(const AttentionShape &l, const AttentionStep &p, Precision type, hipStream_t s);
// A block of rows of one sequence at positions base..
struct AttentionBlock {
    const float *mixed;
    int rows, base, seq;
    int first_key, keys, keys_p;             // keys first_key .. base + rows - 1; keys_p: rounded up to 64
    void *q;                                 // [heads][rows rounded up to 32][dim_p]
    void *k, *vt;                            // [keys_p][kv_heads * dim_p], [kv_heads * vdim_p][keys_p]
    void *act;
    int ld_act;
};
hipError_t launch_attention_block(const AttentionShape &l, const AttentionBlock &p, Precision type, hipStream_t s);

// ---- latent attention (latent_attention.hip) ----------------------------------------------------------------
struct LatentShape {
    int heads, dim, vdim, rot_dim, kv_rank;
    int dim_p, vdim_p, rot_p, rank_p;        // a cached row is rank_p + rot_p elements
    int rot_dims, window;
    int ld_mix, dkv_at, gate_at;             // columns of the mixed rows: q | latent, rotated key part (dkv_at < 0: none) | gates
    int max_seq, ring;                       // the cache holds position p at row p % ring
    float scale, eps;
    const float *cos, *sin;                  // [max_seq][rot_dims / 2], pair i = (2i, 2i + 1), YaRN's factor included
    const float *latent_norm, *sink;
    const uint16_t *uk, *uv;                 // [heads * dim_p][rank_p], [heads * vdim_p][rank_p]
    void *cache;                             // [sequence][ring][rank_p + rot_p]
};
// Rows' latents and rotated key parts into the cache (layers with dkv_at >= 0); for blocks, a step does it itself.
hipError_t launch_latent_store(const LatentShape &l, const float *mixed, const int *pos, const int *seq, int rows, Precision type, hipStream_t s);
// One query per row (rows of different sequences): the row's own latent into the cache where the layer has one, queries through W_uk
// into the latent space, attention over the cached latents, values through W_uv.
constexpr int kLatentMaxRank = 1024;
int latent_step_splits(const LatentShape &l);
struct LatentStep {
    const float *mixed;
    const int *pos, *seq;
    float *absorbed;                         // [rows][heads][rank_p + rot_p]
    float *partial, *partial_ml;             // [rows][splits][heads][rank_p], [rows][splits][heads][2]
    int splits, rows;
    float *mix;                              // fp32 out [rows][heads * vdim_p], or
    void *act;                               // `type` out, rows of ld_act
    int ld_act;
};
hipError_t launch_latent_step(const LatentShape &l, const LatentStep &p, Precision type, hipStream_t s);
// A block of rows of one sequence at positions base..: the latents of every key the block can see are gathered, projected to
// keys and values by the caller's products (K [T][heads * dim_p], V^T [heads * vdim_p][T_p]), and attended to tile by tile.
struct LatentBlock {
    const float *mixed;
    int rows, base, seq;
    int first_key, keys, keys_p;             // keys first_key .. base + rows - 1; keys_p: rounded up to 64
    void *q;                                 // [heads][rows rounded up to 32][dim_p + rot_p]
    void *latents, *key_rot;                 // [keys_p][rank_p], [keys_p][rot_p]
    const void *k, *vt;
    void *act;
    int ld_act;
};
hipError_t launch_latent_gather(const LatentShape &l, const LatentBlock &p, Precision type, hipStream_t s);
hipError_t launch_latent_queries(const LatentShape &l, const LatentBlock &p, Precision type, hipStream_t s);
hipError_t launch_latent_block(const LatentShape &l, const LatentBlock &p, Precision type, hipStream_t s);

}  // namespace esp
