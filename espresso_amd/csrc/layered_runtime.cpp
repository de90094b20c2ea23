#include "layered_runtime.h"

#include <algorithm>
#include <cmath>
#include <cstring>

#include "layered_layout.h"

namespace esp {
using layered::place_rows;
using layered::up;

int LayeredRuntime::create(const LayeredConfig &config, const LayeredOptions &options, LayeredWeights &weights, LayeredRuntime **out) {
    *out = nullptr;
    if (config.layers.empty() || config.vocab < 1 || config.width < 1) return fail(ESP_ERR_INVALID_ARGUMENT, "layered config: no layers, vocabulary or width");
    if (options.max_seq < 1) return fail(ESP_ERR_INVALID_ARGUMENT, "layered runtime: max_seq must be positive");
    if (options.max_sequences < 1 || options.max_sequences > kMaxStepRows)
        return fail(ESP_ERR_INVALID_ARGUMENT, "layered runtime: max_sequences must be 1..%d", kMaxStepRows);
    for (size_t i = 0; i < config.layers.size(); i++) {
        const LayerSpec &S = config.layers[i];
        const struct { bool wrong; const char *what; int value, most; } limits[] = {
            {S.mixer == MixerKind::latent_attention && up(S.kv_rank, 64) > kLatentMaxRank, "latent values", S.kv_rank, kLatentMaxRank},
            {S.mixer == MixerKind::attention && std::max(S.dim, S.vdim) > kAttentionMaxHead, "values per attention head", std::max(S.dim, S.vdim), kAttentionMaxHead},
            {S.mixer == MixerKind::mamba2 && S.state > kMamba2MaxState, "values of a state", S.state, kMamba2MaxState},
            {S.mixer == MixerKind::mamba2 && S.conv > kMamba2MaxTaps, "taps of a convolution", S.conv, kMamba2MaxTaps},
            {S.mixer == MixerKind::mamba2 && S.norm_groups > kMamba2MaxNormGroups, "parts of a norm", S.norm_groups, kMamba2MaxNormGroups},
        };
        for (const auto &l : limits) if (l.wrong) return fail(ESP_ERR_UNSUPPORTED, "layer %zu: %d %s exceed %d", i, l.value, l.what, l.most);
    }
    int rc = ensure_init();
    if (rc != ESP_OK) return rc;
    LayeredRuntime *rt = new LayeredRuntime();
    rt->c_ = config;
    rt->precision_ = options.precision;
    rt->shape_.d_model = config.width; rt->shape_.vocab = config.vocab; rt->shape_.max_seq = options.max_seq;
    rt->shape_.max_sequences = options.max_sequences; rt->shape_.eos_token = options.eos_token;
    if ((rc = rt->build(weights)) != ESP_OK) { delete rt; return rc; }
    *out = rt;
    return ESP_OK;
}

LayeredRuntime::~LayeredRuntime() {
    if (!c_.tied_head) free_device(embedding_);
    free_device(embed_norm_); free_device(final_norm_); free_device(head_.w);
    for (Layer &L : layers_) {
        for (DenseMatrix *m : {&L.in, &L.out, &L.up, &L.down, &L.uk, &L.uv}) free_device(m->w);
        for (float *p : L.vectors) free_device(p);
        for (int *p : L.tables) free_device(p);
        free_device(L.norm1); free_device(L.norm2); free_device(L.state); free_device(L.inputs); free_device(L.cache);
    }
    for (RotaryTable &t : rotary_) { free_device(t.cos); free_device(t.sin); }
    for (float *p : {stream_, branch_, mixed_, act32_, mix32_, squares_, absorbed_, partial_, partial_ml_, workspace_, r_log_hi_, r_log_lo_, r_step_}) free_device(p);
    for (void *p : {n1_, n2_, act_, r_q_, r_k_, r_kt_hi_, r_kt_lo_, r_vt_, r_vs_hi_, r_vs_lo_, r_states_hi_, r_states_lo_, l_q_, l_latents_, l_key_rot_, l_k_, l_vt_}) free_device(p);
}

int LayeredRuntime::upload_matrix(const std::vector<uint16_t> &host, int rows, int ld, DenseMatrix *out) {
    out->rows = rows; out->ld = ld;
    const int rc = device_alloc(&out->w, host.size());
    if (rc != ESP_OK) return rc;
    ESP_HIP_TRY(hipMemcpy(out->w, host.data(), host.size() * 2, hipMemcpyHostToDevice));
    weight_bytes_ += host.size() * 2;
    return ESP_OK;
}

int LayeredRuntime::upload_floats(const std::vector<float> &host, float **out) {
    const int rc = device_alloc(out, host.size());
    if (rc != ESP_OK) return rc;
    ESP_HIP_TRY(hipMemcpy(*out, host.data(), host.size() * 4, hipMemcpyHostToDevice));
    return ESP_OK;
}

int LayeredRuntime::padded_vector(LayeredWeights &weights, const std::string &name, int count, int padded, float **out) {
    std::vector<float> v;
    const int rc = weights.vector(name, count, &v);
    if (rc != ESP_OK) return rc;
    v.resize(padded, 0.0f);
    return upload_floats(v, out);
}

int LayeredRuntime::head_vector(LayeredWeights &weights, const std::string &name, int heads, int size, int padded, float **out) {
    std::vector<float> v, p((size_t)heads * padded, 0.0f);
    const int rc = weights.vector(name, heads * size, &v);
    if (rc != ESP_OK) return rc;
    for (int h = 0; h < heads; h++) std::copy_n(v.begin() + (size_t)h * size, size, p.begin() + (size_t)h * padded);
    return upload_floats(p, out);
}

// Cosines and sines of every position, computed in double and rounded once.
int LayeredRuntime::rotary_table(const RotarySpec &spec, float **cos, float **sin) {
    for (const RotaryTable &t : rotary_)
        if (t.spec == spec) { *cos = t.cos; *sin = t.sin; return ESP_OK; }
    std::vector<double> f;
    double amplitude = 1.0;
    spec.frequencies(&f, &amplitude);
    const size_t half = f.size();
    std::vector<float> c((size_t)shape_.max_seq * half), s(c.size());
    for (int p = 0; p < shape_.max_seq; p++)
        for (size_t i = 0; i < half; i++) {
            c[p * half + i] = (float)(std::cos(p * f[i]) * amplitude);
            s[p * half + i] = (float)(std::sin(p * f[i]) * amplitude);
        }
    RotaryTable t{spec, nullptr, nullptr};
    int rc = upload_floats(c, &t.cos);
    if (rc == ESP_OK) rc = upload_floats(s, &t.sin);
    if (rc != ESP_OK) { free_device(t.cos); return rc; }
    rotary_.push_back(t);
    *cos = t.cos; *sin = t.sin;
    return ESP_OK;
}

int LayeredRuntime::build(LayeredWeights &weights) {
    width_p_ = up(c_.width, 64);
    int rc;
    std::vector<uint16_t> m, p;
    if ((rc = weights.matrix("embed", c_.vocab, c_.width, &m)) != ESP_OK) return rc;
    if (!c_.tied_head) {
        if ((rc = device_alloc(&embedding_, m.size())) != ESP_OK) return rc;
        ESP_HIP_TRY(hipMemcpy(embedding_, m.data(), m.size() * 2, hipMemcpyHostToDevice));
        embedding_ld_ = c_.width;
        if ((rc = weights.matrix("head", c_.vocab, c_.width, &m)) != ESP_OK) return rc;
    }
    if (c_.embed_norm && (rc = padded_vector(weights, "embed.norm", c_.width, width_p_, &embed_norm_)) != ESP_OK) return rc;
    if ((rc = padded_vector(weights, "final.norm", c_.width, width_p_, &final_norm_)) != ESP_OK) return rc;
    const int head_rows = up(c_.vocab, 32);
    p.assign((size_t)head_rows * width_p_, 0);
    place_rows(m, c_.width, 0, c_.vocab, &p, width_p_, 0);
    if ((rc = upload_matrix(p, head_rows, width_p_, &head_)) != ESP_OK) return rc;
    if (c_.tied_head) { embedding_ = head_.w; embedding_ld_ = head_.ld; }
    layers_.resize(c_.layers.size());
    for (size_t i = 0; i < layers_.size(); i++)
        if ((rc = build_layer(i, weights)) != ESP_OK) return rc;
    // a layer that reads another one's cache takes its ring
    for (size_t i = 0; i < layers_.size(); i++) {
        const int from = c_.layers[i].kv_from;
        if (!has_cache(c_.layers[i].mixer) || from < 0) continue;
        Layer &L = layers_[i];
        L.latent.cache = L.attention.cache = layers_[from].cache;
        L.latent.ring = L.attention.ring = layers_[from].ring;
    }
    if ((rc = allocate_common(kPrefillBlockRows, width_p_)) != ESP_OK) return rc;
    if ((rc = allocate_scratch()) != ESP_OK) return rc;
    return finish_finalize();
}

int LayeredRuntime::build_layer(size_t index, LayeredWeights &weights) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    const bool parallel = c_.block == BlockKind::parallel_two_norms;
    const std::string p = "l" + std::to_string(index) + ".";
    const int d = c_.width, vp = up(S.vdim, 32), H = S.heads, ffp = S.ff ? up(S.ff, 64) : 0;
    int rc;
    L.mixer = S.mixer;
    L.gate_function = S.activation == Activation::gelu_tanh ? GateFunction::gelu_tanh : GateFunction::silu;
    if ((rc = padded_vector(weights, p + "norm1", d, width_p_, &L.norm1)) != ESP_OK) return rc;
    if (S.ff && (rc = padded_vector(weights, p + "norm2", d, width_p_, &L.norm2)) != ESP_OK) return rc;

    // ---- input side: the mixer's projections head by head; gate and up rows in pairs ----
    L.mix_rows = up(mixer_rows(S), 128);
    const int in_rows = L.mix_rows + (parallel ? 2 * ffp : 0);
    std::vector<uint16_t> in((size_t)in_rows * width_p_, 0), pairs, m;
    if ((rc = place_mixer_rows(index, weights, &in)) != ESP_OK) return rc;
    if (S.ff) {
        if (!parallel) pairs.assign((size_t)2 * ffp * width_p_, 0);
        std::vector<uint16_t> &dst = parallel ? in : pairs;
        for (int half = 0; half < 2; half++) {
            if ((rc = weights.matrix(p + (half ? "mlp.up" : "mlp.gate"), S.ff, d, &m)) != ESP_OK) return rc;
            for (int i = 0; i < S.ff; i++) place_rows(m, d, i, 1, &dst, width_p_, (parallel ? L.mix_rows : 0) + 2 * i + half);
        }
    }
    if ((rc = upload_matrix(in, in_rows, width_p_, &L.in)) != ESP_OK) return rc;
    if (!pairs.empty() && (rc = upload_matrix(pairs, 2 * ffp, width_p_, &L.up)) != ESP_OK) return rc;
    std::vector<uint16_t>().swap(in);
    std::vector<uint16_t>().swap(pairs);

    // ---- output side: W_o, with W_down beside it (one product over [mixer | feed-forward]) or on its own ----
    L.mix_cols = up(H * vp, 64);
    const int out_cols = L.mix_cols + (parallel ? ffp : 0);
    std::vector<uint16_t> out((size_t)width_p_ * out_cols, 0);
    if ((rc = weights.matrix(p + "mix.o", d, H * S.vdim, &m)) != ESP_OK) return rc;
    for (int r = 0; r < d; r++)
        for (int h = 0; h < H; h++) std::memcpy(out.data() + (size_t)r * out_cols + h * vp, m.data() + (size_t)r * H * S.vdim + h * S.vdim, (size_t)S.vdim * 2);
    if (S.ff) {
        if ((rc = weights.matrix(p + "mlp.down", d, S.ff, &m)) != ESP_OK) return rc;
        if (parallel) {
            place_rows(m, S.ff, 0, d, &out, out_cols, 0, L.mix_cols);
        } else {
            std::vector<uint16_t> down((size_t)width_p_ * ffp, 0);
            place_rows(m, S.ff, 0, d, &down, ffp, 0);
            if ((rc = upload_matrix(down, width_p_, ffp, &L.down)) != ESP_OK) return rc;
        }
    }
    if ((rc = upload_matrix(out, width_p_, out_cols, &L.out)) != ESP_OK) return rc;
    std::vector<uint16_t>().swap(out);

    mix_max_ = std::max(mix_max_, L.mix_rows);
    out_cols_max_ = std::max(out_cols_max_, std::max(out_cols, ffp));
    return build_mixer(index, weights);
}

int LayeredRuntime::allocate_scratch() {
    const size_t R = block_rows_, E = precision_bytes(precision_);
    size_t act32 = 64;
    for (const Layer &L : layers_) act32 = std::max(act32, (size_t)std::max(L.out.ld - L.mix_cols, L.down.ld));
    int rc;
    auto bytes = [&](void **p, size_t n) -> int {
        uint8_t *q = nullptr;
        const int r = device_alloc(&q, n);
        *p = q;
        return r;
    };
    if ((rc = device_alloc(&stream_, (size_t)width_p_)) != ESP_OK || (rc = device_alloc(&branch_, (size_t)width_p_)) != ESP_OK ||
        (rc = device_alloc(&mixed_, R * mix_max_)) != ESP_OK || (rc = device_alloc(&act32_, act32)) != ESP_OK || (rc = bytes(&n1_, R * width_p_ * E)) != ESP_OK ||
        (rc = bytes(&n2_, R * width_p_ * E)) != ESP_OK || (rc = bytes(&act_, R * out_cols_max_ * E)) != ESP_OK)
        return rc;
    // columns of an output product's input that no head fills meet zero weights, so they only have to be finite
    ESP_HIP_TRY(hipMemset(act_, 0, R * out_cols_max_ * E));
    workspace_floats_ = std::max(kGemmWorkspaceFloats, R * width_p_);
    if ((rc = device_alloc(&workspace_, workspace_floats_)) != ESP_OK) return rc;
    return allocate_mixer_scratch();
}

int LayeredRuntime::clear_state() {
    const size_t n = shape_.max_sequences;
    for (Layer &L : layers_) {
        if (L.state) ESP_HIP_TRY(hipMemsetAsync(L.state, 0, n * L.state_floats * 4, context().stream));
        if (L.inputs) ESP_HIP_TRY(hipMemsetAsync(L.inputs, 0, n * L.input_floats * 4, context().stream));
        if (L.cache) ESP_HIP_TRY(hipMemsetAsync(L.cache, 0, n * L.ring * L.cache_row_bytes, context().stream));
    }
    return ESP_OK;
}

// `embedded` changes nothing here: the trunk always fetches (and norms) the embedding from the rows' tokens.
int LayeredRuntime::enqueue_trunk(int rows, bool, float *final_out) {
    ESP_HIP_TRY(launch_embed_norm(embedding_, embedding_ld_, d_tokens_, embed_norm_, (float)c_.norm_eps, rows, c_.width, width_p_, hidden_, context().stream));
    return rows == 1 ? enqueue_step(final_out) : enqueue_block(rows, -1, 0, final_out);
}

// One row: three launches per recurrent layer, four or five per attention layer, two more for a feed-forward of its own.
int LayeredRuntime::enqueue_step(float *final_out) {
    if (c_.block == BlockKind::sequential_post_norms) return enqueue_step_sequential(final_out);
    hipStream_t s = context().stream;
    const float eps = (float)c_.norm_eps, mult = (float)c_.residual_mult;
    int rc;
    for (size_t i = 0; i < layers_.size(); i++) {
        Layer &L = layers_[i];
        DenseGemvIn in;
        in.w = L.in; in.mix_rows = L.mix_rows; in.x = hidden_; in.norm1 = L.norm1; in.norm2 = L.norm2; in.width = c_.width; in.eps = eps; in.y = mixed_; in.act = act32_; in.gate_function = L.gate_function;
        if ((rc = time_begin(K_IN)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_dense_gemv_in(in, s));
        if ((rc = time_end()) != ESP_OK) return rc;
        DenseGemvOut out;
        out.w = L.out; out.act_at = L.mix_cols; out.act_cols = L.out.ld - L.mix_cols; out.mix = mix32_; out.act = act32_; out.mult = mult; out.eps = eps; out.rows = width_p_;
        out.residual = hidden_; out.out = final_out && i + 1 == layers_.size() ? final_out : hidden_;
        if ((rc = mixer_step(L, &out)) != ESP_OK) return rc;
        if ((rc = time_begin(K_OUT)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_dense_gemv_out(out, s));
        if ((rc = time_end()) != ESP_OK) return rc;
    }
    return ESP_OK;
}

// Every branch is normed as it joins the stream, and the norm needs the whole branch: the next product's staging does both, in every
// workgroup, and its first workgroup writes the new stream to the other of two copies.
int LayeredRuntime::enqueue_step_sequential(float *final_out) {
    hipStream_t s = context().stream;
    const float eps = (float)c_.norm_eps;
    const float *x = hidden_, *norm = nullptr;   // norm: of the branch that has not joined yet
    int rc;
    auto input = [&](const Layer &L, const DenseMatrix &w, int mix_rows) -> int {
        DenseGemvIn in;
        in.w = w; in.mix_rows = mix_rows; in.x = x; in.width = c_.width; in.eps = eps; in.y = mixed_; in.act = act32_; in.gate_function = L.gate_function;
        if (norm) {
            in.branch = branch_; in.branch_norm = norm;
            in.x_out = x == hidden_ ? stream_ : hidden_;
            x = in.x_out;
        }
        int r = time_begin(K_IN);
        if (r != ESP_OK) return r;
        ESP_HIP_TRY(launch_dense_gemv_in(in, s));
        return time_end();
    };
    auto output = [&](DenseGemvOut &out, const DenseMatrix &w) -> int {
        out.w = w; out.act_at = w.ld; out.eps = eps; out.rows = width_p_; out.out = branch_;
        int r = time_begin(K_OUT);
        if (r != ESP_OK) return r;
        ESP_HIP_TRY(launch_dense_gemv_out(out, s));
        return time_end();
    };
    for (Layer &L : layers_) {
        if ((rc = input(L, L.in, L.mix_rows)) != ESP_OK) return rc;
        DenseGemvOut out;
        out.mix = mix32_;
        if ((rc = mixer_step(L, &out)) != ESP_OK || (rc = output(out, L.out)) != ESP_OK) return rc;
        norm = L.norm1;
        if (!L.up.w) continue;
        if ((rc = input(L, L.up, 0)) != ESP_OK) return rc;
        DenseGemvOut down;
        down.mix = act32_; down.mix_cols = L.down.ld;
        if ((rc = output(down, L.down)) != ESP_OK) return rc;
        norm = L.norm2;
    }
    BranchNorm n;
    n.x = const_cast<float *>(x); n.final_x = final_out ? final_out : hidden_;
    n.rows = 1; n.width = c_.width; n.ld = width_p_; n.planes = branch_; n.splits = 1; n.plane = width_p_; n.eps = eps; n.norm = norm;
    if ((rc = time_begin(K_NORM)) != ESP_OK) return rc;
    ESP_HIP_TRY(launch_branch_norm(n, precision_, s));
    return time_end();
}

int LayeredRuntime::enqueue_planes(const DenseMatrix &w, int rows, int *splits) {
    DenseGemm o;
    o.a = act_; o.a_type = precision_; o.lda = w.ld; o.b = w.w; o.ldb = w.ld; o.m = rows; o.n = width_p_; o.k = w.ld;
    o.out = GemmOut::planes; o.y = workspace_; o.ldy = width_p_; o.splits = gemm_planes_splits(rows, width_p_, w.ld, workspace_floats_);
    const int rc = time_begin(K_OUT);
    if (rc != ESP_OK) return rc;
    ESP_HIP_TRY(launch_dense_gemm(o, context().stream));
    *splits = o.splits;
    return time_end();
}

int LayeredRuntime::enqueue_block(int rows, int seq, int base, float *final_out) {
    if (c_.block == BlockKind::sequential_post_norms) return enqueue_block_sequential(rows, seq, base, final_out);
    hipStream_t s = context().stream;
    const float eps = (float)c_.norm_eps;
    const size_t E = precision_bytes(precision_);
    int rc;
    ResidualNorm n;
    n.x = hidden_; n.rows = rows; n.width = c_.width; n.ld = width_p_; n.mult = (float)c_.residual_mult; n.eps = eps; n.out1 = n1_; n.out2 = n2_;
    n.norm1 = layers_.front().norm1; n.norm2 = layers_.front().norm2;
    if ((rc = time_begin(K_NORM)) != ESP_OK) return rc;
    ESP_HIP_TRY(launch_residual_norm(n, precision_, s));
    if ((rc = time_end()) != ESP_OK) return rc;
    for (size_t i = 0; i < layers_.size(); i++) {
        Layer &L = layers_[i];
        const int ld_act = L.out.ld;
        DenseGemm g;
        g.a = n1_; g.a2 = n2_; g.a_type = precision_; g.lda = width_p_; g.b = L.in.w; g.ldb = width_p_; g.m = rows; g.n = L.in.rows; g.k = width_p_;
        g.out = GemmOut::mix_gated; g.y = mixed_; g.ldy = L.mix_rows; g.mix_cols = L.mix_rows; g.ld_act = ld_act; g.gate_function = L.gate_function;
        g.act = static_cast<uint8_t *>(act_) + (size_t)L.mix_cols * E;
        if ((rc = time_begin(K_IN)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_dense_gemm(g, s));
        if ((rc = time_end()) != ESP_OK) return rc;
        if ((rc = mixer_block(L, rows, seq, base)) != ESP_OK || (rc = enqueue_planes(L.out, rows, &n.splits)) != ESP_OK) return rc;
        const bool last = i + 1 == layers_.size();
        n.planes = workspace_; n.plane = (size_t)rows * width_p_;
        n.norm1 = last ? nullptr : layers_[i + 1].norm1; n.norm2 = last ? nullptr : layers_[i + 1].norm2;
        n.final_x = last ? final_out : nullptr;
        if ((rc = time_begin(K_NORM)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_residual_norm(n, precision_, s));
        if ((rc = time_end()) != ESP_OK) return rc;
        if (layer_observer_) layer_observer_((int)i);
    }
    return ESP_OK;
}

int LayeredRuntime::enqueue_block_sequential(int rows, int seq, int base, float *final_out) {
    hipStream_t s = context().stream;
    int rc;
    BranchNorm n;
    n.x = hidden_; n.rows = rows; n.width = c_.width; n.ld = width_p_; n.eps = (float)c_.norm_eps; n.out = n1_;
    auto join = [&]() -> int {
        int r = time_begin(K_NORM);
        if (r != ESP_OK) return r;
        ESP_HIP_TRY(launch_branch_norm(n, precision_, s));
        return time_end();
    };
    auto input = [&](const Layer &L, const DenseMatrix &w, int mix_cols) -> int {
        DenseGemm g;
        g.a = g.a2 = n1_; g.a_type = precision_; g.lda = width_p_; g.b = w.w; g.ldb = width_p_; g.m = rows; g.n = w.rows; g.k = width_p_;
        g.out = GemmOut::mix_gated; g.y = mixed_; g.ldy = mix_cols; g.mix_cols = mix_cols; g.act = act_; g.ld_act = L.down.ld; g.gate_function = L.gate_function;
        int r = time_begin(K_IN);
        if (r != ESP_OK) return r;
        ESP_HIP_TRY(launch_dense_gemm(g, s));
        return time_end();
    };
    if ((rc = join()) != ESP_OK) return rc;   // nothing joins yet: the products' copy of the embeddings
    n.planes = workspace_; n.plane = (size_t)rows * width_p_;
    for (size_t i = 0; i < layers_.size(); i++) {
        Layer &L = layers_[i];
        const bool last = i + 1 == layers_.size();
        if ((rc = input(L, L.in, L.mix_rows)) != ESP_OK || (rc = mixer_block(L, rows, seq, base)) != ESP_OK || (rc = enqueue_planes(L.out, rows, &n.splits)) != ESP_OK) return rc;
        n.norm = L.norm1;
        n.final_x = last && !L.up.w ? final_out : nullptr;
        if ((rc = join()) != ESP_OK) return rc;
        if (L.up.w) {
            if ((rc = input(L, L.up, 0)) != ESP_OK || (rc = enqueue_planes(L.down, rows, &n.splits)) != ESP_OK) return rc;
            n.norm = L.norm2;
            n.final_x = last ? final_out : nullptr;
            if ((rc = join()) != ESP_OK) return rc;
        }
        if (layer_observer_) layer_observer_((int)i);
    }
    return ESP_OK;
}

int LayeredRuntime::prefill_block(int seq, const uint32_t *tokens, int rows, int base) {
    const int rc = upload_block_rows(seq, tokens, rows, base);
    if (rc != ESP_OK) return rc;
    ESP_HIP_TRY(launch_embed_norm(embedding_, embedding_ld_, d_tokens_, embed_norm_, (float)c_.norm_eps, rows, c_.width, width_p_, hidden_, context().stream));
    return enqueue_block(rows, seq, base, nullptr);
}

int LayeredRuntime::run_head(const float *hidden_rows, int count, bool want_logits) {
    hipStream_t s = context().stream;
    int rc;
    if ((rc = time_begin(K_HEAD)) != ESP_OK) return rc;
    if (count == 1) {
        DenseGemvHead h;
        h.w = head_; h.x = hidden_rows; h.norm = final_norm_; h.width = c_.width; h.vocab = c_.vocab; h.eps = (float)c_.norm_eps; h.cap = (float)c_.logit_softcap;
        if (want_logits) h.logits = logits_;
        else { h.best_value = argmax_scratch_.part_value; h.best_index = argmax_scratch_.part_index; }
        ESP_HIP_TRY(launch_dense_gemv_head(h, s));
    } else {
        ResidualNorm n;
        n.x = const_cast<float *>(hidden_rows); n.rows = count; n.width = c_.width; n.ld = width_p_; n.eps = (float)c_.norm_eps; n.norm1 = final_norm_; n.out1 = n1_;
        ESP_HIP_TRY(launch_residual_norm(n, precision_, s));
        DenseGemm g;
        g.a = n1_; g.a_type = precision_; g.lda = width_p_; g.b = head_.w; g.ldb = width_p_; g.m = count; g.n = head_.rows; g.k = width_p_;
        g.out = GemmOut::logits; g.y = logits_; g.ldy = c_.vocab; g.n_store = c_.vocab; g.cap = (float)c_.logit_softcap;
        ESP_HIP_TRY(launch_dense_gemm(g, s));
    }
    if ((rc = time_end()) != ESP_OK) return rc;
    if (want_logits) return ESP_OK;
    if (count == 1) ESP_HIP_TRY(launch_argmax_final(argmax_scratch_, dense_gemv_head_workgroups(head_), 1, d_out_tokens_, s));
    else ESP_HIP_TRY(launch_argmax(logits_, count, c_.vocab, d_out_tokens_, nullptr, argmax_scratch_, s));
    return ESP_OK;
}

int LayeredRuntime::enqueue_greedy_token(int seq) {
    hipStream_t s = context().stream;
    DenseGemvHead h;
    h.w = head_; h.x = device_last_hidden(seq); h.norm = final_norm_; h.width = c_.width; h.vocab = c_.vocab; h.eps = (float)c_.norm_eps; h.cap = (float)c_.logit_softcap;
    h.best_value = argmax_scratch_.part_value; h.best_index = argmax_scratch_.part_index;
    ESP_HIP_TRY(launch_dense_gemv_head(h, s));
    ESP_HIP_TRY(launch_greedy_tail(argmax_scratch_, dense_gemv_head_workgroups(head_), d_out_tokens_, seq, d_visible_, d_tokens_, d_pos_, d_seq_, d_log_, d_log_count_,
                                   shape_.max_seq, nullptr, false, c_.width, hidden_, shape_.eos_token, s));
    return ESP_OK;
}

size_t LayeredRuntime::kernel_bytes(int kernel_class) const {
    size_t n = 0;
    auto matrix = [](const DenseMatrix &m) { return (size_t)m.rows * m.ld * 2; };
    for (const Layer &L : layers_) {
        const size_t window = has_cache(L.mixer) ? (L.mixer == MixerKind::attention ? L.attention.window : L.latent.window) : 0;
        if (kernel_class == K_IN) n += matrix(L.in) + matrix(L.up);
        else if (kernel_class == K_OUT) n += matrix(L.out) + matrix(L.down);
        else if (kernel_class == K_RETENTION && L.mixer == MixerKind::retention) n += L.state_floats * 8;
        else if (kernel_class == K_MAMBA2 && L.mixer == MixerKind::mamba2) n += L.state_floats * 8 + L.input_floats * 4;
        else if (kernel_class == K_LATENT && L.mixer == MixerKind::latent_attention) n += matrix(L.uk) + matrix(L.uv) + window * L.cache_row_bytes;
        else if (kernel_class == K_ATTENTION && L.mixer == MixerKind::attention) n += window * L.cache_row_bytes;
    }
    if (kernel_class == K_HEAD) n = matrix(head_);
    return n;
}

}  // namespace esp
