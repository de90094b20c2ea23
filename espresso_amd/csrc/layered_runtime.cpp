#include "layered_runtime.h"

#include <algorithm>
#include <cmath>
#include <cstring>

namespace esp {
namespace {
int up(int v, int to) { return (v + to - 1) / to * to; }

// Copies rows [first, first + count) of a host matrix [..][cols] to rows at.. of dst [..][ld].
void place_rows(const std::vector<uint16_t> &src, int cols, int first, int count, std::vector<uint16_t> *dst, int ld, int at, int at_col = 0) {
    for (int r = 0; r < count; r++)
        std::memcpy(dst->data() + (size_t)(at + r) * ld + at_col, src.data() + (size_t)(first + r) * cols, (size_t)cols * 2);
}
}  // namespace

int LayeredRuntime::create(const LayeredConfig &config, const LayeredOptions &options, LayeredWeights &weights, LayeredRuntime **out) {
    *out = nullptr;
    if (config.layers.empty() || config.vocab < 1 || config.width < 1) return fail(ESP_ERR_INVALID_ARGUMENT, "layered config: no layers, vocabulary or width");
    if (options.max_seq < 1) return fail(ESP_ERR_INVALID_ARGUMENT, "layered runtime: max_seq must be positive");
    if (options.max_sequences < 1 || options.max_sequences > kMaxStepRows)
        return fail(ESP_ERR_INVALID_ARGUMENT, "layered runtime: max_sequences must be 1..%d", kMaxStepRows);
    if (config.block != BlockKind::parallel_two_norms) return fail(ESP_ERR_UNSUPPORTED, "layered runtime: this kind of layer has no kernels");
    for (size_t i = 0; i < config.layers.size(); i++)
        if (config.layers[i].mixer == MixerKind::latent_attention && up(config.layers[i].kv_rank, 64) > kLatentMaxRank)
            return fail(ESP_ERR_UNSUPPORTED, "layer %zu: latents of %d values exceed %d", i, config.layers[i].kv_rank, kLatentMaxRank);
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
    free_device(embedding_); free_device(embed_norm_); free_device(final_norm_); free_device(head_.w);
    for (Layer &L : layers_) {
        free_device(L.norm1); free_device(L.norm2); free_device(L.in.w); free_device(L.out.w); free_device(L.uk.w); free_device(L.uv.w);
        free_device(L.decay); free_device(L.powers); free_device(L.latent_norm); free_device(L.sink); free_device(L.state); free_device(L.cache);
    }
    for (RotaryTable &t : rotary_) { free_device(t.cos); free_device(t.sin); }
    for (float *p : {mixed_, act32_, mix32_, squares_, absorbed_, partial_, partial_ml_, workspace_}) free_device(p);
    for (void *p : {n1_, n2_, act_, r_q_, r_k_, r_kt_hi_, r_kt_lo_, r_vt_, r_states_hi_, r_states_lo_, l_q_, l_latents_, l_key_rot_, l_k_, l_vt_}) free_device(p);
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
    if ((rc = device_alloc(&embedding_, m.size())) != ESP_OK) return rc;
    ESP_HIP_TRY(hipMemcpy(embedding_, m.data(), m.size() * 2, hipMemcpyHostToDevice));
    if ((rc = padded_vector(weights, "embed.norm", c_.width, width_p_, &embed_norm_)) != ESP_OK) return rc;
    if ((rc = padded_vector(weights, "final.norm", c_.width, width_p_, &final_norm_)) != ESP_OK) return rc;
    if ((rc = weights.matrix("head", c_.vocab, c_.width, &m)) != ESP_OK) return rc;
    const int head_rows = up(c_.vocab, 32);
    p.assign((size_t)head_rows * width_p_, 0);
    place_rows(m, c_.width, 0, c_.vocab, &p, width_p_, 0);
    if ((rc = upload_matrix(p, head_rows, width_p_, &head_)) != ESP_OK) return rc;
    layers_.resize(c_.layers.size());
    for (size_t i = 0; i < layers_.size(); i++)
        if ((rc = build_layer(i, weights)) != ESP_OK) return rc;
    // a layer that reads another one's latents takes its cache and ring
    for (size_t i = 0; i < layers_.size(); i++) {
        const int from = c_.layers[i].kv_from;
        if (c_.layers[i].mixer != MixerKind::latent_attention || from < 0) continue;
        layers_[i].latent.cache = layers_[from].cache;
        layers_[i].latent.ring = layers_[from].ring;
    }
    if ((rc = allocate_common(kPrefillBlockRows, width_p_)) != ESP_OK) return rc;
    if ((rc = allocate_scratch()) != ESP_OK) return rc;
    return finish_finalize();
}

int LayeredRuntime::build_layer(size_t index, LayeredWeights &weights) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    const std::string p = "l" + std::to_string(index) + ".", x = p + "mix.";
    const int d = c_.width, dp = up(S.dim, 32), vp = up(S.vdim, 32), H = S.heads, ffp = S.ff ? up(S.ff, 64) : 0;
    int rc;
    if ((rc = padded_vector(weights, p + "norm1", d, width_p_, &L.norm1)) != ESP_OK) return rc;
    if (S.ff && (rc = padded_vector(weights, p + "norm2", d, width_p_, &L.norm2)) != ESP_OK) return rc;

    // ---- input side: the mixer's projections head by head, then gate and up rows in pairs ----
    const int rp = up(S.rot_dim, 32), kp = up(S.kv_rank, 64);
    const bool retention = S.mixer == MixerKind::retention, own = !retention && S.kv_from < 0;
    int used = retention ? 2 * H * (dp + vp) : H * (dp + rp) + (own ? kp + rp : 0) + up(H, 32);
    L.mix_rows = up(used, 128);
    const int in_rows = L.mix_rows + 2 * ffp;
    std::vector<uint16_t> in((size_t)in_rows * width_p_, 0), m;
    // projection `name` of heads of `size` rows: rows of head h to row at + h * stride
    auto heads_in = [&](const char *name, int size, int at, int stride) -> int {
        const int r = weights.matrix(x + name, H * size, d, &m);
        if (r != ESP_OK) return r;
        for (int h = 0; h < H; h++) place_rows(m, d, h * size, size, &in, width_p_, at + h * stride);
        return ESP_OK;
    };
    if (retention) {
        recurrent_ = true;
        if ((rc = heads_in("q", S.dim, 0, dp)) != ESP_OK || (rc = heads_in("k", S.dim, H * dp, dp)) != ESP_OK || (rc = heads_in("v", S.vdim, 2 * H * dp, vp)) != ESP_OK ||
            (rc = heads_in("g", S.vdim, 2 * H * dp + H * vp, vp)) != ESP_OK)
            return rc;
    } else {
        if ((rc = weights.matrix(x + "q", H * (S.dim + S.rot_dim), d, &m)) != ESP_OK) return rc;
        for (int h = 0; h < H; h++) {
            place_rows(m, d, h * (S.dim + S.rot_dim), S.dim, &in, width_p_, h * (dp + rp));
            place_rows(m, d, h * (S.dim + S.rot_dim) + S.dim, S.rot_dim, &in, width_p_, h * (dp + rp) + dp);
        }
        int at = H * (dp + rp);
        L.latent.dkv_at = -1;
        if (own) {
            if ((rc = weights.matrix(x + "dkv", S.kv_rank + S.rot_dim, d, &m)) != ESP_OK) return rc;
            place_rows(m, d, 0, S.kv_rank, &in, width_p_, at);
            place_rows(m, d, S.kv_rank, S.rot_dim, &in, width_p_, at + kp);
            L.latent.dkv_at = at;
            at += kp + rp;
        }
        if ((rc = weights.matrix(x + "g", H, d, &m)) != ESP_OK) return rc;
        place_rows(m, d, 0, H, &in, width_p_, at);
        L.latent.gate_at = at;
    }
    if (S.ff) {
        for (int half = 0; half < 2; half++) {
            if ((rc = weights.matrix(p + (half ? "mlp.up" : "mlp.gate"), S.ff, d, &m)) != ESP_OK) return rc;
            for (int i = 0; i < S.ff; i++) place_rows(m, d, i, 1, &in, width_p_, L.mix_rows + 2 * i + half);
        }
    }
    if ((rc = upload_matrix(in, in_rows, width_p_, &L.in)) != ESP_OK) return rc;
    std::vector<uint16_t>().swap(in);

    // ---- output side: W_o beside W_down, one product over [mixer | feed-forward] ----
    L.mix_cols = up(H * vp, 64);
    const int out_cols = L.mix_cols + ffp;
    std::vector<uint16_t> out((size_t)width_p_ * out_cols, 0);
    if ((rc = weights.matrix(x + "o", d, H * S.vdim, &m)) != ESP_OK) return rc;
    for (int r = 0; r < d; r++)
        for (int h = 0; h < H; h++) std::memcpy(out.data() + (size_t)r * out_cols + h * vp, m.data() + (size_t)r * H * S.vdim + h * S.vdim, (size_t)S.vdim * 2);
    if (S.ff) {
        if ((rc = weights.matrix(p + "mlp.down", d, S.ff, &m)) != ESP_OK) return rc;
        place_rows(m, S.ff, 0, d, &out, out_cols, 0, L.mix_cols);
    }
    if ((rc = upload_matrix(out, width_p_, out_cols, &L.out)) != ESP_OK) return rc;
    std::vector<uint16_t>().swap(out);

    mix_max_ = std::max(mix_max_, L.mix_rows);
    out_cols_max_ = std::max(out_cols_max_, out_cols);
    if ((rc = rotary_table(S.rot, &L.cos, &L.sin)) != ESP_OK) return rc;
    const int n_seq = shape_.max_sequences;
    if (retention) {
        std::vector<float> decay(H), powers((size_t)H * (kRetentionChunk + 1));
        for (int h = 0; h < H; h++) {
            decay[h] = (float)S.decay[h];
            for (int i = 0; i <= kRetentionChunk; i++) powers[h * (kRetentionChunk + 1) + i] = (float)std::pow(S.decay[h], i);
        }
        if ((rc = upload_floats(decay, &L.decay)) != ESP_OK || (rc = upload_floats(powers, &L.powers)) != ESP_OK) return rc;
        const size_t per_seq = (size_t)H * dp * vp;
        if ((rc = device_alloc(&L.state, per_seq * n_seq)) != ESP_OK) return rc;
        sequence_bytes_ += per_seq * 4;
        RetentionShape &r = L.retention;
        r.heads = H; r.dim = S.dim; r.vdim = S.vdim; r.dim_p = dp; r.vdim_p = vp; r.rot_dims = S.rot.dims; r.ld_mix = L.mix_rows;
        r.max_seq = shape_.max_seq; r.cos = L.cos; r.sin = L.sin; r.decay = L.decay; r.powers = L.powers; r.state = L.state;
        return ESP_OK;
    }
    auto up_projection = [&](const char *name, int size, int padded, DenseMatrix *dst) -> int {
        int r = weights.matrix(x + name, H * size, S.kv_rank, &m);
        if (r != ESP_OK) return r;
        std::vector<uint16_t> w((size_t)H * padded * kp, 0);
        for (int h = 0; h < H; h++) place_rows(m, S.kv_rank, h * size, size, &w, kp, h * padded);
        return upload_matrix(w, H * padded, kp, dst);
    };
    if ((rc = up_projection("uk", S.dim, dp, &L.uk)) != ESP_OK) return rc;
    if ((rc = up_projection("uv", S.vdim, vp, &L.uv)) != ESP_OK) return rc;
    if ((rc = padded_vector(weights, x + "sink", H, up(H, 32), &L.sink)) != ESP_OK) return rc;
    if (own) {
        if ((rc = padded_vector(weights, x + "dkv.norm", S.kv_rank, kp, &L.latent_norm)) != ESP_OK) return rc;
        // the ring holds what the widest window over these latents can see, beside a whole block of new rows
        int window = 1;
        for (size_t j = index; j < c_.layers.size(); j++)
            if (c_.layers[j].mixer == MixerKind::latent_attention && (j == index || c_.layers[j].kv_from == (int)index)) window = std::max(window, c_.layers[j].window);
        L.ring = (int)std::min<long long>(shape_.max_seq, (long long)window - 1 + kPrefillBlockRows);
        const size_t per_seq = (size_t)L.ring * (kp + rp) * precision_bytes(precision_);
        uint8_t *cache = nullptr;
        if ((rc = device_alloc(&cache, per_seq * n_seq)) != ESP_OK) return rc;
        L.cache = cache;
        sequence_bytes_ += per_seq;
    }
    LatentShape &l = L.latent;
    l.heads = H; l.dim = S.dim; l.vdim = S.vdim; l.rot_dim = S.rot_dim; l.kv_rank = S.kv_rank; l.dim_p = dp; l.vdim_p = vp; l.rot_p = rp; l.rank_p = kp;
    l.rot_dims = S.rot.dims; l.window = S.window; l.ld_mix = L.mix_rows; l.max_seq = shape_.max_seq; l.ring = L.ring; l.scale = (float)S.scale; l.eps = (float)c_.norm_eps;
    l.cos = L.cos; l.sin = L.sin; l.latent_norm = L.latent_norm; l.sink = L.sink; l.uk = L.uk.w; l.uv = L.uv.w; l.cache = L.cache;
    L.splits = latent_step_splits(l);
    return ESP_OK;
}

void LayeredRuntime::latent_key_range(const Layer &L, int rows, int base, LatentBlock *b) const {
    b->first_key = std::max(0, base - L.latent.window + 1);
    b->keys = base + rows - b->first_key;
    b->keys_p = up(b->keys, 64);
}

int LayeredRuntime::allocate_scratch() {
    const size_t R = block_rows_, RS = kMaxStepRows, E = precision_bytes(precision_);
    size_t act32 = 64, squares = 1, absorbed = 1, partial = 1, partial_ml = 1, rq = 1, rv = 1, states = 1, lq = 1, latents = 1, key_rot = 1, lk = 1, lvt = 1, mix32 = 64;
    for (const Layer &L : layers_) {
        act32 = std::max(act32, (size_t)(L.out.ld - L.mix_cols));
        if (L.retention.heads) {
            const RetentionShape &r = L.retention;
            squares = std::max(squares, RS * r.heads * retention_step_parts(r.vdim_p));
            rq = std::max(rq, (size_t)r.heads * r.dim_p * R);
            rv = std::max(rv, (size_t)r.heads * r.vdim_p * R);
            states = std::max(states, (size_t)(R / kRetentionChunk) * r.heads * r.dim_p * r.vdim_p);
            mix32 = std::max(mix32, R * r.heads * r.vdim_p);
        } else {
            const LatentShape &l = L.latent;
            const size_t T = up((int)std::min<long long>(shape_.max_seq, (long long)l.window - 1 + block_rows_), 64);
            absorbed = std::max(absorbed, RS * l.heads * (l.rank_p + l.rot_p));
            partial = std::max(partial, RS * L.splits * l.heads * l.rank_p);
            partial_ml = std::max(partial_ml, RS * L.splits * l.heads * 2);
            lq = std::max(lq, R * l.heads * (l.dim_p + l.rot_p));
            latents = std::max(latents, T * l.rank_p);
            key_rot = std::max(key_rot, T * l.rot_p);
            lk = std::max(lk, T * l.heads * l.dim_p);
            lvt = std::max(lvt, T * l.heads * l.vdim_p);
            mix32 = std::max(mix32, RS * l.heads * l.vdim_p);
        }
    }
    int rc;
    auto bytes = [&](void **p, size_t n) -> int {
        uint8_t *q = nullptr;
        const int r = device_alloc(&q, n);
        *p = q;
        return r;
    };
    if ((rc = device_alloc(&mixed_, R * mix_max_)) != ESP_OK || (rc = device_alloc(&act32_, act32)) != ESP_OK || (rc = device_alloc(&mix32_, mix32)) != ESP_OK ||
        (rc = device_alloc(&squares_, squares)) != ESP_OK || (rc = device_alloc(&absorbed_, absorbed)) != ESP_OK || (rc = device_alloc(&partial_, partial)) != ESP_OK ||
        (rc = device_alloc(&partial_ml_, partial_ml)) != ESP_OK)
        return rc;
    if ((rc = bytes(&n1_, R * width_p_ * E)) != ESP_OK || (rc = bytes(&n2_, R * width_p_ * E)) != ESP_OK || (rc = bytes(&act_, R * out_cols_max_ * E)) != ESP_OK ||
        (rc = bytes(&r_q_, rq * E)) != ESP_OK || (rc = bytes(&r_k_, rq * E)) != ESP_OK || (rc = bytes(&r_kt_hi_, rq * E)) != ESP_OK || (rc = bytes(&r_kt_lo_, rq * E)) != ESP_OK ||
        (rc = bytes(&r_vt_, rv * E)) != ESP_OK || (rc = bytes(&r_states_hi_, states * E)) != ESP_OK || (rc = bytes(&r_states_lo_, states * E)) != ESP_OK ||
        (rc = bytes(&l_q_, lq * E)) != ESP_OK || (rc = bytes(&l_latents_, latents * E)) != ESP_OK || (rc = bytes(&l_key_rot_, key_rot * E)) != ESP_OK ||
        (rc = bytes(&l_k_, lk * E)) != ESP_OK || (rc = bytes(&l_vt_, lvt * E)) != ESP_OK)
        return rc;
    // columns of an output product's input that no head fills meet zero weights, so they only have to be finite
    ESP_HIP_TRY(hipMemset(act_, 0, R * out_cols_max_ * E));
    workspace_floats_ = std::max(kGemmWorkspaceFloats, R * width_p_);
    return device_alloc(&workspace_, workspace_floats_);
}

int LayeredRuntime::clear_state() {
    for (size_t i = 0; i < layers_.size(); i++) {
        Layer &L = layers_[i];
        const size_t n = shape_.max_sequences;
        if (L.state) ESP_HIP_TRY(hipMemsetAsync(L.state, 0, n * L.retention.heads * L.retention.dim_p * L.retention.vdim_p * 4, context().stream));
        if (L.cache) ESP_HIP_TRY(hipMemsetAsync(L.cache, 0, n * L.ring * (L.latent.rank_p + L.latent.rot_p) * precision_bytes(precision_), context().stream));
    }
    return ESP_OK;
}

// `embedded` changes nothing here: the embedding is normed, so the trunk always fetches it from the rows' tokens.
int LayeredRuntime::enqueue_trunk(int rows, bool, float *final_out) {
    ESP_HIP_TRY(launch_embed_norm(embedding_, d_tokens_, embed_norm_, (float)c_.norm_eps, rows, c_.width, width_p_, hidden_, context().stream));
    return rows == 1 ? enqueue_step(final_out) : enqueue_block(rows, -1, 0, final_out);
}

// One row: three launches per retention layer, five per attention layer.
int LayeredRuntime::enqueue_step(float *final_out) {
    hipStream_t s = context().stream;
    const float eps = (float)c_.norm_eps, mult = (float)c_.residual_mult;
    int rc;
    for (size_t i = 0; i < layers_.size(); i++) {
        Layer &L = layers_[i];
        DenseGemvIn in;
        in.w = L.in; in.mix_rows = L.mix_rows; in.x = hidden_; in.norm1 = L.norm1; in.norm2 = L.norm2; in.width = c_.width; in.eps = eps; in.y = mixed_; in.act = act32_;
        if ((rc = time_begin(K_IN)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_dense_gemv_in(in, s));
        if ((rc = time_end()) != ESP_OK) return rc;
        DenseGemvOut out;
        out.w = L.out; out.act_at = L.mix_cols; out.act_cols = L.out.ld - L.mix_cols; out.mix = mix32_; out.act = act32_; out.mult = mult; out.eps = eps; out.rows = width_p_;
        out.residual = hidden_; out.out = final_out && i + 1 == layers_.size() ? final_out : hidden_;
        if (L.retention.heads) {
            const RetentionShape &r = L.retention;
            // a replay after the stop token must leave the states alone (the other kernels recompute what they computed last)
            RetentionStep st{mixed_, d_pos_, d_seq_, capturing_ ? d_log_count_ + 1 : nullptr, mix32_, squares_, 1};
            if ((rc = time_begin(K_RETENTION)) != ESP_OK) return rc;
            ESP_HIP_TRY(launch_retention_step(r, st, s));
            if ((rc = time_end()) != ESP_OK) return rc;
            out.mix_cols = r.heads * r.vdim_p; out.squares = squares_; out.gate = mixed_ + 2 * r.heads * r.dim_p + r.heads * r.vdim_p;
            out.parts = retention_step_parts(r.vdim_p); out.vdim = r.vdim; out.vdim_p = r.vdim_p;
        } else {
            const LatentShape &l = L.latent;
            if ((rc = time_begin(K_LATENT)) != ESP_OK) return rc;
            LatentStep st{mixed_, d_pos_, d_seq_, absorbed_, partial_, partial_ml_, L.splits, 1, mix32_, nullptr, 0};
            ESP_HIP_TRY(launch_latent_step(l, st, precision_, s));
            if ((rc = time_end()) != ESP_OK) return rc;
            out.mix_cols = l.heads * l.vdim_p;
        }
        if ((rc = time_begin(K_OUT)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_dense_gemv_out(out, s));
        if ((rc = time_end()) != ESP_OK) return rc;
    }
    return ESP_OK;
}

int LayeredRuntime::enqueue_block(int rows, int seq, int base, float *final_out) {
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
        g.out = GemmOut::mix_swiglu; g.y = mixed_; g.ldy = L.mix_rows; g.mix_cols = L.mix_rows; g.ld_act = ld_act;
        g.act = static_cast<uint8_t *>(act_) + (size_t)L.mix_cols * E;
        if ((rc = time_begin(K_IN)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_dense_gemm(g, s));
        if ((rc = time_end()) != ESP_OK) return rc;
        if (L.retention.heads) {
            const RetentionShape &r = L.retention;
            if ((rc = time_begin(K_RETENTION)) != ESP_OK) return rc;
            if (seq >= 0) {
                RetentionBlock b{mixed_, rows, base, seq, r_q_, r_k_, r_kt_hi_, r_kt_lo_, r_vt_, r_states_hi_, r_states_lo_, mix32_};
                ESP_HIP_TRY(launch_retention_block(r, b, precision_, s));
            } else {
                RetentionStep st{mixed_, d_pos_, d_seq_, nullptr, mix32_, squares_, rows};
                ESP_HIP_TRY(launch_retention_step(r, st, s));
            }
            ESP_HIP_TRY(launch_retention_gate(r, mix32_, mixed_, rows, eps, act_, ld_act, precision_, s));
            if ((rc = time_end()) != ESP_OK) return rc;
        } else {
            const LatentShape &l = L.latent;
            if ((rc = time_begin(K_LATENT)) != ESP_OK) return rc;
            if (seq >= 0) {
                if (l.dkv_at >= 0) ESP_HIP_TRY(launch_latent_store(l, mixed_, d_pos_, d_seq_, rows, precision_, s));
                LatentBlock b{};
                b.mixed = mixed_; b.rows = rows; b.base = base; b.seq = seq;
                latent_key_range(L, rows, base, &b);
                b.q = l_q_; b.latents = l_latents_; b.key_rot = l_key_rot_; b.k = l_k_; b.vt = l_vt_; b.act = act_; b.ld_act = ld_act;
                ESP_HIP_TRY(launch_latent_gather(l, b, precision_, s));
                ESP_HIP_TRY(launch_latent_queries(l, b, precision_, s));
                DenseGemm k;   // keys [T][heads * dim_p]
                k.a = l_latents_; k.a_type = precision_; k.lda = l.rank_p; k.b = L.uk.w; k.ldb = l.rank_p; k.m = b.keys_p; k.n = L.uk.rows; k.k = l.rank_p;
                k.out = GemmOut::elems; k.y = l_k_; k.ldy = L.uk.rows;
                ESP_HIP_TRY(launch_dense_gemm(k, s));
                DenseGemm v;   // values transposed [heads * vdim_p][T]
                v.a = L.uv.w; v.lda = l.rank_p; v.b = l_latents_; v.b_type = precision_; v.ldb = l.rank_p; v.m = L.uv.rows; v.n = b.keys_p; v.k = l.rank_p;
                v.out = GemmOut::elems; v.y = l_vt_; v.ldy = b.keys_p;
                ESP_HIP_TRY(launch_dense_gemm(v, s));
                ESP_HIP_TRY(launch_latent_block(l, b, precision_, s));
            } else {
                LatentStep st{mixed_, d_pos_, d_seq_, absorbed_, partial_, partial_ml_, L.splits, rows, nullptr, act_, ld_act};
                ESP_HIP_TRY(launch_latent_step(l, st, precision_, s));
            }
            if ((rc = time_end()) != ESP_OK) return rc;
        }
        DenseGemm o;
        o.a = act_; o.a_type = precision_; o.lda = ld_act; o.b = L.out.w; o.ldb = ld_act; o.m = rows; o.n = width_p_; o.k = ld_act;
        o.out = GemmOut::planes; o.y = workspace_; o.ldy = width_p_; o.splits = gemm_planes_splits(rows, width_p_, ld_act, workspace_floats_);
        if ((rc = time_begin(K_OUT)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_dense_gemm(o, s));
        if ((rc = time_end()) != ESP_OK) return rc;
        const bool last = i + 1 == layers_.size();
        n.planes = workspace_; n.splits = o.splits; n.plane = (size_t)rows * width_p_;
        n.norm1 = last ? nullptr : layers_[i + 1].norm1; n.norm2 = last ? nullptr : layers_[i + 1].norm2;
        n.final_x = last ? final_out : nullptr;
        if ((rc = time_begin(K_NORM)) != ESP_OK) return rc;
        ESP_HIP_TRY(launch_residual_norm(n, precision_, s));
        if ((rc = time_end()) != ESP_OK) return rc;
        if (layer_observer_) layer_observer_((int)i);
    }
    return ESP_OK;
}

int LayeredRuntime::prefill_block(int seq, const uint32_t *tokens, int rows, int base) {
    const int rc = upload_block_rows(seq, tokens, rows, base);
    if (rc != ESP_OK) return rc;
    ESP_HIP_TRY(launch_embed_norm(embedding_, d_tokens_, embed_norm_, (float)c_.norm_eps, rows, c_.width, width_p_, hidden_, context().stream));
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
    for (const Layer &L : layers_) {
        if (kernel_class == K_IN) n += (size_t)L.in.rows * L.in.ld * 2;
        else if (kernel_class == K_OUT) n += (size_t)L.out.rows * L.out.ld * 2;
        else if (kernel_class == K_RETENTION && L.retention.heads) n += (size_t)L.retention.heads * L.retention.dim_p * L.retention.vdim_p * 8;
        else if (kernel_class == K_LATENT && !L.retention.heads)
            n += ((size_t)L.uk.rows + L.uv.rows) * L.uk.ld * 2 + (size_t)L.latent.window * (L.latent.rank_p + L.latent.rot_p) * precision_bytes(precision_);
    }
    if (kernel_class == K_HEAD) n = (size_t)head_.rows * head_.ld * 2;
    return n;
}

}  // namespace esp
