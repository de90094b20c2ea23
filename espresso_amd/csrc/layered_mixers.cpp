// The mixers of layered runtimes: where their projections sit in a layer's input matrix, their parameters, states and caches, and the
// launches of a step and of a block.
#include <algorithm>
#include <cmath>

#include "layered_layout.h"
#include "layered_runtime.h"

namespace esp {
using layered::place_rows;
using layered::up;

namespace {
std::string mixer_prefix(size_t index) { return "l" + std::to_string(index) + ".mix."; }
}  // namespace

// ---- layout of the mixed rows ----------------------------------------------------------------------------
int LayeredRuntime::mixer_rows(const LayerSpec &S) {
    const int H = S.heads, dp = up(S.dim, 32), vp = up(S.vdim, 32);
    switch (S.mixer) {
        case MixerKind::retention: return 2 * H * (dp + vp);                        // q | k | v | gate
        case MixerKind::latent_attention: {                                         // q | latent, rotated key part | gates
            const int rp = up(S.rot_dim, 32), kp = up(S.kv_rank, 64);
            return H * (dp + rp) + (S.kv_from < 0 ? kp + rp : 0) + up(H, 32);
        }
        case MixerKind::attention: return H * dp + (S.kv_from < 0 ? S.kv_heads * (dp + vp) : 0);   // q | k | v
        case MixerKind::mamba2: return 2 * H * vp + 2 * S.groups * up(S.state, 32) + H;           // z | x | B | C | dt
    }
    return 0;
}

int LayeredRuntime::place_mixer_rows(size_t index, LayeredWeights &weights, std::vector<uint16_t> *in) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    const std::string x = mixer_prefix(index);
    const int d = c_.width, H = S.heads, dp = up(S.dim, 32), vp = up(S.vdim, 32);
    std::vector<uint16_t> m;
    int rc = ESP_OK, at = 0;
    // `count` heads (or groups) of `size` rows from row `first` of m, `stride` rows apart from row `at`
    auto heads = [&](int first, int count, int size, int stride) {
        for (int h = 0; h < count; h++) place_rows(m, d, first + h * size, size, in, width_p_, at + h * stride);
        at += count * stride;
    };
    auto projection = [&](const char *name, int count, int size, int stride) -> int {
        const int r = weights.matrix(x + name, count * size, d, &m);
        if (r == ESP_OK) heads(0, count, size, stride);
        return r;
    };
    switch (S.mixer) {
        case MixerKind::retention:
            if ((rc = projection("q", H, S.dim, dp)) != ESP_OK || (rc = projection("k", H, S.dim, dp)) != ESP_OK || (rc = projection("v", H, S.vdim, vp)) != ESP_OK) return rc;
            return projection("g", H, S.vdim, vp);
        case MixerKind::attention:
            if ((rc = projection("q", H, S.dim, dp)) != ESP_OK) return rc;
            L.attention.k_at = S.kv_from < 0 ? at : -1;
            if (S.kv_from >= 0) return ESP_OK;
            if ((rc = projection("k", S.kv_heads, S.dim, dp)) != ESP_OK) return rc;
            return projection("v", S.kv_heads, S.vdim, vp);
        case MixerKind::mamba2: {
            const int inner = H * S.vdim, shared = S.groups * S.state, sp = up(S.state, 32);
            if ((rc = weights.matrix(x + "in", 2 * inner + 2 * shared + H, d, &m)) != ESP_OK) return rc;
            heads(0, H, S.vdim, vp);
            heads(inner, H, S.vdim, vp);
            heads(2 * inner, S.groups, S.state, sp);
            heads(2 * inner + shared, S.groups, S.state, sp);
            heads(2 * inner + 2 * shared, H, 1, 1);
            return ESP_OK;
        }
        case MixerKind::latent_attention: {
            const int rp = up(S.rot_dim, 32), kp = up(S.kv_rank, 64);
            if ((rc = weights.matrix(x + "q", H * (S.dim + S.rot_dim), d, &m)) != ESP_OK) return rc;
            for (int h = 0; h < H; h++) {
                place_rows(m, d, h * (S.dim + S.rot_dim), S.dim, in, width_p_, h * (dp + rp));
                place_rows(m, d, h * (S.dim + S.rot_dim) + S.dim, S.rot_dim, in, width_p_, h * (dp + rp) + dp);
            }
            at = H * (dp + rp);
            L.latent.dkv_at = -1;
            if (S.kv_from < 0) {
                if ((rc = weights.matrix(x + "dkv", S.kv_rank + S.rot_dim, d, &m)) != ESP_OK) return rc;
                place_rows(m, d, 0, S.kv_rank, in, width_p_, at);
                place_rows(m, d, S.kv_rank, S.rot_dim, in, width_p_, at + kp);
                L.latent.dkv_at = at;
                at += kp + rp;
            }
            L.latent.gate_at = at;
            return projection("g", H, 1, 1);
        }
    }
    return rc;
}

// ---- parameters, states and caches -------------------------------------------------------------------------
int LayeredRuntime::build_mixer(size_t index, LayeredWeights &weights) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    int rc;
    if (S.mixer != MixerKind::mamba2 && (rc = rotary_table(S.rot, &L.cos, &L.sin)) != ESP_OK) return rc;
    switch (S.mixer) {
        case MixerKind::retention: rc = build_retention(index, weights); break;
        case MixerKind::latent_attention: rc = build_latent(index, weights); break;
        case MixerKind::attention: rc = build_attention(index, weights); break;
        case MixerKind::mamba2: rc = build_mamba2(index, weights); break;
    }
    if (rc != ESP_OK) return rc;
    if (!has_cache(S.mixer)) {
        recurrent_ = true;
        if ((rc = device_alloc(&L.state, L.state_floats * shape_.max_sequences)) != ESP_OK) return rc;
        if (L.input_floats && (rc = device_alloc(&L.inputs, L.input_floats * shape_.max_sequences)) != ESP_OK) return rc;
        sequence_bytes_ += (L.state_floats + L.input_floats) * 4;
        L.retention.state = L.mamba2.state_of = L.state;
        L.mamba2.inputs = L.inputs;
    }
    return ESP_OK;
}

// The ring holds what the widest window over this layer's cache can see, beside a whole block of new rows.
int LayeredRuntime::allocate_cache(size_t index, size_t row_elements) {
    Layer &L = layers_[index];
    int window = 1;
    for (size_t j = index; j < c_.layers.size(); j++)
        if (has_cache(c_.layers[j].mixer) && (j == index || c_.layers[j].kv_from == (int)index)) window = std::max(window, c_.layers[j].window);
    L.ring = (int)std::min<long long>(shape_.max_seq, (long long)window - 1 + kPrefillBlockRows);
    L.cache_row_bytes = row_elements * precision_bytes(precision_);
    uint8_t *cache = nullptr;
    const int rc = device_alloc(&cache, L.ring * L.cache_row_bytes * shape_.max_sequences);
    L.cache = cache;
    sequence_bytes_ += L.ring * L.cache_row_bytes;
    return rc;
}

int LayeredRuntime::build_retention(size_t index, LayeredWeights &) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    const int H = S.heads, stride = kRecurrenceChunk + 1;
    std::vector<float> decay(H), powers((size_t)H * stride);
    for (int h = 0; h < H; h++) {
        decay[h] = (float)S.decay[h];
        for (int i = 0; i < stride; i++) powers[h * stride + i] = (float)std::pow(S.decay[h], i);
    }
    L.vectors.assign(2, nullptr);
    int rc;
    if ((rc = upload_floats(decay, &L.vectors[0])) != ESP_OK || (rc = upload_floats(powers, &L.vectors[1])) != ESP_OK) return rc;
    RetentionShape &r = L.retention;
    r.heads = H; r.dim = S.dim; r.vdim = S.vdim; r.dim_p = up(S.dim, 32); r.vdim_p = up(S.vdim, 32); r.rot_dims = S.rot.dims; r.ld_mix = L.mix_rows;
    r.max_seq = shape_.max_seq; r.cos = L.cos; r.sin = L.sin; r.decay = L.vectors[0]; r.powers = L.vectors[1];
    L.state_floats = (size_t)H * r.dim_p * r.vdim_p;
    return ESP_OK;
}

int LayeredRuntime::build_latent(size_t index, LayeredWeights &weights) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    const std::string x = mixer_prefix(index);
    const int H = S.heads, dp = up(S.dim, 32), vp = up(S.vdim, 32), rp = up(S.rot_dim, 32), kp = up(S.kv_rank, 64);
    std::vector<uint16_t> m;
    int rc;
    auto up_projection = [&](const char *name, int size, int padded, DenseMatrix *dst) -> int {
        int r = weights.matrix(x + name, H * size, S.kv_rank, &m);
        if (r != ESP_OK) return r;
        std::vector<uint16_t> w((size_t)H * padded * kp, 0);
        for (int h = 0; h < H; h++) place_rows(m, S.kv_rank, h * size, size, &w, kp, h * padded);
        return upload_matrix(w, H * padded, kp, dst);
    };
    if ((rc = up_projection("uk", S.dim, dp, &L.uk)) != ESP_OK || (rc = up_projection("uv", S.vdim, vp, &L.uv)) != ESP_OK) return rc;
    L.vectors.assign(2, nullptr);
    if ((rc = padded_vector(weights, x + "sink", H, up(H, 32), &L.vectors[0])) != ESP_OK) return rc;
    if (S.kv_from < 0 && ((rc = padded_vector(weights, x + "dkv.norm", S.kv_rank, kp, &L.vectors[1])) != ESP_OK || (rc = allocate_cache(index, kp + rp)) != ESP_OK)) return rc;
    if (S.kv_from >= 0) L.cache_row_bytes = layers_[S.kv_from].cache_row_bytes;
    LatentShape &l = L.latent;
    l.heads = H; l.dim = S.dim; l.vdim = S.vdim; l.rot_dim = S.rot_dim; l.kv_rank = S.kv_rank; l.dim_p = dp; l.vdim_p = vp; l.rot_p = rp; l.rank_p = kp;
    l.rot_dims = S.rot.dims; l.window = S.window; l.ld_mix = L.mix_rows; l.max_seq = shape_.max_seq; l.ring = L.ring; l.scale = (float)S.scale; l.eps = (float)c_.norm_eps;
    l.cos = L.cos; l.sin = L.sin; l.sink = L.vectors[0]; l.latent_norm = L.vectors[1]; l.uk = L.uk.w; l.uv = L.uv.w; l.cache = L.cache;
    L.splits = latent_step_splits(l);
    return ESP_OK;
}

int LayeredRuntime::build_attention(size_t index, LayeredWeights &weights) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    const std::string x = mixer_prefix(index);
    const int dp = up(S.dim, 32), vp = up(S.vdim, 32);
    int rc;
    L.vectors.assign(2, nullptr);
    if ((rc = head_vector(weights, x + "q.norm", S.heads, S.dim, dp, &L.vectors[0])) != ESP_OK) return rc;
    if (S.kv_from < 0 && ((rc = head_vector(weights, x + "k.norm", S.kv_heads, S.dim, dp, &L.vectors[1])) != ESP_OK || (rc = allocate_cache(index, (size_t)S.kv_heads * (dp + vp))) != ESP_OK))
        return rc;
    if (S.kv_from >= 0) L.cache_row_bytes = layers_[S.kv_from].cache_row_bytes;
    AttentionShape &l = L.attention;   // k_at is set
    l.heads = S.heads; l.kv_heads = S.kv_heads; l.dim = S.dim; l.vdim = S.vdim; l.dim_p = dp; l.vdim_p = vp; l.rot_dims = S.rot.dims; l.window = S.window; l.ld_mix = L.mix_rows;
    l.max_seq = shape_.max_seq; l.ring = L.ring; l.scale = (float)S.scale; l.eps = (float)c_.norm_eps; l.cos = L.cos; l.sin = L.sin;
    l.q_norm = L.vectors[0]; l.k_norm = L.vectors[1]; l.cache = L.cache;
    L.splits = attention_step_splits(l);
    return ESP_OK;
}

int LayeredRuntime::build_mamba2(size_t index, LayeredWeights &weights) {
    const LayerSpec &S = c_.layers[index];
    Layer &L = layers_[index];
    const std::string x = mixer_prefix(index);
    const int H = S.heads, G = S.groups, vp = up(S.vdim, 32), sp = up(S.state, 32), inner = H * S.vdim, channels = inner + 2 * G * S.state;
    const size_t values = (size_t)H * vp, channels_p = values + (size_t)2 * G * sp;
    int rc;
    L.vectors.assign(6, nullptr);
    L.tables.assign(2, nullptr);
    // channel c of x | B | C, at its place in the padded layout
    auto padded = [&](int c) -> size_t {
        if (c < inner) return (size_t)(c / S.vdim) * vp + c % S.vdim;
        return values + (size_t)((c - inner) / S.state) * sp + (c - inner) % S.state;
    };
    std::vector<uint16_t> taps;
    std::vector<float> v, conv(channels_p * S.conv, 0.0f), bias(channels_p, 0.0f);
    if ((rc = weights.matrix(x + "conv", channels, S.conv, &taps)) != ESP_OK || (rc = weights.vector(x + "conv.b", channels, &v)) != ESP_OK) return rc;
    for (int c = 0; c < channels; c++) {
        bias[padded(c)] = v[c];
        for (int j = 0; j < S.conv; j++) {
            const uint32_t wide = (uint32_t)taps[(size_t)c * S.conv + j] << 16;
            std::memcpy(&conv[j * channels_p + padded(c)], &wide, 4);
        }
    }
    if ((rc = upload_floats(conv, &L.vectors[0])) != ESP_OK || (rc = upload_floats(bias, &L.vectors[1])) != ESP_OK) return rc;
    if ((rc = padded_vector(weights, x + "dt_bias", H, H, &L.vectors[2])) != ESP_OK || (rc = weights.vector(x + "A_log", H, &v)) != ESP_OK) return rc;
    for (float &a : v) a = (float)std::exp((double)a);
    if ((rc = upload_floats(v, &L.vectors[3])) != ESP_OK || (rc = padded_vector(weights, x + "D", H, H, &L.vectors[4])) != ESP_OK ||
        (rc = head_vector(weights, x + "norm", H, S.vdim, vp, &L.vectors[5])) != ESP_OK)
        return rc;
    // equal parts of the values as they are, in the padded layout: a part may end within a head
    const int part_size = inner / S.norm_groups;
    std::vector<int> part(values), starts(S.norm_groups + 1, (int)values);
    for (size_t k = 0; k < values; k++) part[k] = std::min((int)(k / vp * S.vdim + std::min<size_t>(k % vp, S.vdim - 1)) / part_size, S.norm_groups - 1);
    bool by_eight = true;
    for (int g = 0; g < S.norm_groups; g++) {
        starts[g] = (int)padded(g * part_size);
        by_eight = by_eight && starts[g] % 8 == 0;
    }
    for (int i = 0; i < 2; i++) {
        const std::vector<int> &t = i ? starts : part;
        if ((rc = device_alloc(&L.tables[i], t.size())) != ESP_OK) return rc;
        ESP_HIP_TRY(hipMemcpy(L.tables[i], t.data(), t.size() * sizeof(int), hipMemcpyHostToDevice));
    }
    Mamba2Shape &r = L.mamba2;
    r.heads = H; r.vdim = S.vdim; r.state = S.state; r.groups = G; r.taps = S.conv; r.norm_groups = S.norm_groups; r.vdim_p = vp; r.state_p = sp; r.ld_mix = L.mix_rows;
    r.max_seq = shape_.max_seq; r.conv = L.vectors[0]; r.conv_bias = L.vectors[1]; r.dt_bias = L.vectors[2]; r.rate = L.vectors[3]; r.skip = L.vectors[4]; r.norm = L.vectors[5];
    r.norm_part = L.tables[0]; r.norm_starts = L.tables[1]; r.norm_by_eight = by_eight;
    L.state_floats = values * sp;
    L.input_floats = channels_p * S.conv;
    return ESP_OK;
}

LayeredRuntime::KeyRange LayeredRuntime::visible_keys(int window, int rows, int base) {
    const int first = std::max(0, base - window + 1), keys = base + rows - first;
    return {first, keys, up(keys, 64)};
}

// What the mixers of all layers need for a step of every sequence and for a block of one.
int LayeredRuntime::allocate_mixer_scratch() {
    const size_t R = block_rows_, RS = kMaxStepRows, E = precision_bytes(precision_), chunks = R / kRecurrenceChunk;
    size_t mix32 = 64, squares = 1, absorbed = 1, partial = 1, partial_ml = 1, rq = 1, rkt = 1, rv = 1, rvs = 1, logs = 1, states = 1, lq = 1, latents = 1, key_rot = 1, lk = 1, lvt = 1;
    auto most = [](size_t &have, size_t n) { have = std::max(have, n); };
    for (const Layer &L : layers_) {
        const size_t window = has_cache(L.mixer) ? (L.mixer == MixerKind::attention ? L.attention.window : L.latent.window) : 1;
        const size_t T = up((int)std::min<long long>(shape_.max_seq, (long long)window - 1 + block_rows_), 64);
        switch (L.mixer) {
            case MixerKind::retention: {
                const RetentionShape &r = L.retention;
                most(squares, RS * r.heads * retention_step_parts(r.vdim_p));
                most(rq, (size_t)r.heads * r.dim_p * R);
                most(rkt, (size_t)r.heads * r.dim_p * R);
                most(rv, (size_t)r.heads * r.vdim_p * R);
                most(states, chunks * L.state_floats);
                most(mix32, R * r.heads * r.vdim_p);
                break;
            }
            case MixerKind::mamba2: {
                const Mamba2Shape &r = L.mamba2;
                most(rq, (size_t)r.groups * r.state_p * R);
                most(rkt, (size_t)r.groups * r.state_p * R);
                most(rv, (size_t)r.heads * r.vdim_p * R);
                most(rvs, (size_t)r.heads * r.vdim_p * R);
                most(logs, (size_t)r.heads * R);
                most(states, chunks * L.state_floats);
                most(mix32, R * r.heads * r.vdim_p);
                break;
            }
            case MixerKind::latent_attention: {
                const LatentShape &l = L.latent;
                most(absorbed, RS * l.heads * (l.rank_p + l.rot_p));
                most(partial, RS * L.splits * l.heads * l.rank_p);
                most(partial_ml, RS * L.splits * l.heads * 2);
                most(lq, R * l.heads * (l.dim_p + l.rot_p));
                most(latents, T * l.rank_p);
                most(key_rot, T * l.rot_p);
                most(lk, T * l.heads * l.dim_p);
                most(lvt, T * l.heads * l.vdim_p);
                most(mix32, RS * l.heads * l.vdim_p);
                break;
            }
            case MixerKind::attention: {
                const AttentionShape &l = L.attention;
                most(partial, RS * L.splits * l.heads * l.vdim_p);
                most(partial_ml, RS * L.splits * l.heads * 2);
                most(lq, R * l.heads * l.dim_p);
                most(lk, T * l.kv_heads * l.dim_p);
                most(lvt, T * l.kv_heads * l.vdim_p);
                most(mix32, RS * l.heads * l.vdim_p);
                break;
            }
        }
    }
    auto bytes = [&](void **p, size_t n) -> int {
        uint8_t *q = nullptr;
        const int r = device_alloc(&q, n);
        *p = q;
        return r;
    };
    int rc;
    const struct { float **p; size_t n; } floats[] = {{&mix32_, mix32}, {&squares_, squares}, {&absorbed_, absorbed}, {&partial_, partial}, {&partial_ml_, partial_ml},
                                                      {&r_log_hi_, logs}, {&r_log_lo_, logs}, {&r_step_, logs}};
    for (const auto &b : floats) if ((rc = device_alloc(b.p, b.n)) != ESP_OK) return rc;
    const struct { void **p; size_t n; } operands[] = {{&r_q_, rq}, {&r_k_, rq}, {&r_kt_hi_, rkt}, {&r_kt_lo_, rkt}, {&r_vt_, rv}, {&r_vs_hi_, rvs}, {&r_vs_lo_, rvs}, {&r_states_hi_, states},
                                                       {&r_states_lo_, states}, {&l_q_, lq}, {&l_latents_, latents}, {&l_key_rot_, key_rot}, {&l_k_, lk}, {&l_vt_, lvt}};
    for (const auto &b : operands) if ((rc = bytes(b.p, b.n * E)) != ESP_OK) return rc;
    return ESP_OK;
}

// ---- launches ------------------------------------------------------------------------------------------------
int LayeredRuntime::mixer_step(Layer &L, DenseGemvOut *out) {
    hipStream_t s = context().stream;
    // a replay after the stop token must leave the states alone (the other kernels recompute what they computed last)
    const int *halt = capturing_ ? d_log_count_ + 1 : nullptr;
    int rc;
    switch (L.mixer) {
        case MixerKind::retention: {
            const RetentionShape &r = L.retention;
            RetentionStep st{mixed_, d_pos_, d_seq_, halt, mix32_, squares_, 1};
            if ((rc = time_begin(K_RETENTION)) != ESP_OK) return rc;
            ESP_HIP_TRY(launch_retention_step(r, st, s));
            out->mix_cols = r.heads * r.vdim_p; out->squares = squares_; out->gate = mixed_ + 2 * r.heads * r.dim_p + r.heads * r.vdim_p;
            out->parts = retention_step_parts(r.vdim_p); out->vdim = r.vdim; out->vdim_p = r.vdim_p;
            break;
        }
        case MixerKind::mamba2: {
            const Mamba2Shape &r = L.mamba2;
            Mamba2Step st{mixed_, d_pos_, d_seq_, halt, mix32_, 1};
            if ((rc = time_begin(K_MAMBA2)) != ESP_OK) return rc;
            ESP_HIP_TRY(launch_mamba2_step(r, st, s));
            out->mix_cols = r.heads * r.vdim_p; out->part_of = r.norm_part; out->part_starts = r.norm_starts; out->part_norm = r.norm;
            out->part_count = r.norm_groups; out->part_size = (float)(r.heads * r.vdim / r.norm_groups); out->part_by_eight = r.norm_by_eight;
            break;
        }
        case MixerKind::latent_attention: {
            const LatentShape &l = L.latent;
            LatentStep st{mixed_, d_pos_, d_seq_, absorbed_, partial_, partial_ml_, L.splits, 1, mix32_, nullptr, 0};
            if ((rc = time_begin(K_LATENT)) != ESP_OK) return rc;
            ESP_HIP_TRY(launch_latent_step(l, st, precision_, s));
            out->mix_cols = l.heads * l.vdim_p;
            break;
        }
        case MixerKind::attention: {
            const AttentionShape &l = L.attention;
            AttentionStep st{mixed_, d_pos_, d_seq_, partial_, partial_ml_, L.splits, 1, mix32_, nullptr, 0};
            if ((rc = time_begin(K_ATTENTION)) != ESP_OK) return rc;
            ESP_HIP_TRY(launch_attention_step(l, st, precision_, s));
            out->mix_cols = l.heads * l.vdim_p;
            break;
        }
    }
    return time_end();
}

int LayeredRuntime::mixer_block(Layer &L, int rows, int seq, int base) {
    hipStream_t s = context().stream;
    const float eps = (float)c_.norm_eps;
    const int ld_act = L.out.ld;
    int rc;
    switch (L.mixer) {
        case MixerKind::retention: {
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
            break;
        }
        case MixerKind::mamba2: {
            const Mamba2Shape &r = L.mamba2;
            if ((rc = time_begin(K_MAMBA2)) != ESP_OK) return rc;
            if (seq >= 0) {
                Mamba2Block b{mixed_, rows, base, seq, r_q_, r_k_, r_kt_hi_, r_vt_, r_vs_hi_, r_vs_lo_, r_log_hi_, r_log_lo_, r_step_, r_states_hi_, r_states_lo_, mix32_};
                ESP_HIP_TRY(launch_mamba2_block(r, b, precision_, s));
            } else {
                Mamba2Step st{mixed_, d_pos_, d_seq_, nullptr, mix32_, rows};
                ESP_HIP_TRY(launch_mamba2_step(r, st, s));
            }
            Mamba2Norm n{mix32_, act_, ld_act, eps, seq >= 0 ? rows : 0, base, seq, mixed_, 0};
            ESP_HIP_TRY(launch_mamba2_norm(r, n, rows, precision_, s));
            break;
        }
        case MixerKind::latent_attention: {
            const LatentShape &l = L.latent;
            if ((rc = time_begin(K_LATENT)) != ESP_OK) return rc;
            if (seq < 0) {
                LatentStep st{mixed_, d_pos_, d_seq_, absorbed_, partial_, partial_ml_, L.splits, rows, nullptr, act_, ld_act};
                ESP_HIP_TRY(launch_latent_step(l, st, precision_, s));
                break;
            }
            if (l.dkv_at >= 0) ESP_HIP_TRY(launch_latent_store(l, mixed_, d_pos_, d_seq_, rows, precision_, s));
            const KeyRange range = visible_keys(l.window, rows, base);
            LatentBlock b{mixed_, rows, base, seq, range.first, range.keys, range.keys_p, l_q_, l_latents_, l_key_rot_, l_k_, l_vt_, act_, ld_act};
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
            break;
        }
        case MixerKind::attention: {
            const AttentionShape &l = L.attention;
            if ((rc = time_begin(K_ATTENTION)) != ESP_OK) return rc;
            if (seq < 0) {
                AttentionStep st{mixed_, d_pos_, d_seq_, partial_, partial_ml_, L.splits, rows, nullptr, act_, ld_act};
                ESP_HIP_TRY(launch_attention_step(l, st, precision_, s));
                break;
            }
            const KeyRange range = visible_keys(l.window, rows, base);
            AttentionBlock b{mixed_, rows, base, seq, range.first, range.keys, range.keys_p, l_q_, l_k_, l_vt_, act_, ld_act};
            ESP_HIP_TRY(launch_attention_block(l, b, precision_, s));
            break;
        }
    }
    return time_end();
}

}  // namespace esp
