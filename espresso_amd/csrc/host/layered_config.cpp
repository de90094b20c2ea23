#include "layered_config.h"

#include <cmath>

#include "json_min.h"
#include "model_support.h"

namespace esp {

void RotarySpec::frequencies(std::vector<double> *f, double *amplitude) const {
    const int pairs = dims / 2;
    f->resize(pairs);
    *amplitude = 1.0;
    for (int i = 0; i < pairs; i++) (*f)[i] = std::pow(base, -2.0 * i / dims);
    if (scaling == Scaling::linear)
        for (double &v : *f) v /= factor;
    if (scaling != Scaling::yarn) return;
    const double two_pi = 6.283185307179586476925286766559;
    // the pair whose wave makes `turns` turns over the original context
    auto pair_at = [&](double turns) { return dims * std::log(original / (two_pi * turns)) / (2.0 * std::log(base)); };
    const double lo = std::fmax(std::floor(pair_at(fast)), 0.0), hi = std::fmin(std::ceil(pair_at(slow)), dims - 1.0);
    for (int i = 0; i < pairs; i++) {
        const double ramp = std::fmin(std::fmax((i - lo) / std::fmax(hi - lo, 0.001), 0.0), 1.0);
        (*f)[i] = (*f)[i] / factor * ramp + (*f)[i] * (1.0 - ramp);
    }
    *amplitude = 0.1 * std::log(factor) + 1.0;
}

bool RotarySpec::operator==(const RotarySpec &o) const {
    return dims == o.dims && base == o.base && interleaved == o.interleaved && scaling == o.scaling && factor == o.factor &&
           original == o.original && fast == o.fast && slow == o.slow;
}

std::vector<LayeredConfig::TensorSpec> LayeredConfig::tensors() const {
    std::vector<TensorSpec> t = {{"embed", vocab, width}};
    if (embed_norm) t.push_back({"embed.norm", width, 0});
    for (size_t i = 0; i < layers.size(); i++) {
        const LayerSpec &L = layers[i];
        const std::string p = "l" + std::to_string(i) + ".", x = p + "mix.";
        t.push_back({p + "norm1", width, 0});
        if (L.ff) t.push_back({p + "norm2", width, 0});
        if (L.mixer == MixerKind::retention) {
            t.push_back({x + "q", L.heads * L.dim, width});
            t.push_back({x + "k", L.heads * L.dim, width});
            t.push_back({x + "v", L.heads * L.vdim, width});
            t.push_back({x + "g", L.heads * L.vdim, width});
        } else if (L.mixer == MixerKind::attention) {
            t.push_back({x + "q", L.heads * L.dim, width});
            t.push_back({x + "q.norm", L.heads * L.dim, 0});
            if (L.kv_from < 0) {
                t.push_back({x + "k", L.kv_heads * L.dim, width});
                t.push_back({x + "k.norm", L.kv_heads * L.dim, 0});
                t.push_back({x + "v", L.kv_heads * L.vdim, width});
            }
        } else if (L.mixer == MixerKind::mamba2) {
            const int inner = L.heads * L.vdim, channels = inner + 2 * L.groups * L.state;
            t.push_back({x + "in", inner + channels + L.heads, width});
            t.push_back({x + "conv", channels, L.conv});
            t.push_back({x + "conv.b", channels, 0});
            for (const char *name : {"dt_bias", "A_log", "D"}) t.push_back({x + name, L.heads, 0});
            t.push_back({x + "norm", inner, 0});
        } else {
            t.push_back({x + "q", L.heads * (L.dim + L.rot_dim), width});
            if (L.kv_from < 0) {
                t.push_back({x + "dkv", L.kv_rank + L.rot_dim, width});
                t.push_back({x + "dkv.norm", L.kv_rank, 0});
            }
            t.push_back({x + "uk", L.heads * L.dim, L.kv_rank});
            t.push_back({x + "uv", L.heads * L.vdim, L.kv_rank});
            t.push_back({x + "sink", L.heads, 0});
            t.push_back({x + "g", L.heads, width});
        }
        t.push_back({x + "o", width, L.heads * L.vdim});
        if (L.ff) {
            t.push_back({p + "mlp.gate", L.ff, width});
            t.push_back({p + "mlp.up", L.ff, width});
            t.push_back({p + "mlp.down", width, L.ff});
        }
    }
    t.push_back({"final.norm", width, 0});
    if (!tied_head) t.push_back({"head", vocab, width});
    return t;
}

namespace {

// Typed access to the members of one JSON object, with the member's path in every message.
class Fields {
  public:
    Fields(const JsonNode *node, std::string path, std::string *error) : node_(node), path_(std::move(path)), error_(error) {}
    bool ok() const { return ok_; }
    const JsonNode *member(const char *key) const {
        const JsonNode *n = node_ && node_->is(JsonNode::Object) ? node_->find(key) : nullptr;
        return n && n->is(JsonNode::Null) ? nullptr : n;
    }
    double number(const char *key) {
        const JsonNode *n = member(key);
        if (!n || !n->is(JsonNode::Number)) { complain(key, "is not a number"); return 0; }
        return n->number;
    }
    double number_or(const char *key, double fallback) { return member(key) ? number(key) : fallback; }
    int count(const char *key, int least = 1) {
        const double v = number(key);
        if (ok_ && (v != std::floor(v) || v < least || v > 2147483647.0)) complain(key, "is not a usable count");
        return ok_ ? (int)v : 0;
    }
    std::string string(const char *key) {
        const JsonNode *n = member(key);
        if (!n || !n->is(JsonNode::String)) { complain(key, "is not a string"); return ""; }
        return n->text;
    }
    Fields object(const char *key) {
        const JsonNode *n = member(key);
        if (!n || !n->is(JsonNode::Object)) complain(key, "is not an object");
        return Fields(n, path_ + key + ".", error_);
    }
    void complain(const char *key, const char *what) {
        if (ok_ && error_) *error_ = "config.json: " + path_ + key + " " + what;
        ok_ = false;
    }
    bool take(const Fields &inner) { ok_ = ok_ && inner.ok_; return ok_; }

  private:
    const JsonNode *node_;
    std::string path_;
    std::string *error_;
    bool ok_ = true;
};

// `scaling`: what an object of that name means in this architecture.
bool parse_rotary(Fields &mixer, bool interleaved, RotarySpec::Scaling scaling, int head_size, RotarySpec *r) {
    Fields f = mixer.object("rot");
    if (!mixer.take(f)) return false;
    r->dims = f.count("dims");
    r->base = f.number("base");
    r->interleaved = interleaved;
    if (f.ok() && (r->dims % 2 != 0 || r->dims > head_size)) f.complain("dims", "is odd or larger than what it rotates");
    if (f.ok() && !(r->base > 0)) f.complain("base", "is not positive");
    if (f.ok() && f.member("scaling")) {
        Fields s = f.object("scaling");
        if (f.take(s)) {
            r->scaling = scaling;
            r->factor = s.number("factor");
            if (s.ok() && !(r->factor > 0)) s.complain("factor", "is not positive");
            if (scaling == RotarySpec::Scaling::yarn) {
                r->original = s.number("original");
                r->fast = s.number("fast");
                r->slow = s.number("slow");
                if (s.ok() && !(r->original > 0 && r->fast > 0 && r->slow > 0)) s.complain("original", "or one of its neighbours is not positive");
            }
            f.take(s);
        }
    }
    return mixer.take(f);
}

bool parse_window(Fields &mixer, LayerSpec *L) {
    Fields m = mixer.object("mask");
    if (!mixer.take(m)) return false;
    L->window = m.count("size");
    return mixer.take(m);
}

bool parse_retention(Fields &x, LayerSpec *L) {
    L->mixer = MixerKind::retention;
    L->dim = x.count("dim");
    L->vdim = x.count("vdim");
    if (!x.ok() || !parse_rotary(x, false, RotarySpec::Scaling::yarn, L->dim, &L->rot)) return false;
    const JsonNode *d = x.member("decay");
    if (!d || !d->is(JsonNode::Array) || (int)d->items.size() != L->heads) { x.complain("decay", "does not list one decay per head"); return false; }
    for (const JsonNode &v : d->items) {
        if (!v.is(JsonNode::Number) || v.number < 0) { x.complain("decay", "holds something other than a decay"); return false; }
        L->decay.push_back(v.number);
    }
    return true;
}

bool parse_latent_attention(Fields &x, LayerSpec *L) {
    L->mixer = MixerKind::latent_attention;
    L->dim = x.count("dim");
    L->vdim = x.count("vdim");
    L->kv_rank = x.count("kv_rank");
    L->rot_dim = x.count("rot_dim");
    L->scale = x.number("scale");
    if (!x.ok() || !parse_rotary(x, true, RotarySpec::Scaling::yarn, L->rot_dim, &L->rot) || !parse_window(x, L)) return false;
    if (x.member("kv_from")) L->kv_from = x.count("kv_from", 0);
    return x.ok();
}

// Grouped heads, normed queries and keys, rotation of a part of a head in halves, a sliding window.
bool parse_attention(Fields &x, LayerSpec *L) {
    L->mixer = MixerKind::attention;
    L->dim = x.count("dim");
    L->vdim = x.count("vdim");
    L->kv_heads = x.count("kv_heads");
    L->scale = x.number("scale");
    if (x.ok() && L->heads % L->kv_heads) x.complain("kv_heads", "does not divide the query heads");
    if (!x.ok() || !parse_rotary(x, false, RotarySpec::Scaling::linear, L->dim, &L->rot) || !parse_window(x, L)) return false;
    if (x.member("kv_from")) L->kv_from = x.count("kv_from", 0);
    return x.ok();
}

bool parse_mamba2(Fields &x, LayerSpec *L) {
    L->mixer = MixerKind::mamba2;
    L->vdim = x.count("vdim");
    L->state = x.count("state");
    L->groups = x.count("groups");
    L->conv = x.count("conv");
    L->norm_groups = x.count("norm_groups");
    if (x.ok() && L->heads % L->groups) x.complain("groups", "does not divide the heads");
    if (x.ok() && (long long)L->heads * L->vdim % L->norm_groups) x.complain("norm_groups", "does not divide the values of all heads");
    return x.ok();
}

struct MixerReader {
    const char *type;
    bool (*parse)(Fields &mixer, LayerSpec *L);
};

// The members every architecture's layers have: a mixer of one of the given types, and a gated feed-forward or none.
bool parse_layer(const JsonNode &node, size_t index, const std::vector<MixerReader> &mixers, Activation activation, LayerSpec *L, std::string *error) {
    Fields f(&node, "layers[" + std::to_string(index) + "].", error);
    const std::string type = f.string("type");
    Fields x = f.object("mixer");
    if (!f.ok()) return false;
    L->heads = x.count("heads");
    if (!x.ok()) return false;
    const MixerReader *reader = nullptr;
    for (const MixerReader &r : mixers) if (type == r.type) reader = &r;
    if (!reader) { f.complain("type", ("names no mixer of this architecture: " + type).c_str()); return false; }
    if (!reader->parse(x, L) || !x.ok()) return false;
    if (f.member("mlp")) {
        Fields m = f.object("mlp");
        if (!f.take(m)) return false;
        if (m.string("kind") != "dense" && m.ok()) m.complain("kind", "is not dense");
        L->ff = m.count("ff");
        L->activation = activation;
        if (!m.ok()) return false;
    }
    return true;
}

// Whether a layer can read the other one's cache.
bool cache_fits(const LayerSpec &L, const LayerSpec &source) {
    if (source.mixer != L.mixer || source.kv_from >= 0 || !(source.rot == L.rot)) return false;
    if (L.mixer == MixerKind::latent_attention) return source.kv_rank == L.kv_rank && source.rot_dim == L.rot_dim;
    return source.heads == L.heads && source.kv_heads == L.kv_heads && source.dim == L.dim && source.vdim == L.vdim;
}

bool parse_model(Fields &f, const std::vector<MixerReader> &mixers, Activation activation, LayeredConfig *c, std::string *error) {
    c->vocab = f.count("vocab");
    c->width = f.count("width");
    Fields n = f.object("norm");
    if (!f.take(n)) return false;
    c->norm_eps = n.number("eps");
    if (!f.take(n)) return false;
    const JsonNode *layers = f.member("layers");
    if (!layers || !layers->is(JsonNode::Array) || layers->items.empty()) { f.complain("layers", "is not a list of layers"); return false; }
    for (size_t i = 0; i < layers->items.size(); i++) {
        LayerSpec L;
        if (!parse_layer(layers->items[i], i, mixers, activation, &L, error)) return false;
        if (L.kv_from >= 0) {
            const std::string at = "config.json: layers[" + std::to_string(i) + "].mixer.kv_from ";
            if (L.kv_from >= (int)i) { if (error) *error = at + "does not name an earlier layer"; return false; }
            if (!cache_fits(L, c->layers[L.kv_from])) { if (error) *error = at + "names a layer without a fitting cache of its own"; return false; }
        }
        c->layers.push_back(L);
    }
    return true;
}

bool parse_ranavik(const JsonNode &root, LayeredConfig *c, std::string *error) {
    Fields f(&root, "", error);
    c->block = BlockKind::parallel_two_norms;
    c->residual_mult = f.number("residual_mult");
    c->logit_softcap = f.number_or("logit_softcap", 0.0);
    return parse_model(f, {{"retention", parse_retention}, {"latent_attention", parse_latent_attention}}, Activation::silu, c, error);
}

// Mamba-2 layers come in two kinds of equal mechanism, each with sizes of its own.
bool parse_forovik(const JsonNode &root, LayeredConfig *c, std::string *error) {
    Fields f(&root, "", error);
    c->block = BlockKind::sequential_post_norms;
    c->embed_norm = false;
    c->tied_head = true;
    return parse_model(f, {{"attention", parse_attention}, {"mamba2", parse_mamba2}, {"mamba2_2", parse_mamba2}}, Activation::gelu_tanh, c, error);
}

}  // namespace

const std::vector<LayeredArchitecture> &layered_architectures() {
    static const std::vector<LayeredArchitecture> table = {{"Ranavik", parse_ranavik}, {"Forovik", parse_forovik}};
    return table;
}

const LayeredArchitecture *find_layered_architecture(const std::string &name) {
    for (const LayeredArchitecture &a : layered_architectures()) if (name == a.name) return &a;
    return nullptr;
}

bool parse_layered_config(const std::string &text, LayeredConfig *out, std::string *error) {
    JsonNode root;
    std::string perr;
    if (!json_parse(text, &root, &perr) || !root.is(JsonNode::Object)) { if (error) *error = "config.json is not a JSON object: " + perr; return false; }
    const JsonNode *name = root.find("architecture");
    if (!name || !name->is(JsonNode::String)) { if (error) *error = "config.json: architecture is missing"; return false; }
    const LayeredArchitecture *a = find_layered_architecture(name->text);
    if (!a) { if (error) *error = "config.json: unknown architecture " + name->text; return false; }
    LayeredConfig c;
    c.architecture = name->text;
    if (!a->parse(root, &c, error)) return false;
    *out = c;
    return true;
}

bool load_layered_config(const std::string &model_dir, LayeredConfig *out, std::string *error) {
    std::vector<uint8_t> raw;
    const std::string path = joinPath(model_dir, "config.json");
    if (!fileExists(path) || !readFile(path, &raw)) { if (error) *error = "Failed to read " + path; return false; }
    return parse_layered_config(std::string(raw.begin(), raw.end()), out, error);
}

bool is_layered_model_dir(const std::string &model_dir) {
    std::vector<uint8_t> raw;
    const std::string path = joinPath(model_dir, "config.json");
    JsonNode root;
    std::string perr;
    if (!fileExists(path) || !readFile(path, &raw) || !json_parse(std::string(raw.begin(), raw.end()), &root, &perr) || !root.is(JsonNode::Object)) return false;
    const JsonNode *name = root.find("architecture");
    return name && name->is(JsonNode::String) && find_layered_architecture(name->text);
}

}  // namespace esp
