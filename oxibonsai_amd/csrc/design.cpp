// design.cpp — configuration readers and the registry of designs (see design.h).
#include "design.h"

#include <cmath>

namespace oxb {

namespace {

// Typed access to one JSON object; the first problem is kept and names the key.
struct Fields {
    const Json* j;
    std::string where;
    std::string* err;
    bool ok = true;

    bool bad(const std::string& what) {
        if (ok) *err = where + what;
        return ok = false;
    }
    const Json* need(const char* key) {
        const Json* v = j ? j->get(key) : nullptr;
        if (!v) bad(std::string(key) + " is missing");
        return v;
    }
    uint32_t u32(const char* key, uint32_t lo = 1, uint32_t hi = 1u << 30) {
        const Json* v = need(key);
        if (!v) return 0;
        if (v->type != Json::Number || v->num != (double)(int64_t)v->num || v->num < (double)lo || v->num > (double)hi)
            return bad(std::string(key) + " is not a whole number in range"), 0;
        return (uint32_t)v->num;
    }
    double real(const char* key) {
        const Json* v = need(key);
        if (!v) return 0;
        if (v->type != Json::Number) return bad(std::string(key) + " is not a number"), 0;
        return v->num;
    }
    std::string text(const char* key) {
        const Json* v = need(key);
        if (!v) return {};
        if (v->type != Json::String) return bad(std::string(key) + " is not a string"), std::string();
        return v->s;
    }
    Fields object(const char* key) {
        const Json* v = need(key);
        if (v && v->type != Json::Object) bad(std::string(key) + " is not an object"), v = nullptr;
        return Fields{v, where + key + ".", err, ok};
    }
};

bool read_rope(Fields& f, uint32_t room, RopeConfig* out) {
    Fields r = f.object("rot");
    out->base = r.real("base");
    out->dims = r.u32("dims", 2, 4096);
    if (!f.ok || !r.ok) return false;
    if (out->dims % 2 || out->dims > room) return r.bad("dims must be even and within the rotated part");
    if (!(out->base > 0)) return r.bad("base must be positive");
    const Json* scaling = r.j->get("scaling");
    if (!scaling || scaling->is_null()) return true;
    Fields s = r.object("scaling");
    out->factor = s.real("factor");
    out->low = s.real("low");
    out->high = s.real("high");
    out->original = s.real("original");
    if (s.ok && (!(out->factor > 0) || !(out->low > 0) || !(out->high >= out->low) || !(out->original > 0)))
        return s.bad("factor, low and original must be positive and high at least low");
    return s.ok;
}

bool read_latent_attention(Fields f, MixerConfig* m) {
    m->kind = MixerKind::LatentAttention;
    m->heads = f.u32("heads", 1, 4096);
    m->dim = f.u32("dim", 1, 4096);
    m->rot_dim = f.u32("rot_dim", 1, 4096);
    m->vdim = f.u32("vdim", 1, 4096);
    m->kv_rank = f.u32("kv_rank", 1, 65536);
    m->scale = (float)f.real("scale");
    if (!read_rope(f, m->rot_dim, &m->rope)) return false;
    return f.ok;
}

bool read_grouped_attention(Fields f, MixerConfig* m) {
    m->kind = MixerKind::GroupedAttention;
    m->heads = f.u32("heads", 1, 4096);
    m->kv_heads = f.u32("kv_heads", 1, 4096);
    m->dim = f.u32("dim", 1, 4096);
    m->vdim = f.u32("vdim", 1, 4096);
    m->scale = (float)f.real("scale");
    if (f.ok && m->heads % m->kv_heads) return f.bad("heads must be a multiple of kv_heads");
    return f.ok && read_rope(f, m->dim, &m->rope);
}

bool read_state_space(Fields f, MixerConfig* m) {
    m->kind = MixerKind::StateSpace;
    m->heads = f.u32("heads", 1, 4096);
    m->vdim = f.u32("vdim", 1, 4096);
    m->state = f.u32("state", 1, 4096);
    m->groups = f.u32("groups", 1, 4096);
    m->norm_groups = f.u32("norm_groups", 1, 1u << 20);
    m->conv = f.u32("conv", 1, 64);
    if (f.ok && m->heads % m->groups) return f.bad("heads must be a multiple of groups");
    if (f.ok && (m->heads * m->vdim) % m->norm_groups) return f.bad("norm_groups must divide heads x vdim");
    return f.ok;
}

bool read_gated_delta(Fields f, MixerConfig* m) {
    m->kind = MixerKind::GatedDelta;
    m->heads = f.u32("heads", 1, 4096);
    m->kv_heads = f.u32("kv_heads", 1, 4096);
    m->dim = f.u32("dim", 1, 4096);
    m->vdim = f.u32("vdim", 1, 4096);
    m->conv = f.u32("conv", 1, 64);
    if (f.ok && m->heads % m->kv_heads) return f.bad("heads must be a multiple of kv_heads");
    return f.ok;
}

// Grouped attention (left) beside a state space (right).
bool read_attention_and_state(Fields f, MixerConfig* m) {
    m->kind = MixerKind::Parallel;
    m->parts.resize(2);
    Fields left = f.object("left");
    if (!left.ok || !read_grouped_attention(left, &m->parts[0])) return false;
    Fields right = f.object("right");
    if (!right.ok || !read_state_space(right, &m->parts[1])) return false;
    m->part_scales = {(float)f.real("left_scale"), (float)f.real("right_scale")};
    m->part_names = {"left.", "right."};
    return f.ok;
}

bool read_dense_mlp(Fields f, MlpConfig* m) {
    m->kind = MlpKind::Dense;
    m->ff = f.u32("ff");
    return f.ok;
}

bool read_gated_mlp(Fields f, MlpConfig* m) {
    m->kind = MlpKind::Gated;
    m->ff = f.u32("ff");
    return f.ok;
}

// The kinds a design's layers may name, with their readers.
struct MixerReader { const char* name; bool (*read)(Fields, MixerConfig*); };
struct MlpReader { const char* name; bool (*read)(Fields, MlpConfig*); };
struct LayerKinds {
    std::vector<MixerReader> mixers;
    std::vector<MlpReader> mlps;
};

bool read_layer(Fields f, const LayerKinds& kinds, LayerConfig* l) {
    const std::string type = f.text("type");
    if (!f.ok) return false;
    const MixerReader* mr = nullptr;
    for (const MixerReader& r : kinds.mixers)
        if (type == r.name) mr = &r;
    if (!mr) return f.bad("type \"" + type + "\" is unknown");
    Fields mixer = f.object("mixer");
    if (!mixer.ok || !mr->read(mixer, &l->mixer)) return false;
    const Json* mlp = f.j->get("mlp");
    if (!mlp || mlp->is_null()) return true;
    Fields ff = f.object("mlp");
    const std::string kind = ff.text("kind");
    if (!ff.ok) return false;
    for (const MlpReader& r : kinds.mlps)
        if (kind == r.name) return l->has_mlp = true, r.read(ff, &l->mlp);
    return ff.bad("kind \"" + kind + "\" is unknown");
}

// Sizes, the norm's eps and the list of layers.
bool read_common(Fields& f, const LayerKinds& kinds, DesignConfig* c) {
    c->vocab = f.u32("vocab");
    c->width = f.u32("width");
    Fields n = f.object("norm");
    if (f.ok && n.ok) c->eps = (float)n.real("eps");
    const Json* layers = f.need("layers");
    if (!f.ok || !n.ok) return false;
    if (layers->type != Json::Array || layers->a.empty() || layers->a.size() > 4096) return f.bad("layers is not a list of layers");
    for (size_t i = 0; i < layers->a.size(); i++) {
        LayerConfig l;
        if (!read_layer(Fields{&layers->a[i], "layers[" + std::to_string(i) + "].", f.err}, kinds, &l)) return false;
        c->layers.push_back(l);
    }
    return true;
}

// Fulirax: latent attention with sinks, dynamic-tanh norms, dense tanh-GELU feed-forwards, a loop that mixes the embedding
// output back in, logits through the embedding table.
bool read_fulirax(const Json& j, DesignConfig* c, std::string* err) {
    static const LayerKinds kinds = {{{"latent_attention", read_latent_attention}}, {{"dense", read_dense_mlp}}};
    Fields f{&j, "", err};
    c->norm = NormKind::DynamicTanh;
    c->block = BlockKind::Sequential;
    c->logit_scale = (float)f.real("logit_scale");
    if (!read_common(f, kinds, c)) return false;
    const Json* loop = j.get("loop");
    if (loop && !loop->is_null()) {
        Fields lf = f.object("loop");
        c->loop.start = lf.u32("start", 0, (uint32_t)c->layers.size());
        c->loop.stop = lf.u32("stop", 0, (uint32_t)c->layers.size());
        c->loop.times = lf.u32("times", 1, 4096);
        if (!lf.ok) return false;
        if (c->loop.start >= c->loop.stop) return lf.bad("stop must lie behind start");
    }
    return true;
}

// Muvonex: layers of a gated delta rule, or of grouped attention beside a state space; mixer and gated feed-forward read one
// norm and join the stream together; logits through the embedding table.
bool read_muvonex(const Json& j, DesignConfig* c, std::string* err) {
    static const LayerKinds kinds = {{{"delta", read_gated_delta}, {"parallel", read_attention_and_state}}, {{"dense", read_gated_mlp}}};
    Fields f{&j, "", err};
    c->norm = NormKind::RmsAroundOne;
    c->block = BlockKind::Parallel;
    c->residual_mult = (float)f.real("residual_mult");
    Fields e = f.object("embedding");
    if (f.ok && e.ok) c->embed_scale = (float)e.real("scale");
    return e.ok && read_common(f, kinds, c);
}

}  // namespace

const std::vector<Design>& designs() {
    static const std::vector<Design> all = {{"Fulirax", read_fulirax}, {"Muvonex", read_muvonex}};
    return all;
}

bool read_design(const std::string& text, DesignConfig* c, std::string* err) {
    Json j;
    if (!json_parse(text.data(), text.size(), &j, err)) {
        *err = "config.json: " + *err;
        return false;
    }
    const Json* a = j.get("architecture");
    if (!a || a->type != Json::String) {
        *err = "config.json: architecture is missing";
        return false;
    }
    for (const Design& d : designs())
        if (a->s == d.architecture) {
            *c = DesignConfig();
            c->architecture = a->s;
            if (d.read(j, c, err)) return true;
            *err = "config.json: " + *err;
            return false;
        }
    std::string known;
    for (const Design& d : designs()) known += std::string(known.empty() ? "" : ", ") + d.architecture;
    *err = "config.json: architecture \"" + a->s + "\" is unknown (known: " + known + ")";
    return false;
}

double rope_frequency(const RopeConfig& r, uint32_t i) {
    const double f = std::pow(r.base, -2.0 * (double)i / (double)r.dims);
    if (r.factor == 0) return f;
    const double turn = 2.0 * 3.14159265358979323846 / f;   // positions per full turn
    if (turn < r.original / r.high) return f;
    if (turn > r.original / r.low) return f / r.factor;
    const double s = (r.original / turn - r.low) / (r.high - r.low);
    return (1.0 - s) * f / r.factor + s * f;
}

std::vector<LayerRun> layer_runs(const DesignConfig& c) {
    std::vector<LayerRun> out;
    const uint32_t n = (uint32_t)c.layers.size();
    for (uint32_t i = 0; i < n;) {
        if (c.loop.times && i == c.loop.start) {
            for (uint32_t t = 0; t < c.loop.times; t++)
                for (uint32_t L = c.loop.start; L < c.loop.stop; L++) out.push_back({L, (int)t, L == c.loop.start});
            i = c.loop.stop;
        } else {
            out.push_back({i++, -1, false});
        }
    }
    return out;
}

}  // namespace oxb
