// design.cpp — configuration readers and the registry of designs (see design.h).
#include "design.h"

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

bool read_latent_attention(Fields f, MixerConfig* m) {
    m->kind = MixerKind::LatentAttention;
    m->heads = f.u32("heads", 1, 4096);
    m->dim = f.u32("dim", 1, 4096);
    m->rot_dim = f.u32("rot_dim", 1, 4096);
    m->vdim = f.u32("vdim", 1, 4096);
    m->kv_rank = f.u32("kv_rank", 1, 65536);
    m->scale = (float)f.real("scale");
    Fields r = f.object("rot");
    m->rot_base = r.real("base");
    m->rot_dims = r.u32("dims", 2, 4096);
    if (f.ok && r.ok && (m->rot_dims % 2 || m->rot_dims > m->rot_dim)) return r.bad("dims must be even and at most rot_dim");
    if (f.ok && r.ok && !(m->rot_base > 0)) return r.bad("base must be positive");
    return f.ok && r.ok;
}

bool read_dense_mlp(Fields f, MlpConfig* m) {
    m->kind = MlpKind::Dense;
    m->ff = f.u32("ff");
    return f.ok;
}

// The readers of the kinds a layer may name; designs share them.
struct MixerReader { const char* name; bool (*read)(Fields, MixerConfig*); };
const MixerReader kMixers[] = {{"latent_attention", read_latent_attention}};
struct MlpReader { const char* name; bool (*read)(Fields, MlpConfig*); };
const MlpReader kMlps[] = {{"dense", read_dense_mlp}};

bool read_layer(Fields f, LayerConfig* l) {
    const std::string type = f.text("type");
    if (!f.ok) return false;
    const MixerReader* mr = nullptr;
    for (const MixerReader& r : kMixers)
        if (type == r.name) mr = &r;
    if (!mr) return f.bad("type \"" + type + "\" is unknown");
    Fields mixer = f.object("mixer");
    if (!mixer.ok || !mr->read(mixer, &l->mixer)) return false;
    const Json* mlp = f.j->get("mlp");
    if (!mlp || mlp->is_null()) return true;
    Fields ff = f.object("mlp");
    const std::string kind = ff.text("kind");
    if (!ff.ok) return false;
    for (const MlpReader& r : kMlps)
        if (kind == r.name) return l->has_mlp = true, r.read(ff, &l->mlp);
    return ff.bad("kind \"" + kind + "\" is unknown");
}

// Fulirax: latent attention with sinks, dynamic-tanh norms, dense tanh-GELU feed-forwards, a loop that mixes the embedding
// output back in, logits through the embedding table.
bool read_fulirax(const Json& j, DesignConfig* c, std::string* err) {
    Fields f{&j, "", err};
    c->norm = NormKind::DynamicTanh;
    c->vocab = f.u32("vocab");
    c->width = f.u32("width");
    c->logit_scale = (float)f.real("logit_scale");
    Fields n = f.object("norm");
    if (f.ok && n.ok) c->eps = (float)n.real("eps");
    const Json* layers = f.need("layers");
    if (!f.ok || !n.ok) return false;
    if (layers->type != Json::Array || layers->a.empty() || layers->a.size() > 4096) return f.bad("layers is not a list of layers");
    for (size_t i = 0; i < layers->a.size(); i++) {
        LayerConfig l;
        if (!read_layer(Fields{&layers->a[i], "layers[" + std::to_string(i) + "].", err}, &l)) return false;
        c->layers.push_back(l);
    }
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

}  // namespace

const std::vector<Design>& designs() {
    static const std::vector<Design> all = {{"Fulirax", read_fulirax}};
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
