// program_mixers.hip — parallel blocks of a layer program: mixers (grouped attention, state space, gated delta rule; any
// number side by side) and a gated feed-forward that all read one RMS norm of the stream and join it together.
//
// One product brings the columns of every mixer and the feed-forward's (gate, up) pairs, whose activation its epilogue forms;
// one product takes all results side by side along its k and adds them to the stream.  The factors of the results are
// multiplied in by whoever writes that operand.
#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>

#include "mixer_kernels.h"
#include "program_internal.h"

namespace oxb {

uint32_t grouped_splits(const Model& m, const ProgramBranch& b, uint32_t rows) {
    return decode_splits(m, 2 * g_rt.n_cus, rows * b.kv_heads * oxb_row_head_tiles(b.heads / b.kv_heads));
}

int check_parallel_layer(const Program& p, const ProgramLayer& l) {
    int rc = OXB_HIP_OK;
    for (const ProgramBranch& b : l.branches) {
        auto vec = [&](uint64_t id, uint32_t n, const char* what) {
            if (!rc && id) vec_ptr(id, n, what, &rc);
        };
        if (b.kind == MixerKind::GroupedAttention) {
            vec(b.sink, b.heads, "sink");
            continue;
        }
        vec(b.conv_w, b.r.channels * b.r.taps, "convolution");
        vec(b.conv_b, b.r.channels, "convolution bias");
        vec(b.neg_a, b.r.heads, "decay");
        vec(b.dt_bias, b.r.heads, "decay bias");
        vec(b.skip, b.r.heads, "skip");
        vec(b.norm_w, b.r.norm_shared ? b.r.norm_len : b.r.heads * b.r.dv, "output norm");
    }
    if (!rc) dense_ptr(l.in, "input product", &rc);
    if (!rc) dense_ptr(l.out, "output product", &rc);
    return rc;
}

// Parameters of a grouped attention branch: the new tokens' store, and the attention with what follows it.
static int attention_params(Model& m, const ProgramBranch& b, ActBuf& a, const OxbRows& rows, OxbGroupedStore* s, OxbRowAttnParams* q) {
    Program& p = *m.prog;
    int rc = OXB_HIP_OK;
    memset(s, 0, sizeof *s);
    memset(q, 0, sizeof *q);
    q->sink = vec_ptr(b.sink, b.heads, "sink", &rc);
    if (rc) return rc;
    const size_t slots = m.n_pages ? (size_t)m.n_pages << m.page_shift : (size_t)m.d.batch * m.row_stride;
    s->rows = q->rows = rows;
    s->lin = a.qkv;
    s->ld_lin = p.ld_qkv;
    s->col_q = b.col_q, s->col_k = b.col_k, s->col_v = b.col_v;
    s->heads = b.heads, s->kv_heads = b.kv_heads;
    s->dim = b.dim, s->dim_p = b.dim_p, s->vdim = b.vdim, s->vdim_p = b.vdim_p;
    s->rot_dims = p.rope[b.rope].r.dims;
    s->eps = p.c.eps;
    s->cos_t = p.rope[b.rope].cos_t;
    s->sin_t = p.rope[b.rope].sin_t;
    s->q = a.q_abs;
    s->cache = (uint8_t*)m.k_cache + b.cache_off * slots * oxb_dt_bytes(p.dt);
    s->kv = kv_layout(m);
    s->kv.n_layers = 1;
    s->kv.nkv = b.kv_heads;
    q->kv = s->kv;
    q->q = a.q_abs;
    q->heads = b.heads;
    q->rep = b.heads / b.kv_heads;
    q->cache = s->cache;
    q->ld = b.dim_p + b.vdim_p;
    q->ks = q->v0 = b.dim_p / 32;
    q->nt = b.vdim_p / 16;
    q->scale = b.att_scale;
    q->part_o = p.part_o;
    q->part_ml = p.part_ml;
    q->n_splits = grouped_splits(m, b, rows.m);
    q->out = a.attn;
    q->ld_out = p.ld_attn;
    q->out_col = b.out_col;
    q->out_scale = b.scale;
    return OXB_HIP_OK;
}

static int recurrent_params(Model& m, const ProgramBranch& b, ActBuf& a, const OxbRows& rows, OxbRecurParams* r) {
    Program& p = *m.prog;
    int rc = OXB_HIP_OK;
    auto vec = [&](uint64_t id, uint32_t n, const char* what) { return rc || !id ? nullptr : vec_ptr(id, n, what, &rc); };
    memset(r, 0, sizeof *r);
    r->d = b.r;
    r->rows = rows;
    r->lin = a.qkv;
    r->ld_lin = p.ld_qkv;
    r->conv_w = vec(b.conv_w, b.r.channels * b.r.taps, "convolution");
    r->conv_b = vec(b.conv_b, b.r.channels, "convolution bias");
    r->neg_a = vec(b.neg_a, b.r.heads, "decay");
    r->dt_bias = vec(b.dt_bias, b.r.heads, "decay bias");
    r->skip = vec(b.skip, b.r.heads, "skip");
    r->norm_w = vec(b.norm_w, b.r.norm_shared ? b.r.norm_len : b.r.heads * b.r.dv, "output norm");
    r->memory = p.memory + b.memory_off;
    r->seq_stride = p.memory_floats;
    r->o = a.rec;
    r->out = a.attn;
    r->ld_out = p.ld_attn;
    r->out_col = b.out_col;
    r->out_fill = b.out_fill;
    return rc;
}

static int encode_attention(Model& m, const ProgramBranch& b, ActBuf& a, const OxbRows& rows, bool step) {
    const int dt = m.prog->dt;
    hipStream_t st = g_rt.stream;
    OxbGroupedStore s;
    OxbRowAttnParams q;
    OXB_TRY(attention_params(m, b, a, rows, &s, &q));
    OXB_TRY_HIP(oxb_launch_grouped_store(s, dt, st), "kernel launch failed: grouped_store");
    if (!step) {
        OXB_TRY_HIP(oxb_launch_row_prefill(q, dt, st), "kernel launch failed: row_prefill");
        return OXB_HIP_OK;
    }
    OXB_TRY_HIP(oxb_launch_row_decode(q, 1, dt, st), "kernel launch failed: row_decode");
    OXB_TRY_HIP(oxb_launch_row_merge(q, dt, st), "kernel launch failed: row_merge");
    return OXB_HIP_OK;
}

static int encode_recurrent(Model& m, const ProgramBranch& b, ActBuf& a, const OxbRows& rows, bool step) {
    Program& p = *m.prog;
    hipStream_t st = g_rt.stream;
    OxbRecurParams r;
    OXB_TRY(recurrent_params(m, b, a, rows, &r));
    if (step) {
        OXB_TRY_HIP(oxb_launch_recur_step(r, p.dt, st), "kernel launch failed: recur_step");
        if (oxb_recur_step_finishes(b.r)) return OXB_HIP_OK;
    } else {
        for (uint32_t at = 0; at < rows.m; at += OXB_RECUR_SEGMENT) {
            r.first = at;
            r.n = std::min(rows.m - at, OXB_RECUR_SEGMENT);
            (void)oxb_recur_scratch(b.r, r.n, (float*)p.scan_ws.ptr, &r.s);
            OXB_TRY_HIP(oxb_launch_recur_chunked(r, st), "kernel launch failed: recur_chunked");
        }
    }
    OXB_TRY_HIP(oxb_launch_recur_finish(r, !step, p.dt, st), "kernel launch failed: recur_finish");
    return OXB_HIP_OK;
}

// All mixers of a block.  A decode step of attention beside a recurrence shares launches between the two.
static int encode_branches(Model& m, const ProgramLayer& l, ActBuf& a, const OxbRows& rows, bool step) {
    const int dt = m.prog->dt;
    hipStream_t st = g_rt.stream;
    if (step && l.branches.size() == 2 && l.branches[0].kind == MixerKind::GroupedAttention && l.branches[1].kind != MixerKind::GroupedAttention) {
        OxbGroupedStore s;
        OxbRowAttnParams q;
        OxbRecurParams r;
        OXB_TRY(attention_params(m, l.branches[0], a, rows, &s, &q));
        OXB_TRY(recurrent_params(m, l.branches[1], a, rows, &r));
        if (oxb_pair_ok(s, r)) {
            OXB_TRY_HIP(oxb_launch_pair_enter(s, r, dt, st), "kernel launch failed: pair_enter");
            OXB_TRY_HIP(oxb_launch_row_decode(q, 1, dt, st), "kernel launch failed: row_decode");
            OXB_TRY_HIP(oxb_launch_pair_leave(q, r, dt, st), "kernel launch failed: pair_leave");
            return OXB_HIP_OK;
        }
    }
    for (const ProgramBranch& b : l.branches) {
        if (b.kind == MixerKind::GroupedAttention) OXB_TRY(encode_attention(m, b, a, rows, step));
        else OXB_TRY(encode_recurrent(m, b, a, rows, step));
    }
    return OXB_HIP_OK;
}

int encode_parallel_layers(Model& m, ActBuf& a, float* x, const OxbRows& rows, bool step) {
    Program& p = *m.prog;
    const uint32_t w = p.c.width;
    int rc = OXB_HIP_OK;
    auto norm = [&](const ProgramNorm& n, float in_scale) -> int {
        const float* nw = vec_ptr(n.w, w, "norm", &rc);
        if (rc) return rc;
        OXB_TRY_HIP(oxb_launch_row_norm(x, w, rows.m, in_scale, nw, p.c.eps, a.act, p.ld_act, oxb_dense_pad(w), p.dt, g_rt.stream), "kernel launch failed: row_norm");
        return OXB_HIP_OK;
    };
    // The norm between two layers is split over the products on either side where both take the few-row kernel.
    const uint32_t w_pad = oxb_dense_pad(w);
    auto few = [&](uint64_t id) {
        const DenseWeight* d = dense_ptr(id, "weight", &rc);
        return d && oxb_dense_few_rows(d->n_pad, d->k_pad, rows.m, g_rt.n_cus);
    };
    bool half_normed = false;   // a.act holds x * weight, a.ssq the sums of squares
    for (size_t i = 0; i < p.layers.size(); i++) {
        const ProgramLayer& l = p.layers[i];
        if (!half_normed) OXB_TRY(norm(l.norm1, i ? 1.0f : p.c.embed_scale));
        OxbEpilogue e = epilogue(l.n_lin);
        e.out32 = a.qkv;
        e.ld32 = p.ld_qkv;
        if (half_normed) {
            e.ssq_in = a.ssq;
            e.n_ssq = w_pad / 16;
            e.ssq_width = w;
            e.ssq_eps = p.c.eps;
        }
        if (l.has_mlp) {
            e.glu = l.n_lin;
            e.glu_out = (uint8_t*)a.attn + (size_t)l.mid_col * oxb_dt_bytes(p.dt);
            e.ld_glu = p.ld_attn;
            e.n_glu = oxb_dense_pad(l.ff);
        }
        OXB_TRY(product(p, l.in, a.act, p.ld_act, rows.m, e, "kernel launch failed: input product"));
        OXB_TRY(encode_branches(m, l, a, rows, step));
        OxbEpilogue o = epilogue(w);
        o.scale = p.c.residual_mult;
        o.resid = o.out32 = x;
        o.ld32 = w;
        half_normed = i + 1 < p.layers.size() && few(l.out) && few(p.layers[i + 1].in);
        if (half_normed) {
            o.nw = vec_ptr(p.layers[i + 1].norm1.w, w, "norm", &rc);
            o.norm = OXB_NORM_SCALE;
            o.out_t = a.act;
            o.ld_t = p.ld_act;
            o.fill = w_pad;
            o.ssq_out = a.ssq;
        }
        if (rc) return rc;
        OXB_TRY(product(p, l.out, a.attn, p.ld_attn, rows.m, o, "kernel launch failed: output product"));
    }
    return norm(p.final_norm, 1.0f);
}

// ---------------------------------------------------------------------------
// Loading
// ---------------------------------------------------------------------------
namespace {

// Rows of the input product and columns of the output product of one block, collected over its parts.
struct BlockMaps {
    Loader& ld;
    uint32_t width;
    std::vector<const TensorView*> in_src, out_src;
    int64_t in_at = 0, out_at = 0;                   // elements of the sources so far
    std::vector<int64_t> in_rows, out_cols, out_muls;

    // Source [n][width] of the input product -> its first element.
    int input(const std::string& name, uint64_t n, int64_t* first) {
        const TensorView* t;
        OXB_TRY(ld.get(name, {n, width}, &t));
        in_src.push_back(t);
        *first = in_at;
        in_at += (int64_t)t->elements();
        return OXB_HIP_OK;
    }
    // `count` rows of a source from row `row` on, the columns of the product they become; padded to a multiple of 4.
    uint32_t columns(int64_t first, uint64_t row, uint64_t count) {
        const uint32_t col = (uint32_t)in_rows.size();
        for (uint64_t i = 0; i < (count + 3) / 4 * 4; i++) in_rows.push_back(i < count ? first + (int64_t)((row + i) * width) : -1);
        return col;
    }
    // Source [width][n] of the output product: `groups` groups of n / groups columns, each padded to `padded`, the whole to a
    // multiple of 32 -> its first column.
    int output(const std::string& name, uint64_t n, uint64_t groups, uint32_t padded, uint32_t* col, uint32_t* fill) {
        const TensorView* t;
        OXB_TRY(ld.get(name, {width, n}, &t));
        out_src.push_back(t);
        *col = (uint32_t)out_cols.size();
        const uint64_t each = n / groups;
        for (uint64_t g = 0; g < groups; g++)
            for (uint32_t i = 0; i < padded; i++) {
                out_cols.push_back(i < each ? out_at + (int64_t)(g * each + i) : -1);
                out_muls.push_back((int64_t)n);
            }
        while (out_cols.size() % 32) out_cols.push_back(-1), out_muls.push_back(0);
        *fill = (uint32_t)out_cols.size() - *col;
        out_at += (int64_t)t->elements();
        return OXB_HIP_OK;
    }
};

double plain_value(double v) { return v; }
double negative_exp(double v) { return -exp(v); }

int load_attention(BlockMaps& b, Model& m, const MixerConfig& c, const std::string& name, ProgramBranch* o) {
    Program& p = *m.prog;
    o->heads = c.heads, o->kv_heads = c.kv_heads;
    o->dim = c.dim, o->dim_p = oxb_pad32(c.dim);
    o->vdim = c.vdim, o->vdim_p = oxb_pad32(c.vdim);
    o->att_scale = c.scale;
    if (const char* why = oxb_grouped_check(c.heads, c.kv_heads, c.dim, c.vdim, c.rope.dims, p.dt))
        return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: %s: %s", name.c_str(), why);
    int64_t q, k, v;
    OXB_TRY(b.input(name + "q", (uint64_t)c.heads * c.dim, &q));
    OXB_TRY(b.input(name + "k", (uint64_t)c.kv_heads * c.dim, &k));
    OXB_TRY(b.input(name + "v", (uint64_t)c.kv_heads * c.vdim, &v));
    o->col_q = b.columns(q, 0, (uint64_t)c.heads * c.dim);
    o->col_k = b.columns(k, 0, (uint64_t)c.kv_heads * c.dim);
    o->col_v = b.columns(v, 0, (uint64_t)c.kv_heads * c.vdim);
    OXB_TRY(b.ld.vector(name + "sink", c.heads, &o->sink));
    OXB_TRY(b.output(name + "o", (uint64_t)c.heads * c.vdim, c.heads, o->vdim_p, &o->out_col, &o->out_fill));
    o->cache_off = p.row_elems;
    p.row_elems += (size_t)c.kv_heads * (o->dim_p + o->vdim_p);
    return rope_table(m, p, c.rope, &o->rope);
}

// Convolution weights [channels][taps] -> [taps][channels].
int upload_taps(BlockMaps& b, const std::vector<float>& w, uint32_t taps, uint64_t* id) {
    std::vector<float> t(w.size());
    const size_t channels = w.size() / taps;
    for (size_t c = 0; c < channels; c++)
        for (size_t k = 0; k < taps; k++) t[k * channels + c] = w[c * taps + k];
    return b.ld.upload(t, id);
}

// Sizes both recurrent mixers derive from the ones their configuration gives.
int finish_recurrent(BlockMaps& b, Program& p, const std::string& name, ProgramBranch* o) {
    OxbRecurDims& d = o->r;
    d.dk_p = oxb_pad32(d.dk);
    d.slices = (d.dv + 31) / 32;
    d.ring = 1;
    while (d.ring < d.taps - 1 + OXB_RECUR_STEP_TOKENS) d.ring *= 2;
    d.eps = p.c.eps;
    d.out_scale = o->scale;
    if (const char* why = oxb_recur_check(d)) return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: %s: %s", name.c_str(), why);
    OXB_TRY(b.ld.vector(name + "A_log", d.heads, negative_exp, &o->neg_a));
    OXB_TRY(b.ld.vector(name + "dt_bias", d.heads, &o->dt_bias));
    const uint32_t inner = d.heads * d.dv;
    OXB_TRY(b.ld.vector(name + "norm", d.norm_shared ? d.norm_len : inner, &o->norm_w));
    OXB_TRY(b.output(name + "o", inner, 1, inner, &o->out_col, &o->out_fill));
    o->memory_off = p.memory_floats;
    p.memory_floats += (oxb_recur_floats(d) + 63) / 64 * 64;
    return OXB_HIP_OK;
}

int load_state_space(BlockMaps& b, Program& p, const MixerConfig& c, const std::string& name, ProgramBranch* o) {
    OxbRecurDims& d = o->r;
    const uint32_t inner = c.heads * c.vdim, gn = c.groups * c.state;
    d.heads = c.heads, d.qk_heads = c.groups, d.dk = c.state, d.dv = c.vdim, d.taps = c.conv;
    d.channels = inner + 2 * gn;
    d.ch_v = 0, d.ch_k = inner, d.ch_q = inner + gn;
    d.q_scale = 1.0f;
    d.norm_len = inner / c.norm_groups;
    d.gate_first = 1;
    int64_t in;
    OXB_TRY(b.input(name + "in", (uint64_t)inner + d.channels + c.heads, &in));
    d.col_z = b.columns(in, 0, inner);
    d.col_conv = b.columns(in, inner, d.channels);
    d.col_a = d.col_b = b.columns(in, (uint64_t)inner + d.channels, c.heads);
    std::vector<float> w;
    OXB_TRY(b.ld.values(name + "conv", {d.channels, d.taps}, plain_value, &w));
    OXB_TRY(upload_taps(b, w, d.taps, &o->conv_w));
    OXB_TRY(b.ld.vector(name + "conv.b", d.channels, &o->conv_b));
    OXB_TRY(b.ld.vector(name + "D", c.heads, &o->skip));
    return finish_recurrent(b, p, name, o);
}

int load_gated_delta(BlockMaps& b, Program& p, const MixerConfig& c, const std::string& name, ProgramBranch* o) {
    OxbRecurDims& d = o->r;
    const uint32_t inner = c.heads * c.vdim, qk = c.kv_heads * c.dim;
    d.delta = 1;
    d.heads = c.heads, d.qk_heads = c.kv_heads, d.dk = c.dim, d.dv = c.vdim, d.taps = c.conv;
    d.channels = 2 * qk + inner;
    d.ch_q = 0, d.ch_k = qk, d.ch_v = 2 * qk;
    d.q_scale = (float)(1.0 / sqrt((double)c.dim));
    d.norm_len = c.vdim;
    d.norm_shared = 1;
    int64_t q, k, v, g, beta, a;
    OXB_TRY(b.input(name + "q", qk, &q));
    OXB_TRY(b.input(name + "k", qk, &k));
    OXB_TRY(b.input(name + "v", inner, &v));
    OXB_TRY(b.input(name + "g", inner, &g));
    OXB_TRY(b.input(name + "b", c.heads, &beta));
    OXB_TRY(b.input(name + "a", c.heads, &a));
    // (the channels lie side by side without padding: the three sources follow each other)
    d.col_conv = b.columns(q, 0, (uint64_t)d.channels);
    d.col_z = b.columns(g, 0, inner);
    d.col_b = b.columns(beta, 0, c.heads);
    d.col_a = b.columns(a, 0, c.heads);
    std::vector<float> w;
    OXB_TRY(b.ld.values(name + "q.conv", {qk, d.taps}, plain_value, &w));
    OXB_TRY(b.ld.values(name + "k.conv", {qk, d.taps}, plain_value, &w));
    OXB_TRY(b.ld.values(name + "v.conv", {inner, d.taps}, plain_value, &w));
    OXB_TRY(upload_taps(b, w, d.taps, &o->conv_w));
    return finish_recurrent(b, p, name, o);
}

int load_branch(BlockMaps& b, Model& m, const MixerConfig& c, const std::string& name, float scale, ProgramLayer* l) {
    ProgramBranch o;
    memset(&o.r, 0, sizeof o.r);
    o.kind = c.kind;
    o.scale = scale;
    switch (c.kind) {
    case MixerKind::GroupedAttention: OXB_TRY(load_attention(b, m, c, name, &o)); break;
    case MixerKind::StateSpace: OXB_TRY(load_state_space(b, *m.prog, c, name, &o)); break;
    case MixerKind::GatedDelta: OXB_TRY(load_gated_delta(b, *m.prog, c, name, &o)); break;
    default: return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: %s: a mixer that parallel blocks do not take", name.c_str());
    }
    l->branches.push_back(o);
    return OXB_HIP_OK;
}

}  // namespace

int load_parallel_layer(Loader& ld, Model& m, const LayerConfig& c, const std::string& name, ProgramLayer* l) {
    const uint32_t w = m.prog->c.width;
    memset(&l->d, 0, sizeof l->d);
    BlockMaps b{ld, w};
    OXB_TRY(ld.vector(name + "norm1", w, [](double v) { return 1.0 + v; }, &l->norm1.w));
    if (c.mixer.kind == MixerKind::Parallel) {
        for (size_t i = 0; i < c.mixer.parts.size(); i++)
            OXB_TRY(load_branch(b, m, c.mixer.parts[i], name + "mix." + c.mixer.part_names[i], c.mixer.part_scales[i], l));
    } else {
        OXB_TRY(load_branch(b, m, c.mixer, name + "mix.", 1.0f, l));
    }
    while (b.in_rows.size() % OXB_DENSE_PAD) b.in_rows.push_back(-1);
    l->n_lin = (uint32_t)b.in_rows.size();
    l->has_mlp = c.has_mlp;
    if (c.has_mlp) {
        l->ff = c.mlp.ff;
        int64_t gate, up;
        OXB_TRY(b.input(name + "mlp.gate", l->ff, &gate));
        OXB_TRY(b.input(name + "mlp.up", l->ff, &up));
        for (uint32_t j = 0; j < oxb_dense_pad(l->ff); j++) {
            b.in_rows.push_back(j < l->ff ? gate + (int64_t)j * w : -1);
            b.in_rows.push_back(j < l->ff ? up + (int64_t)j * w : -1);
        }
        uint32_t fill;
        OXB_TRY(b.output(name + "mlp.down", l->ff, 1, oxb_dense_pad(l->ff), &l->mid_col, &fill));
    }
    l->n_out = (uint32_t)b.out_cols.size();
    OXB_TRY(ld.matrix(b.in_src, b.in_rows, Loader::range(w, 1), &l->in));
    return ld.matrix(b.out_src, Loader::range(w, 1), b.out_cols, &l->out, &b.out_muls);
}

}  // namespace oxb
