// program.hip — layer programs: weights of a configured design in the handle tables, and the kernel sequence of a decode
// step and of a prefill portion.
//
// The residual stream x is fp32 and updated in place by the epilogues of the products that end a sub-layer; the same
// epilogue leaves the next product's input (its dynamic-tanh norm, or the plain stream at the start of a loop pass) behind,
// so a layer is: input product, latent store / absorb, attention, merge + value product, output product, up, down - and
// nothing else.  A repeated layer's runs share weights and differ in their cache regions.
#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>
#include <cstdlib>
#include <cstring>

#include "layer_kernels.h"
#include "program_internal.h"

namespace oxb {

Model::Model() = default;
Model::~Model() = default;

const DenseWeight* dense_ptr(uint64_t id, const char* what, int* rc) {
    auto it = g_rt.dense.find(id);
    if (it != g_rt.dense.end()) return &it->second;
    if (!*rc) *rc = fail(OXB_HIP_WEIGHT_NOT_FOUND, "weight handle %llu (%s) not found", (unsigned long long)id, what);
    return nullptr;
}

void program_release(Program& p) {
    p.k_exp.release();
    p.v_exp.release();
    p.want_act.release();
    p.scan_ws.release();
    for (void* q : p.pf_allocs) (void)hipFree(q);
    p.pf_allocs.clear();
    p.pf = ActBuf();
}

// ---------------------------------------------------------------------------
// Recurrent memory follows its sequence: it can go on where it stands, or start again at position 0.
// ---------------------------------------------------------------------------
int program_begin(Model& m, uint32_t seq, uint32_t pos) {
    Program& p = *m.prog;
    if (!p.memory_floats) return OXB_HIP_OK;
    if (pos && p.at[seq] != pos) {
        if (p.at[seq] == kNoPosition)
            return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: the recurrent state of sequence %u was lost in a failed call: it starts again at position 0", seq);
        return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: the recurrent state of sequence %u stands at position %u: it goes on there or starts again at 0, not at %u",
                    seq, p.at[seq], pos);
    }
    return OXB_HIP_OK;
}
void program_commit(Model& m, uint32_t seq, uint32_t next) { m.prog->at[seq] = next; }

size_t program_cache_row_bytes(const Program& p) { return p.row_elems * oxb_dt_bytes(p.dt); }

int program_check_handles(Model& m) {
    Program& p = *m.prog;
    const uint32_t w = p.c.width;
    int rc = OXB_HIP_OK;
    auto norm = [&](const ProgramNorm& n, const char* what) {
        if (!rc) vec_ptr(n.w, w, what, &rc);
        if (!rc && p.c.norm == NormKind::DynamicTanh) vec_ptr(n.b, w, what, &rc);
    };
    for (const ProgramLayer& l : p.layers) {
        norm(l.norm1, "norm1");
        if (p.c.block == BlockKind::Parallel) {
            if (!rc) rc = check_parallel_layer(p, l);
            continue;
        }
        if (l.has_mlp) norm(l.norm2, "norm2");
        if (!rc) vec_ptr(l.c_norm, l.d.rank, "latent norm", &rc);
        if (!rc) vec_ptr(l.sink, l.d.heads, "sink", &rc);
        dense_ptr(l.qkv, "input product", &rc);
        dense_ptr(l.uk_t, "key product", &rc);
        dense_ptr(l.uk, "key product", &rc);
        dense_ptr(l.uv, "value product", &rc);
        dense_ptr(l.o, "output product", &rc);
        if (l.has_mlp) {
            dense_ptr(l.up, "up", &rc);
            dense_ptr(l.down, "down", &rc);
        }
    }
    norm(p.final_norm, "final norm");
    if (p.loop_in) dense_ptr(p.loop_in, "loop input product", &rc);
    for (uint64_t s : p.loop_step)
        if (!rc) vec_ptr(s, w, "loop step", &rc);
    dense_ptr(p.head, "output head", &rc);
    return rc;
}

uint32_t decode_splits(const Model& m, uint32_t wgs, uint32_t rows) {
    const uint32_t most = oxb_max_splits(m.d.max_seq);
    uint32_t s = (wgs + rows - 1) / rows;
    if (s > most) s = most;
    if (const char* e = getenv("OXB_HIP_ATTN_SLOTS")) {  // measurement aid: a fixed slot count (long walks per workgroup)
        const long v = strtol(e, nullptr, 10);
        if (v > 0 && (uint32_t)v < s) s = (uint32_t)v;
    }
    if (s > 8) s = s / 8 * 8;   // head tiles of a split then share an XCD's L2
    return s ? s : 1;
}
static uint32_t latent_splits(const Model& m, const OxbLatentDims& d, uint32_t rows) {
    const uint32_t per = 16 * oxb_latent_head_tiles(d, rows), tiles = (d.heads + per - 1) / per;
    return decode_splits(m, g_rt.n_cus, rows * tiles);
}

OxbEpilogue epilogue(uint32_t n) {
    OxbEpilogue e;
    memset(&e, 0, sizeof e);
    e.scale = 1.0f;
    e.n = n;
    return e;
}

// The part of an epilogue that leaves the input of what follows run i (-1: the embedding) behind: the next layer's first
// norm, the plain stream in front of a loop pass, or the final norm.
static int feed_next(const Program& p, int i, const ActBuf& a, OxbEpilogue* e) {
    const uint32_t w = p.c.width;
    int rc = OXB_HIP_OK;
    const size_t next = (size_t)(i + 1);
    if (next < p.runs.size() && p.runs[next].r.first) {
        e->out_t = a.cat;
        e->ld_t = p.ld_cat;
        e->fill = w;            // the columns behind are the embedding output's
        e->norm = OXB_NORM_NONE;
        return rc;
    }
    const ProgramNorm& n = next < p.runs.size() ? p.layers[p.runs[next].r.layer].norm1 : p.final_norm;
    e->out_t = a.act;
    e->ld_t = p.ld_act;
    e->fill = oxb_dense_pad(w);
    e->norm = OXB_NORM_DYT;
    e->nw = vec_ptr(n.w, w, "norm", &rc);
    if (!rc) e->nb = vec_ptr(n.b, w, "norm", &rc);
    e->alpha = n.alpha;
    return rc;
}

int product(const Program& p, uint64_t id, const void* x, uint32_t ldx, uint32_t m, const OxbEpilogue& e, const char* what) {
    int rc = OXB_HIP_OK;
    const DenseWeight* w = dense_ptr(id, what, &rc);
    if (rc) return rc;
    OxbDenseParams q;
    memset(&q, 0, sizeof q);
    q.w = w->d;
    q.n_pad = w->n_pad;
    q.k_pad = w->k_pad;
    q.x = x;
    q.ldx = ldx;
    q.m = m;
    q.e = e;
    OXB_TRY_HIP(oxb_launch_dense(q, p.dt, g_rt.n_cus, g_rt.stream), what);
    return OXB_HIP_OK;
}

// Keys and values of every head for positions 0 .. kv_len - 1 of one sequence, from the cached latents.
static int expand(Model& m, const ProgramLayer& l, OxbLatentParams& lp, uint32_t seq, uint32_t kv_len) {
    Program& p = *m.prog;
    int rc = OXB_HIP_OK;
    const DenseWeight *uk = dense_ptr(l.uk, "key product", &rc), *uv = dense_ptr(l.uv, "value product", &rc);
    if (rc) return rc;
    OxbDenseParams q;
    memset(&q, 0, sizeof q);
    q.x = lp.cache;
    q.ldx = lp.ld;
    q.m = kv_len;
    if (m.n_pages) {
        q.row_table = m.d_table + (size_t)seq * m.table_stride;
        q.row_shift = m.page_shift;
    } else {
        q.row0 = (size_t)seq * m.row_stride;
    }
    q.w = uk->d;
    q.n_pad = uk->n_pad;
    q.k_pad = uk->k_pad;
    q.e = epilogue(l.d.heads * l.d.dim_p);
    q.e.out_t = p.k_exp.ptr;
    q.e.ld_t = oxb_act_ld(uk->n_pad);
    q.e.fill = uk->n_pad;
    OXB_TRY_HIP(oxb_launch_dense(q, p.dt, g_rt.n_cus, g_rt.stream), "kernel launch failed: key product");
    lp.k_exp = p.k_exp.ptr;
    lp.ld_k = q.e.ld_t;
    q.w = uv->d;
    q.n_pad = uv->n_pad;
    q.k_pad = uv->k_pad;
    q.e = epilogue(l.d.heads * l.d.vdim_p);
    q.e.out_t = p.v_exp.ptr;
    q.e.ld_t = oxb_act_ld((kv_len + 127u) / 128u * 128u);
    OXB_TRY_HIP(oxb_launch_dense_gemm_t(q, p.dt, g_rt.n_cus, g_rt.stream), "kernel launch failed: value product");
    lp.v_exp_t = p.v_exp.ptr;
    lp.ld_v = q.e.ld_t;
    return OXB_HIP_OK;
}

// All layer runs for rows.m token rows whose embedding rows are in x (fp32, updated in place); leaves the final norm of
// every row in a.act.  absorbed: latent rows alone (any mix of sequences); otherwise one sequence's consecutive positions.
static int encode_layers(Model& m, ActBuf& a, float* x, const OxbRows& rows, bool absorbed) {
    Program& p = *m.prog;
    hipStream_t st = g_rt.stream;
    const uint32_t w = p.c.width, M = rows.m;
    int rc = OXB_HIP_OK;
    if (p.c.block == BlockKind::Parallel) return encode_parallel_layers(m, a, x, rows, absorbed);
    {
        OxbEpilogue e = epilogue(w);
        OXB_TRY(feed_next(p, -1, a, &e));
        OXB_TRY_HIP(oxb_launch_stream_enter(x, w, M, p.loop_in ? a.cat : nullptr, p.ld_cat, w, oxb_dense_pad(2 * w), e, p.dt, st), "kernel launch failed: stream_enter");
    }
    for (size_t i = 0; i < p.runs.size(); i++) {
        const ProgramRun& run = p.runs[i];
        const ProgramLayer& l = p.layers[run.r.layer];
        if (run.r.first) {   // start of a loop pass: x <- W_in [x; x0] + step
            OxbEpilogue e = epilogue(w);
            e.add = vec_ptr(p.loop_step[(size_t)run.r.pass], w, "loop step", &rc);
            e.nw = rc ? nullptr : vec_ptr(l.norm1.w, w, "norm1", &rc);
            e.nb = rc ? nullptr : vec_ptr(l.norm1.b, w, "norm1", &rc);
            if (rc) return rc;
            e.out32 = x;
            e.ld32 = w;
            e.out_t = a.act;
            e.ld_t = p.ld_act;
            e.fill = oxb_dense_pad(w);
            e.norm = OXB_NORM_DYT;
            e.alpha = l.norm1.alpha;
            OXB_TRY(product(p, p.loop_in, a.cat, p.ld_cat, M, e, "kernel launch failed: loop input product"));
        }
        {   // queries of all heads, latent and rotated key part: one product
            OxbEpilogue e = epilogue(l.n_qkv);
            e.out32 = a.qkv;
            e.ld32 = p.ld_qkv;
            OXB_TRY(product(p, l.qkv, a.act, p.ld_act, M, e, "kernel launch failed: input product"));
        }
        const DenseWeight *ukt = dense_ptr(l.uk_t, "key product", &rc), *uv = dense_ptr(l.uv, "value product", &rc);
        OxbLatentParams lp;
        memset(&lp, 0, sizeof lp);
        lp.d = l.d;
        lp.rows = rows;
        lp.qkv = a.qkv;
        lp.ld_qkv = p.ld_qkv;
        lp.cos_t = p.rope[l.rope].cos_t;
        lp.sin_t = p.rope[l.rope].sin_t;
        lp.c_norm = rc ? nullptr : vec_ptr(l.c_norm, l.d.rank, "latent norm", &rc);
        lp.sink = rc ? nullptr : vec_ptr(l.sink, l.d.heads, "sink", &rc);
        if (rc) return rc;
        lp.w_uk_t = ukt->d;
        lp.k_uk = ukt->k_pad;
        lp.w_uv = uv->d;
        lp.k_uv = uv->k_pad;
        lp.q_abs = a.q_abs;
        const size_t slots = m.n_pages ? (size_t)m.n_pages << m.page_shift : (size_t)m.d.batch * m.row_stride;
        lp.cache = (uint8_t*)m.k_cache + run.cache_off * slots * oxb_dt_bytes(p.dt);
        lp.ld = run.ld;
        lp.kv = kv_layout(m);
        lp.kv.n_layers = lp.kv.nkv = 1;
        lp.part_o = p.part_o;
        lp.part_ml = p.part_ml;
        lp.n_splits = latent_splits(m, l.d, M);
        lp.out = a.attn;
        lp.ld_out = oxb_act_ld(l.d.heads * l.d.vdim_p);
        OXB_TRY_HIP(oxb_launch_latent_store(lp, absorbed, p.dt, st), "kernel launch failed: latent_store");
        if (absorbed) {
            OXB_TRY_HIP(oxb_launch_latent_decode(lp, p.dt, st), "kernel launch failed: latent_decode");
            OXB_TRY_HIP(oxb_launch_latent_merge(lp, p.dt, st), "kernel launch failed: latent_merge");
        } else {
            OXB_TRY(expand(m, l, lp, rows.seq0, rows.pos0 + M));
            OXB_TRY_HIP(oxb_launch_latent_prefill(lp, p.dt, st), "kernel launch failed: latent_prefill");
        }
        OxbEpilogue e = epilogue(w);
        e.resid = e.out32 = x;
        e.ld32 = w;
        if (l.has_mlp) {
            e.out_t = a.act;
            e.ld_t = p.ld_act;
            e.fill = oxb_dense_pad(w);
            e.norm = OXB_NORM_DYT;
            e.nw = vec_ptr(l.norm2.w, w, "norm2", &rc);
            e.nb = rc ? nullptr : vec_ptr(l.norm2.b, w, "norm2", &rc);
            if (rc) return rc;
            e.alpha = l.norm2.alpha;
        } else {
            OXB_TRY(feed_next(p, (int)i, a, &e));
        }
        OXB_TRY(product(p, l.o, a.attn, lp.ld_out, M, e, "kernel launch failed: output product"));
        if (!l.has_mlp) continue;
        OxbEpilogue eu = epilogue(l.ff);
        eu.act = OXB_ACT_GELU_TANH;
        eu.out_t = a.mid;
        eu.ld_t = oxb_act_ld(l.ff);
        eu.fill = oxb_dense_pad(l.ff);
        OXB_TRY(product(p, l.up, a.act, p.ld_act, M, eu, "kernel launch failed: up product"));
        OxbEpilogue ed = epilogue(w);
        ed.resid = ed.out32 = x;
        ed.ld32 = w;
        OXB_TRY(feed_next(p, (int)i, a, &ed));
        OXB_TRY(product(p, l.down, a.mid, eu.ld_t, M, ed, "kernel launch failed: down product"));
    }
    return OXB_HIP_OK;
}

static int encode_head(const Program& p, const void* act, uint32_t rows, float* logits) {
    OxbEpilogue e = epilogue(p.c.vocab);
    e.scale = p.c.logit_scale;
    e.out32 = logits;
    e.ld32 = p.c.vocab;
    return product(p, p.head, act, p.ld_act, rows, e, "kernel launch failed: output head");
}

int program_decode_step(Model& m) {
    Program& p = *m.prog;
    const OxbRows rows = {m.pos, 0, 0, 1, m.d.batch};
    OXB_TRY(encode_layers(m, p.dec, m.hidden, rows, true));
    OXB_TRY(encode_head(p, p.dec.act, m.d.batch, m.logits));
    OXB_TRY_HIP(oxb_launch_argmax(m.logits, m.d.vocab, m.d.batch, m.tokens, m.argmax_ws, g_rt.stream, m.h_tokens), "kernel launch failed: argmax");
    return OXB_HIP_OK;
}

// Portions up to this many tokens take the absorbed form.
#define OXB_PROGRAM_SHORT 16u

int program_prefill(Model& m, uint32_t seq, uint32_t M, uint32_t pos_start, const uint32_t* want, uint32_t n_want, float* d_logits) {
    Program& p = *m.prog;
    const bool small = M <= OXB_PROGRAM_SHORT;
    ActBuf& a = small ? p.dec : p.pf;
    const OxbRows rows = {nullptr, pos_start, seq, 0, M};
    OXB_TRY(encode_layers(m, a, m.pf_hidden, rows, small));
    if (!n_want) return OXB_HIP_OK;
    const size_t row = (size_t)p.ld_act * oxb_dt_bytes(p.dt);
    if (!want) return encode_head(p, (const uint8_t*)a.act + (M - 1) * row, 1, d_logits);
    OXB_TRY(p.want_act.ensure(n_want * row));
    OXB_TRY(m.want_rows.ensure((size_t)n_want * 4));
    OXB_TRY_HIP(hipMemcpyAsync(m.want_rows.ptr, want, (size_t)n_want * 4, hipMemcpyHostToDevice, g_rt.stream), "row index upload");
    OXB_TRY_HIP(oxb_launch_gather_rows(a.act, p.ld_act, (const uint32_t*)m.want_rows.ptr, n_want, p.want_act.ptr, p.dt, g_rt.stream), "kernel launch failed: gather_rows");
    return encode_head(p, p.want_act.ptr, n_want, d_logits);
}

// ---------------------------------------------------------------------------
// Buffers
// ---------------------------------------------------------------------------
// Zeroed: rows are written whole by their producers, but a matrix's columns past the last written one must be finite.
static int alloc_act(const Program& p, ActBuf* a, uint32_t rows, bool absorbed, std::vector<void*>* allocs) {
    const size_t es = oxb_dt_bytes(p.dt), R = rows;
    struct { void** ptr; size_t bytes; } bufs[] = {{&a->act, R * p.ld_act * es}, {&a->cat, p.loop_in ? R * p.ld_cat * es : 0},
                                                  {&a->q_abs, absorbed ? R * p.n_q_abs * es : 0}, {&a->attn, R * p.ld_attn * es},
                                                  {&a->mid, R * p.ld_mid * es}, {(void**)&a->qkv, R * p.ld_qkv * 4}, {(void**)&a->rec, R * p.n_rec * 4},
                                                  {(void**)&a->ssq, R * (oxb_dense_pad(p.c.width) / 16) * 4}};
    for (auto& b : bufs) {
        *b.ptr = nullptr;
        if (!b.bytes) continue;
        if (hipMalloc(b.ptr, b.bytes) != hipSuccess)
            return fail(OXB_HIP_OUT_OF_MEMORY, "out of device memory: requested %zu bytes on device %d", b.bytes, g_rt.device);
        allocs->push_back(*b.ptr);
        OXB_TRY_HIP(hipMemset(*b.ptr, 0, b.bytes), "activation clear");
    }
    a->rows = rows;
    return OXB_HIP_OK;
}

int program_prefill_buffers(Model& m, uint32_t rows, uint32_t pos_start) {
    Program& p = *m.prog;
    const bool small = rows <= OXB_PROGRAM_SHORT;
    if (rows > m.pf_cap) {
        OXB_TRY_HIP(hipStreamSynchronize(g_rt.stream), "synchronize");
        for (void* q : m.pf_allocs) (void)hipFree(q);
        m.pf_allocs.clear();
        m.pf_cap = 0;
        const size_t bytes = ((size_t)rows + 127) / 128 * 128 * p.c.width * 4;
        if (hipMalloc((void**)&m.pf_hidden, bytes) != hipSuccess)
            return fail(OXB_HIP_OUT_OF_MEMORY, "out of device memory: requested %zu bytes on device %d", bytes, g_rt.device);
        m.pf_allocs.push_back(m.pf_hidden);
        m.pf_cap = (rows + 127u) / 128u * 128u;
    }
    if (small) return OXB_HIP_OK;
    if (rows > p.pf.rows) {
        OXB_TRY_HIP(hipStreamSynchronize(g_rt.stream), "synchronize");
        for (void* q : p.pf_allocs) (void)hipFree(q);
        p.pf_allocs.clear();
        p.pf = ActBuf();
        ActBuf a;
        const int rc = alloc_act(p, &a, (rows + 127u) / 128u * 128u, p.c.block == BlockKind::Parallel, &p.pf_allocs);
        if (rc) {
            for (void* q : p.pf_allocs) (void)hipFree(q);
            p.pf_allocs.clear();
            return rc;
        }
        p.pf = a;
    }
    if (p.c.block == BlockKind::Parallel) {
        size_t floats = 0;
        for (const ProgramLayer& l : p.layers)
            for (const ProgramBranch& b : l.branches)
                if (b.kind != MixerKind::GroupedAttention)
                    floats = std::max(floats, oxb_recur_scratch(b.r, std::min(rows, OXB_RECUR_SEGMENT), nullptr, nullptr));
        OXB_TRY_HIP(hipStreamSynchronize(g_rt.stream), "synchronize");
        return floats ? p.scan_ws.ensure(floats * 4) : OXB_HIP_OK;
    }
    const size_t keys = ((size_t)pos_start + rows + 127) / 128 * 128, es = oxb_dt_bytes(p.dt);
    size_t k = 0, v = 0;
    for (const ProgramLayer& l : p.layers) {
        const size_t nk = oxb_act_ld(l.d.heads * l.d.dim_p), nv = (size_t)l.d.heads * l.d.vdim_p;
        if (nk > k) k = nk;
        if (nv > v) v = nv;
    }
    OXB_TRY_HIP(hipStreamSynchronize(g_rt.stream), "synchronize");
    OXB_TRY(p.k_exp.ensure(keys * k * es));
    OXB_TRY(p.v_exp.ensure((size_t)oxb_act_ld((uint32_t)keys) * v * es));
    return OXB_HIP_OK;
}

// ---------------------------------------------------------------------------
// Loading
// ---------------------------------------------------------------------------
static int load_layer(Loader& ld, Program& p, const LayerConfig& c, const std::string& name, ProgramLayer* l) {
    const MixerConfig& mx = c.mixer;
    const uint32_t w = p.c.width;
    OxbLatentDims& d = l->d;
    memset(&d, 0, sizeof d);
    d.heads = mx.heads;
    d.dim = mx.dim, d.dim_p = oxb_pad32(mx.dim);
    d.rot = mx.rot_dim, d.rot_p = oxb_pad32(mx.rot_dim);
    d.rank = mx.kv_rank, d.rank_p = oxb_pad32(mx.kv_rank);
    d.vdim = mx.vdim, d.vdim_p = oxb_pad32(mx.vdim);
    d.rot_dims = mx.rope.dims;
    d.scale = mx.scale;
    d.eps = p.c.eps;
    if (const char* why = oxb_latent_check(d, p.dt)) return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: %s: %s", name.c_str(), why);
    OXB_TRY(ld.norm(name + "norm1", w, &l->norm1));
    OXB_TRY(ld.vector(name + "mix.dkv.norm", d.rank, &l->c_norm));
    OXB_TRY(ld.vector(name + "mix.sink", d.heads, &l->sink));
    const TensorView *q, *dkv, *uk, *uv, *o;
    OXB_TRY(ld.get(name + "mix.q", {(uint64_t)d.heads * (d.dim + d.rot), w}, &q));
    OXB_TRY(ld.get(name + "mix.dkv", {(uint64_t)d.rank + d.rot, w}, &dkv));
    OXB_TRY(ld.get(name + "mix.uk", {(uint64_t)d.heads * d.dim, d.rank}, &uk));
    OXB_TRY(ld.get(name + "mix.uv", {(uint64_t)d.heads * d.vdim, d.rank}, &uv));
    OXB_TRY(ld.get(name + "mix.o", {w, (uint64_t)d.heads * d.vdim}, &o));
    // a source row (or column) per packed row (column): `count` of them from `first` on, zeros up to `padded`
    auto put = [](std::vector<int64_t>* v, int64_t first, int64_t stride, uint32_t count, uint32_t padded) {
        for (uint32_t i = 0; i < padded; i++) v->push_back(i < count ? first + (int64_t)i * stride : -1);
    };
    {   // [heads x (dim_p | rot_p)], latent, key part
        std::vector<int64_t> rows;
        const int64_t dkv0 = (int64_t)q->elements();
        for (uint32_t h = 0; h < d.heads; h++) {
            put(&rows, (int64_t)h * (d.dim + d.rot) * w, w, d.dim, d.dim_p);
            put(&rows, ((int64_t)h * (d.dim + d.rot) + d.dim) * w, w, d.rot, d.rot_p);
        }
        put(&rows, dkv0, w, d.rank, d.rank_p);
        put(&rows, dkv0 + (int64_t)d.rank * w, w, d.rot, d.rot_p);
        l->n_qkv = (uint32_t)rows.size();
        OXB_TRY(ld.matrix({q, dkv}, rows, Loader::range(w, 1), &l->qkv));
    }
    std::vector<int64_t> r_uk, c_rank, r_ukt, c_ukt, r_uv, c_o;
    put(&c_rank, 0, 1, d.rank, d.rank_p);
    put(&c_ukt, 0, d.rank, d.dim, d.dim_p);
    for (uint32_t h = 0; h < d.heads; h++) {
        put(&r_uk, (int64_t)h * d.dim * d.rank, d.rank, d.dim, d.dim_p);
        put(&r_ukt, (int64_t)h * d.dim * d.rank, 1, d.rank, d.rank_p);
        put(&r_uv, (int64_t)h * d.vdim * d.rank, d.rank, d.vdim, d.vdim_p);
        put(&c_o, (int64_t)h * d.vdim, 1, d.vdim, d.vdim_p);
    }
    OXB_TRY(ld.matrix({uk}, r_uk, c_rank, &l->uk));
    OXB_TRY(ld.matrix({uk}, r_ukt, c_ukt, &l->uk_t));
    OXB_TRY(ld.matrix({uv}, r_uv, c_rank, &l->uv));
    OXB_TRY(ld.matrix({o}, Loader::range(w, (int64_t)d.heads * d.vdim), c_o, &l->o));
    l->has_mlp = c.has_mlp;
    if (c.has_mlp) {
        l->ff = c.mlp.ff;
        OXB_TRY(ld.norm(name + "norm2", w, &l->norm2));
        OXB_TRY(ld.plain(name + "mlp.up", l->ff, w, &l->up));
        OXB_TRY(ld.plain(name + "mlp.down", w, l->ff, &l->down));
    }
    return OXB_HIP_OK;
}

// Angles position * frequency, formed in double and rounded once.
int rope_table(Model& m, Program& p, const RopeConfig& r, uint32_t* index) {
    for (size_t i = 0; i < p.rope.size(); i++)
        if (p.rope[i].r == r) {
            *index = (uint32_t)i;
            return OXB_HIP_OK;
        }
    const size_t half = r.dims / 2, n = (size_t)m.d.max_seq * half;
    std::vector<float> c(n), s(n);
    for (size_t i = 0; i < half; i++) {
        const double f = rope_frequency(r, (uint32_t)i);
        for (size_t pos = 0; pos < m.d.max_seq; pos++) {
            c[pos * half + i] = (float)cos((double)pos * f);
            s[pos * half + i] = (float)sin((double)pos * f);
        }
    }
    RopeTable t = {r, nullptr, nullptr};
    OXB_TRY(dev_alloc(m, (void**)&t.cos_t, n * 4));
    OXB_TRY(dev_alloc(m, (void**)&t.sin_t, n * 4));
    OXB_TRY_HIP(hipMemcpy(t.cos_t, c.data(), n * 4, hipMemcpyHostToDevice), "rope table upload");
    OXB_TRY_HIP(hipMemcpy(t.sin_t, s.data(), n * 4, hipMemcpyHostToDevice), "rope table upload");
    *index = (uint32_t)p.rope.size();
    p.rope.push_back(t);
    return OXB_HIP_OK;
}

static int load_all(Model& m, const DesignConfig& c, const TensorMap& tensors, int dt, uint64_t* embedding) {
    Program& p = *m.prog;
    Loader ld{tensors, dt, m};
    const uint32_t w = c.width;
    OXB_TRY_HIP(c.block == BlockKind::Parallel ? oxb_row_attention_prepare(dt) : oxb_latent_prepare(dt), "kernel preparation");
    const TensorView* emb;
    OXB_TRY(ld.get("embed", {c.vocab, w}, &emb));
    OXB_TRY(ld.plain("embed", c.vocab, w, &p.head));
    const bool parallel = c.block == BlockKind::Parallel;
    if (parallel) OXB_TRY(ld.vector("final.norm", w, [](double v) { return 1.0 + v; }, &p.final_norm.w));
    else OXB_TRY(ld.norm("final.norm", w, &p.final_norm));
    if (c.loop.times) {
        OXB_TRY(ld.plain("loop.in", w, 2 * w, &p.loop_in));
        const TensorView* step;
        OXB_TRY(ld.get("loop.step", {c.loop.times, w}, &step));
        p.loop_step.resize(c.loop.times);
        for (uint32_t t = 0; t < c.loop.times; t++) OXB_TRY(ld.upload_vector(*step, (uint64_t)t * w, w, &p.loop_step[t]));
    }
    p.layers.resize(c.layers.size());
    for (size_t i = 0; i < c.layers.size(); i++) {
        const std::string name = "l" + std::to_string(i) + ".";
        if (parallel) {
            OXB_TRY(load_parallel_layer(ld, m, c.layers[i], name, &p.layers[i]));
            continue;
        }
        OXB_TRY(load_layer(ld, p, c.layers[i], name, &p.layers[i]));
        OXB_TRY(rope_table(m, p, c.layers[i].mixer.rope, &p.layers[i].rope));
    }
    p.ld_act = oxb_act_ld(w);
    p.ld_cat = oxb_act_ld(2 * w);
    const size_t R = m.d.batch > OXB_PROGRAM_SHORT ? m.d.batch : OXB_PROGRAM_SHORT;
    size_t part = 0, ml = 0;
    auto grow = [](auto* v, size_t n) { if (n > *v) *v = (std::remove_pointer_t<decltype(v)>)n; };
    for (const ProgramLayer& l : p.layers) {
        if (parallel) {
            grow(&p.ld_qkv, oxb_dense_pad(l.n_lin));
            grow(&p.ld_attn, oxb_act_ld(l.n_out));
            for (const ProgramBranch& b : l.branches) {
                if (b.kind != MixerKind::GroupedAttention) {
                    grow(&p.n_rec, (size_t)b.r.heads * b.r.dv);
                    continue;
                }
                grow(&p.n_q_abs, (size_t)b.heads * b.dim_p);
                for (uint32_t r = 1; r <= R; r++) {
                    const size_t slots = (size_t)r * b.kv_heads * oxb_row_head_tiles(b.heads / b.kv_heads) * grouped_splits(m, b, r);
                    grow(&part, slots * 16 * b.vdim_p);
                    grow(&ml, slots * 32);
                }
            }
            continue;
        }
        const OxbLatentDims& d = l.d;
        grow(&p.ld_qkv, oxb_dense_pad(l.n_qkv));
        grow(&p.ld_attn, oxb_act_ld(d.heads * d.vdim_p));
        grow(&p.n_q_abs, d.heads * (d.rank_p + d.rot_p));
        if (l.has_mlp) grow(&p.ld_mid, oxb_act_ld(l.ff));
        const size_t tiles = (d.heads + 15) / 16;
        for (uint32_t r = 1; r <= R; r++) {
            const size_t slots = (size_t)r * tiles * latent_splits(m, d, r);
            if (slots * 16 * d.rank_p > part) part = slots * 16 * d.rank_p;
            if (slots * 32 > ml) ml = slots * 32;
        }
    }
    for (const LayerRun& r : layer_runs(c)) {
        const OxbLatentDims& d = p.layers[r.layer].d;
        ProgramRun run;
        run.r = r;
        run.cache_off = p.row_elems;
        run.ld = d.rank_p + d.rot_p;
        if (!parallel) p.row_elems += run.ld;   // (a parallel block's branches have taken theirs)
        p.runs.push_back(run);
    }
    OXB_TRY(alloc_act(p, &p.dec, (uint32_t)R, true, &m.allocs));
    OXB_TRY(dev_alloc(m, (void**)&p.part_o, std::max<size_t>(part, 4) * 4));
    OXB_TRY(dev_alloc(m, (void**)&p.part_ml, std::max<size_t>(ml, 4) * 4));
    if (p.memory_floats) OXB_TRY(dev_alloc(m, (void**)&p.memory, m.d.batch * p.memory_floats * 4));
    p.at.assign(m.d.batch, 0);
    const size_t B = m.d.batch;
    OXB_TRY(dev_alloc(m, (void**)&m.hidden, B * w * 4));
    OXB_TRY(dev_alloc(m, (void**)&m.logits, B * c.vocab * 4));
    OXB_TRY(dev_alloc(m, (void**)&m.tokens, B * 4));
    OXB_TRY(dev_alloc(m, (void**)&m.pos, B * 4));
    OXB_TRY(dev_alloc(m, &m.argmax_ws, B * OXB_ARGMAX_MAX_PARTS * 8));
    OXB_TRY_HIP(hipHostMalloc((void**)&m.h_hidden, B * w * 4, hipHostMallocCoherent), "pinned staging");
    OXB_TRY_HIP(hipHostMalloc((void**)&m.h_pos, B * 2 * 4, hipHostMallocCoherent), "pinned staging");
    m.h_tokens = m.h_pos + B;
    m.logits_cap = B * c.vocab;
    return oxb_hip_upload_embedding(embedding, emb->data, (size_t)emb->bytes, emb->type, c.vocab, w);
}

int program_create(const DesignConfig& c, const TensorMap& tensors, int dt, uint32_t max_seq, uint32_t batch, uint64_t* model,
                   uint64_t* embedding) {
    if (dt != OXB_DT_BF16 && dt != OXB_DT_F32) return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: unknown compute type %d", dt);
    if (!max_seq || !batch) return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: context and batch must not be 0");
    OXB_TRY(ensure_init());
    auto mp = std::make_unique<Model>();
    Model& m = *mp;
    memset(&m.d, 0, sizeof m.d);
    m.prog = std::make_unique<Program>();
    Program& p = *m.prog;
    p.c = c;
    p.dt = dt;
    m.d.fmt = -1;
    m.d.h = c.width;
    m.d.vocab = c.vocab;
    m.d.max_seq = max_seq;
    m.d.batch = batch;
    m.d.eps = c.eps;
    uint64_t emb = 0;
    int rc = load_all(m, c, tensors, dt, &emb);
    m.d.n_layers = (uint32_t)p.runs.size();
    m.d.lm_head = p.head;
    if (!rc) rc = model_alloc_cache(m, 0, 0);
    if (!rc) rc = program_check_handles(m);
    if (rc) {
        if (emb) (void)oxb_hip_free_embedding(emb);
        const std::vector<uint64_t> mats = std::move(m.owned_mats), vecs = std::move(m.owned_vecs);
        free_model(m);
        const std::string why = oxb_hip_last_error();
        for (uint64_t id : mats) (void)oxb_hip_free_weight(id);
        for (uint64_t id : vecs) (void)oxb_hip_free_f32(id);
        return fail(rc, "%s", why.c_str());
    }
    m.checked_gen = g_rt.weights_gen;
    const char* no_graph = getenv("OXB_HIP_DISABLE_GRAPH");
    m.graph_failed = no_graph && no_graph[0] == '1';
    *model = add_model(std::move(mp));
    *embedding = emb;
    return OXB_HIP_OK;
}

}  // namespace oxb
