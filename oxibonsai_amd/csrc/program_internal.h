// program_internal.h — layer programs as the translation units that load and encode them share them.
#pragma once
#include <hip/hip_fp16.h>
#include <hip/hip_runtime.h>

#include <cstring>

#include "dense_kernels.h"
#include "gguf.h"
#include "latent_kernels.h"
#include "program.h"
#include "recurrent_kernels.h"
#include "row_attention.h"

namespace oxb {

struct ProgramNorm {
    uint64_t w = 0, b = 0;
    float alpha = 1.0f;
};

// A mixer of a parallel block.
struct ProgramBranch {
    MixerKind kind;
    float scale;                          // of its result
    uint32_t out_col = 0, out_fill = 0;   // its columns in the operand of the block's output product
    // grouped attention
    uint32_t heads = 0, kv_heads = 0, dim = 0, dim_p = 0, vdim = 0, vdim_p = 0;
    uint32_t col_q = 0, col_k = 0, col_v = 0;
    float att_scale = 1.0f;
    uint32_t rope = 0;
    uint64_t sink = 0;
    size_t cache_off = 0;                 // elements per cache row slot in front of its rows
    // recurrent mixers
    OxbRecurDims r;
    uint64_t conv_w = 0, conv_b = 0, neg_a = 0, dt_bias = 0, skip = 0, norm_w = 0;
    size_t memory_off = 0;                // floats of a sequence's memory in front of its own
};

struct ProgramLayer {
    bool has_mlp = false;
    OxbLatentDims d;
    uint32_t n_qkv = 0, ff = 0;           // columns of the input product; feed-forward width
    ProgramNorm norm1, norm2;
    uint64_t qkv = 0, uk_t = 0, uk = 0, uv = 0, o = 0, up = 0, down = 0;   // dense matrices
    uint64_t c_norm = 0, sink = 0;        // vectors
    uint32_t rope = 0;                    // index into Program::rope
    // parallel blocks: one product in front of all mixers and the feed-forward, one behind them
    std::vector<ProgramBranch> branches;
    uint64_t in = 0, out = 0;             // dense matrices; in: [columns of the branches | gate / up pairs]
    uint32_t n_lin = 0;                   // columns in front of the pairs
    uint32_t mid_col = 0, n_out = 0;      // the feed-forward's place in, and the width of, the operand of `out`
};

struct ProgramRun {
    LayerRun r;
    size_t cache_off = 0;                 // elements in front of this run's rows, per cache row slot (times row count)
    uint32_t ld = 0;                      // elements per cache row
};

struct RopeTable {
    RopeConfig r;
    float *cos_t, *sin_t;                 // [max_seq][dims / 2]
};

// Activations of up to `rows` token rows.
struct ActBuf {
    uint32_t rows = 0;
    void *act = nullptr, *cat = nullptr, *q_abs = nullptr, *attn = nullptr, *mid = nullptr;
    float *qkv = nullptr, *rec = nullptr;   // input product; outputs of a recurrence
    float* ssq = nullptr;                   // sums of squares of a norm between two products
};

struct Program {
    DesignConfig c;
    int dt = OXB_DT_BF16;
    std::vector<ProgramLayer> layers;
    std::vector<ProgramRun> runs;
    std::vector<RopeTable> rope;
    ProgramNorm final_norm;
    uint64_t loop_in = 0;
    std::vector<uint64_t> loop_step;      // one vector per pass
    uint64_t head = 0;                    // embedding table as the output product
    uint32_t ld_act = 0, ld_cat = 0, ld_mid = 0, ld_attn = 0, ld_qkv = 0, n_q_abs = 0, n_rec = 0;
    size_t row_elems = 0;                 // cache elements per position over all runs
    ActBuf dec, pf;
    std::vector<void*> pf_allocs;
    float *part_o = nullptr, *part_ml = nullptr;
    DevBuf k_exp, v_exp, want_act, scan_ws;
    // recurrent layers' memory [sequence][memory_floats], and per sequence the position its memory stands at: 0 none yet,
    // kNoPosition unknown (a call failed half way)
    float* memory = nullptr;
    size_t memory_floats = 0;
    std::vector<uint32_t> at;
};

const DenseWeight* dense_ptr(uint64_t id, const char* what, int* rc);
OxbEpilogue epilogue(uint32_t n);
// y = W x for m rows through the epilogue; `what` names the launch in errors.
int product(const Program& p, uint64_t id, const void* x, uint32_t ldx, uint32_t m, const OxbEpilogue& e, const char* what);
// Splits of the attention over cached rows: about one workgroup per CU over heads and rows, no more than a full context has chunks.
uint32_t decode_splits(const Model& m, uint32_t wgs, uint32_t rows);
// .. and of a grouped attention branch: two workgroups per CU.
uint32_t grouped_splits(const Model& m, const ProgramBranch& b, uint32_t rows);
int rope_table(Model& m, Program& p, const RopeConfig& r, uint32_t* index);

inline std::string shape_text(const std::vector<uint64_t>& s) {
    std::string t = "[";
    for (size_t i = 0; i < s.size(); i++) t += (i ? ", " : "") + std::to_string(s[i]);
    return t + "]";
}

struct Loader {
    const TensorMap& tensors;
    int dt;
    Model& owner;   // collects what was uploaded

    int get(const std::string& name, const std::vector<uint64_t>& shape, const TensorView** out) {
        auto it = tensors.find(name);
        if (it == tensors.end()) return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: tensor not found: %s", name.c_str());
        const TensorView& t = it->second;
        if (t.type != (int)GGUF_F32 && t.type != (int)GGUF_F16 && t.type != (int)GGUF_BF16)
            return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: tensor %s is not of a floating-point type this tier reads", name.c_str());
        if (t.shape != shape || !t.data || t.bytes != t.elements() * tensor_type_bytes(t.type))
            return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: tensor %s has shape %s, expected %s", name.c_str(), shape_text(t.shape).c_str(),
                        shape_text(shape).c_str());
        *out = &t;
        return OXB_HIP_OK;
    }
    static float element(const TensorView& t, uint64_t i) {
        if (t.type == (int)GGUF_F32) {
            float f;
            memcpy(&f, t.data + 4 * i, 4);
            return f;
        }
        uint16_t h;
        memcpy(&h, t.data + 2 * i, 2);
        if (t.type == (int)GGUF_F16) return __half2float(__ushort_as_half(h));
        const uint32_t b = (uint32_t)h << 16;
        float f;
        memcpy(&f, &b, 4);
        return f;
    }
    int upload_vector(const TensorView& t, uint64_t first, uint32_t n, uint64_t* id) {
        std::vector<float> v(n);
        for (uint32_t i = 0; i < n; i++) v[i] = element(t, first + i);
        return upload(v, id);
    }
    int upload(const std::vector<float>& v, uint64_t* id) {
        const uint32_t n = (uint32_t)v.size();
        *id = 0;
        OXB_TRY(oxb_hip_upload_f32(id, v.data(), n));
        owner.owned_vecs.push_back(*id);
        return OXB_HIP_OK;
    }
    int vector(const std::string& name, uint32_t n, uint64_t* id) {
        const TensorView* t;
        OXB_TRY(get(name, {n}, &t));
        return upload_vector(*t, 0, n, id);
    }
    // Values of a tensor through f, appended to out.
    template <typename F> int values(const std::string& name, const std::vector<uint64_t>& shape, F f, std::vector<float>* out) {
        const TensorView* t;
        OXB_TRY(get(name, shape, &t));
        for (uint64_t i = 0; i < t->elements(); i++) out->push_back((float)f((double)element(*t, i)));
        return OXB_HIP_OK;
    }
    template <typename F> int vector(const std::string& name, uint32_t n, F f, uint64_t* id) {
        std::vector<float> v;
        OXB_TRY(values(name, {n}, f, &v));
        return upload(v, id);
    }
    int norm(const std::string& name, uint32_t n, ProgramNorm* out) {
        const TensorView* t;
        OXB_TRY(vector(name, n, &out->w));
        OXB_TRY(vector(name + ".b", n, &out->b));
        auto a = tensors.find(name + ".alpha");   // a scalar; a vector of one value will do
        const bool one = a != tensors.end() && a->second.shape.size() == 1;
        OXB_TRY(get(name + ".alpha", one ? std::vector<uint64_t>{1} : std::vector<uint64_t>{}, &t));
        out->alpha = element(*t, 0);
        return OXB_HIP_OK;
    }
    // Packed matrix from the concatenated source tensors (all of one type): element (n, k) = source[rows[n] + cols[k]], with
    // `muls` source[rows[n] * muls[k] + cols[k]].
    int matrix(const std::vector<const TensorView*>& src, const std::vector<int64_t>& rows, const std::vector<int64_t>& cols, uint64_t* id,
               const std::vector<int64_t>* muls = nullptr) {
        const uint32_t n_pad = oxb_dense_pad((uint32_t)rows.size()), k_pad = oxb_dense_pad((uint32_t)cols.size());
        std::vector<int64_t> ro(rows), co(cols);
        ro.resize(n_pad, -1);
        co.resize(k_pad, -1);
        std::vector<int64_t> mu(k_pad, 0);
        if (muls) std::copy(muls->begin(), muls->end(), mu.begin());
        size_t bytes = 0;
        for (const TensorView* t : src) {
            if (t->type != src[0]->type) return fail(OXB_HIP_INVALID_ARGUMENT, "invalid argument: matrices that are packed together differ in type");
            bytes += t->bytes;
        }
        DevBuf raw, off;
        DenseWeight w;
        w.dt = dt;
        w.n_pad = n_pad;
        w.k_pad = k_pad;
        int rc = OXB_HIP_OK;
        if (!(rc = raw.ensure(bytes)) && !(rc = off.ensure(((size_t)n_pad + 2 * k_pad) * 8))) {
            hipError_t e = hipSuccess;
            size_t at = 0;
            for (const TensorView* t : src) {
                if (e == hipSuccess) e = hipMemcpy((uint8_t*)raw.ptr + at, t->data, t->bytes, hipMemcpyHostToDevice);
                at += t->bytes;
            }
            int64_t* d_ro = (int64_t*)off.ptr;
            if (e == hipSuccess) e = hipMemcpy(d_ro, ro.data(), (size_t)n_pad * 8, hipMemcpyHostToDevice);
            if (e == hipSuccess) e = hipMemcpy(d_ro + n_pad, co.data(), (size_t)k_pad * 8, hipMemcpyHostToDevice);
            if (e == hipSuccess) e = hipMemcpy(d_ro + n_pad + k_pad, mu.data(), (size_t)k_pad * 8, hipMemcpyHostToDevice);
            if (e == hipSuccess && hipMalloc(&w.d, (n_pad / 16) * oxb_tile_stride(k_pad, oxb_dt_bytes(dt)) * oxb_dt_bytes(dt)) != hipSuccess)
                rc = fail(OXB_HIP_OUT_OF_MEMORY, "out of device memory: a %u x %u matrix on device %d", n_pad, k_pad, g_rt.device);
            if (!rc && e == hipSuccess) e = oxb_launch_dense_pack(raw.ptr, src[0]->type, d_ro, d_ro + n_pad, muls ? d_ro + n_pad + k_pad : nullptr, n_pad, k_pad, dt, w.d, g_rt.stream);
            if (e == hipSuccess) e = hipStreamSynchronize(g_rt.stream);
            if (!rc && e != hipSuccess) rc = hip_fail(e, "matrix upload");
        }
        raw.release();
        off.release();
        if (rc) {
            if (w.d) (void)hipFree(w.d);
            return rc;
        }
        *id = g_rt.next_id++;
        g_rt.dense[*id] = w;
        owner.owned_mats.push_back(*id);
        return OXB_HIP_OK;
    }
    static std::vector<int64_t> range(uint32_t n, int64_t stride) {
        std::vector<int64_t> v(n);
        for (uint32_t i = 0; i < n; i++) v[i] = (int64_t)i * stride;
        return v;
    }
    int plain(const std::string& name, uint32_t n, uint32_t k, uint64_t* id) {
        const TensorView* t;
        OXB_TRY(get(name, {n, k}, &t));
        return matrix({t}, range(n, k), range(k, 1), id);
    }
};

// Parallel blocks (program_mixers.hip).
int load_parallel_layer(Loader& ld, Model& m, const LayerConfig& c, const std::string& name, ProgramLayer* l);
int check_parallel_layer(const Program& p, const ProgramLayer& l);
// decode: one token per sequence; otherwise consecutive positions of one sequence.
int encode_parallel_layers(Model& m, ActBuf& a, float* x, const OxbRows& rows, bool step);

}  // namespace oxb
