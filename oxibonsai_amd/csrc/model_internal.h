// model_internal.h — a resident model as the translation units behind the model entry points share it: handles, decode
// buffers, KV cache with its page bookkeeping, captured decode graph, sampler state.
#pragma once
#include <hip/hip_runtime.h>

#include <memory>
#include <vector>

#include "../../include/oxb_hip.h"
#include "gemv_kernels.h"
#include "kv_quant_device.h"
#include "runtime_internal.h"

namespace oxb {

struct Program;

struct Model {
    oxb_model_desc d;
    std::vector<oxb_layer_ids> layers;
    // activations
    float *hidden = nullptr, *qkv = nullptr, *attn_part = nullptr, *attn_out = nullptr,
          *gu = nullptr, *act = nullptr, *logits = nullptr;  // gu: [batch][2 inter] gate || up sums, act: [batch][inter] SwiGLU output
    uint32_t *tokens = nullptr, *pos = nullptr;
    // pinned host staging of a decode call's small transfers (embedding rows and positions in, tokens out): copies from
    // and to pageable memory go through the runtime's own staging and cost about 10 us per call more
    float* h_hidden = nullptr;
    uint32_t *h_pos = nullptr, *h_tokens = nullptr;
    uint32_t* attn_done = nullptr;  // [batch][nkv] arrival counters of the attention workgroups, 0 between launches
    void* argmax_ws = nullptr;
    // KV cache: rows of hd fp16 values or one-byte codes, a quantised cache also one f32 scale per row.  Contiguous:
    // [batch][n_layers][nkv][row_stride] rows; paged: a pool [n_pages][n_layers][nkv][2^page_shift] rows and, per
    // sequence, a table of page numbers (kv_quant_device.h: OxbKvLayout)
    void *k_cache = nullptr, *v_cache = nullptr;
    float *k_scale = nullptr, *v_scale = nullptr;
    uint32_t kv_mode = OXB_KV_F16, row_stride = 0, window = 0, sinks = 0;
    uint32_t page_shift = 0, n_pages = 0, table_stride = 0;   // n_pages 0: contiguous
    std::vector<uint32_t> free_pages;                          // stack of free physical pages
    std::vector<std::vector<uint32_t>> seq_pages;              // pages of each sequence slot, in position order
    std::vector<uint32_t> h_table;                             // [batch][table_stride], mirrored in d_table
    uint32_t* d_table = nullptr;
    bool table_dirty = false;
    float *cos_t = nullptr, *sin_t = nullptr;
    uint32_t chunk = 0, n_splits = 0;
    // graph
    hipGraphExec_t graph_exec = nullptr;
    uint64_t checked_gen = 0;  // g_rt.weights_gen when every handle was last looked up
    uint64_t graph_gen = 0;  // g_rt.weights_gen at capture: the graph holds the weights' device pointers of that moment
    bool graph_failed = false;
    bool want_logits_in_graph = true;
    size_t logits_cap = 0;  // floats m.logits holds
    std::vector<void*> allocs;
    // prefill activations for up to pf_cap token rows (allocated on first use)
    uint32_t pf_cap = 0;
    float *pf_hidden = nullptr, *pf_qkv = nullptr, *pf_attn = nullptr, *pf_gu = nullptr;
    std::vector<void*> pf_allocs;
    GemmWorkspace gws;  // GEMM scratch of the captured large-batch decode step: sized at creation, never moved
    DevBuf gpack;       // quantised activation vectors of the captured GEMV-based step (batches of two to eight): likewise
    DevBuf gpack_o;     // the O projection's quantised input where the attention kernel writes it itself; starts as zeros (= zero vectors) and
                        // nothing else writes it, so the slots of a last vector group's absent vectors stay zero vectors
    // a model loaded from a file owns the weights it uploaded
    std::vector<uint64_t> owned_mats, owned_vecs;
    DevBuf tok_hist, tok_ids;  // token history of the on-device generation loop; prompt ids of a token prefill
    DevBuf sample_ws, rng;     // sampler scratch and per-sequence xorshift64 states
    DevBuf want_rows;          // rows of a portion whose logits are asked for
    // a model of a configured design: its layer program (program.hip) replaces the fixed Qwen3 sequence behind the same
    // entry points; null otherwise
    std::unique_ptr<Program> prog;

    Model();
    ~Model();
};

struct Embedding {  // token embedding table in its stored form
    void* d = nullptr;
    int type = 0;   // GGUF tensor type id: 0 F32, 1 F16, 41 Q1_0_g128, 42 TQ2_0_g128
    uint32_t vocab = 0, h = 0;
    size_t bytes = 0;
};
int dev_alloc(Model& m, void** p, size_t bytes);       // device memory that lives as long as the model
const float* vec_ptr(uint64_t id, uint32_t n, const char* what, int* rc);
OxbKvLayout kv_layout(const Model& m);
uint64_t add_model(std::unique_ptr<Model> m);
void free_model(Model& m);
// (Re)allocates a program model's cache, contiguous (n_pages 0) or paged.
int model_alloc_cache(Model& m, uint32_t page_size, uint32_t n_pages);

}  // namespace oxb

#define OXB_TRY_HIP(expr, what)                               \
    do {                                                      \
        hipError_t e_ = (expr);                               \
        if (e_ != hipSuccess) return hip_fail(e_, what);      \
    } while (0)
#define OXB_TRY(expr)            \
    do {                         \
        int rc_ = (expr);        \
        if (rc_) return rc_;     \
    } while (0)

