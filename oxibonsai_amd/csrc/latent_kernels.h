// latent_kernels.h — latent attention: keys and values of all heads are linear images of one short latent row per token,
// so that row (plus one rotated key part shared by the heads) is all the cache holds.
//
// Cache row of `ld` elements (bf16 or fp32): [latent c: rank, zeros to rank_p | rotated key part: rot, zeros to rot_p],
// rank_p and rot_p multiples of 32.  Rows are placed by OxbKvLayout like those of the other caches (one "layer", one
// "head": every layer run has a region of its own).
//
// Two forms of the same attention:
//   absorbed   q . (W_uk c) = (W_uk^T q) . c and sum p (W_uv c) = W_uv (sum p c): the kernel works on latent rows alone, all
//              heads share one read of the cache.  Decode steps and short portions.
//   expanded   keys and values of every head are formed once per portion by two GEMMs over the cached rows, and attention
//              runs on them with the small per-head sizes.  Prompts.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "row_attention.h"

struct OxbLatentDims {
    uint32_t heads, dim, dim_p, rot, rot_p, rank, rank_p, vdim, vdim_p;  // *_p: padded to multiples of 32
    uint32_t rot_dims;                                                    // rotated elements of the rot part (even)
    float scale, eps;
};

struct OxbLatentParams {
    OxbLatentDims d;
    OxbRows rows;
    const float* qkv;        // [m][ld_qkv] fp32: heads x [dim_p | rot_p], then latent (rank_p), then key part (rot_p)
    uint32_t ld_qkv;
    const float *cos_t, *sin_t;   // [max_seq][rot_dims / 2]
    const float* c_norm;     // [rank]
    const float* sink;       // [heads]
    const void* w_uk_t;      // operand units of the absorbed form: rows head x rank_p, k = dim (k_uk = padded k)
    uint32_t k_uk;
    const void* w_uv;        // operand units: rows head x vdim_p, k = rank (k_uv = padded k)
    uint32_t k_uv;
    void* q_abs;             // [m][heads][rank_p + rot_p]
    void* cache;             // this layer run's rows
    uint32_t ld;             // rank_p + rot_p
    OxbKvLayout kv;          // n_layers = nkv = 1
    float* part_o;           // [m][head tiles][splits][16][rank_p]
    float* part_ml;          // [m][head tiles][splits][16][2]
    uint32_t n_splits;
    void* out;               // [m][ld_out]: heads x vdim_p
    uint32_t ld_out;
    // expanded form
    const void* k_exp;       // [key][ld_k]: heads x dim_p
    uint32_t ld_k;
    const void* v_exp_t;     // [heads x vdim_p][ld_v]: keys contiguous, ld_v a multiple of 128 and > the last key
    uint32_t ld_v;
};

// Norm + rotate the new tokens' latent rows into the cache; rotate (and with `absorb` also absorb) their queries into q_abs.
hipError_t oxb_launch_latent_store(const OxbLatentParams& p, bool absorb, int dt, hipStream_t st);
// Absorbed form: split-key attention over the cache, then merge of the splits with the sink and the value product.
hipError_t oxb_launch_latent_decode(const OxbLatentParams& p, int dt, hipStream_t st);
hipError_t oxb_launch_latent_merge(const OxbLatentParams& p, int dt, hipStream_t st);
// Expanded form, rows of one sequence (seq_step 0) at consecutive positions.
hipError_t oxb_launch_latent_prefill(const OxbLatentParams& p, int dt, hipStream_t st);
// Once per process and type, before the first launch.
hipError_t oxb_latent_prepare(int dt);
// Whether the kernels can take these sizes, and why not.
const char* oxb_latent_check(const OxbLatentDims& d, int dt);
// Head tiles (of 16 heads) a workgroup of the absorbed form takes: two share the cache reads where the rows alone keep the
// GPU busy, one finishes a lone sequence sooner.
static inline uint32_t oxb_latent_head_tiles(const OxbLatentDims& d, uint32_t rows) { return d.heads > 16 && rows >= 8 ? 2u : 1u; }
