// row_attention.h — softmax attention with a learned sink per head over cached rows that hold a token's key and value side by
// side: row = [key: 32 ks elements | ..], the value beginning 32 v0 elements into the row (it may overlap the key: a latent
// row is both).  Rows are placed by OxbKvLayout (one "layer": every layer run has a region of its own), one row per kv head
// and position; `rep` query heads share a kv head.
//
//   store    new tokens: rotation and RMS norm of queries and keys per head, keys and values into the cache (grouped heads)
//   decode   split keys: every split leaves sums and maxima behind, `merge` joins them with the sink
//   prefill  portions of one sequence
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "kv_quant_device.h"
#include "token_rows.h"

struct OxbRowAttnParams {
    OxbRows rows;
    OxbKvLayout kv;          // n_layers = 1, nkv = kv heads
    const void* q;           // [m][heads][32 ks], rotated and normed
    uint32_t heads, rep;     // query heads; query heads per kv head
    const void* cache;       // this layer run's rows
    uint32_t ld;             // elements per row, a multiple of 32
    uint32_t ks, v0, nt;     // k units of the key; units in front of the value; 16-wide tiles of the value (even)
    float scale;
    const float* sink;       // [heads]
    float* part_o;           // [m][kv heads x head tiles][splits][16][16 nt]
    float* part_ml;          // [m][kv heads x head tiles][splits][16][2]
    uint32_t n_splits;
    void* out;               // merge, prefill: [m][ld_out], head h at out_col + 16 nt h
    uint32_t ld_out, out_col;
    float out_scale;
};
static inline uint32_t oxb_row_head_tiles(uint32_t rep) { return (rep + 15) / 16; }

// Grouped heads: queries, keys and values of new tokens out of the input product.
struct OxbGroupedStore {
    OxbRows rows;
    const float* lin;        // [m][ld_lin]
    uint32_t ld_lin, col_q, col_k, col_v;
    uint32_t heads, kv_heads, dim, dim_p, vdim, vdim_p, rot_dims;
    float eps;
    const float *cos_t, *sin_t;   // [max_seq][rot_dims / 2]
    void* q;                 // [m][heads][dim_p]
    void* cache;             // rows [key dim_p | value vdim_p]
    OxbKvLayout kv;
};

hipError_t oxb_launch_grouped_store(const OxbGroupedStore& p, int dt, hipStream_t st);
// head_tiles: tiles of 16 heads of one kv head that a workgroup takes (1 or 2).
hipError_t oxb_launch_row_decode(const OxbRowAttnParams& p, uint32_t head_tiles, int dt, hipStream_t st);
hipError_t oxb_launch_row_merge(const OxbRowAttnParams& p, int dt, hipStream_t st);
hipError_t oxb_launch_row_prefill(const OxbRowAttnParams& p, int dt, hipStream_t st);
bool oxb_grouped_store_ok(const OxbGroupedStore& p, int dt);
bool oxb_row_merge_ok(const OxbRowAttnParams& p, int dt);
// Once per process and type, before the first launch.
hipError_t oxb_row_attention_prepare(int dt);
// Whether rows of `units` 32-element units and grouped heads of these sizes fit the kernels, and why not.
const char* oxb_row_check(uint32_t units, int dt);
const char* oxb_grouped_check(uint32_t heads, uint32_t kv_heads, uint32_t dim, uint32_t vdim, uint32_t rot_dims, int dt);

#define OXB_MAX_SPLITS 128u
#define OXB_KEY_CHUNK 32u
// Splits in use at a position: two chunks each at least.
#if defined(__HIPCC__)
__host__ __device__
#endif
static inline uint32_t oxb_used_splits(uint32_t pos, uint32_t n_splits) {
    const uint32_t pairs = (pos / OXB_KEY_CHUNK + 2) / 2;
    return pairs < n_splits ? pairs : n_splits;
}
// Splits a context of max_seq positions can keep busy.
static inline uint32_t oxb_max_splits(uint32_t max_seq) { return oxb_used_splits(max_seq - 1, OXB_MAX_SPLITS); }
