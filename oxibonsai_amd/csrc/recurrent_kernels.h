// recurrent_kernels.h — layers whose memory is a matrix per head that every token decays and writes to, behind short causal
// convolutions: the gated delta rule, and the state-space recurrence of Mamba-2.  Both are, per head with state S [dk][dv],
//
//   S <- a S + k u^T        o = S^T q        u = beta v                    (state space: k = B, q = C, v = x, beta = dt)
//                                            u = beta (v - (a S)^T k)      (delta rule)
//
// with a scalar decay a per token and head.  Everything in them is fp32 in every compute type, products included.
//
// What a sequence keeps, per layer (floats): the states [heads][dv / 32 slices][dk_p][32], then a ring of convolution inputs
// [ring][channels], the inputs of position p in row p % ring (ring a power of two).  Neither is ever cleared: position 0 starts from zeros without
// reading, and a convolution reads no position before 0.
//
// Forms:
//   step   a workgroup per sequence and head (or 32 columns of one) walks its tokens with the state in registers: decode
//          steps, portions of up to OXB_RECUR_STEP_TOKENS.
//   chunks of 64 tokens: `prepare` (convolutions, unit norms, decays), `chunk` (what needs no state, all chunks at once: decay
//          matrices, and for the delta rule the inverse of its unit lower triangular system), `scan` (chunk after chunk, a
//          workgroup per head and 16 columns): prompts.
// `finish` gates and norms the outputs into the next product's operand for both.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "token_rows.h"

#define OXB_RECUR_STEP_TOKENS 16u
#define OXB_RECUR_CHUNK 64u
#define OXB_RECUR_SEGMENT 2048u   // tokens a chunked pass takes at a time (bounds its scratch)

struct OxbRecurDims {
    uint32_t delta;                    // 1: gated delta rule, 0: state space
    uint32_t heads, qk_heads;          // head h uses q/k head h / (heads / qk_heads)
    uint32_t dk, dk_p, dv, slices;     // dk_p: padded to 32; slices of 32 columns
    uint32_t taps, channels, ring;     // ring >= taps - 1 + OXB_RECUR_STEP_TOKENS rows
    uint32_t ch_q, ch_k, ch_v;         // first convolution channel of each
    uint32_t col_conv, col_z, col_a, col_b;   // columns of the input product: convolution channels, output gate, decay / step, beta
    uint32_t norm_len;                 // outputs that share a root mean square
    uint32_t norm_shared;              // 1: one weight vector [norm_len] for all parts, 0: [heads * dv]
    uint32_t gate_first;               // 1: gate, then norm; 0: norm, then gate
    float q_scale, eps, out_scale;
};
#if defined(__HIPCC__)
__host__ __device__
#endif
static inline size_t oxb_recur_state(const OxbRecurDims& d) { return (size_t)d.heads * d.slices * d.dk_p * 32; }
static inline size_t oxb_recur_floats(const OxbRecurDims& d) { return oxb_recur_state(d) + (size_t)d.ring * d.channels; }

// Scratch of a chunked pass over n tokens (floats), carved out of one allocation.
struct OxbRecurScratch {
    float *q, *k, *v;                  // [n][qk_heads][dk_p], [n][heads][dv_p] after convolution (and unit norm)
    float *la, *beta;                  // [n][heads] logarithm of the decay; beta
    float *gam, *fwd;                  // [chunk][head][64]: decay from the chunk's start; from the token to the chunk's end
    float *P, *W, *Kt, *U0;            // operand units, per chunk and head (Kt: per q/k head)
};
size_t oxb_recur_scratch(const OxbRecurDims& d, uint32_t n, float* base, OxbRecurScratch* s);   // -> floats

struct OxbRecurParams {
    OxbRecurDims d;
    OxbRows rows;                      // rows of the whole launch (finish, step)
    const float* lin;                  // [rows.m][ld_lin] input product
    uint32_t ld_lin;
    const float *conv_w, *conv_b;      // [taps][channels], last tap the current token's; [channels] or null
    const float *neg_a, *dt_bias;      // [heads]: -exp(A_log); bias
    const float* skip;                 // [heads] or null: o += skip v
    const float* norm_w;
    float* memory;                     // sequence 0's floats of this layer
    size_t seq_stride;                 // floats from one sequence's to the next
    float* o;                          // [rows.m][heads * dv]
    void* out;                         // finish: [rows.m][ld_out] in the compute type
    uint32_t ld_out, out_col, out_fill;   // columns out_col ..; out_fill columns from there on are written (zeros past the end)
    // chunked: rows first .. first + n - 1
    uint32_t first, n;
    OxbRecurScratch s;
};

// One token per sequence (rows.seq_step 1), or all rows.m <= OXB_RECUR_STEP_TOKENS of one sequence (seq_step 0).
// Where it finishes a head's output by itself (oxb_recur_step_finishes) p.out is written and no `finish` follows.
hipError_t oxb_launch_recur_step(const OxbRecurParams& p, int dt, hipStream_t st);
bool oxb_recur_step_finishes(const OxbRecurDims& d);
hipError_t oxb_launch_recur_chunked(const OxbRecurParams& p, hipStream_t st);
// keep_conv: also bring the last convolution inputs of a chunked portion into the ring.
hipError_t oxb_launch_recur_finish(const OxbRecurParams& p, bool keep_conv, int dt, hipStream_t st);
bool oxb_recur_params_ok(const OxbRecurParams& p);
bool oxb_recur_finish_ok(const OxbRecurParams& p);
const char* oxb_recur_check(const OxbRecurDims& d);
