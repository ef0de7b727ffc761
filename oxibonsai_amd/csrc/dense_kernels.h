// dense_kernels.h — linear layers with dense (bf16 or fp32) weights: resident layout, launch interface.
//
// Resident layout, "operand units": the matrix W [n][k] (y = W x) is cut into units of 16 rows x 32 columns, row tiles
// outermost, and a unit holds its 512 elements in the order a wave64 feeds them to the matrix cores: lane
// l = 16 g + r keeps row r, columns 8 g .. 8 g + 7.  bf16: the lane's eight elements are its 16 bytes at 16 l (1 KiB per
// unit).  Row tiles lie 256 bytes further apart than their units need, so that workgroups walking different tiles in step
// do not all draw on the same memory channels.  fp32: its first four are 16 bytes at 16 l, its last four 16 bytes at 1024 + 16 l (2 KiB per unit), so both
// types load a unit with fully coalesced 16-byte lane loads.  Rows and columns pad with zeros to multiples of 64.
//
// Activations are row-major [token][ld], bf16 or fp32 like the weights, ld a multiple of 64.  Whoever writes an
// activation row writes all of its columns up to `fill`, zeros past the last valid one, so a consumer may read whole
// units.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

enum { OXB_DT_BF16 = 0, OXB_DT_F32 = 1 };
static inline uint32_t oxb_dt_bytes(int dt) { return dt == OXB_DT_BF16 ? 2u : 4u; }

#define OXB_DENSE_PAD 64u
static inline uint32_t oxb_dense_pad(uint32_t n) { return (n + OXB_DENSE_PAD - 1) / OXB_DENSE_PAD * OXB_DENSE_PAD; }
// Elements from one row tile of a packed matrix to the next.
#if defined(__HIPCC__)
__host__ __device__
#endif
static inline size_t oxb_tile_stride(uint32_t k_pad, uint32_t elem_bytes) { return (size_t)(k_pad / 32u) * 512u + 256u / elem_bytes; }
// Row stride of an activation matrix of n columns: padded columns, and 128 elements more where rows would otherwise start a
// multiple of 1 KiB apart (the 16 rows of an operand would all come out of one or two L2 channels).
static inline uint32_t oxb_act_ld(uint32_t n) { const uint32_t p = oxb_dense_pad(n); return p % 512u ? p : p + 128u; }
#define OXB_DENSE_GEMV_MAX_ROWS 64u   // token rows up to which the few-row kernel is used (four column tiles)

// What happens to y[m][n] behind the product, in this order:
//   y = product * scale (+ add[n]) ; act(y) ; (+ resid[m][n]) -> out32[m][n] ; norm(y)[m][n] -> out_t (weights' type)
struct OxbEpilogue {
    float scale;
    const float* add;        // [n] or null
    uint32_t act;            // OXB_ACT_*
    const float* resid;      // [m][ld32] or null
    float* out32;            // [m][ld32] or null
    uint32_t ld32;
    void* out_t;             // [m][ld_t] or null: the next product's activation
    uint32_t ld_t, fill;     // columns n .. fill - 1 of out_t become zeros
    uint32_t norm;           // OXB_NORM_*
    const float *nw, *nb;    // [n] norm weight and bias
    float alpha;             // dynamic tanh
    uint32_t n;              // valid columns
    // RMS norm over a whole row, its two halves in the products on either side (few-row kernel): the one that completes the
    // row leaves y * nw in out_t and sums of squares, one per 16 columns, in ssq_out[m][n_pad / 16]; the one that consumes
    // it multiplies its products by 1 / sqrt(sum(ssq_in[m][0 .. n_ssq)) / ssq_width + ssq_eps) in front of everything else.
    float* ssq_out;
    const float* ssq_in;
    uint32_t n_ssq, ssq_width;
    float ssq_eps;
    // gated pairs (null: none): columns glu .. hold (gate, up) pairs and only those; gelu_tanh(gate) * up -> glu_out[m][pair]
    uint32_t glu;            // a multiple of 4, >= n
    void* glu_out;           // weights' type
    uint32_t ld_glu, n_glu;  // pairs, even
};
enum { OXB_ACT_NONE = 0, OXB_ACT_GELU_TANH = 1 };
enum { OXB_NORM_NONE = 0, OXB_NORM_DYT = 1, OXB_NORM_SCALE = 2 };   // dynamic tanh: tanh(alpha x) * w + b, elementwise; x * w

struct OxbDenseParams {
    const void* w;           // operand units
    uint32_t n_pad, k_pad;   // multiples of 64
    const void* x;           // [m][ldx] in the weights' type
    uint32_t ldx, m;
    // rows of x through a page table (null: row t is row0 + t): row of token t = (table[t >> shift] << shift) + low bits
    const uint32_t* row_table;
    uint32_t row_shift;
    size_t row0;
    OxbEpilogue e;
    // transposed store (oxb_launch_dense_gemm_t): out_t[n][ld_t] with the token contiguous, all columns of the token
    // tiles written (rows past m repeat the last one)
};

// src: row-major source elements on the device (gguf-style type ids: 0 F32, 1 F16, 30 BF16); element (n, k) of the packed
// matrix is src[row_off[n] + col_off[k]], or zero where either offset is negative.  row_off [n_pad], col_off [k_pad].
// With col_mul [k_pad] it is src[row_off[n] * col_mul[k] + col_off[k]]: columns out of matrices of different row lengths.
hipError_t oxb_launch_dense_pack(const void* src, int src_type, const int64_t* row_off, const int64_t* col_off, const int64_t* col_mul,
                                 uint32_t n_pad, uint32_t k_pad, int dt, void* dst, hipStream_t st);
// y = W x for any m: up to OXB_DENSE_GEMV_MAX_ROWS through the few-row kernel (weights streamed once, K split over the waves of a
// workgroup), more through the tiled GEMM.
hipError_t oxb_launch_dense(const OxbDenseParams& p, int dt, uint32_t n_cus, hipStream_t st);
// Whether a product of this size takes the few-row kernel, for m rows.
bool oxb_dense_few_rows(uint32_t n_pad, uint32_t k_pad, uint32_t m, uint32_t n_cus);
hipError_t oxb_launch_dense_gemm_t(const OxbDenseParams& p, int dt, uint32_t n_cus, hipStream_t st);
// Start of a forward on fp32 rows x [m][width]: optional copy of the rows into the second half of a [x; x0] buffer
// (x0_out + column x0_col, padded with zeros to x0_fill), and the first consumer's activation through the epilogue.
hipError_t oxb_launch_stream_enter(const float* x, uint32_t width, uint32_t m, void* x0_out, uint32_t ld_x0, uint32_t x0_col,
                                   uint32_t x0_fill, const OxbEpilogue& e, int dt, hipStream_t st);
// out[i][0 .. ld) = in[rows[i]][0 .. ld)
hipError_t oxb_launch_gather_rows(const void* in, uint32_t ld, const uint32_t* rows, uint32_t n, void* out, int dt, hipStream_t st);
// RMS norm of fp32 rows x [m][width] into activation rows: out = x / sqrt(mean(x^2) + eps) * w, zeros up to `fill`.
// in_scale != 1 multiplies x in front of it and is written back.
hipError_t oxb_launch_row_norm(float* x, uint32_t width, uint32_t m, float in_scale, const float* w, float eps, void* out, uint32_t ld,
                               uint32_t fill, int dt, hipStream_t st);
