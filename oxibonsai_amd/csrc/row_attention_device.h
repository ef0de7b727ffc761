// row_attention_device.h — device helpers of the attention kernels over cached rows.
#pragma once
#include "dense_device.h"
#include "row_attention.h"

// Element i of a rotated part v (rot elements, the first rot_dims of them in pairs (i, i + rot_dims / 2)).
__device__ __forceinline__ float rotated(const float* v, uint32_t i, uint32_t rot_dims, const float* cs, const float* sn) {
    const uint32_t half = rot_dims >> 1;
    if (i < half) return v[i] * cs[i] - v[i + half] * sn[i];
    if (i < rot_dims) return v[i] * cs[i - half] + v[i - half] * sn[i - half];
    return v[i];
}

// Grouped heads, new tokens: a wave per head and ROWS rows, E elements per lane: queries and keys are rotated, then divided by
// their root mean square; values are copied.  Workgroup (rb, hb): rows ROWS rb .., heads 4 hb ...
template <typename T, int E, int ROWS> __device__ __forceinline__ void grouped_store(const OxbGroupedStore& p, uint32_t rb, uint32_t hb) {
    const uint32_t lane = threadIdx.x & 63u, hd = hb * 4 + (threadIdx.x >> 6);
    if (hd >= p.heads + 2 * p.kv_heads) return;
    const uint32_t half = p.rot_dims >> 1, kvh = hd < p.heads ? 0 : (hd - p.heads) % p.kv_heads;
    const bool is_q = hd < p.heads, is_v = hd >= p.heads + p.kv_heads;
    const uint32_t len = is_v ? p.vdim : p.dim, pad = is_v ? p.vdim_p : p.dim_p;
    const uint32_t col = is_q ? p.col_q + hd * p.dim : is_v ? p.col_v + kvh * p.vdim : p.col_k + kvh * p.dim;
    // the partner of each element in its rotation, the sign of the partner's share, and the angle's index
    uint32_t partner[E], angle[E];
    float sign[E];
#pragma unroll
    for (int e = 0; e < E; e++) {
        const uint32_t i = lane + 64 * e;
        const bool low = i < half, turns = !is_v && i < p.rot_dims;
        partner[e] = turns ? (low ? i + half : i - half) : min(i, len - 1);
        angle[e] = turns ? (low ? i : i - half) : 0;
        sign[e] = turns ? (low ? -1.f : 1.f) : 0.f;
    }
    float x[ROWS][E], y[ROWS][E], cs[ROWS][E], sn[ROWS][E];
#pragma unroll
    for (int t = 0; t < ROWS; t++) {
        const uint32_t m = min(rb * ROWS + t, p.rows.m - 1);
        const size_t at = (size_t)row_pos(p.rows, m) * half;
        const float* src = p.lin + (size_t)m * p.ld_lin + col;
#pragma unroll
        for (int e = 0; e < E; e++) {
            x[t][e] = src[min(lane + 64 * e, len - 1)];
            if (is_v) continue;
            y[t][e] = src[partner[e]];
            cs[t][e] = p.cos_t[at + angle[e]];
            sn[t][e] = p.sin_t[at + angle[e]];
        }
    }
#pragma unroll
    for (int t = 0; t < ROWS; t++) {
        const uint32_t m = rb * ROWS + t;
        float f = 1.0f;
        if (!is_v) {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < E; e++) {
                if (sign[e] != 0.f) x[t][e] = x[t][e] * cs[t][e] + sign[e] * y[t][e] * sn[t][e];
                if (lane + 64 * e < len) ss = fmaf(x[t][e], x[t][e], ss);
            }
            f = 1.0f / sqrtf(wave_sum_f32(ss) / (float)len + p.eps);
        }
        if (m >= p.rows.m) continue;
        T* dst = is_q ? reinterpret_cast<T*>(p.q) + ((size_t)m * p.heads + hd) * p.dim_p
                      : reinterpret_cast<T*>(p.cache) + kv_row(p.kv, row_seq(p.rows, m), 0, kvh, row_pos(p.rows, m)) * (p.dim_p + p.vdim_p) + (is_v ? p.dim_p : 0);
#pragma unroll
        for (int e = 0; e < E; e++)
            if (lane + 64 * e < pad) dst[lane + 64 * e] = lane + 64 * e < len ? (T)(x[t][e] * f) : (T)0.f;
    }
}

// Merge of one head's splits - the sink joins the denominator here, once.  One workgroup of at least 256 threads (values have at
// most 256 elements).
template <typename T> __device__ __forceinline__ void row_merge(const OxbRowAttnParams& p, uint32_t head, uint32_t m) {
    __shared__ float wgt[OXB_MAX_SPLITS];
    const uint32_t tid = threadIdx.x, lane = tid & 63u;
    const uint32_t n_ht = (p.rep + 15) / 16, kvh = head / p.rep, local = head % p.rep, col = local % 16;
    const uint32_t used = oxb_used_splits(row_pos(p.rows, m), p.n_splits), dim = 16 * p.nt;
    const size_t slot0 = ((size_t)m * p.kv.nkv * n_ht + kvh * n_ht + local / 16) * p.n_splits;
    const float sink = p.sink[head] * 1.4426950408889634f;   // (maxima are in units of log2(e))
    float ms[2], ls[2], M = sink;
#pragma unroll
    for (int i = 0; i < 2; i++) {
        const uint32_t s = lane + 64 * i;
        ms[i] = s < used ? p.part_ml[(slot0 + s) * 32 + col * 2] : -INFINITY;
        ls[i] = s < used ? p.part_ml[(slot0 + s) * 32 + col * 2 + 1] : 0.f;
        M = fmaxf(M, ms[i]);
    }
    M = wave_max_f32(M);
    float w[2], L = 0.f;
#pragma unroll
    for (int i = 0; i < 2; i++) {
        w[i] = ms[i] == -INFINITY ? 0.f : exp2_of<T>(ms[i] - M);
        L += w[i] * ls[i];
    }
    L = wave_sum_f32(L) + exp2_of<T>(sink - M);
    if (tid < 64) {
#pragma unroll
        for (int i = 0; i < 2; i++)
            if (lane + 64 * i < used) wgt[lane + 64 * i] = w[i] / L * p.out_scale;
    }
    __syncthreads();
    // a thread per value element, the threads beyond take further shares of the splits
    __shared__ float sums[1024];
    const uint32_t shares = min(max(blockDim.x / dim, 1u), 8u), share = tid / dim;
    const float* po = p.part_o + (slot0 * 16 + col) * dim;
    if (share < shares) {
        const uint32_t i = tid % dim;
        float y = 0.f;
        for (uint32_t s0 = share; s0 < used; s0 += 8 * shares) {
            float v[8];
#pragma unroll
            for (int k = 0; k < 8; k++) v[k] = po[(size_t)min(s0 + k * shares, used - 1) * 16 * dim + i];
#pragma unroll
            for (int k = 0; k < 8; k++)
                if (s0 + k * shares < used) y = fmaf(v[k], wgt[s0 + k * shares], y);
        }
        sums[tid] = y;
    }
    __syncthreads();
    T* out = reinterpret_cast<T*>(p.out) + (size_t)m * p.ld_out + p.out_col + head * dim;
    if (tid < dim) {
        float y = sums[tid];
        for (uint32_t k = 1; k < shares; k++) y += sums[k * dim + tid];
        out[tid] = (T)y;
    }
}
