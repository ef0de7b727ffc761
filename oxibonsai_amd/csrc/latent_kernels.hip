// latent_kernels.hip — latent attention on the matrix cores (see latent_kernels.h for the two forms).
//
// Precision: scores, softmax and sums are fp32.  Probabilities meet bf16 values as a bf16 hi + lo pair (two products), so
// a weight keeps 16 bits; the fp32 kernels use fp32 operands throughout.
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <cstring>

#include "dense_device.h"
#include "latent_kernels.h"
#include "row_attention_device.h"

// ---------------------------------------------------------------------------
// New tokens.  The first n_abs blocks of a grid row absorb queries (4 waves, one 16-row tile of (head, latent) each); the
// blocks behind them belong to the 16 token rows in turn: block 0 of a row brings the RMS-normed latent and the rotated key
// part into the cache, the others rotate 1024 elements of the row's query parts into q_abs.
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(OxbLatentParams p, uint32_t n_abs, uint32_t tiles_per_head, uint32_t per_row) {
    typedef typename Dt<T>::frag frag;
    const OxbLatentDims& d = p.d;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, m0 = blockIdx.y * 16;
    const uint32_t kl = d.rank_p + d.rot_p, qh = d.dim_p + d.rot_p;
    T* q_abs = reinterpret_cast<T*>(p.q_abs);
    if (blockIdx.x < n_abs) {
        constexpr int UN = 4;
        const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
        const uint32_t tile = blockIdx.x * 4 + wave, c = lane & 15u, g = lane >> 4;
        if (tile >= d.heads * tiles_per_head) return;
        const uint32_t head = tile / tiles_per_head, rt = tile % tiles_per_head, nu = d.dim_p / 32;
        const T* w = reinterpret_cast<const T*>(p.w_uk_t) + tile * oxb_tile_stride(p.k_uk, sizeof(T));
        const bool have = m0 + c < p.rows.m;
        const float* q = p.qkv + (size_t)(have ? m0 + c : 0) * p.ld_qkv + head * qh + 8 * g;
        v4f acc = {0.f, 0.f, 0.f, 0.f};
        for (uint32_t u0 = 0; u0 < nu; u0 += UN) {
            frag a[UN], b[UN];
#pragma unroll
            for (int i = 0; i < UN; i++) {
                const uint32_t u = min(u0 + i, nu - 1);
                a[i] = load_unit(w + (size_t)u * 512, lane);
                const v8f x = load_row8(q + 32 * u);
#pragma unroll
                for (int e = 0; e < 8; e++) b[i][e] = have && u0 + i < nu ? (T)x[e] : (T)0.f;
            }
#pragma unroll
            for (int i = 0; i < UN; i++) acc = mfma32(a[i], b[i], acc);
        }
        if (have) {
            typename Dt<T>::quad o;
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] = (T)acc[i];
            *reinterpret_cast<typename Dt<T>::quad*>(q_abs + ((size_t)(m0 + c) * d.heads + head) * kl + rt * 16 + 4 * g) = o;
        }
        return;
    }
    const uint32_t m = m0 + (blockIdx.x - n_abs) / per_row, part = (blockIdx.x - n_abs) % per_row;
    if (m >= p.rows.m) return;
    const uint32_t pos = row_pos(p.rows, m), half = d.rot_dims >> 1;
    const float* cs = p.cos_t + (size_t)pos * half;
    const float* sn = p.sin_t + (size_t)pos * half;
    const float* row = p.qkv + (size_t)m * p.ld_qkv;
    if (part) {
#pragma unroll
        for (int k = 0; k < 4; k++) {
            const uint32_t i = (part - 1) * 1024 + k * 256 + tid;
            if (i >= d.heads * d.rot_p) break;
            const uint32_t head = i / d.rot_p, j = i % d.rot_p;
            q_abs[((size_t)m * d.heads + head) * kl + d.rank_p + j] =
                (T)(j < d.rot ? rotated(row + head * qh + d.dim_p, j, d.rot_dims, cs, sn) : 0.f);
        }
        return;
    }
    const float* lat = row + d.heads * qh;
    __shared__ float red[4];
    float ss = 0.f;
    for (uint32_t i = tid; i < d.rank; i += 256) ss = fmaf(lat[i], lat[i], ss);
    ss = wave_sum_f32(ss);
    if (lane == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)d.rank + d.eps);
    T* dst = reinterpret_cast<T*>(p.cache) + kv_row(p.kv, row_seq(p.rows, m), 0, 0, pos) * p.ld;
    for (uint32_t i = tid; i < kl; i += 256) {
        float v = 0.f;
        if (i < d.rank) v = lat[i] * inv * p.c_norm[i];
        else if (i >= d.rank_p && i - d.rank_p < d.rot) v = rotated(lat + d.rank_p, i - d.rank_p, d.rot_dims, cs, sn);
        dst[i] = (T)v;
    }
}

// ---------------------------------------------------------------------------
// Merge of one head's splits - the sink joins the denominator here, once - and the value product W_uv (sum p c).
// Grid (head, token row), 8 waves, a tile of 16 value rows each; UN units of the product's weights are in flight per wave.
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(512) void latent_merge_kernel(OxbLatentParams p) {
    typedef typename Dt<T>::frag frag;
    constexpr int UN = 8;
    extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
    __shared__ float wgt[OXB_MAX_SPLITS];
    const OxbLatentDims& d = p.d;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, c = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t head = blockIdx.x, m = blockIdx.y, ht = head / 16, col = head % 16, n_ht = (d.heads + 15) / 16;
    const uint32_t used = oxb_used_splits(row_pos(p.rows, m), p.n_splits);
    const size_t slot0 = ((size_t)m * n_ht + ht) * p.n_splits;
    const float sink = p.sink[head] * 1.4426950408889634f;   // (maxima are in units of log2(e))
    const uint32_t nu = p.k_uv / 32, tiles = d.vdim_p / 16;
    const size_t ts = oxb_tile_stride(p.k_uv, sizeof(T));
    const T* w_head = reinterpret_cast<const T*>(p.w_uv) + head * tiles * ts;
    frag a0[UN];   // the wave's first weights travel while the splits are merged
#pragma unroll
    for (int i = 0; i < UN; i++) a0[i] = load_unit(w_head + min(wave, tiles - 1) * ts + (size_t)min((uint32_t)i, nu - 1) * 512, lane);
    T* lat = reinterpret_cast<T*>(smem);  // [k_uv]
    {
        // every wave forms the weights (at most two splits per lane); wave 0 leaves them in LDS
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
        if (wave == 0) {
#pragma unroll
            for (int i = 0; i < 2; i++)
                if (lane + 64 * i < used) wgt[lane + 64 * i] = w[i] / L;
        }
    }
    __syncthreads();
    // four consecutive latent elements per thread; the threads beyond rank_p / 4 take further shares of the splits
    {
        const float* po = p.part_o + (slot0 * 16 + col) * d.rank_p;
        const uint32_t cols = d.rank_p / 4, shares = 512 / cols > 8 ? 8 : (512 / cols ? 512 / cols : 1), share = tid / cols;
        float* sums = reinterpret_cast<float*>(smem + p.k_uv * sizeof(T));   // [shares][rank_p]
        for (uint32_t c0 = 0; c0 < cols; c0 += 512) {
            const uint32_t i = shares > 1 ? tid % cols : c0 + tid;
            if (i < cols && share < shares) {
                v4f y = {0.f, 0.f, 0.f, 0.f};
                for (uint32_t s0 = shares > 1 ? share : 0; s0 < used; s0 += 8 * shares) {
                    v4f v[8];
#pragma unroll
                    for (int k = 0; k < 8; k++) v[k] = *reinterpret_cast<const v4f*>(po + (size_t)min(s0 + k * shares, used - 1) * 16 * d.rank_p + 4 * i);
#pragma unroll
                    for (int k = 0; k < 8; k++)
                        if (s0 + k * shares < used) y += v[k] * wgt[s0 + k * shares];
                }
                *reinterpret_cast<v4f*>(sums + (shares > 1 ? share : 0) * d.rank_p + 4 * i) = y;
            }
        }
        __syncthreads();
        for (uint32_t i = tid; i < p.k_uv; i += 512) {
            float y = 0.f;
            if (i < d.rank_p)
                for (uint32_t k = 0; k < shares; k++) y += sums[k * d.rank_p + i];
            lat[i] = (T)y;
        }
    }
    __syncthreads();
    T* out = reinterpret_cast<T*>(p.out) + (size_t)m * p.ld_out;
    for (uint32_t t = wave; t < tiles; t += 8) {
        const T* w = w_head + t * ts;
        v4f acc = {0.f, 0.f, 0.f, 0.f};
        for (uint32_t u0 = 0; u0 < nu; u0 += UN) {
            if (u0 || t != wave) {
#pragma unroll
                for (int i = 0; i < UN; i++) a0[i] = load_unit(w + (size_t)min(u0 + i, nu - 1) * 512, lane);
            }
#pragma unroll
            for (int i = 0; i < UN; i++) {
                const frag b = c == 0 && u0 + i < nu ? load_row8(lat + 32 * min(u0 + i, nu - 1) + 8 * g) : zero_frag((const T*)nullptr);
                acc = mfma32(a0[i], b, acc);
            }
        }
        if (c == 0) {
            typename Dt<T>::quad o;
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] = (T)acc[i];
            *reinterpret_cast<typename Dt<T>::quad*>(out + head * d.vdim_p + t * 16 + 4 * g) = o;
        }
    }
    if (head == d.heads - 1)
        for (uint32_t i = d.heads * d.vdim_p + tid; i < p.ld_out; i += 512) out[i] = (T)0.f;
}

// ---------------------------------------------------------------------------
// Expanded attention: a wave owns 16 QT queries of one head, the four waves of a workgroup take consecutive query tiles
// and share the keys and values of each 32-key block through LDS (two buffers if they fit; memory -> LDS copies of block
// i + 1 run under block i).  Keys enter the score product in the order that leaves lane (query, g) with keys
// 8 g .. 8 g + 7 of the block - row 4 a + v of key tile t is key 8 a + 4 t + v - which is exactly the k order in which
// the transposed values are read, 16 bytes per lane.
// ---------------------------------------------------------------------------
template <typename T, int QT, int KS, int VT>
__global__ __launch_bounds__(256, QT == 2 && !Dt<T>::is_f32 ? 2 : 1) void latent_prefill_kernel(OxbLatentParams p, uint32_t n_buf) {
    typedef typename Dt<T>::frag frag;
    constexpr int NU = (2 * KS + VT + 3) / 4;   // units a wave brings in per block, at most
    constexpr float kLazy = 8.0f;               // the running maximum follows once it is 2^8 behind
    extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
    const OxbLatentDims& d = p.d;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, qi = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t n_qb = (p.rows.m + 64 * QT - 1) / (64 * QT);
    const uint32_t qb = n_qb - 1 - blockIdx.x / d.heads, head = blockIdx.x % d.heads;   // long (late) query blocks first
    const uint32_t kd = d.dim_p / 32, kr = d.rot_p / 32, ks = kd + kr, vt = d.vdim_p / 16;
    const uint32_t kl = d.rank_p + d.rot_p, qh = d.dim_p + d.rot_p, half = d.rot_dims >> 1;
    const uint32_t units = 2 * ks + vt, slot = staged_slot(qi, g), sr = stage_row(lane), sc = 8 * stage_col(lane);
    T* lds = reinterpret_cast<T*>(smem);
    const T* cache = reinterpret_cast<const T*>(p.cache);
    const uint32_t q_last = min((qb + 1) * 64 * QT, p.rows.m) - 1;
    const uint32_t kv_len = p.rows.pos0 + q_last + 1;   // keys the workgroup's last query sees
    const float c2 = d.scale * 1.4426950408889634f;

    // Unit un of a block: key tile un / ks, k unit un % ks for the first 2 ks; value tile un - 2 ks behind them.  A wave
    // keeps one running address per unit it brings in.  (Keys past the last one are whatever lies behind it in its buffer or
    // page, inside the allocation: their scores are masked.)
    const T* src[NU];
    uint32_t step[NU], rot_key[NU];             // rot_key: the unit comes out of a paged cache, by key
    const bool paged = p.kv.page_table != nullptr;
#pragma unroll
    for (int i = 0; i < NU; i++) {
        const uint32_t un = wave + 4 * i;
        src[i] = nullptr;
        step[i] = rot_key[i] = 0;
        if (un >= units) continue;
        if (un < 2 * ks) {
            const uint32_t t = un >= ks ? 1u : 0u, s = un - t * ks, key = 8 * (sr >> 2) + 4 * t + (sr & 3u);
            if (s < kd) {
                src[i] = reinterpret_cast<const T*>(p.k_exp) + (size_t)key * p.ld_k + head * d.dim_p + 32 * s + sc;
                step[i] = 32 * p.ld_k;
            } else {
                src[i] = cache + d.rank_p + 32 * (s - kd) + sc;
                if (paged) rot_key[i] = key + 1;
                else src[i] += kv_row(p.kv, p.rows.seq0, 0, 0, key) * kl, step[i] = 32 * kl;
            }
        } else {
            src[i] = reinterpret_cast<const T*>(p.v_exp_t) + (size_t)(head * d.vdim_p + (un - 2 * ks) * 16 + sr) * p.ld_v + sc;
            step[i] = 32;
        }
    }
    auto stage = [&](uint32_t key0, uint32_t buf) {
        T* base = lds + ((size_t)buf * units + wave) * 512;
#pragma unroll
        for (int i = 0; i < NU; i++) {
            if (wave + 4 * i >= units) break;
            const T* a = src[i];
            if (paged && rot_key[i]) a += kv_row(p.kv, p.rows.seq0, 0, 0, key0 + rot_key[i] - 1) * kl;
            stage_unit(a, base + (size_t)i * 2048);
            src[i] += step[i];
        }
    };
    stage(0, 0);

    // queries of this wave, rotated, in operand order; rows past the end repeat the last one and are not stored
    frag q[QT][KS];
    uint32_t qpos[QT];
#pragma unroll
    for (int t = 0; t < QT; t++) {
        const uint32_t row = min(qb * 64 * QT + (wave * QT + t) * 16 + qi, p.rows.m - 1);
        qpos[t] = p.rows.pos0 + row;
        const float* qs = p.qkv + (size_t)row * p.ld_qkv + head * qh;
        const float* cs = p.cos_t + (size_t)qpos[t] * half;
        const float* sn = p.sin_t + (size_t)qpos[t] * half;
#pragma unroll
        for (int s = 0; s < KS; s++) {
            q[t][s] = zero_frag((const T*)nullptr);
            if ((uint32_t)s >= ks) continue;
            if ((uint32_t)s < kd) {
                const v8f x = load_row8(qs + 32 * s + 8 * g);
#pragma unroll
                for (int e = 0; e < 8; e++) q[t][s][e] = (T)x[e];
            } else {
                const float* rp = qs + d.dim_p;
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const uint32_t i = 32 * (s - kd) + 8 * g + e;
                    q[t][s][e] = (T)(i < d.rot ? rotated(rp, i, d.rot_dims, cs, sn) : 0.f);
                }
            }
        }
    }
    const uint32_t q_first = p.rows.pos0 + min(qb * 64 * QT + wave * QT * 16, p.rows.m - 1);   // blocks up to here are wholly visible to the wave
    v4f O[QT][VT];
    float m_run[QT], l_run[QT];   // maximum (times c2) and this lane's share of the sum
#pragma unroll
    for (int t = 0; t < QT; t++) {
        m_run[t] = -INFINITY, l_run[t] = 0.f;
#pragma unroll
        for (int i = 0; i < VT; i++) O[t][i] = (v4f){0.f, 0.f, 0.f, 0.f};
    }
    uint32_t buf = 0;
    for (uint32_t key0 = 0; key0 < kv_len; key0 += 32) {
        wait_lds_copies();
        __syncthreads();
        if (n_buf > 1 && key0 + 32 < kv_len) stage(key0 + 32, buf ^ 1u);
        const T* kb = lds + (size_t)buf * units * 512;
        const T* vb = kb + (size_t)2 * ks * 512;
        v4f s0[QT], s1[QT];
#pragma unroll
        for (int t = 0; t < QT; t++) s0[t] = s1[t] = (v4f){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s2 = 0; s2 < KS; s2 += 2)
            if ((uint32_t)s2 < ks) {
#pragma unroll
                for (int j = 0; j < 2; j++) {
                    const uint32_t s = min((uint32_t)(s2 + j), ks - 1);   // (past the end: against zero queries)
                    const frag k0 = load_staged(kb + (size_t)s * 512, slot), k1 = load_staged(kb + (size_t)(ks + s) * 512, slot);
#pragma unroll
                    for (int t = 0; t < QT; t++) {
                        s0[t] = mfma32(k0, q[t][s2 + j], s0[t]);
                        s1[t] = mfma32(k1, q[t][s2 + j], s1[t]);
                    }
                }
            }
        const bool whole = key0 + 31 <= q_first;
        float sv[QT][8];
        bool behind = false;
#pragma unroll
        for (int t = 0; t < QT; t++) {
            float mx = -INFINITY;
#pragma unroll
            for (int e = 0; e < 8; e++) {
                sv[t][e] = (e < 4 ? s0[t][e & 3] : s1[t][e & 3]) * c2;
                if (!whole && key0 + 8 * g + e > qpos[t]) sv[t][e] = -INFINITY;
                mx = fmaxf(mx, sv[t][e]);
            }
            s0[t][0] = mx = max_rows4(mx);
            behind |= mx > m_run[t] + kLazy;   // (the first block: key 0 is visible to every query, -inf is behind)
        }
        if (__any(behind)) {
#pragma unroll
            for (int t = 0; t < QT; t++) {
                const float m_new = fmaxf(m_run[t], s0[t][0]), alpha = exp2_of<T>(m_run[t] - m_new);
                m_run[t] = m_new;
                l_run[t] *= alpha;
#pragma unroll
                for (int i = 0; i < VT; i++) O[t][i] *= alpha;
            }
        }
        frag hi[QT], lo[QT];
#pragma unroll
        for (int t = 0; t < QT; t++) {
            float pe[8];
#pragma unroll
            for (int e = 0; e < 8; e++) {
                pe[e] = exp2_of<T>(sv[t][e] - m_run[t]);
                l_run[t] += pe[e];
            }
            split_hi_lo(pe, hi[t], lo[t]);
        }
#pragma unroll
        for (int i2 = 0; i2 < VT; i2 += 2)
            if ((uint32_t)i2 < vt) {   // (vt is even)
#pragma unroll
                for (int j = 0; j < 2; j++) {
                    const frag a = load_staged(vb + (size_t)(i2 + j) * 512, slot);
#pragma unroll
                    for (int t = 0; t < QT; t++) {
                        O[t][i2 + j] = mfma32(a, hi[t], O[t][i2 + j]);
                        if constexpr (!Dt<T>::is_f32) O[t][i2 + j] = mfma32(a, lo[t], O[t][i2 + j]);
                    }
                }
            }
        if (n_buf > 1) {
            buf ^= 1u;
        } else if (key0 + 32 < kv_len) {
            __syncthreads();
            stage(key0 + 32, 0);
        }
    }
    const float sink = p.sink[head] * 1.4426950408889634f;
#pragma unroll
    for (int t = 0; t < QT; t++) {
        const uint32_t row = qb * 64 * QT + (wave * QT + t) * 16 + qi;
        const float l = sum_rows4(l_run[t]);
        if (row >= p.rows.m) continue;
        const float M = fmaxf(m_run[t], sink), f = exp2_of<T>(m_run[t] - M);
        const float inv = f / (l * f + exp2_of<T>(sink - M));
        T* o = reinterpret_cast<T*>(p.out) + (size_t)row * p.ld_out + head * d.vdim_p + 4 * g;
#pragma unroll
        for (int i = 0; i < VT; i++)
            if ((uint32_t)i < vt) {
                typename Dt<T>::quad w;
#pragma unroll
                for (int v = 0; v < 4; v++) w[v] = (T)(O[t][i][v] * inv);
                *reinterpret_cast<typename Dt<T>::quad*>(o + 16 * i) = w;
            }
        if (head == d.heads - 1)
            for (uint32_t i = d.heads * d.vdim_p + g; i < p.ld_out; i += 4) reinterpret_cast<T*>(p.out)[(size_t)row * p.ld_out + i] = (T)0.f;
    }
}

// ---------------------------------------------------------------------------
static constexpr uint32_t kLdsMax = 160u << 10;

static uint32_t prefill_block_bytes(const OxbLatentDims& d, int dt) {
    return (2 * (d.dim_p + d.rot_p) / 32 + d.vdim_p / 16) * 512 * oxb_dt_bytes(dt);
}
const char* oxb_latent_check(const OxbLatentDims& d, int dt) {
    if (!d.heads || !d.dim || !d.rot || !d.rank || !d.vdim) return "a latent attention size is 0";
    if (d.rot_dims > d.rot || d.rot_dims % 2) return "rotated dimensions must be even and within the rotated part";
    if (d.rank > 1024 || d.rot > 128) return "latent size beyond 1024 or rotated part beyond 128";
    if (d.dim_p + d.rot_p > 512 || d.vdim > 512) return "head size beyond 512";
    if (const char* why = oxb_row_check((d.rank_p + d.rot_p) / 32, dt)) return why;
    if (prefill_block_bytes(d, dt) > kLdsMax) return "a block of keys and values exceeds the LDS";
    return nullptr;
}

static bool rows_ok(const OxbLatentParams& p) {
    const OxbLatentDims& d = p.d;
    return p.rows.m && p.cache && p.qkv && p.cos_t && p.sin_t && p.c_norm && p.sink && p.ld == d.rank_p + d.rot_p &&
           p.ld_qkv >= d.heads * (d.dim_p + d.rot_p) + d.rank_p + d.rot_p && p.kv.n_layers == 1 && p.kv.nkv == 1 &&
           (!p.kv.page_table || (p.kv.page_shift >= 4 && p.kv.page_shift <= 7));
}

hipError_t oxb_launch_latent_store(const OxbLatentParams& p, bool absorb, int dt, hipStream_t st) {
    if (!rows_ok(p) || (absorb && (!p.q_abs || !p.w_uk_t || p.k_uk < p.d.dim_p || p.k_uk % 32))) return hipErrorInvalidValue;
    OxbLatentParams q = p;
    if (!absorb) q.q_abs = nullptr;
    const uint32_t tph = p.d.rank_p / 16, n_abs = absorb ? (p.d.heads * tph + 3) / 4 : 0;
    const uint32_t per_row = absorb ? 1 + (p.d.heads * p.d.rot_p + 1023) / 1024 : 1;
    const dim3 grid(n_abs + per_row * (p.rows.m < 16 ? p.rows.m : 16), (p.rows.m + 15) / 16);
    if (dt == OXB_DT_BF16) hipLaunchKernelGGL((latent_store_kernel<__bf16>), grid, dim3(256), 0, st, q, n_abs, tph, per_row);
    else hipLaunchKernelGGL((latent_store_kernel<float>), grid, dim3(256), 0, st, q, n_abs, tph, per_row);
    return hipGetLastError();
}

hipError_t oxb_launch_latent_decode(const OxbLatentParams& p, int dt, hipStream_t st) {
    if (!rows_ok(p) || oxb_latent_check(p.d, dt) || !p.q_abs) return hipErrorInvalidValue;
    OxbRowAttnParams a;
    memset(&a, 0, sizeof a);
    a.rows = p.rows;
    a.kv = p.kv;
    a.q = p.q_abs;
    a.heads = a.rep = p.d.heads;
    a.cache = p.cache;
    a.ld = p.ld;
    a.ks = p.ld / 32;
    a.nt = p.d.rank_p / 16;
    a.scale = p.d.scale;
    a.sink = p.sink;
    a.part_o = p.part_o;
    a.part_ml = p.part_ml;
    a.n_splits = p.n_splits;
    return oxb_launch_row_decode(a, oxb_latent_head_tiles(p.d, p.rows.m), dt, st);
}

hipError_t oxb_launch_latent_merge(const OxbLatentParams& p, int dt, hipStream_t st) {
    if (!rows_ok(p) || !p.part_o || !p.part_ml || !p.out || !p.w_uv || p.k_uv < p.d.rank_p || p.k_uv % 32 || p.ld_out < p.d.heads * p.d.vdim_p ||
        !p.n_splits || p.n_splits > OXB_MAX_SPLITS)
        return hipErrorInvalidValue;
    const dim3 grid(p.d.heads, p.rows.m);
    const uint32_t cols = p.d.rank_p / 4, shares = 512 / cols > 8 ? 8 : 512 / cols ? 512 / cols : 1;
    const uint32_t lds = p.k_uv * oxb_dt_bytes(dt) + shares * p.d.rank_p * 4;
    if (dt == OXB_DT_BF16) hipLaunchKernelGGL((latent_merge_kernel<__bf16>), grid, dim3(512), lds, st, p);
    else hipLaunchKernelGGL((latent_merge_kernel<float>), grid, dim3(512), lds, st, p);
    return hipGetLastError();
}

template <typename T, int QT, int KS, int VT>
static hipError_t launch_prefill(const OxbLatentParams& p, uint32_t block_bytes, hipStream_t st) {
    const uint32_t n_buf = 2 * block_bytes <= kLdsMax ? 2u : 1u, n_qb = (p.rows.m + 64 * QT - 1) / (64 * QT);
    hipLaunchKernelGGL((latent_prefill_kernel<T, QT, KS, VT>), dim3(n_qb * p.d.heads), dim3(256), n_buf * block_bytes, st, p, n_buf);
    return hipGetLastError();
}

template <typename T>
static hipError_t pick_prefill(const OxbLatentParams& p, uint32_t bytes, hipStream_t st) {
    const uint32_t ks = (p.d.dim_p + p.d.rot_p) / 32, vt = p.d.vdim_p / 16;
    if (ks <= 4 && vt <= 8) return launch_prefill<T, 2, 4, 8>(p, bytes, st);
    if (ks <= 6 && vt <= 8) return launch_prefill<T, 2, 6, 8>(p, bytes, st);
    if (ks <= 8 && vt <= 16) return launch_prefill<T, 1, 8, 16>(p, bytes, st);
    return launch_prefill<T, 1, 16, 32>(p, bytes, st);
}

// Dynamic LDS beyond 64 KB has to be asked for, per kernel; done ahead of any launch so that none has to do it inside a
// stream capture.
template <typename T>
static hipError_t raise_lds() {
    const void* prefill[] = {(const void*)&latent_prefill_kernel<T, 2, 4, 8>, (const void*)&latent_prefill_kernel<T, 2, 6, 8>,
                             (const void*)&latent_prefill_kernel<T, 1, 8, 16>, (const void*)&latent_prefill_kernel<T, 1, 16, 32>};
    hipError_t e = hipSuccess;
    for (const void* f : prefill)
        if (e == hipSuccess) e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsMax);
    return e;
}
hipError_t oxb_latent_prepare(int dt) {
    const hipError_t e = oxb_row_attention_prepare(dt);
    if (e != hipSuccess) return e;
    return dt == OXB_DT_BF16 ? raise_lds<__bf16>() : raise_lds<float>();
}

hipError_t oxb_launch_latent_prefill(const OxbLatentParams& p, int dt, hipStream_t st) {
    if (!rows_ok(p) || oxb_latent_check(p.d, dt) || p.rows.pos || p.rows.seq_step || !p.k_exp || !p.v_exp_t || !p.out ||
        p.ld_k < p.d.heads * p.d.dim_p || p.ld_v % 32 || p.ld_v < p.rows.pos0 + p.rows.m || p.ld_out < p.d.heads * p.d.vdim_p)
        return hipErrorInvalidValue;
    const uint32_t bytes = prefill_block_bytes(p.d, dt);
    return dt == OXB_DT_BF16 ? pick_prefill<__bf16>(p, bytes, st) : pick_prefill<float>(p, bytes, st);
}
