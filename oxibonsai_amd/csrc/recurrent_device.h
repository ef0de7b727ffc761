// recurrent_device.h — device bodies of the recurrences' step and finish, shared by the kernels that launch them alone and
// beside attention.
#pragma once
#include "dense_device.h"
#include "recurrent_kernels.h"

// z / (1 + e^-z) on the hardware exponential and reciprocal (a few ulp where the result is not negligible beside z).
__device__ __forceinline__ float silu_of(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.4426950408889634f)); }
__device__ __forceinline__ float softplus_of(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ v4f load4(const float* p) { return *reinterpret_cast<const v4f*>(p); }

// Short convolution and its activation: channel ch of the token in row `row` of the input product, at position pos; `back`
// earlier rows of the same sequence lie in front of it there, older inputs in the ring.
__device__ __forceinline__ float conv_of(const OxbRecurParams& p, const float* ring, uint32_t row, uint32_t back, uint32_t pos, uint32_t ch) {
    // (bases are the same for all lanes, the channel is every load's offset)
    const OxbRecurDims& d = p.d;
    const float* x = p.lin + (size_t)row * p.ld_lin + d.col_conv;
    const float* w = p.conv_w + (size_t)(d.taps - 1) * d.channels;
    const uint32_t n = min(d.taps - 1, pos);   // inputs there are behind this one
    auto past = [&](uint32_t j) {   // (no branch around the loads: they all travel together)
        const uint32_t k = min(j, n);
        const float* at = k <= back ? x - (size_t)k * p.ld_lin : ring + (size_t)((pos - k) & (d.ring - 1u)) * d.channels;
        const float y = at[ch] * (w - (size_t)k * d.channels)[ch];
        return j <= n ? y : 0.f;
    };
    const float x0 = x[ch] * w[ch], x1 = past(1), x2 = past(2), x3 = past(3);
    float v = (p.conv_b ? p.conv_b[ch] : 0.f) + x0 + x1 + x2 + x3;
#pragma unroll 1
    for (uint32_t j = 4; j <= n; j++) v += past(j);
    return silu_of(v);
}

// Logarithm of the decay and beta of one head from its columns of the input product.
__device__ __forceinline__ void gates_of(const OxbRecurParams& p, uint32_t row, uint32_t head, float* la, float* beta) {
    const float* x = p.lin + (size_t)row * p.ld_lin;
    const float sp = softplus_of(x[p.d.col_a + head] + p.dt_bias[head]);
    *la = p.neg_a[head] * sp;
    *beta = p.d.delta ? 1.0f / (1.0f + expf(-x[p.d.col_b + head])) : sp;
}

// ---------------------------------------------------------------------------
// Step.  Workgroup (hb, sb): head x slice group, sequence; 256 threads per slice of 32 columns.  Thread (rg, cl) = (tid / 8 %
// 32, tid % 8) holds rows rg + 32 j and columns 4 cl .. + 3 of its slice of the state.  S^T k and S^T q come out of the state as
// it was, in one pass: with the write k u^T, o = a (S^T q) + (k . q) u.  With every slice of a head in the workgroup (FINISH) the
// head's output is gated and normed here as well.
// ---------------------------------------------------------------------------
template <typename T, int RPT, int SL, bool FINISH, bool ONE>
__device__ __forceinline__ void recur_step(const OxbRecurParams& p, uint32_t n_tokens, uint32_t hb, uint32_t sb) {
    const OxbRecurDims& d = p.d;
    const uint32_t tokens = ONE ? 1 : n_tokens;
    __shared__ __attribute__((aligned(16))) float conv[512 + 32 * SL], os[32 * SL];   // queries, keys, values behind their convolutions
    __shared__ __attribute__((aligned(16))) float part[4 * SL][8][8];
    __shared__ float gates[2];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, cl = tid & 7u, rg = (tid >> 3) & 31u;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6)), mine = wave >> 2;   // slice of the workgroup's
    const uint32_t groups = (d.slices + SL - 1) / SL, head = hb / groups, slice = hb % groups * SL + mine;
    const uint32_t row0 = sb * tokens, rep = d.heads / d.qk_heads, qk = head / rep, pos0 = row_pos(p.rows, row0);
    float* mem = p.memory + (size_t)row_seq(p.rows, row0) * p.seq_stride;
    float* state = mem + ((size_t)head * d.slices + min(slice, d.slices - 1)) * d.dk_p * 32 + rg * 32 + 4 * cl;
    float* ring = mem + oxb_recur_state(d);
    v4f s[RPT];
#pragma unroll
    for (int j = 0; j < RPT; j++) s[j] = load4(state + min(1024u * j, (d.dk_p - 32) * 32));
    const bool own_qk = head % rep == 0 && hb % groups == 0;
    const float *qs = conv, *ks = conv + d.dk_p, *vs = conv + 2 * d.dk_p;
    const uint32_t n_conv = 2 * d.dk_p + 32 * SL, vcol = hb % groups * SL * 32;
    constexpr int ROUNDS = (512 + 32 * SL + 256 * SL - 1) / (256 * SL);
    for (uint32_t t = 0; t < tokens; t++) {
        const uint32_t row = row0 + t, pos = pos0 + t;
        const float* lin = p.lin + (size_t)row * p.ld_lin;
        // the last wave forms the gates, the one before it what the finished output is multiplied by: neither has much of the
        // convolutions to do
        constexpr uint32_t GATES = 4 * SL - 1, LAST = 4 * SL - 2;
        constexpr int E = (SL + 1) / 2;
        float gate[E];
        if constexpr (FINISH) {
            if (wave == LAST) {
#pragma unroll
                for (int e = 0; e < E; e++) {
                    const uint32_t i = min(lane + 64 * e, d.dv - 1);
                    gate[e] = p.norm_w[i] * silu_of(lin[d.col_z + head * d.dv + i]);
                }
            }
        }
        if (wave == GATES) {
            float la, beta;
            gates_of(p, row, head, &la, &beta);
            if (lane == 0) gates[0] = expf(la), gates[1] = beta;
        }
#pragma unroll
        for (int k = 0; k < ROUNDS; k++) {
            const uint32_t it = tid + 256 * SL * k;
            if (it >= n_conv) break;
            const bool is_v = it >= 2 * d.dk_p, is_k = !is_v && it >= d.dk_p;
            const uint32_t i = is_v ? it - 2 * d.dk_p + vcol : is_k ? it - d.dk_p : it, len = is_v ? d.dv : d.dk;
            const uint32_t ch = (is_v ? d.ch_v + head * d.dv : (is_k ? d.ch_k : d.ch_q) + qk * d.dk) + i;
            conv[it] = i < len ? conv_of(p, ring, row, t, pos, ch) : 0.f;
            // inputs that later tokens convolve
            if (d.taps > 1 && t + d.taps > tokens && i < len && (is_v || own_qk)) ring[(size_t)(pos & (d.ring - 1u)) * d.channels + ch] = lin[d.col_conv + ch];
        }
        if (t == 0) {
#pragma unroll
            for (int j = 0; j < RPT; j++)
                if (!pos0) s[j] = (v4f){0.f, 0.f, 0.f, 0.f};
        }
        __syncthreads();
        const float a = gates[0], beta = gates[1];
        float qq = 0.f, kk = 0.f, kq = 0.f;   // (every wave for itself)
        #pragma unroll 1
        for (uint32_t i = lane; i < d.dk_p; i += 64) {
            const float q = qs[i], k = ks[i];
            qq = fmaf(q, q, qq), kk = fmaf(k, k, kk), kq = fmaf(k, q, kq);
        }
        float rq = 1.0f, rk = 1.0f;
        if (d.delta) {
            rq = d.q_scale / sqrtf(wave_sum_f32(qq) + 1e-6f);
            rk = 1.0f / sqrtf(wave_sum_f32(kk) + 1e-6f);
        }
        const float dot = wave_sum_f32(kq) * rq * rk;
        v4f sk = {0.f, 0.f, 0.f, 0.f}, sq = sk;
#pragma unroll
        for (int j = 0; j < RPT; j++)
            if (32u * j < d.dk_p) {
                sk += s[j] * ks[rg + 32 * j];
                sq += s[j] * qs[rg + 32 * j];
            }
#pragma unroll
        for (int i = 0; i < 4; i++) {   // over the wave's eight row groups
            sk[i] = sum_rows4(sk[i] + dpp_f32<0x128>(sk[i]));
            sq[i] = sum_rows4(sq[i] + dpp_f32<0x128>(sq[i]));
        }
        if (lane < 8) {
            *reinterpret_cast<v4f*>(&part[wave][cl][0]) = sk;
            *reinterpret_cast<v4f*>(&part[wave][cl][4]) = sq;
        }
        __syncthreads();
        const uint32_t w0 = 4 * mine;
        sk = load4(&part[w0][cl][0]) + load4(&part[w0 + 1][cl][0]) + load4(&part[w0 + 2][cl][0]) + load4(&part[w0 + 3][cl][0]);
        sq = load4(&part[w0][cl][4]) + load4(&part[w0 + 1][cl][4]) + load4(&part[w0 + 2][cl][4]) + load4(&part[w0 + 3][cl][4]);
        const v4f v = load4(&vs[32 * mine + 4 * cl]);
        const v4f u = d.delta ? (v - sk * (a * rk)) * beta : v * beta, uk = u * rk;
#pragma unroll
        for (int j = 0; j < RPT; j++)
            if (32u * j < d.dk_p) s[j] = s[j] * a + uk * ks[rg + 32 * j];
        if (rg == 0) {
            v4f o = sq * (a * rq) + u * dot;
            if (p.skip) o += v * p.skip[head];
            if constexpr (FINISH) {
                *reinterpret_cast<v4f*>(&os[32 * mine + 4 * cl]) = o;
            } else {
                float* dst = p.o + (size_t)row * d.heads * d.dv + head * d.dv + slice * 32 + 4 * cl;
#pragma unroll
                for (int i = 0; i < 4; i++)
                    if (slice * 32 + 4 * cl + i < d.dv) dst[i] = o[i];
            }
        }
        if (FINISH || t + 1 < tokens) __syncthreads();
        if constexpr (FINISH) {
            if (wave == LAST) {
                float y[E], ss = 0.f;
#pragma unroll
                for (int e = 0; e < E; e++) {
                    y[e] = lane + 64 * e < d.dv ? os[lane + 64 * e] : 0.f;
                    ss = fmaf(y[e], y[e], ss);
                }
                const float inv = d.out_scale / sqrtf(wave_sum_f32(ss) / (float)d.dv + d.eps);
                T* out = reinterpret_cast<T*>(p.out) + (size_t)row * p.ld_out + p.out_col;
#pragma unroll
                for (int e = 0; e < E; e++)
                    if (lane + 64 * e < d.dv) out[head * d.dv + lane + 64 * e] = (T)(y[e] * inv * gate[e]);
                if (head == 0)
                    for (uint32_t i = d.heads * d.dv + lane; i < p.out_fill; i += 64) out[i] = (T)0.f;
            }
        }
    }
    if (slice < d.slices) {
#pragma unroll
        for (int j = 0; j < RPT; j++)
            if (32u * j < d.dk_p) *reinterpret_cast<v4f*>(state + 1024 * j) = s[j];
    }
}

// ---------------------------------------------------------------------------
// Finish: gate and norm of each part of a row's outputs, values in registers.  Short parts (E values per lane): a wave per
// part, ROWS rows each.  Long ones: 1024 threads per part, eight values each (parts beyond 8192 are read again).
// ---------------------------------------------------------------------------
__device__ __forceinline__ void keep_inputs(const OxbRecurParams& p, uint32_t back, uint32_t first, uint32_t step) {
    const uint32_t row = p.rows.m - 1 - back, pos = p.rows.pos0 + row;
    float* keep = p.memory + (size_t)p.rows.seq0 * p.seq_stride + oxb_recur_state(p.d) + (size_t)(pos & (p.d.ring - 1u)) * p.d.channels;
    const float* x = p.lin + (size_t)row * p.ld_lin + p.d.col_conv;
    for (uint32_t i = first; i < p.d.channels; i += step) keep[i] = x[i];
}

template <typename T, int E, int ROWS>
__device__ __forceinline__ void recur_finish(const OxbRecurParams& p, uint32_t rb, uint32_t pb) {
    const OxbRecurDims& d = p.d;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, inner = d.heads * d.dv, parts = inner / d.norm_len;
    const uint32_t row0 = rb * ROWS, part = pb * 4 + (tid >> 6);
    if (pb == 0)
        for (uint32_t t = 0; t < ROWS && row0 + t < p.rows.m; t++)
            for (uint32_t i = inner + tid; i < p.out_fill; i += 256) reinterpret_cast<T*>(p.out)[(size_t)(row0 + t) * p.ld_out + p.out_col + i] = (T)0.f;
    if (part >= parts) return;
    float o[ROWS][E], z[ROWS][E], w[E];
#pragma unroll
    for (int t = 0; t < ROWS; t++) {
        const uint32_t row = min(row0 + t, p.rows.m - 1);
#pragma unroll
        for (int e = 0; e < E; e++) {
            const uint32_t i = min(lane + 64 * e, d.norm_len - 1);
            o[t][e] = p.o[(size_t)row * inner + (size_t)part * d.norm_len + i];
            z[t][e] = p.lin[(size_t)row * p.ld_lin + d.col_z + (size_t)part * d.norm_len + i];
        }
    }
#pragma unroll
    for (int e = 0; e < E; e++) w[e] = p.norm_w[(d.norm_shared ? 0 : (size_t)part * d.norm_len) + min(lane + 64 * e, d.norm_len - 1)];
#pragma unroll
    for (int t = 0; t < ROWS; t++) {
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < E; e++) {
            z[t][e] = silu_of(z[t][e]);
            const float y = d.gate_first ? o[t][e] * z[t][e] : o[t][e];
            if (lane + 64 * e < d.norm_len) ss = fmaf(y, y, ss);
        }
        const float inv = d.out_scale / sqrtf(wave_sum_f32(ss) / (float)d.norm_len + d.eps);
        if (row0 + t >= p.rows.m) continue;
        T* out = reinterpret_cast<T*>(p.out) + (size_t)(row0 + t) * p.ld_out + p.out_col + (size_t)part * d.norm_len;
#pragma unroll
        for (int e = 0; e < E; e++)
            if (lane + 64 * e < d.norm_len) out[lane + 64 * e] = (T)(o[t][e] * inv * w[e] * z[t][e]);
    }
}

template <typename T> __device__ __forceinline__ void recur_finish_long(const OxbRecurParams& p, uint32_t row, uint32_t part) {
    constexpr int KEEP = 8;
    const OxbRecurDims& d = p.d;
    __shared__ float red[16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, inner = d.heads * d.dv;
    T* out = reinterpret_cast<T*>(p.out) + (size_t)row * p.ld_out + p.out_col;
    if (part == 0)
        for (uint32_t i = inner + tid; i < p.out_fill; i += 1024) out[i] = (T)0.f;
    const float* o = p.o + (size_t)row * inner + (size_t)part * d.norm_len;
    const float* z = p.lin + (size_t)row * p.ld_lin + d.col_z + (size_t)part * d.norm_len;
    const float* w = p.norm_w + (d.norm_shared ? 0 : (size_t)part * d.norm_len);
    float y[KEEP], g[KEEP], nw[KEEP], ss = 0.f;
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
        const uint32_t i = tid + 1024 * k;
        y[k] = g[k] = nw[k] = 0.f;
        if (i < d.norm_len) y[k] = o[i], g[k] = z[i], nw[k] = w[i];
    }
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
        g[k] = silu_of(g[k]);
        const float v = d.gate_first ? y[k] * g[k] : y[k];
        ss = fmaf(v, v, ss);
    }
    for (uint32_t i = tid + 1024 * KEEP; i < d.norm_len; i += 1024) {
        const float v = d.gate_first ? o[i] * silu_of(z[i]) : o[i];
        ss = fmaf(v, v, ss);
    }
    ss = wave_sum_f32(ss);
    if (lane == 0) red[tid >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int k = 0; k < 16; k++) ss += red[k];
    const float inv = d.out_scale / sqrtf(ss / (float)d.norm_len + d.eps);
    out += (size_t)part * d.norm_len;
#pragma unroll
    for (int k = 0; k < KEEP; k++)
        if (tid + 1024 * k < d.norm_len) out[tid + 1024 * k] = (T)(y[k] * inv * nw[k] * g[k]);
    for (uint32_t i = tid + 1024 * KEEP; i < d.norm_len; i += 1024) out[i] = (T)(o[i] * inv * w[i] * silu_of(z[i]));
}
