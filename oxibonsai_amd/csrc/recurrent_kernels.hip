// recurrent_kernels.hip — gated linear recurrences: step form, chunked form, output gate and norm (see recurrent_kernels.h).
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "dense_device.h"
#include "recurrent_kernels.h"

__device__ __forceinline__ float silu_of(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_of(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ v4f load4(const float* p) { return *reinterpret_cast<const v4f*>(p); }

// Short convolution and its activation: channel ch of the token in row `row` of the input product, at position pos; `back`
// earlier rows of the same sequence lie in front of it there, older inputs in the ring.
__device__ __forceinline__ float conv_of(const OxbRecurParams& p, const float* ring, uint32_t row, uint32_t back, uint32_t pos, uint32_t ch) {
    const OxbRecurDims& d = p.d;
    const float* w = p.conv_w + (size_t)ch * d.taps;
    const float* x = p.lin + (size_t)row * p.ld_lin + d.col_conv + ch;
    auto past = [&](uint32_t j) {
        const float* at = j <= back ? x - (size_t)j * p.ld_lin : ring + (size_t)((pos - j) & (d.ring - 1u)) * d.channels + ch;
        return *at * w[d.taps - 1 - j];
    };
    const uint32_t n = min(d.taps - 1, pos);   // inputs there are behind this one
    const float x0 = x[0] * w[d.taps - 1], x1 = n >= 1 ? past(1) : 0.f, x2 = n >= 2 ? past(2) : 0.f, x3 = n >= 3 ? past(3) : 0.f;
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
// Step.  Grid (head x slice group, sequence), 256 threads per slice of 32 columns: thread (rg, cl) = (tid / 8 % 32, tid % 8)
// holds rows rg + 32 j and columns 4 cl .. + 3 of its slice of the state.  S^T k and S^T q come out of the state as it was, in
// one pass: with the write k u^T, o = a (S^T q) + (k . q) u.  With every slice of a head in the workgroup (FINISH) the head's
// output is gated and normed here as well.
// ---------------------------------------------------------------------------
template <typename T, int RPT, int SL, bool FINISH, bool ONE>
__global__ __launch_bounds__(256 * SL, ONE && RPT <= 4 ? 8 : 4) void recur_step_kernel(OxbRecurParams p, uint32_t n_tokens) {
    const OxbRecurDims& d = p.d;
    const uint32_t tokens = ONE ? 1 : n_tokens;
    __shared__ __attribute__((aligned(16))) float qs[256], ks[256], vs[32 * SL], os[32 * SL];
    __shared__ __attribute__((aligned(16))) float part[4 * SL][8][8];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, cl = tid & 7u, rg = (tid >> 3) & 31u;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6)), mine = wave >> 2;   // slice of the workgroup's
    const uint32_t groups = (d.slices + SL - 1) / SL, head = blockIdx.x / groups, slice = blockIdx.x % groups * SL + mine;
    const uint32_t row0 = blockIdx.y * tokens, rep = d.heads / d.qk_heads, qk = head / rep, pos0 = row_pos(p.rows, row0);
    float* mem = p.memory + (size_t)row_seq(p.rows, row0) * p.seq_stride;
    float* state = mem + ((size_t)head * d.slices + min(slice, d.slices - 1)) * d.dk_p * 32 + rg * 32 + 4 * cl;
    float* ring = mem + oxb_recur_state(d);
    v4f s[RPT];
#pragma unroll
    for (int j = 0; j < RPT; j++) s[j] = pos0 && 32u * j < d.dk_p ? load4(state + 1024 * j) : (v4f){0.f, 0.f, 0.f, 0.f};
    const bool own_qk = head % rep == 0 && blockIdx.x % groups == 0;
    // which convolutions a thread brings: queries, keys, values in turn, spread over the workgroup
    const uint32_t qi = tid, ki = SL > 1 ? tid - 256u : tid, vi = SL > 2 ? tid - 512u : 256u * SL - 1 - tid;
    const uint32_t vcol = blockIdx.x % groups * SL * 32 + vi;
    for (uint32_t t = 0; t < tokens; t++) {
        const uint32_t row = row0 + t, pos = pos0 + t;
        const float* lin = p.lin + (size_t)row * p.ld_lin;
        float z[FINISH ? (SL + 1) / 2 : 1], nw[FINISH ? (SL + 1) / 2 : 1];
        if constexpr (FINISH) {
            if (wave == 0) {
#pragma unroll
                for (int e = 0; e < (SL + 1) / 2; e++) {
                    const uint32_t i = min(lane + 64 * e, d.dv - 1);
                    z[e] = lin[d.col_z + head * d.dv + i];
                    nw[e] = p.norm_w[i];
                }
            }
        }
        float la, beta;
        gates_of(p, row, head, &la, &beta);
        const float a = expf(la);
        if (qi < d.dk_p) qs[qi] = qi < d.dk ? conv_of(p, ring, row, t, pos, d.ch_q + qk * d.dk + qi) : 0.f;
        if (ki < d.dk_p) ks[ki] = ki < d.dk ? conv_of(p, ring, row, t, pos, d.ch_k + qk * d.dk + ki) : 0.f;
        if (vi < 32 * SL) vs[vi] = vcol < d.dv ? conv_of(p, ring, row, t, pos, d.ch_v + head * d.dv + vcol) : 0.f;
        if (d.taps > 1 && t + d.taps > tokens) {   // inputs that later tokens convolve
            float* keep = ring + (size_t)(pos & (d.ring - 1u)) * d.channels;
            const float* x = lin + d.col_conv;
            if (own_qk && qi < d.dk) keep[d.ch_q + qk * d.dk + qi] = x[d.ch_q + qk * d.dk + qi];
            if (own_qk && ki < d.dk) keep[d.ch_k + qk * d.dk + ki] = x[d.ch_k + qk * d.dk + ki];
            if (vi < 32 * SL && vcol < d.dv) keep[d.ch_v + head * d.dv + vcol] = x[d.ch_v + head * d.dv + vcol];
        }
        __syncthreads();
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
            if (wave == 0) {
                float y[(SL + 1) / 2], ss = 0.f;
#pragma unroll
                for (int e = 0; e < (SL + 1) / 2; e++) {
                    y[e] = lane + 64 * e < d.dv ? os[lane + 64 * e] : 0.f;
                    ss = fmaf(y[e], y[e], ss);
                }
                const float inv = d.out_scale / sqrtf(wave_sum_f32(ss) / (float)d.dv + d.eps);
                T* out = reinterpret_cast<T*>(p.out) + (size_t)row * p.ld_out + p.out_col;
#pragma unroll
                for (int e = 0; e < (SL + 1) / 2; e++)
                    if (lane + 64 * e < d.dv) out[head * d.dv + lane + 64 * e] = (T)(y[e] * inv * nw[e] * silu_of(z[e]));
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
// Prepare.  A wave takes one head's vector (q, k or v) over 8 tokens; the last vector index stands for the gates of all
// heads.  Grid (tokens / 8, vectors / 4).  E: elements per lane; TAPS: taps of the convolutions, 0 for any number - the rows of
// a known number are all requested ahead and kept in registers.
// ---------------------------------------------------------------------------
template <int E, int TAPS>
__global__ __launch_bounds__(256) void recur_prepare_kernel(OxbRecurParams p, uint32_t dv_p) {
    constexpr int TOKENS = 8;
    const OxbRecurDims& d = p.d;
    const uint32_t lane = threadIdx.x & 63u, vec = blockIdx.y * 4 + (threadIdx.x >> 6), n_vec = 2 * d.qk_heads + d.heads;
    if (vec > n_vec) return;
    const float* ring = p.memory + (size_t)p.rows.seq0 * p.seq_stride + oxb_recur_state(d);
    const uint32_t first = blockIdx.x * TOKENS;
    if (vec == n_vec) {
        for (uint32_t i = lane; i < TOKENS * d.heads; i += 64) {
            const uint32_t m = first + i / d.heads, h = i % d.heads;
            if (m < p.n) gates_of(p, p.first + m, h, p.s.la + (size_t)m * d.heads + h, p.s.beta + (size_t)m * d.heads + h);
        }
        return;
    }
    const bool is_v = vec >= 2 * d.qk_heads, is_k = !is_v && vec >= d.qk_heads;
    const uint32_t hd = is_v ? vec - 2 * d.qk_heads : is_k ? vec - d.qk_heads : vec, len = is_v ? d.dv : d.dk, pad = is_v ? dv_p : d.dk_p;
    const uint32_t ch = (is_v ? d.ch_v : is_k ? d.ch_k : d.ch_q) + hd * len;
    float y[TOKENS][E];
    if constexpr (TAPS > 0) {
        // inputs of the tokens and of the TAPS - 1 in front of them: earlier rows of the portion, the ring, or zeros
        float x[TOKENS + TAPS - 1][E], w[TAPS][E], bias[E];
        const uint32_t row0 = p.first + first, pos0 = p.rows.pos0 + row0;
#pragma unroll
        for (int e = 0; e < E; e++) {
            const uint32_t i = lane + 64 * e, c = ch + (i < len ? i : 0);
#pragma unroll
            for (int j = 0; j < TOKENS + TAPS - 1; j++) {
                const int back = TAPS - 1 - j;   // positive: in front of the first token
                x[j][e] = 0.f;
                if (back > 0) {
                    if ((uint32_t)back <= row0) x[j][e] = p.lin[(size_t)(row0 - back) * p.ld_lin + d.col_conv + c];
                    else if ((uint32_t)back <= pos0) x[j][e] = ring[(size_t)((pos0 - back) & (d.ring - 1u)) * d.channels + c];
                } else {
                    x[j][e] = p.lin[(size_t)(p.first + min(first - back, p.n - 1)) * p.ld_lin + d.col_conv + c];
                }
            }
#pragma unroll
            for (int t = 0; t < TAPS; t++) w[t][e] = p.conv_w[(size_t)c * TAPS + t];
            bias[e] = p.conv_b ? p.conv_b[c] : 0.f;
        }
#pragma unroll
        for (int t = 0; t < TOKENS; t++)
#pragma unroll
            for (int e = 0; e < E; e++) {
                float v = fmaf(w[TAPS - 1][e], x[t + TAPS - 1][e], bias[e]);
#pragma unroll
                for (int j = 1; j < TAPS; j++) v = fmaf(w[TAPS - 1 - j][e], x[t + TAPS - 1 - j][e], v);
                y[t][e] = lane + 64 * e < len ? silu_of(v) : 0.f;
            }
    } else {
#pragma unroll
        for (int t = 0; t < TOKENS; t++) {
            const uint32_t row = p.first + min(first + t, p.n - 1);
#pragma unroll
            for (int e = 0; e < E; e++) y[t][e] = lane + 64 * e < len ? conv_of(p, ring, row, row, p.rows.pos0 + row, ch + lane + 64 * e) : 0.f;
        }
    }
#pragma unroll
    for (int t = 0; t < TOKENS; t++) {
        const uint32_t m = first + t;
        float f = 1.0f;
        if (d.delta && !is_v) {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < E; e++) ss = fmaf(y[t][e], y[t][e], ss);
            f = (is_k ? 1.0f : d.q_scale) / sqrtf(wave_sum_f32(ss) + 1e-6f);
        }
        if (m >= p.n) continue;
        float* dst = is_v ? p.s.v + ((size_t)m * d.heads + hd) * dv_p : (is_k ? p.s.k : p.s.q) + ((size_t)m * d.qk_heads + hd) * d.dk_p;
#pragma unroll
        for (int e = 0; e < E; e++)
            if (lane + 64 * e < pad) dst[lane + 64 * e] = y[t][e] * f;
    }
}

// The order of k in every 32-wide unit of the chunked kernels: lane group g holds k = 4 g .. + 3 and 16 + 4 g .. + 3.  A 16 x
// 16 accumulator tile (lane 16 g + c: column c, rows 4 g .. + 3) is half an operand in that order as it stands.
__device__ __forceinline__ v8f join(v4f a, v4f b) { return (v8f){a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]}; }
// One column of a row-major [token][ld] matrix as such an operand: tokens 32 u + (4 g ..), rows past the end repeat the last.
__device__ __forceinline__ v8f load_column(const float* x, size_t ld, uint32_t m0, uint32_t u, uint32_t g, uint32_t last) {
    v8f f;
#pragma unroll
    for (int e = 0; e < 8; e++) f[e] = x[(size_t)min(m0 + 32 * u + (e & 4) * 4 + 4 * g + (e & 3), last) * ld];
    return f;
}
__device__ __forceinline__ v4f mfma16(v4f a, v4f b, v4f c) {   // 16 x 16 x 16, k = 4 g + e in both operands
#pragma unroll
    for (int e = 0; e < 4; e++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], c, 0, 0, 0);
    return c;
}

// ---------------------------------------------------------------------------
// Chunk.  Grid (head, chunk), 4 waves.  With c_t the decays' logarithms summed from the chunk's start (in double: differences
// of sums are what counts), A_ti = beta_t e^(c_t - c_i) k_t . k_i below the diagonal and T = (1 + A)^-1, leaves behind
//   P_ti = e^(c_t - c_i) q_t . k_i (i <= t)       W = T diag(beta e^c) K      U0 = T diag(beta) V      K^T
// T comes out of 16 x 16 blocks: the diagonal ones by substitution (one per wave), those below by products (one block column
// per wave), T_ij = -T_ii sum_k A_ik T_kj.
// ---------------------------------------------------------------------------
static constexpr uint32_t kLdT = 68;
__global__ __launch_bounds__(256) void recur_chunk_kernel(OxbRecurParams p, uint32_t dv_p) {
    const OxbRecurDims& d = p.d;
    __shared__ __attribute__((aligned(16))) float As[64][kLdT], Ts[64][kLdT];
    __shared__ double cum[64];
    __shared__ __attribute__((aligned(16))) float beta_s[64], bg_s[64];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, c = lane & 15u, g = lane >> 4;
    const uint32_t w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t head = blockIdx.x, chunk = blockIdx.y, m0 = chunk * 64, last = p.n - 1, rep = d.heads / d.qk_heads, qk = head / rep;
    const size_t ld = (size_t)d.qk_heads * d.dk_p, slot = (size_t)chunk * d.heads + head;
    const float *q = p.s.q + qk * d.dk_p, *k = p.s.k + qk * d.dk_p;
    if (w == 0) {
        const bool in = m0 + lane < p.n;
        const float la = in ? p.s.la[(size_t)(m0 + lane) * d.heads + head] : 0.f, b = in ? p.s.beta[(size_t)(m0 + lane) * d.heads + head] : 0.f;
        double s = (double)la;
#pragma unroll
        for (int o = 1; o < 64; o *= 2) {
            const double x = __shfl_up(s, o, 64);
            if ((int)lane >= o) s += x;
        }
        const double end = __shfl(s, 63, 64);
        cum[lane] = s;
        const float ga = expf((float)s);
        beta_s[lane] = b;
        bg_s[lane] = b * ga;
        p.s.gam[slot * 64 + lane] = ga;
        p.s.fwd[slot * 64 + lane] = expf((float)(end - s));
    }
    if (d.delta)
        for (uint32_t i = tid; i < 64 * kLdT; i += 256) (&Ts[0][0])[i] = 0.f;
    v4f ap[4], aa[4];
#pragma unroll
    for (int j = 0; j < 4; j++) ap[j] = aa[j] = (v4f){0.f, 0.f, 0.f, 0.f};
    const size_t at_t = (size_t)min(m0 + 16 * w + c, last) * ld + 8 * g;
    for (uint32_t u = 0; u < d.dk_p / 32; u++) {
        const v8f qf = load_row8(q + at_t + 32 * u), kf = load_row8(k + at_t + 32 * u);
#pragma unroll
        for (int j = 0; j < 4; j++)
            if ((uint32_t)j <= w) {
                const v8f ki = load_row8(k + (size_t)min(m0 + 16 * j + c, last) * ld + 8 * g + 32 * u);
                ap[j] = mfma32(ki, qf, ap[j]);
                if (d.delta) aa[j] = mfma32(ki, kf, aa[j]);
            }
    }
    __syncthreads();
    const uint32_t t = 16 * w + c;
    float* P = p.s.P + slot * 4096 + w * 1024;
#pragma unroll
    for (int j = 0; j < 4; j++) {
        v4f pv, av;
#pragma unroll
        for (int v = 0; v < 4; v++) {
            const uint32_t i = 16 * j + 4 * g + v;
            const float f = i <= t ? expf((float)(cum[t] - cum[i])) : 0.f;
            pv[v] = i <= t ? ap[j][v] * f : 0.f;
            av[v] = i < t ? aa[j][v] * f * beta_s[t] : 0.f;
        }
        *reinterpret_cast<v4f*>(P + (j >> 1) * 512 + (j & 1) * 256 + lane * 4) = pv;
        if (d.delta) *reinterpret_cast<v4f*>(&As[t][16 * j + 4 * g]) = av;
    }
    if (d.delta) {
        __syncthreads();
        {   // column c of the diagonal block's inverse (the lane groups repeat it)
            float col[16];
#pragma unroll
            for (int r = 0; r < 16; r++) {
                float v = (uint32_t)r == c ? 1.0f : 0.f;
#pragma unroll
                for (int i = 0; i < r; i++) v = fmaf(-As[16 * w + r][16 * w + i], col[i], v);
                col[r] = v;
            }
            if (g == 0) {
#pragma unroll
                for (int r = 0; r < 16; r++) Ts[16 * w + r][16 * w + c] = col[r];
            }
        }
        __syncthreads();
        v4f tb[4];   // tb[k]: block (w + k, w) as it stands in the accumulators
#pragma unroll
        for (int v = 0; v < 4; v++) tb[0][v] = Ts[16 * w + 4 * g + v][16 * w + c];
#pragma unroll
        for (int dist = 1; dist < 4; dist++)
            if (w + dist < 4) {
                const uint32_t i = w + dist;
                v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int kk = 0; kk < dist; kk++) acc = mfma16(load4(&As[16 * i + c][16 * (w + kk) + 4 * g]), tb[kk], acc);
                tb[dist] = mfma16(-load4(&Ts[16 * i + c][16 * i + 4 * g]), acc, (v4f){0.f, 0.f, 0.f, 0.f});
#pragma unroll
                for (int v = 0; v < 4; v++) Ts[16 * i + 4 * g + v][16 * w + c] = tb[dist][v];
            }
        __syncthreads();
    }
    // rows of T as operands, shared by all column tiles
    v8f tf[4][2];
    if (d.delta) {
#pragma unroll
        for (int r = 0; r < 4; r++)
#pragma unroll
            for (int u = 0; u <= r / 2; u++) tf[r][u] = join(load4(&Ts[16 * r + c][32 * u + 4 * g]), load4(&Ts[16 * r + c][32 * u + 16 + 4 * g]));
    }
    const uint32_t dkt = d.dk_p / 16;
    if (d.delta || head % rep == 0)
        for (uint32_t tile = w; tile < dkt; tile += 4) {
            v8f kf[2];
#pragma unroll
            for (int u = 0; u < 2; u++) kf[u] = load_column(k + 16 * tile + c, ld, m0, u, g, last);
            if (head % rep == 0) {
                float* kt = p.s.Kt + (((size_t)chunk * d.qk_heads + qk) * dkt + tile) * 1024;
#pragma unroll
                for (int u = 0; u < 2; u++) store_unit(kt + u * 512, lane, kf[u]);
            }
            if (!d.delta) continue;
#pragma unroll
            for (int u = 0; u < 2; u++) kf[u] *= join(load4(&bg_s[32 * u + 4 * g]), load4(&bg_s[32 * u + 16 + 4 * g]));
            float* W = p.s.W + slot * 64 * d.dk_p + (tile >> 1) * 512 + (tile & 1) * 256 + lane * 4;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int u = 0; u <= r / 2; u++) acc = mfma32(kf[u], tf[r][u], acc);
                *reinterpret_cast<v4f*>(W + (size_t)r * 16 * d.dk_p) = acc;
            }
        }
    if (!d.delta) return;
    const uint32_t dvt = dv_p / 16;
    for (uint32_t tile = w; tile < dvt; tile += 4) {
        v8f vf[2];
#pragma unroll
        for (int u = 0; u < 2; u++)
            vf[u] = load_column(p.s.v + head * dv_p + 16 * tile + c, (size_t)d.heads * dv_p, m0, u, g, last) *
                    join(load4(&beta_s[32 * u + 4 * g]), load4(&beta_s[32 * u + 16 + 4 * g]));
        float* U0 = p.s.U0 + (slot * dvt + tile) * 1024 + lane * 4;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            v4f acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int u = 0; u <= r / 2; u++) acc = mfma32(tf[r][u], vf[u], acc);
            *reinterpret_cast<v4f*>(U0 + r * 256) = acc;
        }
    }
}

// ---------------------------------------------------------------------------
// Scan.  Grid (head x 16 columns, the tiles of a head on one XCD: they share its L2), 4 waves: wave w takes token rows 16 w .. of every chunk and the state's row tiles w, w + 4,
// ..; per chunk, with S the state at its start,
//   U = U0 - W S        o = e^c (Q S) + P U        S <- e^(c_end) S + K^T diag(e^(c_end - c)) U
// The operands of the next chunk are requested as soon as this chunk's have been used; the barriers order LDS alone.
// ---------------------------------------------------------------------------
template <int DKU, bool DELTA>
__global__ __launch_bounds__(256) void recur_scan_kernel(OxbRecurParams p, uint32_t dv_p) {
    const OxbRecurDims& d = p.d;
    constexpr int DK = 32 * DKU, TPW = (2 * DKU + 3) / 4;
    __shared__ __attribute__((aligned(16))) float Sx[16][DK + 4], Ux[16][kLdT], Uf[16][kLdT];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, c = lane & 15u, g = lane >> 4;
    const uint32_t w = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t dvt = dv_p / 16, head = (blockIdx.x & 7u) + 8 * ((blockIdx.x >> 3) / dvt), tile = (blockIdx.x >> 3) % dvt;
    if (head >= d.heads) return;
    const uint32_t rep = d.heads / d.qk_heads, qk = head / rep;
    const uint32_t n_chunks = (p.n + 63) / 64, last = p.n - 1, col = 16 * tile + c;
    float* state = p.memory + (size_t)p.rows.seq0 * p.seq_stride + ((size_t)head * d.slices + tile / 2) * DK * 32 + 16 * (tile & 1u) + c;
    const bool fresh = p.rows.pos0 + p.first == 0;
    v4f S[TPW];
#pragma unroll
    for (int j = 0; j < TPW; j++) {
        const uint32_t r0 = 16 * (w + 4 * j) + 4 * g;
        S[j] = (v4f){0.f, 0.f, 0.f, 0.f};
        if (r0 < DK) {
            if (!fresh) {
#pragma unroll
                for (int v = 0; v < 4; v++) S[j][v] = state[(size_t)(r0 + v) * 32];
            }
            *reinterpret_cast<v4f*>(&Sx[c][r0]) = S[j];
        }
    }
    v8f qf[DKU], wf[DELTA ? DKU : 1], pf[2], kf[TPW][2];
    v4f u0, gam, fwd;
    float g_end;
    auto load_qw = [&](uint32_t ch) {
        const float* q = p.s.q + ((size_t)min(ch * 64 + 16 * w + c, last) * d.qk_heads + qk) * DK + 4 * g;
        const float* W = p.s.W + ((size_t)ch * d.heads + head) * 64 * DK + (size_t)w * 16 * DK;
#pragma unroll
        for (int u = 0; u < DKU; u++) {
            qf[u] = join(load4(q + 32 * u), load4(q + 32 * u + 16));
            if constexpr (DELTA) wf[u] = load_unit(W + u * 512, lane);
        }
    };
    auto load_rest = [&](uint32_t ch) {
        const size_t slot = (size_t)ch * d.heads + head;
        const float* P = p.s.P + slot * 4096 + w * 1024;
        const float* kt = p.s.Kt + ((size_t)ch * d.qk_heads + qk) * (2 * DKU) * 1024;
#pragma unroll
        for (int u = 0; u < 2; u++) {
            pf[u] = load_unit(P + u * 512, lane);
#pragma unroll
            for (int j = 0; j < TPW; j++) kf[j][u] = load_unit(kt + (size_t)min(w + 4 * j, 2u * DKU - 1) * 1024 + u * 512, lane);
        }
    };
    auto load_u = [&](uint32_t ch) {
        const size_t slot = (size_t)ch * d.heads + head;
        gam = load4(p.s.gam + slot * 64 + 16 * w + 4 * g);
        fwd = load4(p.s.fwd + slot * 64 + 16 * w + 4 * g);
        g_end = p.s.gam[slot * 64 + 63];
        if constexpr (DELTA) {
            u0 = load4(p.s.U0 + (slot * dvt + tile) * 1024 + w * 256 + lane * 4);
        } else {
#pragma unroll
            for (int v = 0; v < 4; v++) u0[v] = p.s.v[((size_t)min(ch * 64 + 16 * w + 4 * g + v, last) * d.heads + head) * dv_p + col];
        }
    };
    v4f beta = {0.f, 0.f, 0.f, 0.f};
    auto load_beta = [&](uint32_t ch) {
        if constexpr (!DELTA) {
#pragma unroll
            for (int v = 0; v < 4; v++) {
                const uint32_t m = ch * 64 + 16 * w + 4 * g + v;
                beta[v] = m < p.n ? p.s.beta[(size_t)m * d.heads + head] : 0.f;
            }
        }
    };
    load_qw(0);
    load_u(0);
    load_beta(0);
    load_rest(0);
    const float skip = p.skip ? p.skip[head] : 0.f;
    for (uint32_t ch = 0; ch < n_chunks; ch++) {
        lds_barrier();
        v4f oq = {0.f, 0.f, 0.f, 0.f}, ws = oq;
#pragma unroll
        for (int u = 0; u < DKU; u++) {
            const v8f sb = join(load4(&Sx[c][32 * u + 4 * g]), load4(&Sx[c][32 * u + 16 + 4 * g]));
            if constexpr (DELTA) ws = mfma32(wf[u], sb, ws);
            oq = mfma32(qf[u], sb, oq);
        }
        const uint32_t next = min(ch + 1, n_chunks - 1);
        load_qw(next);
        const v4f v = u0, U = DELTA ? u0 - ws : u0 * beta, gc = gam, ge = {g_end, g_end, g_end, g_end};
        *reinterpret_cast<v4f*>(&Ux[c][16 * w + 4 * g]) = U;
        *reinterpret_cast<v4f*>(&Uf[c][16 * w + 4 * g]) = U * fwd;
        load_u(next);
        load_beta(next);
        lds_barrier();
        v4f o = oq * gc;
#pragma unroll
        for (int j = 0; j < TPW; j++) S[j] *= ge;
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const v8f ub = join(load4(&Ux[c][32 * u + 4 * g]), load4(&Ux[c][32 * u + 16 + 4 * g]));
            const v8f uf = join(load4(&Uf[c][32 * u + 4 * g]), load4(&Uf[c][32 * u + 16 + 4 * g]));
            o = mfma32(pf[u], ub, o);
#pragma unroll
            for (int j = 0; j < TPW; j++) S[j] = mfma32(kf[j][u], uf, S[j]);
        }
        load_rest(next);
#pragma unroll
        for (int j = 0; j < TPW; j++) {
            const uint32_t r0 = 16 * (w + 4 * j) + 4 * g;
            if (r0 < DK) *reinterpret_cast<v4f*>(&Sx[c][r0]) = S[j];
        }
        if (col < d.dv) {
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const uint32_t m = ch * 64 + 16 * w + 4 * g + i;
                if (m < p.n) p.o[(size_t)(p.first + m) * d.heads * d.dv + head * d.dv + col] = o[i] + (DELTA ? 0.f : skip * v[i]);
            }
        }
    }
#pragma unroll
    for (int j = 0; j < TPW; j++) {
        const uint32_t r0 = 16 * (w + 4 * j) + 4 * g;
        if (r0 < DK) {
#pragma unroll
            for (int v = 0; v < 4; v++) state[(size_t)(r0 + v) * 32] = S[j][v];
        }
    }
}

// ---------------------------------------------------------------------------
// Finish: gate and norm of each part of a row's outputs, values in registers.  Short parts (E values per lane): a wave per
// part, four rows each, grid (rows / 4, parts / 4).  Long ones: 1024 threads per part, eight values each (parts beyond 8192 are
// read again), grid (row, part).  Blocks behind the token rows bring the portion's last convolution inputs into the ring.
// ---------------------------------------------------------------------------
__device__ __forceinline__ void keep_inputs(const OxbRecurParams& p, uint32_t back, uint32_t first, uint32_t step) {
    const uint32_t row = p.rows.m - 1 - back, pos = p.rows.pos0 + row;
    float* keep = p.memory + (size_t)p.rows.seq0 * p.seq_stride + oxb_recur_state(p.d) + (size_t)(pos & (p.d.ring - 1u)) * p.d.channels;
    const float* x = p.lin + (size_t)row * p.ld_lin + p.d.col_conv;
    for (uint32_t i = first; i < p.d.channels; i += step) keep[i] = x[i];
}

template <typename T, int E, int ROWS>
__global__ __launch_bounds__(256) void recur_finish_kernel(OxbRecurParams p) {
    const OxbRecurDims& d = p.d;
    const uint32_t tid = threadIdx.x, lane = tid & 63u, inner = d.heads * d.dv, parts = inner / d.norm_len, n_rb = (p.rows.m + ROWS - 1) / ROWS;
    if (blockIdx.x >= n_rb) return keep_inputs(p, blockIdx.x - n_rb, blockIdx.y * 256 + tid, gridDim.y * 256);
    const uint32_t row0 = blockIdx.x * ROWS, part = blockIdx.y * 4 + (tid >> 6);
    if (blockIdx.y == 0)
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

template <typename T>
__global__ __launch_bounds__(1024) void recur_finish_long_kernel(OxbRecurParams p) {
    constexpr int KEEP = 8;
    const OxbRecurDims& d = p.d;
    __shared__ float red[16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, inner = d.heads * d.dv, row = blockIdx.x, part = blockIdx.y;
    if (row >= p.rows.m) return keep_inputs(p, row - p.rows.m, blockIdx.y * 1024 + tid, gridDim.y * 1024);
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

// ---------------------------------------------------------------------------
static uint32_t pad16(uint32_t n) { return (n + 15u) / 16u * 16u; }

size_t oxb_recur_scratch(const OxbRecurDims& d, uint32_t n, float* base, OxbRecurScratch* s) {
    const size_t rows = n, chunks = (n + 63) / 64, dv_p = pad16(d.dv);
    size_t at = 0;
    auto take = [&](float** p, size_t floats) {
        if (s) *p = base + at;
        at += (floats + 63) / 64 * 64;
    };
    OxbRecurScratch none;
    OxbRecurScratch& o = s ? *s : none;
    take(&o.q, rows * d.qk_heads * d.dk_p);
    take(&o.k, rows * d.qk_heads * d.dk_p);
    take(&o.v, rows * d.heads * dv_p);
    take(&o.la, rows * d.heads);
    take(&o.beta, rows * d.heads);
    take(&o.gam, chunks * d.heads * 64);
    take(&o.fwd, chunks * d.heads * 64);
    take(&o.P, chunks * d.heads * 4096);
    take(&o.Kt, chunks * d.qk_heads * 64 * d.dk_p);
    take(&o.W, d.delta ? chunks * d.heads * 64 * d.dk_p : 64);
    take(&o.U0, d.delta ? chunks * d.heads * 64 * dv_p : 64);
    return at;
}

const char* oxb_recur_check(const OxbRecurDims& d) {
    if (!d.heads || !d.qk_heads || !d.dk || !d.dv || !d.taps || !d.norm_len) return "a size of a recurrent mixer is 0";
    if (d.heads % d.qk_heads) return "heads must be a multiple of the query / key heads";
    if (d.dk > 256 || d.dv > 256) return "recurrent head size beyond 256";
    if (d.taps > 64 || d.ring < d.taps - 1 + OXB_RECUR_STEP_TOKENS || (d.ring & (d.ring - 1))) return "convolution taps beyond 64";
    if ((d.heads * d.dv) % d.norm_len) return "norm parts must divide the outputs";
    if (d.heads > 65535) return "too many heads";
    return nullptr;
}

static bool params_ok(const OxbRecurParams& p) {
    return p.rows.m && p.lin && p.conv_w && p.neg_a && p.dt_bias && p.norm_w && p.memory && p.o && !oxb_recur_check(p.d) &&
           p.d.slices == (p.d.dv + 31) / 32 && p.d.dk_p == oxb_pad32(p.d.dk) && p.ld_lin >= p.d.col_conv + p.d.channels;
}

bool oxb_recur_step_finishes(const OxbRecurDims& d) { return !d.gate_first && d.norm_shared && d.norm_len == d.dv && d.slices <= 4; }

template <typename T, int SL, bool FINISH>
static void launch_step(const OxbRecurParams& p, uint32_t tokens, hipStream_t st) {
    const dim3 grid(p.d.heads * ((p.d.slices + SL - 1) / SL), p.rows.m / tokens), block(256 * SL);
#define OXB_STEP(RPT)                                                                                                              \
    if (tokens == 1) hipLaunchKernelGGL((recur_step_kernel<T, RPT, SL, FINISH, true>), grid, block, 0, st, p, tokens);             \
    else hipLaunchKernelGGL((recur_step_kernel<T, RPT, SL, FINISH, false>), grid, block, 0, st, p, tokens);
    if (p.d.dk_p <= 64) {
        OXB_STEP(2)
    } else if (p.d.dk_p <= 128) {
        OXB_STEP(4)
    } else {
        OXB_STEP(8)
    }
#undef OXB_STEP
}
template <typename T>
static void pick_step(const OxbRecurParams& p, uint32_t tokens, hipStream_t st) {
    if (!oxb_recur_step_finishes(p.d)) launch_step<float, 1, false>(p, tokens, st);
    else if (p.d.slices == 1) launch_step<T, 1, true>(p, tokens, st);
    else if (p.d.slices == 2) launch_step<T, 2, true>(p, tokens, st);
    else launch_step<T, 4, true>(p, tokens, st);
}

hipError_t oxb_launch_recur_step(const OxbRecurParams& p, int dt, hipStream_t st) {
    const uint32_t tokens = p.rows.seq_step ? 1 : p.rows.m;
    if (!params_ok(p) || tokens > OXB_RECUR_STEP_TOKENS || p.rows.m / tokens > 65535) return hipErrorInvalidValue;
    if (oxb_recur_step_finishes(p.d) && (!p.out || p.out_fill < p.d.heads * p.d.dv || p.out_col + p.out_fill > p.ld_out)) return hipErrorInvalidValue;
    if (dt == OXB_DT_BF16) pick_step<__bf16>(p, tokens, st);
    else pick_step<float>(p, tokens, st);
    return hipGetLastError();
}

template <int DKU>
static void launch_scan(const OxbRecurParams& p, uint32_t dv_p, hipStream_t st) {
    const dim3 grid((p.d.heads + 7) / 8 * 8 * (dv_p / 16));
    if (p.d.delta) hipLaunchKernelGGL((recur_scan_kernel<DKU, true>), grid, dim3(256), 0, st, p, dv_p);
    else hipLaunchKernelGGL((recur_scan_kernel<DKU, false>), grid, dim3(256), 0, st, p, dv_p);
}

template <int E>
static void launch_prepare(const OxbRecurParams& p, uint32_t dv_p, dim3 grid, hipStream_t st) {
    switch (p.d.taps) {
    case 1: hipLaunchKernelGGL((recur_prepare_kernel<E, 1>), grid, dim3(256), 0, st, p, dv_p); break;
    case 2: hipLaunchKernelGGL((recur_prepare_kernel<E, 2>), grid, dim3(256), 0, st, p, dv_p); break;
    case 3: hipLaunchKernelGGL((recur_prepare_kernel<E, 3>), grid, dim3(256), 0, st, p, dv_p); break;
    case 4: hipLaunchKernelGGL((recur_prepare_kernel<E, 4>), grid, dim3(256), 0, st, p, dv_p); break;
    default: hipLaunchKernelGGL((recur_prepare_kernel<E, 0>), grid, dim3(256), 0, st, p, dv_p); break;
    }
}

hipError_t oxb_launch_recur_chunked(const OxbRecurParams& p, hipStream_t st) {
    const OxbRecurDims& d = p.d;
    if (!params_ok(p) || p.rows.pos || p.rows.seq_step || !p.n || p.first + p.n > p.rows.m || p.n > OXB_RECUR_SEGMENT || !p.s.q) return hipErrorInvalidValue;
    const uint32_t dv_p = pad16(d.dv), n_vec = 2 * d.qk_heads + d.heads + 1;
    const uint32_t widest = d.dk_p > dv_p ? d.dk_p : dv_p;
    const dim3 prep((p.n + 7) / 8, (n_vec + 3) / 4);
    if (widest <= 64) launch_prepare<1>(p, dv_p, prep, st);
    else if (widest <= 128) launch_prepare<2>(p, dv_p, prep, st);
    else launch_prepare<4>(p, dv_p, prep, st);
    hipLaunchKernelGGL(recur_chunk_kernel, dim3(d.heads, (p.n + 63) / 64), dim3(256), 0, st, p, dv_p);
    switch (d.dk_p / 32) {
    case 1: launch_scan<1>(p, dv_p, st); break;
    case 2: launch_scan<2>(p, dv_p, st); break;
    case 3: launch_scan<3>(p, dv_p, st); break;
    case 4: launch_scan<4>(p, dv_p, st); break;
    case 5: launch_scan<5>(p, dv_p, st); break;
    case 6: launch_scan<6>(p, dv_p, st); break;
    case 7: launch_scan<7>(p, dv_p, st); break;
    default: launch_scan<8>(p, dv_p, st); break;
    }
    return hipGetLastError();
}

template <typename T, int E>
static void launch_finish_short(const OxbRecurParams& p, uint32_t extra, hipStream_t st) {
    const uint32_t parts = p.d.heads * p.d.dv / p.d.norm_len;
    if (p.rows.m < 64) hipLaunchKernelGGL((recur_finish_kernel<T, E, 1>), dim3(p.rows.m + extra, (parts + 3) / 4), dim3(256), 0, st, p);
    else hipLaunchKernelGGL((recur_finish_kernel<T, E, 4>), dim3((p.rows.m + 3) / 4 + extra, (parts + 3) / 4), dim3(256), 0, st, p);
}
template <typename T>
static void launch_finish(const OxbRecurParams& p, uint32_t extra, hipStream_t st) {
    if (p.d.norm_len <= 64) launch_finish_short<T, 1>(p, extra, st);
    else if (p.d.norm_len <= 128) launch_finish_short<T, 2>(p, extra, st);
    else if (p.d.norm_len <= 256) launch_finish_short<T, 4>(p, extra, st);
    else hipLaunchKernelGGL((recur_finish_long_kernel<T>), dim3(p.rows.m + extra, p.d.heads * p.d.dv / p.d.norm_len), dim3(1024), 0, st, p);
}

hipError_t oxb_launch_recur_finish(const OxbRecurParams& p, bool keep_conv, int dt, hipStream_t st) {
    if (!params_ok(p) || !p.out || p.out_fill < p.d.heads * p.d.dv || p.out_col + p.out_fill > p.ld_out || (keep_conv && (p.rows.pos || p.rows.seq_step)))
        return hipErrorInvalidValue;
    uint32_t extra = keep_conv ? p.d.taps - 1 : 0;
    if (extra > p.rows.m) extra = p.rows.m;
    if (dt == OXB_DT_BF16) launch_finish<__bf16>(p, extra, st);
    else launch_finish<float>(p, extra, st);
    return hipGetLastError();
}
