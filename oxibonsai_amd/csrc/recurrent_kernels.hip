// recurrent_kernels.hip — gated linear recurrences: step form, chunked form, output gate and norm (see recurrent_kernels.h).
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "recurrent_device.h"

// Waves per SIMD that a step is compiled for: as many as its registers allow without spilling.
constexpr int step_waves(int rpt, int sl, bool one) { return !one || rpt > 4 ? 4 : sl < 4 ? 7 : rpt < 4 ? 8 : 4; }

template <typename T, int RPT, int SL, bool FINISH, bool ONE>   // grid (head x slice group, sequence)
__global__ __launch_bounds__(256 * SL, step_waves(RPT, SL, ONE)) void recur_step_kernel(OxbRecurParams p, uint32_t tokens) {
    recur_step<T, RPT, SL, FINISH, ONE>(p, tokens, blockIdx.x, blockIdx.y);
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
            for (int t = 0; t < TAPS; t++) w[t][e] = p.conv_w[(size_t)t * d.channels + c];
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
__global__ __launch_bounds__(256, 4) void recur_chunk_kernel(OxbRecurParams p, uint32_t dv_p) {
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
// Scan.  Grid (head x 16 columns, the tiles of a head on one XCD: they share its L2), 4 waves: wave w takes token rows 16 w ..
// of every chunk and the state's row tiles w, w + 4, ..; per chunk, with S the state at its start,
//   U = U0 - W S        o = e^c (Q S) + P U        S <- e^(c_end) S + K^T diag(e^(c_end - c)) U
// The operands of a later chunk are requested as soon as this chunk's have been used; the barriers order LDS alone.
// ---------------------------------------------------------------------------
template <int DKU, bool DELTA>
__global__ __launch_bounds__(256, 1) void recur_scan_kernel(OxbRecurParams p, uint32_t dv_p) {
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
    constexpr int NS = DKU <= 4 ? 2 : 1;   // chunks whose operands of the first two products are on their way or in registers
    v8f qf[NS][DKU], wf[NS][DELTA ? DKU : 1], pf[2], kf[TPW][2];
    v4f u0[NS], gam[NS], fwd[NS], beta[NS];
    float g_end[NS];
    auto q_at = [&](uint32_t ch) { return p.s.q + ((size_t)min(min(ch, n_chunks - 1) * 64 + 16 * w + c, last) * d.qk_heads + qk) * DK + 4 * g; };
    auto w_at = [&](uint32_t ch) { return p.s.W + ((size_t)min(ch, n_chunks - 1) * d.heads + head) * 64 * DK + (size_t)w * 16 * DK; };
    auto load_qw = [&](const float* q, const float* W, int set, int u) {
        qf[set][u] = join(load4(q + 32 * u), load4(q + 32 * u + 16));
        if constexpr (DELTA) wf[set][u] = load_unit(W + u * 512, lane);
    };
    auto load_u = [&](uint32_t c0, int set) {
        const uint32_t ch = min(c0, n_chunks - 1);
        const size_t slot = (size_t)ch * d.heads + head;
        gam[set] = load4(p.s.gam + slot * 64 + 16 * w + 4 * g);
        fwd[set] = load4(p.s.fwd + slot * 64 + 16 * w + 4 * g);
        g_end[set] = p.s.gam[slot * 64 + 63];
        if constexpr (DELTA) {
            u0[set] = load4(p.s.U0 + (slot * dvt + tile) * 1024 + w * 256 + lane * 4);
        } else {
#pragma unroll
            for (int v = 0; v < 4; v++) {
                const uint32_t m = ch * 64 + 16 * w + 4 * g + v;
                u0[set][v] = p.s.v[((size_t)min(m, last) * d.heads + head) * dv_p + col];
                beta[set][v] = m < p.n ? p.s.beta[(size_t)m * d.heads + head] : 0.f;
            }
        }
    };
    auto p_at = [&](uint32_t ch) { return p.s.P + ((size_t)min(ch, n_chunks - 1) * d.heads + head) * 4096 + w * 1024; };
    auto k_at = [&](uint32_t ch) { return p.s.Kt + ((size_t)min(ch, n_chunks - 1) * d.qk_heads + qk) * (2 * DKU) * 1024; };
    auto load_pk = [&](const float* P, const float* kt, int u) {
        pf[u] = load_unit(P + u * 512, lane);
#pragma unroll
        for (int j = 0; j < TPW; j++) kf[j][u] = load_unit(kt + (size_t)min(w + 4 * j, 2u * DKU - 1) * 1024 + u * 512, lane);
    };
#pragma unroll
    for (int i = 0; i < NS; i++) {
#pragma unroll
        for (int u = 0; u < DKU; u++) load_qw(q_at(i), w_at(i), i, u);
        load_u(i, i);
        __builtin_amdgcn_sched_barrier(0);   // (the loop's order: its waits count requests)
    }
    load_pk(p_at(0), k_at(0), 0);
    load_pk(p_at(0), k_at(0), 1);
    __builtin_amdgcn_sched_barrier(0);
    const float skip = p.skip ? p.skip[head] : 0.f;
    // Stores behind the end fall outside the buffer and are dropped: no branch, so the count of requests in flight stays known
    // and a chunk waits for its own operands alone.
    const uint32_t inner = d.heads * d.dv, o_bytes = p.n * inner * 4u;
    const __amdgpu_buffer_rsrc_t out = make_rsrc(p.o + (size_t)p.first * inner, o_bytes);
    const uint32_t o_at = ((16 * w + 4 * g) * inner + head * d.dv + col) * 4u, o_rows = col < d.dv ? p.n : 0;
    auto step = [&](uint32_t ch, int set) {
        const bool live = ch < n_chunks;   // (the last group of NS chunks may run over the end)
        lds_barrier();
        v4f oq = {0.f, 0.f, 0.f, 0.f}, ws = oq;
        const float *qn = q_at(ch + NS), *wn = w_at(ch + NS), *pn = p_at(ch + 1), *kn = k_at(ch + 1);
        // an operand's successor is requested right behind its last product, so that the requests spread over the products
        auto s_unit = [&](int u) { return join(load4(&Sx[c][32 * u + 4 * g]), load4(&Sx[c][32 * u + 16 + 4 * g])); };
        v8f sb = s_unit(0);
#pragma unroll
        for (int u = 0; u < DKU; u++) {
            const v8f next = s_unit(u + 1 < DKU ? u + 1 : u);
#pragma unroll
            for (int e = 0; e < 8; e++) {
                if constexpr (DELTA) ws = __builtin_amdgcn_mfma_f32_16x16x4f32(wf[set][u][e], sb[e], ws, 0, 0, 0);
                oq = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[set][u][e], sb[e], oq, 0, 0, 0);
            }
            load_qw(qn, wn, set, u);
            __builtin_amdgcn_sched_barrier(0);
            sb = next;
        }
        const v4f v = u0[set];
        v4f U = DELTA ? u0[set] - ws : u0[set] * beta[set];
        if (!live) U = (v4f){0.f, 0.f, 0.f, 0.f};
        *reinterpret_cast<v4f*>(&Ux[c][16 * w + 4 * g]) = U;
        *reinterpret_cast<v4f*>(&Uf[c][16 * w + 4 * g]) = U * fwd[set];
        v4f o = oq * gam[set];
        const float end = live ? g_end[set] : 1.0f;
#pragma unroll
        for (int j = 0; j < TPW; j++) S[j] *= end;
        load_u(ch + NS, set);
        lds_barrier();
        v8f ub[2], uf[2];
#pragma unroll
        for (int u = 0; u < 2; u++) {
            ub[u] = join(load4(&Ux[c][32 * u + 4 * g]), load4(&Ux[c][32 * u + 16 + 4 * g]));
            uf[u] = join(load4(&Uf[c][32 * u + 4 * g]), load4(&Uf[c][32 * u + 16 + 4 * g]));
        }
#pragma unroll
        for (int u = 0; u < 2; u++) {
#pragma unroll
            for (int e = 0; e < 8; e++) {
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(pf[u][e], ub[u][e], o, 0, 0, 0);
#pragma unroll
                for (int j = 0; j < TPW; j++) S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[j][u][e], uf[u][e], S[j], 0, 0, 0);
            }
            load_pk(pn, kn, u);
            __builtin_amdgcn_sched_barrier(0);
        }
#pragma unroll
        for (int j = 0; j < TPW; j++) {
            const uint32_t r0 = 16 * (w + 4 * j) + 4 * g;
            if (4 * (j + 1) <= 2 * DKU || r0 < DK) *reinterpret_cast<v4f*>(&Sx[c][r0]) = S[j];
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t m = ch * 64 + 16 * w + 4 * g + i;
            __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(o[i] + (DELTA ? 0.f : skip * v[i])), out,
                                                  (int)(m < o_rows ? o_at + (ch * 64 + i) * inner * 4u : OXB_OOB), 0, 0);
        }
    };
    for (uint32_t ch = 0; ch < n_chunks; ch += NS)
#pragma unroll
        for (int i = 0; i < NS; i++) step(ch + i, i);
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
// Finish.  Blocks behind the token rows bring the portion's last convolution inputs into the ring.
// ---------------------------------------------------------------------------
template <typename T, int E, int ROWS>
__global__ __launch_bounds__(256) void recur_finish_kernel(OxbRecurParams p) {   // grid (rows / ROWS, parts / 4)
    const uint32_t n_rb = (p.rows.m + ROWS - 1) / ROWS;
    if (blockIdx.x >= n_rb) return keep_inputs(p, blockIdx.x - n_rb, blockIdx.y * 256 + threadIdx.x, gridDim.y * 256);
    recur_finish<T, E, ROWS>(p, blockIdx.x, blockIdx.y);
}

template <typename T>
__global__ __launch_bounds__(1024) void recur_finish_long_kernel(OxbRecurParams p) {   // grid (row, part)
    if (blockIdx.x >= p.rows.m) return keep_inputs(p, blockIdx.x - p.rows.m, blockIdx.y * 1024 + threadIdx.x, gridDim.y * 1024);
    recur_finish_long<T>(p, blockIdx.x, blockIdx.y);
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
    if (d.heads > 65535 || (uint64_t)d.heads * d.dv > (1u << 18)) return "too many heads";
    return nullptr;
}

bool oxb_recur_params_ok(const OxbRecurParams& p) {
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
    if (!oxb_recur_params_ok(p) || tokens > OXB_RECUR_STEP_TOKENS || p.rows.m / tokens > 65535) return hipErrorInvalidValue;
    if (oxb_recur_step_finishes(p.d) && !oxb_recur_finish_ok(p)) return hipErrorInvalidValue;
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
    if (!oxb_recur_params_ok(p) || p.rows.pos || p.rows.seq_step || !p.n || p.first + p.n > p.rows.m || p.n > OXB_RECUR_SEGMENT || !p.s.q) return hipErrorInvalidValue;
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

bool oxb_recur_finish_ok(const OxbRecurParams& p) {
    return oxb_recur_params_ok(p) && p.out && p.out_fill >= p.d.heads * p.d.dv && p.out_col + p.out_fill <= p.ld_out;
}

hipError_t oxb_launch_recur_finish(const OxbRecurParams& p, bool keep_conv, int dt, hipStream_t st) {
    if (!oxb_recur_finish_ok(p) || (keep_conv && (p.rows.pos || p.rows.seq_step))) return hipErrorInvalidValue;
    uint32_t extra = keep_conv ? p.d.taps - 1 : 0;
    if (extra > p.rows.m) extra = p.rows.m;
    if (dt == OXB_DT_BF16) launch_finish<__bf16>(p, extra, st);
    else launch_finish<float>(p, extra, st);
    return hipGetLastError();
}
