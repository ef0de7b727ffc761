// row_attention.hip — attention over cached rows on the matrix cores (see row_attention.h).
//
// Precision: rotation, norms, scores, softmax and sums are fp32.  Probabilities meet bf16 values as a bf16 hi + lo pair (two
// products), so a weight keeps 16 bits; the fp32 kernels use fp32 operands throughout.
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "row_attention_device.h"

// ---------------------------------------------------------------------------
template <typename T, int E, int ROWS>
__global__ __launch_bounds__(256) void grouped_store_kernel(OxbGroupedStore p) {
    grouped_store<T, E, ROWS>(p, blockIdx.x, blockIdx.y);
}

// ---------------------------------------------------------------------------
// Decode.  Grid (split, kv head x head tile, token row), 8 waves; the 16 heads of a tile are the columns of the products, so a
// row is read once for all of them:
//   S^T[key][head] = K[key] . q[head]              operand reads of the staged rows
//   O^T[r][head]  += V[key][r] P[head][key]        the same LDS rows through the transposing read
// A split walks chunks of 32 keys through a ring of LDS buffers (memory -> LDS copies, up to three chunks ahead).  HT head
// tiles share a workgroup, 8 / HT waves each; of those, wave w multiplies key tile w % 2 with every (4 / HT)-th k unit, the
// partial scores meet in LDS, every wave of the tile forms the same probabilities from them and takes its own share of the
// value elements of O.  KSQ: k units per wave, NTW: accumulator tiles per wave.
// ---------------------------------------------------------------------------
static constexpr uint32_t kChunk = OXB_KEY_CHUNK;
// Value operand: keys 4 g .. 4 g + 3 of both key tiles, one value element per lane.  `at` = value_at(..) of the tile.
template <typename T> __device__ __forceinline__ uint32_t value_at(uint32_t sl, uint32_t qi, uint32_t g);
template <> __device__ __forceinline__ uint32_t value_at<__bf16>(uint32_t sl, uint32_t qi, uint32_t g) {
    // four consecutive halves per lane for the transposing read: row 4 g + qi / 4, columns 16 sl + 4 (qi % 4) ..
    return (sl >> 1) * 512 + staged_slot(4 * g + (qi >> 2), (sl & 1u) * 2 + ((qi & 3u) >> 1)) * 8 + (qi & 1u) * 4;
}
template <> __device__ __forceinline__ uint32_t value_at<float>(uint32_t sl, uint32_t qi, uint32_t g) {
    const uint32_t d = 16 * sl + qi, e = d & 7u;   // (the slots of rows 4 g .. 4 g + 3 lie four apart: they share r >> 2)
    return (d >> 5) * 512 + (e >> 2) * 256 + staged_slot(4 * g, (d & 31u) >> 3) * 4 + (e & 3u);
}
__device__ __forceinline__ v8b value_frag(const __bf16* tile0, const __bf16* tile1) {
    const v4b t0 = __builtin_bit_cast(v4b, lds_read_tr16(reinterpret_cast<const _Float16*>(tile0)));
    const v4b t1 = __builtin_bit_cast(v4b, lds_read_tr16(reinterpret_cast<const _Float16*>(tile1)));
    return (v8b){t0[0], t0[1], t0[2], t0[3], t1[0], t1[1], t1[2], t1[3]};
}
__device__ __forceinline__ v8f value_frag(const float* a, const float* b) { return (v8f){a[0], a[16], a[32], a[48], b[0], b[16], b[32], b[48]}; }

// Units 4 j, j < bring <= N, of a lane's row into the LDS units 4 j behind `at`.
template <typename T, int N, int J>
__device__ __forceinline__ void request_units(const T* row, uint32_t at, uint32_t bring) {
    if constexpr (J < N) {
        if ((uint32_t)J < bring) {
            constexpr int PER = 4096 / (128 * (int)sizeof(T));   // units within an immediate offset
            const T* base = row + J / PER * PER * 128;
            copy16_to_lds_at<J % PER * 128 * (int)sizeof(T)>(base, at + J * 4 * Dt<T>::unit_bytes);
            if constexpr (Dt<T>::sub == 2) copy16_to_lds_at<J % PER * 128 * (int)sizeof(T) + 16>(base, at + J * 4 * Dt<T>::unit_bytes + 1024);
        }
        request_units<T, N, J + 1>(row, at, bring);
    }
}

// Waits until at most n of the wave's requests are in flight (n wave-uniform; rounded down where no instruction says n).
__device__ __forceinline__ void wait_requests(uint32_t n) {
#define OXB_WAIT(k) else if (n >= k) asm volatile("s_waitcnt vmcnt(" #k ")" ::: "memory")
    if (n >= 24) asm volatile("s_waitcnt vmcnt(24)" ::: "memory");
    OXB_WAIT(20); OXB_WAIT(18); OXB_WAIT(16); OXB_WAIT(12); OXB_WAIT(10); OXB_WAIT(9); OXB_WAIT(8); OXB_WAIT(6); OXB_WAIT(5);
    OXB_WAIT(4); OXB_WAIT(3); OXB_WAIT(2); OXB_WAIT(1);
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
#undef OXB_WAIT
}

template <typename T, int HT, int KSQ, int NTW, int DQ>
__global__ __launch_bounds__(512) void row_decode_kernel(OxbRowAttnParams p, uint32_t n_buf) {
    typedef typename Dt<T>::frag frag;
    constexpr float kLazy = 8.0f;                 // the running maximum follows once it is 2^8 behind
    constexpr int WPT = 8 / HT, KSPLIT = 4 / HT;  // waves per head tile; waves sharing the k units of a key tile
    constexpr int SUB = Dt<T>::sub;
    extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
    __shared__ __attribute__((aligned(16))) float part_s[HT][KSPLIT][16][kChunk + 4];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, qi = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t n_ht = (p.rep + 15) / 16, per_kv = (n_ht + HT - 1) / HT, kvh = blockIdx.y / per_kv;
    const uint32_t split = blockIdx.x, hw = wave / WPT, ht = blockIdx.y % per_kv * HT + hw, m = blockIdx.z;
    const uint32_t pos = row_pos(p.rows, m), seq = row_seq(p.rows, m), used = oxb_used_splits(pos, p.n_splits);
    if (split >= used) return;
    const uint32_t n_mine = (pos / kChunk - split) / used + 1;   // chunks split, split + used, ...
    const uint32_t units = p.ld / 32, ks = p.ks, nt = p.nt, kt = wave & 1u, kq = (wave >> 1) % KSPLIT, slot = staged_slot(qi, g);
    const uint32_t dq = wave >> 1, bring = dq < units ? (units - dq + 3) / 4 : 0;   // this wave brings in units dq + 4 j of key tile kt
    T* lds = reinterpret_cast<T*>(smem);
    const uint32_t buf_elems = 2 * units * 512, lds0 = lds_address(smem) + (kt * units + dq) * Dt<T>::unit_bytes;
    const T* cache = reinterpret_cast<const T*>(p.cache) + 32 * dq + 8 * stage_col(lane);
    const float c2 = p.scale * 1.4426950408889634f;   // scores in units of log2(e)
    auto request = [&](uint32_t i) {
        // rows past the newest position repeat it; their scores are masked
        const uint32_t key = (split + i * used) * kChunk + kt * 16 + stage_row(lane);
        const T* row = cache + kv_row(p.kv, seq, 0, kvh, min(key, pos)) * p.ld;
        const uint32_t at = lds0 + (i % n_buf) * (2 * units * Dt<T>::unit_bytes);
        request_units<T, DQ, 0>(row, at, bring);
    };
    const uint32_t ahead = n_buf > 1 ? n_buf - 1 : 1;
    for (uint32_t i = 0; i < ahead && i < n_mine; i++) request(i);

    frag q[KSQ];
    {
        const T* src = reinterpret_cast<const T*>(p.q) + ((size_t)m * p.heads + kvh * p.rep + min(ht * 16 + qi, p.rep - 1)) * (32 * ks) + 8 * g;
#pragma unroll
        for (int j = 0; j < KSQ; j++) {
            const uint32_t s = kq + KSPLIT * j;
            q[j] = load_row8(src + 32 * min(s, ks - 1));
            if (s >= ks) q[j] = zero_frag((const T*)nullptr);
        }
    }
    const uint32_t ntw = (nt + WPT - 1) / WPT, t0 = (wave % WPT) * ntw;
    uint32_t v_at[NTW];
    v4f O[NTW];
#pragma unroll
    for (int i = 0; i < NTW; i++) {
        v_at[i] = p.v0 * 512 + value_at<T>(min(t0 + i, nt - 1), qi, g);
        O[i] = (v4f){0.f, 0.f, 0.f, 0.f};
    }
    float m_run = -INFINITY, l_run = 0.f;   // maximum (times c2) and this lane's share of the sum; the same in every wave of a tile

    for (uint32_t i = 0; i < n_mine; i++) {
        const uint32_t key0 = (split + i * used) * kChunk;
        const T* kb = lds + (i % n_buf) * buf_elems;
        const T* tile = kb + (size_t)kt * units * 512;
        // this chunk's copies have arrived; those of later chunks may stay in flight
        wait_requests(n_buf == 1 ? 0 : min(ahead - 1, n_mine - 1 - i) * bring * SUB);
        lds_barrier();   // for every wave; and every wave is through with the chunk before
        if (n_buf > 1 && i + ahead < n_mine) request(i + ahead);
        v4f s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};   // (two chains of dependent products)
#pragma unroll
        for (int j = 0; j < KSQ; j++) s[j & 1] = mfma32(load_staged(tile + (size_t)min(kq + KSPLIT * j, ks - 1) * 512, slot), q[j], s[j & 1]);
        *reinterpret_cast<v4f*>(&part_s[hw][kq][qi][kt * 16 + 4 * g]) = s[0] + s[1];
        lds_barrier();
        float sv[8], mx = -INFINITY;
        {
            v4f a = *reinterpret_cast<const v4f*>(&part_s[hw][0][qi][4 * g]), b = *reinterpret_cast<const v4f*>(&part_s[hw][0][qi][16 + 4 * g]);
#pragma unroll
            for (int k = 1; k < KSPLIT; k++) {
                a += *reinterpret_cast<const v4f*>(&part_s[hw][k][qi][4 * g]);
                b += *reinterpret_cast<const v4f*>(&part_s[hw][k][qi][16 + 4 * g]);
            }
#pragma unroll
            for (int v = 0; v < 4; v++) sv[v] = a[v] * c2, sv[4 + v] = b[v] * c2;
        }
        if (key0 + kChunk - 1 > pos) {
#pragma unroll
            for (int v = 0; v < 4; v++) {
                if (key0 + 4 * g + v > pos) sv[v] = -INFINITY;
                if (key0 + 16 + 4 * g + v > pos) sv[4 + v] = -INFINITY;
            }
        }
#pragma unroll
        for (int e = 0; e < 8; e++) mx = fmaxf(mx, sv[e]);
        mx = max_rows4(mx);  // finite: key0 <= pos
        if (__any(mx > m_run + kLazy)) {
            const float m_new = fmaxf(m_run, mx), alpha = exp2_of<T>(m_run - m_new);
            m_run = m_new;
            l_run *= alpha;
#pragma unroll
            for (int t = 0; t < NTW; t++) O[t] *= alpha;
        }
        float pe[8];
#pragma unroll
        for (int e = 0; e < 8; e++) {
            pe[e] = exp2_of<T>(sv[e] - m_run);
            l_run += pe[e];
        }
        frag hi, lo;
        split_hi_lo(pe, hi, lo);
        frag v[NTW];
#pragma unroll
        for (int t = 0; t < NTW; t++) v[t] = value_frag(kb + v_at[t], kb + v_at[t] + (size_t)units * 512);
#pragma unroll
        for (int t = 0; t < NTW; t++) O[t] = mfma32(v[t], hi, O[t]);
        if constexpr (!Dt<T>::is_f32) {
#pragma unroll
            for (int t = 0; t < NTW; t++) O[t] = mfma32(v[t], lo, O[t]);
        }
        if (n_buf == 1 && i + 1 < n_mine) {
            lds_barrier();   // every wave is through with the buffer
            request(i + 1);
        }
    }
    if (ht >= n_ht) return;
    const size_t part = ((size_t)m * p.kv.nkv * n_ht + kvh * n_ht + ht) * p.n_splits + split;
    float* po = p.part_o + (part * 16 + qi) * 16 * nt + 4 * g;
#pragma unroll
    for (int t = 0; t < NTW; t++)
        if ((uint32_t)t < ntw && t0 + t < nt) *reinterpret_cast<v4f*>(po + 16 * (t0 + t)) = O[t];
    l_run = sum_rows4(l_run);
    if (wave % WPT == 0 && g == 0) {
        p.part_ml[part * 32 + qi * 2] = m_run;
        p.part_ml[part * 32 + qi * 2 + 1] = l_run;
    }
}

// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void row_merge_kernel(OxbRowAttnParams p) {   // grid (head, token row)
    row_merge<T>(p, blockIdx.x, blockIdx.y);
}

// ---------------------------------------------------------------------------
// Prompts: a wave owns 16 QT queries of one head, the four waves of a workgroup take consecutive query tiles and share each
// 32-key block's rows through LDS (two buffers if they fit; memory -> LDS copies of block i + 1 run under block i).  Operand
// order as in decode: values come out of the same rows through the transposing read.
// ---------------------------------------------------------------------------
template <typename T, int QT, int KS, int VT>
__global__ __launch_bounds__(256, QT == 2 && !Dt<T>::is_f32 ? 2 : 1) void row_prefill_kernel(OxbRowAttnParams p, uint32_t n_buf) {
    typedef typename Dt<T>::frag frag;
    constexpr int NU = (2 * KS + VT + 3) / 4;   // units a wave brings in per block, at most
    constexpr float kLazy = 8.0f;               // the running maximum follows once it is 2^8 behind
    extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, qi = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t n_qb = (p.rows.m + 64 * QT - 1) / (64 * QT);
    const uint32_t qb = n_qb - 1 - blockIdx.x / p.heads, head = blockIdx.x % p.heads, kvh = head / p.rep;   // long (late) query blocks first
    const uint32_t units = p.ld / 32, ks = p.ks, vt = p.nt, slot = staged_slot(qi, g), sr = stage_row(lane), sc = 8 * stage_col(lane);
    T* lds = reinterpret_cast<T*>(smem);
    const T* cache = reinterpret_cast<const T*>(p.cache) + sc;
    const uint32_t lds0 = lds_address(smem), q_last = min((qb + 1) * 64 * QT, p.rows.m) - 1;
    const uint32_t kv_len = p.rows.pos0 + q_last + 1;   // keys the workgroup's last query sees
    const float c2 = p.scale * 1.4426950408889634f;

    // Unit un of a block: key tile un / units, unit un % units of its rows; a wave brings in units wave, wave + 4, ..
    // (Keys past the last one repeat it; their scores are masked.)
    auto stage = [&](uint32_t key0, uint32_t buf) {
        const T* r0 = cache + kv_row(p.kv, p.rows.seq0, 0, kvh, min(key0 + sr, kv_len - 1)) * p.ld;
        const T* r1 = cache + kv_row(p.kv, p.rows.seq0, 0, kvh, min(key0 + 16 + sr, kv_len - 1)) * p.ld;
        const uint32_t at = lds0 + (buf * 2 * units + wave) * Dt<T>::unit_bytes;
#pragma unroll
        for (int i = 0; i < NU; i++) {
            const uint32_t un = wave + 4 * i;
            if (un >= 2 * units) break;
            const T* src = un < units ? r0 + 32 * un : r1 + 32 * (un - units);
            copy16_to_lds_at<0>(src, at + i * 4 * Dt<T>::unit_bytes);
            if constexpr (Dt<T>::sub == 2) copy16_to_lds_at<0>(src + 4, at + i * 4 * Dt<T>::unit_bytes + 1024);
        }
    };
    stage(0, 0);

    // queries of this wave in operand order; rows past the end repeat the last one and are not stored
    frag q[QT][KS];
    uint32_t qpos[QT];
#pragma unroll
    for (int t = 0; t < QT; t++) {
        const uint32_t row = min(qb * 64 * QT + (wave * QT + t) * 16 + qi, p.rows.m - 1);
        qpos[t] = p.rows.pos0 + row;
        const T* qs = reinterpret_cast<const T*>(p.q) + ((size_t)row * p.heads + head) * (32 * ks) + 8 * g;
#pragma unroll
        for (int s = 0; s < KS; s++) q[t][s] = (uint32_t)s < ks ? load_row8(qs + 32 * s) : zero_frag((const T*)nullptr);
    }
    const uint32_t q_first = p.rows.pos0 + min(qb * 64 * QT + wave * QT * 16, p.rows.m - 1);   // blocks up to here are wholly visible to the wave
    uint32_t v_at[VT];
    v4f O[QT][VT];
    float m_run[QT], l_run[QT];   // maximum (times c2) and this lane's share of the sum
#pragma unroll
    for (int i = 0; i < VT; i++) v_at[i] = p.v0 * 512 + value_at<T>(min((uint32_t)i, vt - 1), qi, g);
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
        const T* kb = lds + (size_t)buf * 2 * units * 512;
        v4f s0[QT], s1[QT];
#pragma unroll
        for (int t = 0; t < QT; t++) s0[t] = s1[t] = (v4f){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; s++)
            if ((uint32_t)s < ks) {
                const frag k0 = load_staged(kb + (size_t)s * 512, slot), k1 = load_staged(kb + (size_t)(units + s) * 512, slot);
#pragma unroll
                for (int t = 0; t < QT; t++) {
                    s0[t] = mfma32(k0, q[t][s], s0[t]);
                    s1[t] = mfma32(k1, q[t][s], s1[t]);
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
                if (!whole && key0 + (e & 4) * 4 + 4 * g + (e & 3) > qpos[t]) sv[t][e] = -INFINITY;
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
                    const frag a = value_frag(kb + v_at[i2 + j], kb + v_at[i2 + j] + (size_t)units * 512);
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
        const float inv = f / (l * f + exp2_of<T>(sink - M)) * p.out_scale;
        T* o = reinterpret_cast<T*>(p.out) + (size_t)row * p.ld_out + p.out_col + head * 16 * vt + 4 * g;
#pragma unroll
        for (int i = 0; i < VT; i++)
            if ((uint32_t)i < vt) {
                typename Dt<T>::quad w;
#pragma unroll
                for (int v = 0; v < 4; v++) w[v] = (T)(O[t][i][v] * inv);
                *reinterpret_cast<typename Dt<T>::quad*>(o + 16 * i) = w;
            }
    }
}

// ---------------------------------------------------------------------------
static constexpr uint32_t kLdsMax = 160u << 10, kDecodeStatic = 4 * 16 * (kChunk + 4) * 4;   // (decode's partial scores)

// LDS buffers of a decode chunk: four, and where rows are short enough for two workgroups on a CU no more than both can have.
static uint32_t decode_buffers(uint32_t units, int dt) {
    const uint32_t bytes = kChunk * 32 * units * oxb_dt_bytes(dt), n = (kLdsMax - kDecodeStatic) / bytes, both = (kLdsMax / 2 - kDecodeStatic) / bytes;
    if (both >= 2) return both > 4 ? 4 : both;
    return n > 4 ? 4 : n;
}

const char* oxb_row_check(uint32_t units, int dt) { return units && decode_buffers(units, dt) ? nullptr : "a block of cached rows exceeds the LDS"; }
const char* oxb_grouped_check(uint32_t heads, uint32_t kv_heads, uint32_t dim, uint32_t vdim, uint32_t rot_dims, int dt) {
    if (!heads || !kv_heads || !dim || !vdim) return "an attention size is 0";
    if (heads % kv_heads) return "query heads must be a multiple of the key / value heads";
    if (rot_dims % 2 || rot_dims > dim) return "rotated dimensions must be even and within the head";
    if (dim > 256 || vdim > 256) return "head size beyond 256";
    const uint32_t units = (oxb_pad32(dim) + oxb_pad32(vdim)) / 32;
    if (2 * units * 512 * oxb_dt_bytes(dt) > kLdsMax) return "a block of keys and values exceeds the LDS";
    return oxb_row_check(units, dt);
}

template <typename T, int E>
static void launch_store_rows(const OxbGroupedStore& p, hipStream_t st) {
    const uint32_t y = (p.heads + 2 * p.kv_heads + 3) / 4;
    if (p.rows.m < 64) hipLaunchKernelGGL((grouped_store_kernel<T, E, 1>), dim3(p.rows.m, y), dim3(256), 0, st, p);
    else hipLaunchKernelGGL((grouped_store_kernel<T, E, 4>), dim3((p.rows.m + 3) / 4, y), dim3(256), 0, st, p);
}
template <typename T>
static void launch_store(const OxbGroupedStore& p, uint32_t widest, hipStream_t st) {
    if (widest <= 64) launch_store_rows<T, 1>(p, st);
    else if (widest <= 128) launch_store_rows<T, 2>(p, st);
    else launch_store_rows<T, 4>(p, st);
}

bool oxb_grouped_store_ok(const OxbGroupedStore& p, int dt) {
    return p.rows.m && p.lin && p.q && p.cache && p.cos_t && p.sin_t && p.dim_p == oxb_pad32(p.dim) && p.vdim_p == oxb_pad32(p.vdim) &&
           !oxb_grouped_check(p.heads, p.kv_heads, p.dim, p.vdim, p.rot_dims, dt) && p.kv.n_layers == 1 && p.kv.nkv == p.kv_heads;
}

hipError_t oxb_launch_grouped_store(const OxbGroupedStore& p, int dt, hipStream_t st) {
    if (!oxb_grouped_store_ok(p, dt)) return hipErrorInvalidValue;
    const uint32_t widest = p.dim_p > p.vdim_p ? p.dim_p : p.vdim_p;
    if (dt == OXB_DT_BF16) launch_store<__bf16>(p, widest, st);
    else launch_store<float>(p, widest, st);
    return hipGetLastError();
}

static bool rows_ok(const OxbRowAttnParams& p, int dt) {
    return p.rows.m && p.q && p.cache && p.sink && p.rep && p.heads == p.rep * p.kv.nkv && p.kv.n_layers == 1 && p.ks && p.nt && p.nt % 2 == 0 &&
           p.ld % 32 == 0 && p.ks <= p.ld / 32 && p.v0 + p.nt / 2 <= p.ld / 32 && !oxb_row_check(p.ld / 32, dt) &&
           (!p.kv.page_table || (p.kv.page_shift >= 4 && p.kv.page_shift <= 7));
}

template <typename T, int HT, int KSQ, int NTW, int DQ>
static hipError_t launch_decode(const OxbRowAttnParams& p, uint32_t n_buf, hipStream_t st) {
    const uint32_t per_kv = (oxb_row_head_tiles(p.rep) + HT - 1) / HT;
    hipLaunchKernelGGL((row_decode_kernel<T, HT, KSQ, NTW, DQ>), dim3(p.n_splits, p.kv.nkv * per_kv, p.rows.m), dim3(512),
                       n_buf * kChunk * p.ld * (uint32_t)sizeof(T), st, p, n_buf);
    return hipGetLastError();
}

// KSQ k units of the key per wave, NTW value tiles per wave, DQ units of the row brought in per wave.
#define OXB_DECODE_SIZES(F) F(1, 1, 1, 2) F(1, 2, 1, 2) F(1, 2, 2, 4) F(1, 3, 2, 3) F(1, 5, 4, 5) F(1, 9, 8, 9) F(2, 4, 2, 2) F(2, 6, 4, 3) F(2, 10, 8, 5) F(2, 18, 16, 9)

template <typename T>
static hipError_t pick_decode(const OxbRowAttnParams& p, uint32_t ht, uint32_t n_buf, hipStream_t st) {
    const uint32_t ksq = (p.ks + 4 / ht - 1) / (4 / ht), ntw = (p.nt + 8 / ht - 1) / (8 / ht), dq = (p.ld / 32 + 3) / 4;
#define OXB_TRY_SIZE(H, K, N, D) \
    if (ht == H && ksq <= K && ntw <= N && dq <= D) return launch_decode<T, H, K, N, D>(p, n_buf, st);
    OXB_DECODE_SIZES(OXB_TRY_SIZE)
#undef OXB_TRY_SIZE
    return hipErrorInvalidValue;
}

hipError_t oxb_launch_row_decode(const OxbRowAttnParams& p, uint32_t head_tiles, int dt, hipStream_t st) {
    if (!rows_ok(p, dt) || !p.part_o || !p.part_ml || !p.n_splits || p.n_splits > OXB_MAX_SPLITS || (head_tiles != 1 && head_tiles != 2))
        return hipErrorInvalidValue;
    const uint32_t n_buf = decode_buffers(p.ld / 32, dt);
    return dt == OXB_DT_BF16 ? pick_decode<__bf16>(p, head_tiles, n_buf, st) : pick_decode<float>(p, head_tiles, n_buf, st);
}

bool oxb_row_merge_ok(const OxbRowAttnParams& p, int dt) {
    return rows_ok(p, dt) && p.nt <= 16 && p.part_o && p.part_ml && p.out && p.n_splits && p.n_splits <= OXB_MAX_SPLITS && p.out_col + p.heads * 16 * p.nt <= p.ld_out;
}

hipError_t oxb_launch_row_merge(const OxbRowAttnParams& p, int dt, hipStream_t st) {
    if (!oxb_row_merge_ok(p, dt)) return hipErrorInvalidValue;
    const dim3 grid(p.heads, p.rows.m);
    if (dt == OXB_DT_BF16) hipLaunchKernelGGL((row_merge_kernel<__bf16>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((row_merge_kernel<float>), grid, dim3(256), 0, st, p);
    return hipGetLastError();
}

template <typename T, int QT, int KS, int VT>
static hipError_t launch_prefill(const OxbRowAttnParams& p, hipStream_t st) {
    const uint32_t bytes = 2 * (p.ld / 32) * 512 * (uint32_t)sizeof(T);
    const uint32_t n_buf = 2 * bytes <= kLdsMax ? 2u : 1u, n_qb = (p.rows.m + 64 * QT - 1) / (64 * QT);
    hipLaunchKernelGGL((row_prefill_kernel<T, QT, KS, VT>), dim3(n_qb * p.heads), dim3(256), n_buf * bytes, st, p, n_buf);
    return hipGetLastError();
}

hipError_t oxb_launch_row_prefill(const OxbRowAttnParams& p, int dt, hipStream_t st) {
    if (!rows_ok(p, dt) || p.rows.pos || p.rows.seq_step || !p.out || p.out_col + p.heads * 16 * p.nt > p.ld_out || p.ks + p.nt / 2 != p.ld / 32 || p.ks > 8 ||
        p.nt > 16 || p.ld_out % 4 || p.out_col % 4)
        return hipErrorInvalidValue;
    if (p.ks <= 4 && p.nt <= 8) return dt == OXB_DT_BF16 ? launch_prefill<__bf16, 2, 4, 8>(p, st) : launch_prefill<float, 2, 4, 8>(p, st);
    return dt == OXB_DT_BF16 ? launch_prefill<__bf16, 1, 8, 16>(p, st) : launch_prefill<float, 1, 8, 16>(p, st);
}

// Dynamic LDS beyond 64 KB has to be asked for, per kernel; done ahead of any launch so that none has to do it inside a
// stream capture.
template <typename T>
static hipError_t raise_lds() {
    hipError_t e = hipSuccess;
#define OXB_RAISE(H, K, N, D) \
    if (e == hipSuccess)                                                                                                       \
        e = hipFuncSetAttribute((const void*)&row_decode_kernel<T, H, K, N, D>, hipFuncAttributeMaxDynamicSharedMemorySize,  \
                                (int)(kLdsMax - kDecodeStatic));
    OXB_DECODE_SIZES(OXB_RAISE)
#undef OXB_RAISE
    const void* prefill[] = {(const void*)&row_prefill_kernel<T, 2, 4, 8>, (const void*)&row_prefill_kernel<T, 1, 8, 16>};
    for (const void* f : prefill)
        if (e == hipSuccess) e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kLdsMax);
    return e;
}
hipError_t oxb_row_attention_prepare(int dt) { return dt == OXB_DT_BF16 ? raise_lds<__bf16>() : raise_lds<float>(); }
