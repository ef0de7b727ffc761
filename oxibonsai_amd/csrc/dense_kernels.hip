// dense_kernels.hip — products with dense bf16 / fp32 weights on the matrix cores: upload-time packing, the few-row kernel
// of decode steps, the tiled GEMM of prefill, each with the whole tail of a sub-layer (scale, added vector, GELU, residual
// sum in fp32, dynamic-tanh norm of the next sub-layer) in its epilogue.  A norm without row statistics is elementwise, so
// no launch ever exists for it.
#include <hip/hip_runtime.h>
#include <hip/hip_fp16.h>
#include <stdint.h>

#include "dense_device.h"
#include "dense_kernels.h"

// ---------------------------------------------------------------------------
// Upload: row-major source -> operand units.  One workgroup per unit, one thread per element.
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(512) void dense_pack_kernel(const void* __restrict__ src, int type, const int64_t* __restrict__ row_off,
                                                         const int64_t* __restrict__ col_off, const int64_t* __restrict__ col_mul,
                                                         uint32_t n_units_k, T* __restrict__ dst) {
    const uint32_t j = threadIdx.x, lane = j >> 3, e = j & 7u;
    const uint32_t tile = blockIdx.x / n_units_k, u = blockIdx.x % n_units_k;
    const int64_t ro = row_off[tile * 16 + (lane & 15u)], co = col_off[u * 32 + (lane >> 4) * 8 + e];
    float v = 0.f;
    if (ro >= 0 && co >= 0) {
        const int64_t i = (col_mul ? ro * col_mul[u * 32 + (lane >> 4) * 8 + e] : ro) + co;
        if (type == 0) v = static_cast<const float*>(src)[i];
        else if (type == 1) v = __half2float(static_cast<const __half*>(src)[i]);
        else v = __uint_as_float((uint32_t)static_cast<const uint16_t*>(src)[i] << 16);
    }
    T* unit = dst + tile * oxb_tile_stride(n_units_k * 32, sizeof(T)) + (size_t)u * 512;
    if constexpr (Dt<T>::is_f32) unit[(e >> 2) * 256 + lane * 4 + (e & 3u)] = v;
    else unit[lane * 8 + e] = (T)v;
}

hipError_t oxb_launch_dense_pack(const void* src, int src_type, const int64_t* row_off, const int64_t* col_off, const int64_t* col_mul,
                                 uint32_t n_pad, uint32_t k_pad, int dt, void* dst, hipStream_t st) {
    if (!src || !dst || !row_off || !col_off || n_pad % 16 || k_pad % 32 || !n_pad || !k_pad || (src_type != 0 && src_type != 1 && src_type != 30))
        return hipErrorInvalidValue;
    const uint32_t nu = k_pad / 32;
    const uint64_t grid = (uint64_t)(n_pad / 16) * nu;
    if (grid > 0x7FFFFFFFull) return hipErrorInvalidValue;
    if (dt == OXB_DT_BF16)
        hipLaunchKernelGGL((dense_pack_kernel<__bf16>), dim3((uint32_t)grid), dim3(512), 0, st, src, src_type, row_off, col_off, col_mul, nu, (__bf16*)dst);
    else
        hipLaunchKernelGGL((dense_pack_kernel<float>), dim3((uint32_t)grid), dim3(512), 0, st, src, src_type, row_off, col_off, col_mul, nu, (float*)dst);
    return hipGetLastError();
}

__device__ __forceinline__ size_t x_row(const OxbDenseParams& p, uint32_t t) {
    if (p.row_table) return ((size_t)p.row_table[t >> p.row_shift] << p.row_shift) + (t & ((1u << p.row_shift) - 1u));
    return p.row0 + t;
}

// ---------------------------------------------------------------------------
// Few token rows: a workgroup of 8 waves owns RT row tiles and splits K over its waves; wave w takes the units w, w + 8, ...
// so that the workgroup walks its tiles' bytes in order.  The token rows are the columns of the product, CT tiles of 16:
// lane 16 g + c loads eight activations of token c, lanes of absent tokens supply zeros.  UN units are in flight per wave.
// The waves' sums meet in LDS and are added in wave order.
// ---------------------------------------------------------------------------
template <typename T, int RT, int CT, int UN>
__global__ __launch_bounds__(512) void dense_gemv_kernel(OxbDenseParams p) {
    typedef typename Dt<T>::frag frag;
    __shared__ __attribute__((aligned(16))) float red[8][RT * CT][16][20];
    __shared__ float row_scale[16 * CT];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, c = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t nu = p.k_pad / 32, n_tiles = p.n_pad / 16;
    const T* w[RT];
#pragma unroll
    for (int r = 0; r < RT; r++) w[r] = reinterpret_cast<const T*>(p.w) + min(blockIdx.x * RT + r, n_tiles - 1) * oxb_tile_stride(p.k_pad, sizeof(T));
    const T* x[CT];
#pragma unroll
    for (int t = 0; t < CT; t++) x[t] = reinterpret_cast<const T*>(p.x) + x_row(p, min(16u * t + c, p.m - 1)) * p.ldx + 8 * g;
    v4f acc[RT][CT];
#pragma unroll
    for (int r = 0; r < RT; r++)
#pragma unroll
        for (int t = 0; t < CT; t++) acc[r][t] = (v4f){0.f, 0.f, 0.f, 0.f};
    // sums of squares of a consumed norm: the first token's are on their way under the products
    constexpr int PRE = 4;
    float sq[PRE];
    auto load_ssq = [&](uint32_t m, uint32_t i0) {
#pragma unroll
        for (int k = 0; k < PRE; k++) {
            const uint32_t i = i0 + 64 * k + lane;
            sq[k] = i < p.e.n_ssq ? p.e.ssq_in[(size_t)m * p.e.n_ssq + i] : 0.f;
        }
    };
    if (p.e.ssq_in && wave < p.m) load_ssq(wave, 0);
    for (uint32_t u0 = wave; u0 < nu; u0 += 8 * UN) {
        frag b[UN][CT], a[UN][RT];
#pragma unroll
        for (int i = 0; i < UN; i++) {
            const uint32_t u = u0 + 8 * i;
#pragma unroll
            for (int t = 0; t < CT; t++) b[i][t] = u < nu && 16u * t + c < p.m ? load_row8(x[t] + 32 * u) : zero_frag((const T*)nullptr);
        }
#pragma unroll
        for (int i = 0; i < UN; i++) {
            const uint32_t u = min(u0 + 8 * i, nu - 1);  // (past the end: the last unit again, against a zero operand)
#pragma unroll
            for (int r = 0; r < RT; r++) a[i][r] = load_unit(w[r] + (size_t)u * 512, lane);
        }
#pragma unroll
        for (int i = 0; i < UN; i++)
#pragma unroll
            for (int r = 0; r < RT; r++)
#pragma unroll
                for (int t = 0; t < CT; t++) acc[r][t] = mfma32(a[i][r], b[i][t], acc[r][t]);
    }
    // what a finishing thread owns: a quad of outputs of one token
    const uint32_t f = tid >> 6, fq = tid & 3u, ft = (f % CT) * 16 + ((tid & 63u) >> 2), fn = (blockIdx.x * RT + f / CT) * 16 + 4 * fq;
    const bool finish = f < RT * CT && ft < p.m && blockIdx.x * RT + f / CT < n_tiles;
    const v4f resid = finish ? epilogue_resid(p.e, ft, fn) : (v4f){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < RT; r++)
#pragma unroll
        for (int t = 0; t < CT; t++) *reinterpret_cast<v4f*>(&red[wave][r * CT + t][c][4 * g]) = acc[r][t];
    if (p.e.ssq_in) {
        for (uint32_t m = wave; m < p.m; m += 8) {
            float ss = 0.f;
            for (uint32_t i0 = 0; i0 < p.e.n_ssq; i0 += 64 * PRE) {
                if (m != wave || i0) load_ssq(m, i0);
#pragma unroll
                for (int k = 0; k < PRE; k++) ss += sq[k];
            }
            ss = wave_sum_f32(ss);
            if (lane == 0) row_scale[m] = 1.0f / sqrtf(ss / (float)p.e.ssq_width + p.e.ssq_eps);
        }
    }
    __syncthreads();
    if (finish) {
        v4f y = *reinterpret_cast<const v4f*>(&red[0][f][ft & 15u][4 * fq]);
#pragma unroll
        for (int i = 1; i < 8; i++) y += *reinterpret_cast<const v4f*>(&red[i][f][ft & 15u][4 * fq]);
        if (p.e.ssq_in) y *= row_scale[ft];
        y = epilogue4<T>(p.e, ft, fn, y, resid);
        if (p.e.ssq_out) {
            float ss = y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3];   // (the tile's four quads are four neighbouring lanes)
            ss += dpp_f32<0xB1>(ss);
            ss += dpp_f32<0x4E>(ss);
            if (fq == 0) p.e.ssq_out[(size_t)ft * n_tiles + fn / 16] = ss;
        }
    }
}

// ---------------------------------------------------------------------------
// Tiled GEMM: a workgroup of 4 waves owns 64 RT rows x 16 CT tokens.  The weights come from memory already in operand
// order, so each wave loads its own RT tiles straight into registers; the token tile is shared by the waves and goes
// memory -> LDS without registers, as staged units (dense_device.h).  A stage is two units of k; tokens run
// three stages ahead (four LDS buffers; fp32: one, two buffers), weights two (two register sets).  The one barrier of a stage
// sits between its two units: it hands back the buffer of the stage before and admits reads of the next stage, which run
// under the second unit's products.  It waits for the requests of earlier regions alone; what was requested since the last
// barrier stays in flight.  The last stages request their own data again so that the count of requests in flight never
// changes.  SWAP exchanges the operands' roles: the lane then holds four consecutive tokens of one
// output row, which is the transposed store of the value rows of attention.
// ---------------------------------------------------------------------------
template <typename T, int RT, int CT, bool SWAP>
__global__ __launch_bounds__(256, RT == 4 && Dt<T>::is_f32 ? 1 : 2) void dense_gemm_kernel(OxbDenseParams p, uint32_t n_tm, uint32_t n_tn) {
    typedef typename Dt<T>::frag frag;
    constexpr int UK = 2, SUB = Dt<T>::sub;
    constexpr int UNITS = CT * UK;          // LDS units of a stage
    __shared__ __attribute__((aligned(16))) T xs[Dt<T>::is_f32 ? 2 : 4][UNITS * 512];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, c = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    // consecutive workgroups go to different XCDs: give each XCD a contiguous run of tiles with the token tiles innermost,
    // so that the workgroups sharing a row tile's weights share an L2
    const uint32_t total = n_tm * n_tn, per = (total + 7) / 8, id = (blockIdx.x & 7u) * per + (blockIdx.x >> 3);
    if (id >= total || (blockIdx.x >> 3) >= per) return;
    const uint32_t tm = id % n_tm, tn = id / n_tm, slot = staged_slot(c, g);
    const uint32_t nu = p.k_pad / 32, n_tiles = p.n_pad / 16, n_stages = nu / UK;  // (k_pad is a multiple of 64)
    const T* w[RT];
#pragma unroll
    for (int r = 0; r < RT; r++) w[r] = reinterpret_cast<const T*>(p.w) + min((tn * 4 + wave) * RT + r, n_tiles - 1) * oxb_tile_stride(p.k_pad, sizeof(T));
    // the units of the token tile this wave brings in: unit i -> token tile i / UK, k unit i % UK
    constexpr int MINE = UNITS / 4;
    static_assert(UNITS % 4 == 0, "the waves bring in equal shares");
    const T* xr[MINE];
#pragma unroll
    for (int i = 0; i < MINE; i++) {
        const uint32_t un = wave + 4 * i;
        xr[i] = reinterpret_cast<const T*>(p.x) + x_row(p, min(tm * (16 * CT) + (un / UK) * 16 + stage_row(lane), p.m - 1)) * p.ldx + (un % UK) * 32 + 8 * stage_col(lane);
    }
    auto stage_x = [&](uint32_t st, uint32_t buf) {
#pragma unroll
        for (int i = 0; i < MINE; i++) {
            const uint32_t un = wave + 4 * i;
            stage_unit(xr[i] + st * (32 * UK), &xs[buf][un * 512]);
        }
    };
    v4f acc[RT][CT];
#pragma unroll
    for (int r = 0; r < RT; r++)
#pragma unroll
        for (int t = 0; t < CT; t++) acc[r][t] = (v4f){0.f, 0.f, 0.f, 0.f};
    frag a[2][UK][RT], b[CT];
    auto load_w = [&](uint32_t st, int set, int k) {
#pragma unroll
        for (int r = 0; r < RT; r++) a[set][k][r] = load_unit(w[r] + (size_t)(st * UK + k) * 512, lane);
    };
    auto read_x = [&](uint32_t buf, int k, int t) { b[t] = load_staged(&xs[buf][(t * UK + k) * 512], slot); };
    // One half of a stage: the products of unit k; each token operand is replaced by that of the unit behind it (in the
    // second half: the next stage's first) right after its last use.
    auto half = [&](int set, int k, uint32_t next_buf) {
#pragma unroll
        for (int t = 0; t < CT; t++) {
#pragma unroll
            for (int r = 0; r < RT; r++) acc[r][t] = SWAP ? mfma32(b[t], a[set][k][r], acc[r][t]) : mfma32(a[set][k][r], b[t], acc[r][t]);
            read_x(next_buf, k ^ 1, t);
        }
#pragma unroll
        for (int t = 0; t < CT; t++) {
            __builtin_amdgcn_sched_group_barrier(0x008, RT * (Dt<T>::is_f32 ? 8 : 1), 0);   // matrix core
            __builtin_amdgcn_sched_group_barrier(0x100, SUB, 0);                            // LDS read
        }
    };
    auto clamp_st = [&](uint32_t st) { return min(st, n_stages - 1); };
    constexpr uint32_t NB = Dt<T>::is_f32 ? 2 : 4;   // LDS buffers
    constexpr int AHEAD = NB - 1, REGION = (MINE + UK * RT) * SUB;   // stages the tokens run ahead; requests between two barriers
#pragma unroll
    for (int i = 0; i < AHEAD; i++) stage_x(clamp_st(i), i);
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int k = 0; k < UK; k++) load_w(clamp_st(i), i, k);
    asm volatile("s_waitcnt vmcnt(0)\n\ts_barrier" ::: "memory");
#pragma unroll
    for (int t = 0; t < CT; t++) read_x(0, 0, t);
    auto stage = [&](uint32_t st, int set) {
        const uint32_t nxt = clamp_st(st + 2);
        if constexpr (AHEAD == 1) stage_x(clamp_st(st + 1), (st + 1) % NB);   // (everyone is through with the stage before)
        half(set, 0, st % NB);
        load_w(nxt, set, 0);
        __builtin_amdgcn_sched_barrier(0);
        // the next stage's tokens have arrived, and every wave is through with the stage before this one: its buffer can be
        // filled again
        if constexpr (AHEAD == 1) asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
        else asm volatile("s_waitcnt vmcnt(%0)\n\ts_barrier" ::"n"((AHEAD - 2) * REGION) : "memory");
        if constexpr (AHEAD > 1) stage_x(clamp_st(st + AHEAD), (st + AHEAD) % NB);
        __builtin_amdgcn_sched_barrier(0);
        half(set, 1, (st + 1) % NB);
        load_w(nxt, set, 1);
        __builtin_amdgcn_sched_barrier(0);
    };
    uint32_t st = 0;
    for (; st + 1 < n_stages; st += 2) {
        stage(st, 0);
        stage(st + 1, 1);
    }
    if (st < n_stages) stage(st, 0);
    wait_lds_copies();
    if constexpr (SWAP) {
#pragma unroll
        for (int r = 0; r < RT; r++) {
            const uint32_t n = ((tn * 4 + wave) * RT + r) * 16 + c;
#pragma unroll
            for (int t = 0; t < CT; t++) {
                typename Dt<T>::quad q;
#pragma unroll
                for (int i = 0; i < 4; i++) q[i] = (T)(acc[r][t][i] * p.e.scale);
                const uint32_t m = (tm * CT + t) * 16 + 4 * g;
                if (n < p.e.n && m < p.e.ld_t) *reinterpret_cast<typename Dt<T>::quad*>(reinterpret_cast<T*>(p.e.out_t) + (size_t)n * p.e.ld_t + m) = q;
            }
        }
    } else {
        // Through LDS, PT token tiles at a time: a wave then finishes whole runs of one token's outputs, and the epilogue is a
        // short loop instead of RT x CT inlined copies.  Quad q of token t sits at q ^ t (distinct banks).
        constexpr int PT = CT / RT > 0 ? CT / RT : 1, QUADS = 16 * RT, UN = 4;
        float* ys = reinterpret_cast<float*>(&xs[0][0]);
        static_assert(PT * 16 * QUADS * 16 <= (int)NB * UNITS * (int)Dt<T>::unit_bytes && (PT * 16 * QUADS) % (256 * UN) == 0, "the stages' LDS holds a pass");
#pragma unroll 1
        for (int t0 = 0; t0 < CT; t0 += PT) {
            __syncthreads();
#pragma unroll
            for (int s = 0; s < CT; s += PT)
                if (s == t0) {
#pragma unroll
                    for (int r = 0; r < RT; r++)
#pragma unroll
                        for (int t = 0; t < PT; t++)
                            *reinterpret_cast<v4f*>(ys + ((t * 16 + c) * QUADS + (((wave * RT + r) * 4 + g) ^ c)) * 4) = acc[r][s + t];
                }
            __syncthreads();
#pragma unroll 1
            for (uint32_t i0 = tid; i0 < PT * 16 * QUADS; i0 += 256 * UN) {
                v4f resid[UN];
#pragma unroll
                for (int k = 0; k < UN; k++) {
                    const uint32_t i = i0 + 256 * k, m = (tm * CT + t0) * 16 + i / QUADS;
                    resid[k] = m < p.m ? epilogue_resid(p.e, m, tn * 64 * RT + i % QUADS * 4) : (v4f){0.f, 0.f, 0.f, 0.f};
                }
#pragma unroll
                for (int k = 0; k < UN; k++) {
                    const uint32_t i = i0 + 256 * k, t = i / QUADS, q = i % QUADS, m = (tm * CT + t0) * 16 + t;
                    if (m < p.m)
                        epilogue4<T>(p.e, m, tn * 64 * RT + q * 4, *reinterpret_cast<const v4f*>(ys + (t * QUADS + (q ^ (t & 15u))) * 4), resid[k]);
                }
            }
        }
    }
}

static hipError_t check(const OxbDenseParams& p, int dt) {
    if (!p.w || !p.x || !p.m || !p.n_pad || !p.k_pad || p.n_pad % OXB_DENSE_PAD || p.k_pad % OXB_DENSE_PAD || p.ldx < p.k_pad || p.ldx % 8 ||
        (dt != OXB_DT_BF16 && dt != OXB_DT_F32) || p.e.n > p.n_pad || p.e.fill > p.n_pad || (p.row_table && (p.row_shift < 4 || p.row_shift > 7)))
        return hipErrorInvalidValue;
    if (p.e.glu_out && (p.e.glu % 4 || p.e.glu < p.e.n || p.e.n_glu % 2 || p.e.ld_glu % 2 || p.e.n_glu > p.e.ld_glu || p.e.fill > p.e.glu)) return hipErrorInvalidValue;
    return hipSuccess;
}

template <typename T, int RT, int CT, bool SWAP>
static hipError_t launch_gemm(const OxbDenseParams& p, hipStream_t st) {
    const uint32_t n_tm = (p.m + 16 * CT - 1) / (16 * CT), n_tn = (p.n_pad + 64 * RT - 1) / (64 * RT);
    hipLaunchKernelGGL((dense_gemm_kernel<T, RT, CT, SWAP>), dim3((n_tm * n_tn + 7) / 8 * 8), dim3(256), 0, st, p, n_tm, n_tn);
    return hipGetLastError();
}

// Tile choice by measured cost (us for K = 4096): of a workgroup alone on its CU, and per workgroup where a CU gets several.
template <typename T, bool SWAP>
static hipError_t pick_gemm(const OxbDenseParams& p, uint32_t n_cus, hipStream_t st) {
    struct { uint32_t rt, ct; double alone, each; } const opt[] = {{4, 8, 60, 64}, {2, 8, 42, 37.5}, {4, 4, 38, 38}, {2, 4, 28, 23.5}, {1, 4, 24, 19}};
    int best = -1;
    double best_cost = 0;
    for (int i = 0; i < 5; i++) {
        if (Dt<T>::is_f32 && opt[i].ct == 8) continue;   // (fp32 stages are twice as large)
        const uint64_t wgs = (uint64_t)((p.m + 16 * opt[i].ct - 1) / (16 * opt[i].ct)) * ((p.n_pad + 64 * opt[i].rt - 1) / (64 * opt[i].rt));
        const double busy = (double)((wgs + n_cus - 1) / n_cus) * opt[i].each, cost = busy > opt[i].alone ? busy : opt[i].alone;
        if (best < 0 || cost < best_cost) best = i, best_cost = cost;
    }
    if constexpr (!Dt<T>::is_f32) {
        if (best == 0) return launch_gemm<T, 4, 8, SWAP>(p, st);
        if (best == 1) return launch_gemm<T, 2, 8, SWAP>(p, st);
    }
    if (best == 2) return launch_gemm<T, 4, 4, SWAP>(p, st);
    if (best == 3) return launch_gemm<T, 2, 4, SWAP>(p, st);
    return launch_gemm<T, 1, 4, SWAP>(p, st);
}

template <typename T, int RT, int CT, int UN>
static hipError_t launch_gemv(const OxbDenseParams& p, hipStream_t st) {
    hipLaunchKernelGGL((dense_gemv_kernel<T, RT, CT, UN>), dim3((p.n_pad / 16 + RT - 1) / RT), dim3(512), 0, st, p);
    return hipGetLastError();
}

// Where the few-row kernel is the faster one (measured): always up to 16 rows; up to 32 unless the matrix alone fills the
// GPU with GEMM tiles; up to 64 where it has few tiles and long rows.
bool oxb_dense_few_rows(uint32_t n_pad, uint32_t k_pad, uint32_t m, uint32_t n_cus) {
    const uint32_t tiles = n_pad / 16;
    return m <= 16 || (m <= 32 && tiles <= 4 * n_cus) || (m <= OXB_DENSE_GEMV_MAX_ROWS && tiles <= n_cus && k_pad >= 4096);
}

// Two row tiles per workgroup where the matrix has tiles enough for every CU to get several workgroups all the same; units
// in flight per wave within what the registers of two workgroups per CU allow.
template <typename T>
static hipError_t pick_gemv(const OxbDenseParams& p, uint32_t n_cus, hipStream_t st) {
    const bool many = p.n_pad / 16 >= 4 * n_cus;
    const uint32_t per_wave = (p.k_pad / 32 + 7) / 8;
    constexpr int S = Dt<T>::is_f32 ? 2 : 1;
    if (p.m <= 16) {
        if (many) return launch_gemv<T, 2, 1, 4 / S>(p, st);
        return per_wave > 2 ? launch_gemv<T, 1, 1, 8 / S>(p, st) : launch_gemv<T, 1, 1, 2>(p, st);
    }
    if (p.m <= 32) return p.n_pad / 16 > n_cus ? launch_gemv<T, 2, 2, 4 / S>(p, st) : launch_gemv<T, 1, 2, 4 / S>(p, st);
    return launch_gemv<T, 1, 4, 2>(p, st);
}

hipError_t oxb_launch_dense(const OxbDenseParams& p, int dt, uint32_t n_cus, hipStream_t st) {
    const hipError_t e = check(p, dt);
    if (e != hipSuccess) return e;
    if (oxb_dense_few_rows(p.n_pad, p.k_pad, p.m, n_cus)) return dt == OXB_DT_BF16 ? pick_gemv<__bf16>(p, n_cus, st) : pick_gemv<float>(p, n_cus, st);
    if (p.e.ssq_in || p.e.ssq_out) return hipErrorInvalidValue;   // (the few-row kernel's)
    return dt == OXB_DT_BF16 ? pick_gemm<__bf16, false>(p, n_cus, st) : pick_gemm<float, false>(p, n_cus, st);
}

hipError_t oxb_launch_dense_gemm_t(const OxbDenseParams& p, int dt, uint32_t n_cus, hipStream_t st) {
    const hipError_t e = check(p, dt);
    if (e != hipSuccess) return e;
    if (!p.e.out_t || p.e.ld_t % 4) return hipErrorInvalidValue;
    return dt == OXB_DT_BF16 ? pick_gemm<__bf16, true>(p, n_cus, st) : pick_gemm<float, true>(p, n_cus, st);
}

// Grid (1024 columns, token row), four columns per thread.
template <typename T>
__global__ __launch_bounds__(256) void stream_enter_kernel(const float* __restrict__ x, uint32_t width, T* __restrict__ x0, uint32_t ld_x0,
                                                           uint32_t x0_col, uint32_t x0_fill, OxbEpilogue e) {
    const uint32_t m = blockIdx.y, n0 = (blockIdx.x * 256 + threadIdx.x) * 4;
    const float* row = x + (size_t)m * width;
    v4f y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; i++)
        if (n0 + i < width) y[i] = row[n0 + i];
    if (x0) {
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (x0_col + n0 + i < x0_fill) x0[(size_t)m * ld_x0 + x0_col + n0 + i] = (T)y[i];
    }
    epilogue4<T>(e, m, n0, y, epilogue_resid(e, m, n0));
}

hipError_t oxb_launch_stream_enter(const float* x, uint32_t width, uint32_t m, void* x0_out, uint32_t ld_x0, uint32_t x0_col,
                                   uint32_t x0_fill, const OxbEpilogue& e, int dt, hipStream_t st) {
    if (!x || !width || !m || (x0_out && (x0_fill > ld_x0 || x0_col + width > x0_fill)) || !e.out_t || e.n != width) return hipErrorInvalidValue;
    uint32_t cols = e.n > e.fill ? e.n : e.fill;
    if (x0_out && x0_fill - x0_col > cols) cols = x0_fill - x0_col;
    const dim3 grid((cols + 1023) / 1024, m);
    if (dt == OXB_DT_BF16)
        hipLaunchKernelGGL((stream_enter_kernel<__bf16>), grid, dim3(256), 0, st, x, width, (__bf16*)x0_out, ld_x0, x0_col, x0_fill, e);
    else
        hipLaunchKernelGGL((stream_enter_kernel<float>), grid, dim3(256), 0, st, x, width, (float*)x0_out, ld_x0, x0_col, x0_fill, e);
    return hipGetLastError();
}

__global__ __launch_bounds__(256) void gather_rows_kernel(const v4i* __restrict__ in, uint32_t pieces, const uint32_t* __restrict__ rows,
                                                          v4i* __restrict__ out) {
    const size_t src = (size_t)rows[blockIdx.x] * pieces, dst = (size_t)blockIdx.x * pieces;
    for (uint32_t i = threadIdx.x; i < pieces; i += 256) out[dst + i] = in[src + i];
}

hipError_t oxb_launch_gather_rows(const void* in, uint32_t ld, const uint32_t* rows, uint32_t n, void* out, int dt, hipStream_t st) {
    if (!in || !rows || !out || !n || ld % 8) return hipErrorInvalidValue;
    hipLaunchKernelGGL(gather_rows_kernel, dim3(n), dim3(256), 0, st, (const v4i*)in, ld * oxb_dt_bytes(dt) / 16, rows, (v4i*)out);
    return hipGetLastError();
}

// Grid = rows, 256 threads; a thread keeps up to 16 of its row's values, longer rows are read again.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void row_norm_kernel(float* __restrict__ x, uint32_t width, float in_scale, const float* __restrict__ w,
                                                       float eps, T* __restrict__ out, uint32_t ld, uint32_t fill) {
    constexpr int STEP = VEC ? 4 : 1, KEEP = 16 / STEP;
    __shared__ float red[4];
    const uint32_t tid = threadIdx.x;
    float* row = x + (size_t)blockIdx.x * width;
    T* o = out + (size_t)blockIdx.x * ld;
    float v[KEEP][STEP], ss = 0.f;
    auto load = [&](uint32_t i, float (&y)[STEP]) {
        if constexpr (VEC) {
            const v4f q = *reinterpret_cast<const v4f*>(row + i);
#pragma unroll
            for (int e = 0; e < 4; e++) y[e] = q[e];
        } else {
            y[0] = row[i];
        }
    };
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
        const uint32_t i = (k * 256 + tid) * STEP;
#pragma unroll
        for (int e = 0; e < STEP; e++) v[k][e] = 0.f;
        if (i < width) load(i, v[k]);
    }
#pragma unroll
    for (int k = 0; k < KEEP; k++)
#pragma unroll
        for (int e = 0; e < STEP; e++) {
            v[k][e] *= in_scale;
            ss = fmaf(v[k][e], v[k][e], ss);
        }
    for (uint32_t i = (KEEP * 256 + tid) * STEP; i < width; i += 256 * STEP) {
        float y[STEP];
        load(i, y);
#pragma unroll
        for (int e = 0; e < STEP; e++) ss = fmaf(y[e] * in_scale, y[e] * in_scale, ss);
    }
    ss = wave_sum_f32(ss);
    if ((tid & 63u) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)width + eps);
    auto store = [&](uint32_t i, const float (&y)[STEP]) {
        if constexpr (VEC) {
            const v4f g = *reinterpret_cast<const v4f*>(w + i);
            typename Dt<T>::quad q;
#pragma unroll
            for (int e = 0; e < 4; e++) q[e] = (T)(y[e] * inv * g[e]);
            *reinterpret_cast<typename Dt<T>::quad*>(o + i) = q;
            if (in_scale != 1.0f) *reinterpret_cast<v4f*>(row + i) = (v4f){y[0], y[1], y[2], y[3]};
        } else {
            o[i] = (T)(y[0] * inv * w[i]);
            if (in_scale != 1.0f) row[i] = y[0];
        }
    };
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
        const uint32_t i = (k * 256 + tid) * STEP;
        if (i < width) store(i, v[k]);
    }
    for (uint32_t i = (KEEP * 256 + tid) * STEP; i < width; i += 256 * STEP) {
        float y[STEP];
        load(i, y);
#pragma unroll
        for (int e = 0; e < STEP; e++) y[e] *= in_scale;
        store(i, y);
    }
    for (uint32_t i = width + tid; i < fill; i += 256) o[i] = (T)0.f;
}

hipError_t oxb_launch_row_norm(float* x, uint32_t width, uint32_t m, float in_scale, const float* w, float eps, void* out, uint32_t ld,
                               uint32_t fill, int dt, hipStream_t st) {
    if (!x || !width || !m || !w || !out || fill > ld || ld < width || ld % 8) return hipErrorInvalidValue;
    const bool vec = width % 4 == 0;
    if (dt == OXB_DT_BF16) {
        if (vec) hipLaunchKernelGGL((row_norm_kernel<__bf16, true>), dim3(m), dim3(256), 0, st, x, width, in_scale, w, eps, (__bf16*)out, ld, fill);
        else hipLaunchKernelGGL((row_norm_kernel<__bf16, false>), dim3(m), dim3(256), 0, st, x, width, in_scale, w, eps, (__bf16*)out, ld, fill);
    } else {
        if (vec) hipLaunchKernelGGL((row_norm_kernel<float, true>), dim3(m), dim3(256), 0, st, x, width, in_scale, w, eps, (float*)out, ld, fill);
        else hipLaunchKernelGGL((row_norm_kernel<float, false>), dim3(m), dim3(256), 0, st, x, width, in_scale, w, eps, (float*)out, ld, fill);
    }
    return hipGetLastError();
}
