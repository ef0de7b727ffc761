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
                                                         const int64_t* __restrict__ col_off, uint32_t n_units_k, T* __restrict__ dst) {
    const uint32_t j = threadIdx.x, lane = j >> 3, e = j & 7u;
    const uint32_t tile = blockIdx.x / n_units_k, u = blockIdx.x % n_units_k;
    const int64_t ro = row_off[tile * 16 + (lane & 15u)], co = col_off[u * 32 + (lane >> 4) * 8 + e];
    float v = 0.f;
    if (ro >= 0 && co >= 0) {
        const int64_t i = ro + co;
        if (type == 0) v = static_cast<const float*>(src)[i];
        else if (type == 1) v = __half2float(static_cast<const __half*>(src)[i]);
        else v = __uint_as_float((uint32_t)static_cast<const uint16_t*>(src)[i] << 16);
    }
    T* unit = dst + (size_t)blockIdx.x * 512;
    if constexpr (Dt<T>::is_f32) unit[(e >> 2) * 256 + lane * 4 + (e & 3u)] = v;
    else unit[lane * 8 + e] = (T)v;
}

hipError_t oxb_launch_dense_pack(const void* src, int src_type, const int64_t* row_off, const int64_t* col_off, uint32_t n_pad,
                                 uint32_t k_pad, int dt, void* dst, hipStream_t st) {
    if (!src || !dst || !row_off || !col_off || n_pad % 16 || k_pad % 32 || !n_pad || !k_pad || (src_type != 0 && src_type != 1 && src_type != 30))
        return hipErrorInvalidValue;
    const uint32_t nu = k_pad / 32;
    const uint64_t grid = (uint64_t)(n_pad / 16) * nu;
    if (grid > 0x7FFFFFFFull) return hipErrorInvalidValue;
    if (dt == OXB_DT_BF16)
        hipLaunchKernelGGL((dense_pack_kernel<__bf16>), dim3((uint32_t)grid), dim3(512), 0, st, src, src_type, row_off, col_off, nu, (__bf16*)dst);
    else
        hipLaunchKernelGGL((dense_pack_kernel<float>), dim3((uint32_t)grid), dim3(512), 0, st, src, src_type, row_off, col_off, nu, (float*)dst);
    return hipGetLastError();
}

__device__ __forceinline__ size_t x_row(const OxbDenseParams& p, uint32_t t) {
    if (p.row_table) return ((size_t)p.row_table[t >> p.row_shift] << p.row_shift) + (t & ((1u << p.row_shift) - 1u));
    return p.row0 + t;
}

// ---------------------------------------------------------------------------
// Few rows (m <= 16 per grid row): a workgroup of 8 waves owns RT row tiles and splits K over its waves; wave w takes the
// units w, w + 8, ... so that the workgroup walks its tile's bytes in order.  The token rows are the columns of the
// product: lane 16 g + c loads eight activations of token c, lanes of absent tokens supply zeros.  UN units are in flight
// per wave.  The waves' sums meet in LDS and are added in wave order.
// ---------------------------------------------------------------------------
template <typename T, int RT, int UN>
__global__ __launch_bounds__(512) void dense_gemv_kernel(OxbDenseParams p) {
    typedef typename Dt<T>::frag frag;
    __shared__ __attribute__((aligned(16))) float red[8][RT][16][20];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, c = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t nu = p.k_pad / 32, n_tiles = p.n_pad / 16, m0 = blockIdx.y * 16, mc = min(p.m - m0, 16u);
    const T* w[RT];
#pragma unroll
    for (int r = 0; r < RT; r++) w[r] = reinterpret_cast<const T*>(p.w) + (size_t)min(blockIdx.x * RT + r, n_tiles - 1) * nu * 512;
    const bool have = c < mc;
    const T* x = reinterpret_cast<const T*>(p.x) + (have ? x_row(p, m0 + c) : 0) * p.ldx + 8 * g;
    v4f acc[RT];
#pragma unroll
    for (int r = 0; r < RT; r++) acc[r] = (v4f){0.f, 0.f, 0.f, 0.f};
    for (uint32_t u0 = wave; u0 < nu; u0 += 8 * UN) {
        frag b[UN], a[UN][RT];
#pragma unroll
        for (int i = 0; i < UN; i++) {
            const uint32_t u = u0 + 8 * i;
            b[i] = have && u < nu && 32 * u + 8 * g + 8 <= p.ldx ? load_row8(x + 32 * u) : zero_frag((const T*)nullptr);
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
            for (int r = 0; r < RT; r++) acc[r] = mfma32(a[i][r], b[i], acc[r]);
    }
#pragma unroll
    for (int r = 0; r < RT; r++) *reinterpret_cast<v4f*>(&red[wave][r][c][4 * g]) = acc[r];
    __syncthreads();
    if (tid < 64 * RT) {
        const uint32_t r = tid >> 6, q = tid & 3u, t = (tid & 63u) >> 2;
        v4f y = *reinterpret_cast<const v4f*>(&red[0][r][t][4 * q]);
#pragma unroll
        for (int i = 1; i < 8; i++) y += *reinterpret_cast<const v4f*>(&red[i][r][t][4 * q]);
        if (t < mc && blockIdx.x * RT + r < n_tiles) epilogue4<T>(p.e, m0 + t, (blockIdx.x * RT + r) * 16 + 4 * q, y);
    }
}

// ---------------------------------------------------------------------------
// Tiled GEMM: a workgroup of 4 waves owns 64 RT rows x 16 CT tokens.  The weights come from memory already in operand
// order, so each wave loads its own RT tiles straight into registers, one stage ahead; the token tile is shared by the
// waves and goes memory -> LDS without registers, also in operand order (every LDS access is linear in the lane), two
// stages.  A stage is UK units of k (64 values bf16, 32 fp32).  SWAP exchanges the operands' roles: the lane then holds
// four consecutive tokens of one output row, which is the transposed store of the value rows of attention.
// ---------------------------------------------------------------------------
template <typename T, int RT, int CT, bool SWAP>
__global__ __launch_bounds__(256, 2) void dense_gemm_kernel(OxbDenseParams p, uint32_t n_tm, uint32_t n_tn) {
    typedef typename Dt<T>::frag frag;
    constexpr int UK = Dt<T>::is_f32 ? 1 : 2;
    constexpr int UNITS = CT * UK;          // LDS units of a stage
    __shared__ __attribute__((aligned(16))) T xs[2][UNITS * 512];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, c = lane & 15u, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    // consecutive workgroups go to different XCDs: give each XCD a contiguous run of tiles with the token tiles innermost,
    // so that the workgroups sharing a row tile's weights share an L2
    const uint32_t total = n_tm * n_tn, per = (total + 7) / 8, id = (blockIdx.x & 7u) * per + (blockIdx.x >> 3);
    if (id >= total || (blockIdx.x >> 3) >= per) return;
    const uint32_t tm = id % n_tm, tn = id / n_tm;
    const uint32_t nu = p.k_pad / 32, n_tiles = p.n_pad / 16, n_stages = nu / UK;  // (k_pad is a multiple of 64)
    const T* w[RT];
#pragma unroll
    for (int r = 0; r < RT; r++) w[r] = reinterpret_cast<const T*>(p.w) + (size_t)min((tn * 4 + wave) * RT + r, n_tiles - 1) * nu * 512;
    // the units of the token tile this wave brings in: unit i -> token tile i / UK, k unit i % UK
    constexpr int MINE = (UNITS + 3) / 4;
    const T* xr[MINE];
#pragma unroll
    for (int i = 0; i < MINE; i++) {
        const uint32_t un = wave + 4 * i;
        xr[i] = reinterpret_cast<const T*>(p.x) + x_row(p, min(tm * (16 * CT) + (un / UK) * 16 + c, p.m - 1)) * p.ldx;
    }
    auto stage_x = [&](uint32_t st, int buf) {
#pragma unroll
        for (int i = 0; i < MINE; i++) {
            const uint32_t un = wave + 4 * i;
            if (UNITS % 4 == 0 || un < (uint32_t)UNITS) {
                // (columns past the row's end meet zero weights; any finite value will do)
                const uint32_t k = min((st * UK + un % UK) * 32 + 8 * g, p.ldx - 8);
                copy_row8_to_unit(xr[i] + k, &xs[buf][un * 512]);
            }
        }
    };
    v4f acc[RT][CT];
#pragma unroll
    for (int r = 0; r < RT; r++)
#pragma unroll
        for (int t = 0; t < CT; t++) acc[r][t] = (v4f){0.f, 0.f, 0.f, 0.f};
    frag a[UK][RT];
    stage_x(0, 0);
#pragma unroll
    for (int k = 0; k < UK; k++)
#pragma unroll
        for (int r = 0; r < RT; r++) a[k][r] = load_unit(w[r] + (size_t)min((uint32_t)k, nu - 1) * 512, lane);
    for (uint32_t st = 0; st < n_stages; st++) {
        wait_lds_copies();
        __syncthreads();
        const int buf = st & 1u;
        if (st + 1 < n_stages) stage_x(st + 1, buf ^ 1);
#pragma unroll
        for (int k = 0; k < UK; k++) {
#pragma unroll
            for (int t = 0; t < CT; t++) {
                const frag b = load_unit(&xs[buf][(t * UK + k) * 512], lane);
#pragma unroll
                for (int r = 0; r < RT; r++) acc[r][t] = SWAP ? mfma32(b, a[k][r], acc[r][t]) : mfma32(a[k][r], b, acc[r][t]);
            }
            const uint32_t un = min((st + 1) * UK + k, nu - 1);
#pragma unroll
            for (int r = 0; r < RT; r++) a[k][r] = load_unit(w[r] + (size_t)un * 512, lane);
        }
    }
#pragma unroll
    for (int r = 0; r < RT; r++) {
        const uint32_t tile = (tn * 4 + wave) * RT + r;
        if (tile >= n_tiles) continue;
#pragma unroll
        for (int t = 0; t < CT; t++) {
            if constexpr (SWAP) {
                typename Dt<T>::quad q;
#pragma unroll
                for (int i = 0; i < 4; i++) q[i] = (T)(acc[r][t][i] * p.e.scale);
                const uint32_t n = tile * 16 + c, m = (tm * CT + t) * 16 + 4 * g;
                if (n < p.e.n && m < p.e.ld_t) *reinterpret_cast<typename Dt<T>::quad*>(reinterpret_cast<T*>(p.e.out_t) + (size_t)n * p.e.ld_t + m) = q;
            } else {
                const uint32_t m = (tm * CT + t) * 16 + c;
                if (m < p.m) epilogue4<T>(p.e, m, tile * 16 + 4 * g, acc[r][t]);
            }
        }
    }
}

static hipError_t check(const OxbDenseParams& p, int dt) {
    if (!p.w || !p.x || !p.m || !p.n_pad || !p.k_pad || p.n_pad % OXB_DENSE_PAD || p.k_pad % OXB_DENSE_PAD || p.ldx < 32 || p.ldx % 8 ||
        (dt != OXB_DT_BF16 && dt != OXB_DT_F32) || p.e.n > p.n_pad || p.e.fill > p.n_pad || (p.row_table && (p.row_shift < 4 || p.row_shift > 7)))
        return hipErrorInvalidValue;
    return hipSuccess;
}

template <typename T, int RT, int CT, bool SWAP>
static hipError_t launch_gemm(const OxbDenseParams& p, hipStream_t st) {
    const uint32_t n_tm = (p.m + 16 * CT - 1) / (16 * CT), n_tn = (p.n_pad + 64 * RT - 1) / (64 * RT);
    hipLaunchKernelGGL((dense_gemm_kernel<T, RT, CT, SWAP>), dim3((n_tm * n_tn + 7) / 8 * 8), dim3(256), 0, st, p, n_tm, n_tn);
    return hipGetLastError();
}

// Rounds of workgroups over the CUs (two resident per CU) x what one costs: the smallest estimate wins, larger tiles first
// among equals.
template <typename T, bool SWAP>
static hipError_t pick_gemm(const OxbDenseParams& p, uint32_t n_cus, hipStream_t st) {
    struct { int rt, ct; double mac_cost; } const opt[] = {{4, 8, 1.0}, {2, 8, 1.15}, {4, 4, 1.2}, {2, 4, 1.4}, {1, 8, 1.5}, {1, 4, 1.8}};
    int best = 0;
    double best_cost = 0;
    for (int i = 0; i < 6; i++) {
        const double wgs = (double)((p.m + 16 * opt[i].ct - 1) / (16 * opt[i].ct)) * ((p.n_pad + 64 * opt[i].rt - 1) / (64 * opt[i].rt));
        const double slots = n_cus, rounds = wgs <= slots ? 1.0 : (double)(uint64_t)((wgs + slots - 1) / slots);
        const double cost = rounds * opt[i].rt * opt[i].ct * opt[i].mac_cost;
        if (i == 0 || cost < best_cost) best = i, best_cost = cost;
    }
    switch (best) {
        case 0: return launch_gemm<T, 4, 8, SWAP>(p, st);
        case 1: return launch_gemm<T, 2, 8, SWAP>(p, st);
        case 2: return launch_gemm<T, 4, 4, SWAP>(p, st);
        case 3: return launch_gemm<T, 2, 4, SWAP>(p, st);
        case 4: return launch_gemm<T, 1, 8, SWAP>(p, st);
        default: return launch_gemm<T, 1, 4, SWAP>(p, st);
    }
}

template <typename T>
static hipError_t launch_gemv(const OxbDenseParams& p, uint32_t n_cus, hipStream_t st) {
    const uint32_t tiles = p.n_pad / 16, my = (p.m + 15) / 16;
    // units per wave and pass: as many as the wave has, up to what keeps the registers within two workgroups per CU
    const uint32_t per_wave = (p.k_pad / 32 + 7) / 8;
    constexpr int BIG = Dt<T>::is_f32 ? 4 : 8;
    if (tiles >= 4 * n_cus) {
        hipLaunchKernelGGL((dense_gemv_kernel<T, 2, BIG / 2>), dim3((tiles + 1) / 2, my), dim3(512), 0, st, p);
    } else if (per_wave > 2) {
        hipLaunchKernelGGL((dense_gemv_kernel<T, 1, BIG>), dim3(tiles, my), dim3(512), 0, st, p);
    } else {
        hipLaunchKernelGGL((dense_gemv_kernel<T, 1, 2>), dim3(tiles, my), dim3(512), 0, st, p);
    }
    return hipGetLastError();
}

hipError_t oxb_launch_dense(const OxbDenseParams& p, int dt, uint32_t n_cus, hipStream_t st) {
    const hipError_t e = check(p, dt);
    if (e != hipSuccess) return e;
    if (p.m <= OXB_DENSE_GEMV_MAX_ROWS) return dt == OXB_DT_BF16 ? launch_gemv<__bf16>(p, n_cus, st) : launch_gemv<float>(p, n_cus, st);
    return dt == OXB_DT_BF16 ? pick_gemm<__bf16, false>(p, n_cus, st) : pick_gemm<float, false>(p, n_cus, st);
}

hipError_t oxb_launch_dense_gemm_t(const OxbDenseParams& p, int dt, uint32_t n_cus, hipStream_t st) {
    const hipError_t e = check(p, dt);
    if (e != hipSuccess) return e;
    if (!p.e.out_t || p.e.ld_t % 4) return hipErrorInvalidValue;
    return dt == OXB_DT_BF16 ? pick_gemm<__bf16, true>(p, n_cus, st) : pick_gemm<float, true>(p, n_cus, st);
}

template <typename T>
__global__ __launch_bounds__(256) void stream_enter_kernel(const float* __restrict__ x, uint32_t width, T* __restrict__ x0, uint32_t ld_x0,
                                                           uint32_t x0_col, uint32_t x0_fill, OxbEpilogue e) {
    const uint32_t m = blockIdx.x;
    const float* row = x + (size_t)m * width;
    if (x0)
        for (uint32_t i = threadIdx.x; x0_col + i < x0_fill; i += 256) x0[(size_t)m * ld_x0 + x0_col + i] = (T)(i < width ? row[i] : 0.f);
    const uint32_t lim = e.n > e.fill ? e.n : e.fill;
    for (uint32_t n0 = threadIdx.x * 4; n0 < lim; n0 += 1024) {
        v4f y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (n0 + i < width) y[i] = row[n0 + i];
        epilogue4<T>(e, m, n0, y);
    }
}

hipError_t oxb_launch_stream_enter(const float* x, uint32_t width, uint32_t m, void* x0_out, uint32_t ld_x0, uint32_t x0_col,
                                   uint32_t x0_fill, const OxbEpilogue& e, int dt, hipStream_t st) {
    if (!x || !width || !m || (x0_out && (x0_fill > ld_x0 || x0_col + width > x0_fill)) || !e.out_t || e.n != width) return hipErrorInvalidValue;
    if (dt == OXB_DT_BF16)
        hipLaunchKernelGGL((stream_enter_kernel<__bf16>), dim3(m), dim3(256), 0, st, x, width, (__bf16*)x0_out, ld_x0, x0_col, x0_fill, e);
    else
        hipLaunchKernelGGL((stream_enter_kernel<float>), dim3(m), dim3(256), 0, st, x, width, (float*)x0_out, ld_x0, x0_col, x0_fill, e);
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
