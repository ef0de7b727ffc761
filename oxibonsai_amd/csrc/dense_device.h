// dense_device.h — matrix-core operands of 32 k-values in bf16 or fp32, and the scalar functions of the dense designs.
//
// One unit of work is a 16 x 16 x 32 product.  bf16: one v_mfma_f32_16x16x32_bf16, lane 16 g + r holding row r,
// k = 8 g + e.  fp32: eight v_mfma_f32_16x16x4_f32 (full 32-bit multiply and add), step e taking element e of every lane,
// so the four k-values of a step are 8 g + e, g = 0..3: the order of k inside a unit is free as long as both operands use
// the same one, and kernels are written once for both types.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "dense_kernels.h"
#include "device_utils.h"

typedef __bf16 v8b __attribute__((ext_vector_type(8)));
typedef __bf16 v4b __attribute__((ext_vector_type(4)));
typedef float v8f __attribute__((ext_vector_type(8)));

template <typename T> struct Dt;
template <> struct Dt<__bf16> {
    typedef v8b frag;
    typedef v4b quad;
    static constexpr bool is_f32 = false;
    static constexpr uint32_t unit_bytes = 1024, sub = 1;  // 1 KiB pieces per unit
};
template <> struct Dt<float> {
    typedef v8f frag;
    typedef v4f quad;
    static constexpr bool is_f32 = true;
    static constexpr uint32_t unit_bytes = 2048, sub = 2;
};

__device__ __forceinline__ v4f mfma32(v8b a, v8b b, v4f c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ v4f mfma32(v8f a, v8f b, v4f c) {
#pragma unroll
    for (int e = 0; e < 8; e++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], c, 0, 0, 0);
    return c;
}

// The lane's eight elements of a unit in operand order (global or LDS memory).
__device__ __forceinline__ v8b load_unit(const __bf16* unit, uint32_t lane) { return *reinterpret_cast<const v8b*>(unit + lane * 8); }
__device__ __forceinline__ v8f load_unit(const float* unit, uint32_t lane) {
    const v4f a = *reinterpret_cast<const v4f*>(unit + lane * 4), b = *reinterpret_cast<const v4f*>(unit + 256 + lane * 4);
    return (v8f){a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}
__device__ __forceinline__ void store_unit(__bf16* unit, uint32_t lane, v8b v) { *reinterpret_cast<v8b*>(unit + lane * 8) = v; }
__device__ __forceinline__ void store_unit(float* unit, uint32_t lane, v8f v) {
    *reinterpret_cast<v4f*>(unit + lane * 4) = (v4f){v[0], v[1], v[2], v[3]};
    *reinterpret_cast<v4f*>(unit + 256 + lane * 4) = (v4f){v[4], v[5], v[6], v[7]};
}
// Eight consecutive elements of a row.
__device__ __forceinline__ v8b load_row8(const __bf16* p) { return *reinterpret_cast<const v8b*>(p); }
__device__ __forceinline__ v8f load_row8(const float* p) {
    const v4f a = *reinterpret_cast<const v4f*>(p), b = *reinterpret_cast<const v4f*>(p + 4);
    return (v8f){a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}
__device__ __forceinline__ v8b zero_frag(const __bf16*) { return (v8b)(__bf16)0.f; }
__device__ __forceinline__ v8f zero_frag(const float*) { return (v8f)0.f; }

// Memory -> LDS without a trip through registers, 16 bytes per lane: lane l's 16 bytes land at base + 16 l (base is
// wave-uniform).  `src` is the lane's own address.  Written as an instruction, not through the compiler's builtin: the
// builtin makes the compiler wait for every outstanding copy in front of any LDS read that it cannot tell apart from the
// copies' target, and the kernels here read one buffer while the next one fills.  They place the waits themselves
// (wait_lds_copies, or a counted wait), always together with a barrier or before the wave's own reads; those waits carry the
// memory clobber that keeps LDS accesses on their side.
__device__ __forceinline__ void copy16_to_lds(const void* src, void* lds_base) {
    const uint32_t at = (uint32_t)__builtin_amdgcn_readfirstlane((int)(uint32_t)(uintptr_t)(__attribute__((address_space(3))) void*)lds_base);
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(at), "v"(src) : "m0");
}
// The same with the lane's address OFF bytes further on (an immediate of the instruction, which counts for the LDS address
// too and is taken off there) and the LDS address as a number.
template <int OFF>
__device__ __forceinline__ void copy16_to_lds_at(const void* src, uint32_t lds_at) {
    static_assert(OFF >= 0 && OFF < 4096, "immediate offset");
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off offset:%2" ::"s"(lds_at - OFF), "v"(src), "n"(OFF) : "m0");
}
__device__ __forceinline__ uint32_t lds_address(const void* p) {
    return (uint32_t)__builtin_amdgcn_readfirstlane((int)(uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void*)p);
}
// Staged units: 16 rows x 32 columns in LDS, filled by such copies from row-major memory.  Lane l brings columns
// 8 stage_col(l) .. + 7 of row stage_row(l), so four lanes in turn read one row's 64 (128) contiguous bytes, and its 16 bytes
// land in slot l: row r, column group g sits in slot 4 r + (g ^ (r >> 2)).  The exclusive-or keeps the operand reads of the
// matrix cores (16 rows, one column group) on distinct banks.  fp32: the first halves of all groups, then the second.
__device__ __forceinline__ uint32_t stage_row(uint32_t lane) { return lane >> 2; }
__device__ __forceinline__ uint32_t stage_col(uint32_t lane) { return (lane & 3u) ^ (lane >> 4); }
__device__ __forceinline__ uint32_t staged_slot(uint32_t r, uint32_t g) { return r * 4 + (g ^ (r >> 2)); }
__device__ __forceinline__ void stage_unit(const __bf16* row8, __bf16* unit) { copy16_to_lds(row8, unit); }
__device__ __forceinline__ void stage_unit(const float* row8, float* unit) {
    copy16_to_lds(row8, unit);
    copy16_to_lds(row8 + 4, unit + 256);
}
// Operand of lane 16 g + r: `slot` = staged_slot(r, g).
__device__ __forceinline__ v8b load_staged(const __bf16* unit, uint32_t slot) { return *reinterpret_cast<const v8b*>(unit + slot * 8); }
__device__ __forceinline__ v8f load_staged(const float* unit, uint32_t slot) { return load_unit(unit, slot); }
__device__ __forceinline__ void wait_lds_copies() { asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); }

// tanh in fp32: the library's for the fp32 kernels; for bf16 results 1 - 2 / (e^(2|z|) + 1) on the hardware exponential
// (absolute error around 1e-7), with the odd series near zero where that form cancels.
template <typename T> __device__ __forceinline__ float tanh_of(float z) {
    if constexpr (Dt<T>::is_f32) return tanhf(z);
    const float a = fabsf(z);
    const float e = __builtin_amdgcn_exp2f(a * 2.8853900817779268f);
    const float big = 1.0f - 2.0f * __builtin_amdgcn_rcpf(e + 1.0f);
    const float s = a * a;
    const float small = a * (1.0f + s * (-0.33333333333f + s * (0.13333333333f - 0.053968253968f * s)));
    return copysignf(a < 0.125f ? small : big, z);
}
template <typename T> __device__ __forceinline__ float gelu_tanh_of(float z) {
    return 0.5f * z * (1.0f + tanh_of<T>(0.79788456080286536f * (z + 0.044715f * z * z * z)));
}
// 2^z, z <= 0 or little above in every use.
template <typename T> __device__ __forceinline__ float exp2_of(float z) {
    if constexpr (Dt<T>::is_f32) return exp2f(z);
    return __builtin_amdgcn_exp2f(z);
}
// Eight fp32 weights as a matrix-core operand.  bf16: v = hi + lo, hi the upper half of v's bits (exact), lo the rounded
// rest: 16 bits of the weight in two operands.
__device__ __forceinline__ void split_hi_lo(const float (&v)[8], v8b& hi, v8b& lo) {
    typedef uint32_t v4w __attribute__((ext_vector_type(4)));
    v4w h;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const uint32_t a = __float_as_uint(v[2 * i]), b = __float_as_uint(v[2 * i + 1]);
        h[i] = __builtin_amdgcn_perm(b, a, 0x07060302u);
        lo[2 * i] = (__bf16)(v[2 * i] - __uint_as_float(a & 0xFFFF0000u));
        lo[2 * i + 1] = (__bf16)(v[2 * i + 1] - __uint_as_float(b & 0xFFFF0000u));
    }
    hi = __builtin_bit_cast(v8b, h);
}
__device__ __forceinline__ void split_hi_lo(const float (&v)[8], v8f& hi, v8f& lo) {
    hi = (v8f){v[0], v[1], v[2], v[3], v[4], v[5], v[6], v[7]};
    lo = hi;   // (not used)
}

// The residual's four values for outputs y[m][n0 .. n0 + 3], requested ahead of the arithmetic (zeros where epilogue4 fetches
// them itself).
__device__ __forceinline__ bool epilogue_whole(const OxbEpilogue& e, uint32_t n0) { return n0 + 4 <= e.n && (e.ld32 & 3u) == 0; }
__device__ __forceinline__ v4f epilogue_resid(const OxbEpilogue& e, uint32_t m, uint32_t n0) {
    if (!e.resid || !epilogue_whole(e, n0)) return (v4f){0.f, 0.f, 0.f, 0.f};
    return *reinterpret_cast<const v4f*>(e.resid + (size_t)m * e.ld32 + n0);
}
// Four consecutive outputs through the epilogue; resid = epilogue_resid(e, m, n0).  -> the outputs in front of the norm, zeros
// past the last column.
template <typename T> __device__ __forceinline__ v4f epilogue4(const OxbEpilogue& e, uint32_t m, uint32_t n0, v4f y, v4f resid) {
    if (e.glu_out && n0 >= e.glu) {
        const uint32_t j = (n0 - e.glu) >> 1;
        if (j >= e.n_glu) return y;
        y *= e.scale;
        typedef T pair __attribute__((ext_vector_type(2)));
        *reinterpret_cast<pair*>(reinterpret_cast<T*>(e.glu_out) + (size_t)m * e.ld_glu + j) =
            (pair){(T)(gelu_tanh_of<T>(y[0]) * y[1]), (T)(gelu_tanh_of<T>(y[2]) * y[3])};
        return y;
    }
    const uint32_t lim = e.n > e.fill ? e.n : e.fill;
    if (n0 >= lim) return (v4f){0.f, 0.f, 0.f, 0.f};
    y *= e.scale;
    v4f sum = {0.f, 0.f, 0.f, 0.f};
    if (epilogue_whole(e, n0)) {
        if (e.add) y += *reinterpret_cast<const v4f*>(e.add + n0);
        if (e.act == OXB_ACT_GELU_TANH) {
#pragma unroll
            for (int i = 0; i < 4; i++) y[i] = gelu_tanh_of<T>(y[i]);
        }
        const size_t o = (size_t)m * e.ld32 + n0;
        y += resid;
        sum = y;
        if (e.out32) *reinterpret_cast<v4f*>(e.out32 + o) = y;
        if (!e.out_t) return sum;
        if (e.norm == OXB_NORM_SCALE) y *= *reinterpret_cast<const v4f*>(e.nw + n0);
        if (e.norm == OXB_NORM_DYT) {
            const v4f w = *reinterpret_cast<const v4f*>(e.nw + n0), b = *reinterpret_cast<const v4f*>(e.nb + n0);
#pragma unroll
            for (int i = 0; i < 4; i++) y[i] = tanh_of<T>(e.alpha * y[i]) * w[i] + b[i];
        }
    } else {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t n = n0 + i;
            if (n >= e.n) {
                y[i] = 0.f;
                continue;
            }
            float v = y[i];
            if (e.add) v += e.add[n];
            if (e.act == OXB_ACT_GELU_TANH) v = gelu_tanh_of<T>(v);
            const size_t o = (size_t)m * e.ld32 + n;
            if (e.resid) v += e.resid[o];
            sum[i] = v;
            if (e.out32) e.out32[o] = v;
            if (e.norm == OXB_NORM_SCALE) v *= e.nw[n];
            if (e.norm == OXB_NORM_DYT) v = tanh_of<T>(e.alpha * v) * e.nw[n] + e.nb[n];
            y[i] = v;
        }
        if (!e.out_t) return sum;
    }
    T* t = reinterpret_cast<T*>(e.out_t) + (size_t)m * e.ld_t + n0;
    if (n0 + 4 <= e.fill && (((uintptr_t)t) & (sizeof(T) * 4 - 1)) == 0) {
        typename Dt<T>::quad q;
#pragma unroll
        for (int i = 0; i < 4; i++) q[i] = (T)y[i];
        *reinterpret_cast<typename Dt<T>::quad*>(t) = q;
    } else {
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (n0 + i < e.fill) t[i] = (T)y[i];
    }
    return sum;
}
