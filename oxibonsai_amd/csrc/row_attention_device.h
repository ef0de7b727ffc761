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
