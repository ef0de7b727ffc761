// mixer_kernels.hip — attention's and a recurrence's decode work in shared launches (see mixer_kernels.h).
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "mixer_kernels.h"
#include "recurrent_device.h"
#include "row_attention_device.h"

// Grid (step's workgroups, then the store's; token row).
template <typename T, int E, int RPT>
__global__ __launch_bounds__(256, RPT <= 4 ? 7 : 4) void pair_enter_kernel(OxbGroupedStore s, OxbRecurParams r, uint32_t n_step) {
    if (blockIdx.x < n_step) recur_step<float, RPT, 1, false, true>(r, 1, blockIdx.x, blockIdx.y);
    else grouped_store<T, E, 1>(s, blockIdx.y, blockIdx.x - n_step);
}

// Grid (heads, then the recurrence's parts; token row).  E: values per lane of a part, 0: long parts.
template <typename T, int E>
__global__ __launch_bounds__(E ? 256 : 1024) void pair_leave_kernel(OxbRowAttnParams a, OxbRecurParams r) {
    if (blockIdx.x < a.heads) {
        row_merge<T>(a, blockIdx.x, blockIdx.y);
    } else {
        if constexpr (E > 0) recur_finish<T, E, 1>(r, blockIdx.y, blockIdx.x - a.heads);
        else recur_finish_long<T>(r, blockIdx.y, blockIdx.x - a.heads);
    }
}

bool oxb_pair_ok(const OxbGroupedStore& s, const OxbRecurParams& r) {
    return s.rows.seq_step && r.rows.seq_step && s.rows.m == r.rows.m && s.rows.m <= 65535 && !oxb_recur_step_finishes(r.d);
}

template <typename T, int E>
static void launch_enter(const OxbGroupedStore& s, const OxbRecurParams& r, hipStream_t st) {
    const uint32_t n_step = r.d.heads * r.d.slices;
    const dim3 grid(n_step + (s.heads + 2 * s.kv_heads + 3) / 4, s.rows.m);
    if (r.d.dk_p <= 64) hipLaunchKernelGGL((pair_enter_kernel<T, E, 2>), grid, dim3(256), 0, st, s, r, n_step);
    else if (r.d.dk_p <= 128) hipLaunchKernelGGL((pair_enter_kernel<T, E, 4>), grid, dim3(256), 0, st, s, r, n_step);
    else hipLaunchKernelGGL((pair_enter_kernel<T, E, 8>), grid, dim3(256), 0, st, s, r, n_step);
}
template <typename T>
static void pick_enter(const OxbGroupedStore& s, const OxbRecurParams& r, hipStream_t st) {
    const uint32_t widest = s.dim_p > s.vdim_p ? s.dim_p : s.vdim_p;
    if (widest <= 64) launch_enter<T, 1>(s, r, st);
    else if (widest <= 128) launch_enter<T, 2>(s, r, st);
    else launch_enter<T, 4>(s, r, st);
}

hipError_t oxb_launch_pair_enter(const OxbGroupedStore& s, const OxbRecurParams& r, int dt, hipStream_t st) {
    if (!oxb_pair_ok(s, r) || !oxb_grouped_store_ok(s, dt) || !oxb_recur_params_ok(r)) return hipErrorInvalidValue;
    if (dt == OXB_DT_BF16) pick_enter<__bf16>(s, r, st);
    else pick_enter<float>(s, r, st);
    return hipGetLastError();
}

template <typename T>
static void pick_leave(const OxbRowAttnParams& a, const OxbRecurParams& r, hipStream_t st) {
    const uint32_t parts = r.d.heads * r.d.dv / r.d.norm_len;
    const dim3 some(a.heads + (parts + 3) / 4, a.rows.m), each(a.heads + parts, a.rows.m);
    if (r.d.norm_len <= 64) hipLaunchKernelGGL((pair_leave_kernel<T, 1>), some, dim3(256), 0, st, a, r);
    else if (r.d.norm_len <= 128) hipLaunchKernelGGL((pair_leave_kernel<T, 2>), some, dim3(256), 0, st, a, r);
    else if (r.d.norm_len <= 256) hipLaunchKernelGGL((pair_leave_kernel<T, 4>), some, dim3(256), 0, st, a, r);
    else hipLaunchKernelGGL((pair_leave_kernel<T, 0>), each, dim3(1024), 0, st, a, r);
}

hipError_t oxb_launch_pair_leave(const OxbRowAttnParams& a, const OxbRecurParams& r, int dt, hipStream_t st) {
    if (!oxb_row_merge_ok(a, dt) || !oxb_recur_finish_ok(r) || a.rows.m != r.rows.m || a.rows.m > 65535) return hipErrorInvalidValue;
    if (dt == OXB_DT_BF16) pick_leave<__bf16>(a, r, st);
    else pick_leave<float>(a, r, st);
    return hipGetLastError();
}
