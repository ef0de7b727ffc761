// token_rows.h — the token rows of a launch.
#pragma once
#include <stdint.h>

// Row r is the token of sequence seq0 + r * seq_step at position pos[r] (device) or pos0 + r.
struct OxbRows {
    const uint32_t* pos;
    uint32_t pos0, seq0, seq_step, m;
};
static inline uint32_t oxb_pad32(uint32_t n) { return (n + 31u) / 32u * 32u; }
#if defined(__HIPCC__)
__device__ __forceinline__ uint32_t row_pos(const OxbRows& r, uint32_t m) { return r.pos ? r.pos[m] : r.pos0 + m; }
__device__ __forceinline__ uint32_t row_seq(const OxbRows& r, uint32_t m) { return r.seq0 + m * r.seq_step; }
#endif
