// mixer_kernels.h — decode steps of a layer with grouped attention and a recurrence side by side: the work in front of the
// attention (store of the new tokens, step of the states) in one launch, the work behind it (merge of the splits, gate and norm
// of the recurrence) in another.
#pragma once
#include "recurrent_kernels.h"
#include "row_attention.h"

// One token per sequence in both; recurrences that do not finish in their step.
bool oxb_pair_ok(const OxbGroupedStore& s, const OxbRecurParams& r);
hipError_t oxb_launch_pair_enter(const OxbGroupedStore& s, const OxbRecurParams& r, int dt, hipStream_t st);
hipError_t oxb_launch_pair_leave(const OxbRowAttnParams& a, const OxbRecurParams& r, int dt, hipStream_t st);
