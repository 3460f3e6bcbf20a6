// What the attention kernels over the paged cache share: which keys a query sees, what happens to scores and
// outputs, and how the outputs of a head's two softmax maps become one.
#pragma once
#include "common.h"

// The first key a query at position p sees (kept first positions aside).
__device__ __forceinline__ int aw_first_key(int p, int window, int chunk) {
    int lo = window > 0 ? max(0, p + 1 - window) : 0;
    if (chunk > 0) lo = max(lo, p - p % chunk);
    return lo;
}

// What a head's output is multiplied by after the softmax: the sigmoid of one logit a token and head (token t, head h at
// gate[t * stride + h]); no gate: 1.
template <typename T>
struct HeadGate {
    const T* gate;
    int stride;
    __device__ __forceinline__ float at(int t, int head) const {
        return gate ? 1.f / (1.f + expf(-ld_f32(gate + (size_t)t * stride + head))) : 1.f;
    }
};

// How the outputs of a head's two maps become one (maps = 2).
struct DiffHow { float lam, gain, eps; };

// A wave writes a head's output from its two maps' outputs, NC values of each a lane (feature lane + 64 c).
template <typename T, int NC>
__device__ __forceinline__ void aw_write_difference(T* __restrict__ o, const float (&a)[NC], const float (&b)[NC], int dv, int lane, DiffHow how) {
    float y[NC], ss = 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
        y[c] = lane + 64 * c < dv ? a[c] - how.lam * b[c] : 0.f;
        ss = fmaf(y[c], y[c], ss);
    }
    ss = wave_sum(ss);
    const float f = how.gain / sqrtf(ss / (float)dv + how.eps);
#pragma unroll
    for (int c = 0; c < NC; ++c)
        if (lane + 64 * c < dv) st_f32(o + lane + 64 * c, y[c] * f);
}
