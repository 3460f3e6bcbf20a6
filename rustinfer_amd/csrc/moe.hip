// A feed-forward of many small experts of which every token uses a few.
//
//   moe_route           32-bit router logits [T][E] -> weights [T][E]: the softmax probability for the
//                       `top` experts with the largest probabilities (ties: the lower index), 0 for
//                       the others; optionally divided by the chosen ones' sum.
//   moe_swiglu_weighted act[t][e F + i] = weight[t][e] * silu(gu[t][e 2F + i]) * gu[t][e 2F + F + i]:
//                       the experts' activations side by side, each scaled by its token's weight, so
//                       that ONE product with the experts' down matrices side by side is the weighted
//                       sum of the chosen experts' outputs (an expert that was not chosen adds zeros).
//                       A router may also score with a sigmoid of each logit instead of the softmax over all
//                       (the chosen scores divided by their sum + eps if renormalised), and multiply the
//                       weights by a constant.  Fs more columns after the experts' are a shared expert that
//                       every token uses with weight 1: act[t][E F + i] = silu(gu[t][2 E F + i]) * gu[t][2 E F + Fs + i];
//                       columns beyond E F + Fs up to the width given are zeros.
//                       The activation of a pair (g, u) of gate and up values may also be the clipped one:
//                       g' = min(g, limit), u' = clamp(u, -limit, limit), g' sigmoid(slope g') (u' + shift), with a
//                       limit of its own for the shared expert; the weight may multiply the expert's INPUT instead
//                       of its output (both of its pre-activations, then, since they are linear in it); and
//                       one more logit a token may gate the shared expert (its sigmoid in place of weight 1).
//                       Experts may also have no gate at all: act = relu(u)^2 of their up values u, gu then
//                       being [T][E F + Fs], F columns an expert.
//                       The router's logits may have a bias, and the weights may be the softmax over the
//                       chosen experts' logits alone.
//   moe_swiglu_routed   the two in one launch: every block makes its token's weights from the logits
//                       itself (what the engine runs; the two above are its halves, kept for callers
//                       that want the weights).
#include "common.h"
#include <math.h>

namespace {

constexpr int MOE_EPL = 8;       // experts a lane: up to 512 experts

enum { ROUTE_SOFTMAX = 0, ROUTE_SIGMOID = 1, ROUTE_CHOSEN = 2 };

// One wave: the weights of a token's experts from its logits z [E] into wr [E] (global or LDS).
struct RouteHow {
    int score;         // ROUTE_SOFTMAX over all experts, ROUTE_SIGMOID of each logit, ROUTE_CHOSEN: softmax over the chosen logits
    int renorm;        // the chosen scores are divided by their sum + eps
    float eps, scale;  // scale: a factor on every weight
    const float* bias; // [E] added to the logits, or null
};

__device__ __forceinline__ void route_token(const float* __restrict__ z, float* wr, int E, int top, RouteHow how, int lane) {
    const int renorm = how.renorm;
    float s[MOE_EPL];
    float m = -INFINITY;
#pragma unroll
    for (int j = 0; j < MOE_EPL; ++j) {
        const int e = lane + 64 * j;
        s[j] = e < E ? (how.bias ? z[e] + how.bias[e] : z[e]) : -INFINITY;
        m = fmaxf(m, s[j]);
    }
    m = wave_max(m);
    if (how.score == ROUTE_CHOSEN) {
        // ranked by the logits themselves; an expert that is there has a logit above -inf
        unsigned chosen = 0;
        float sum = 0.f;
        for (int n = 0; n < top; ++n) {
            float best = -INFINITY;
            int best_e = 0x7fffffff;
#pragma unroll
            for (int j = 0; j < MOE_EPL; ++j) {
                const int e = lane + 64 * j;
                if (!(chosen >> j & 1u) && e < E && (s[j] > best || (s[j] == best && e < best_e))) { best = s[j]; best_e = e; }
            }
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) {
                const float ob = __shfl_xor(best, o, 64);
                const int oe = __shfl_xor(best_e, o, 64);
                if (ob > best || (ob == best && oe < best_e)) { best = ob; best_e = oe; }
            }
            if (best_e < E && (best_e & 63) == lane) chosen |= 1u << (best_e >> 6);
            sum += expf(best - m);
        }
        const float f = how.scale / sum;
#pragma unroll
        for (int j = 0; j < MOE_EPL; ++j) {
            const int e = lane + 64 * j;
            if (e < E) wr[e] = (chosen >> j & 1u) ? expf(s[j] - m) * f : 0.f;
        }
        return;
    }
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < MOE_EPL; ++j) {
        if (how.score == ROUTE_SIGMOID) s[j] = (lane + 64 * j) < E ? 1.f / (1.f + expf(-s[j])) : -1.f;
        else s[j] = (lane + 64 * j) < E ? expf(s[j] - m) : -1.f;     // scores are >= 0: -1 marks "not there"
        if (s[j] > 0.f) sum += s[j];
    }
    sum = wave_sum(sum);
    const float inv = how.score == ROUTE_SIGMOID ? 1.f : 1.f / sum;
    unsigned chosen = 0;             // bit j: this lane's expert lane + 64 j is chosen
    float kept = 0.f;
    for (int n = 0; n < top; ++n) {
        float best = -1.f;
        int best_e = 0x7fffffff;
#pragma unroll
        for (int j = 0; j < MOE_EPL; ++j) {
            const int e = lane + 64 * j;
            if (!(chosen >> j & 1u) && e < E && (s[j] > best || (s[j] == best && e < best_e))) { best = s[j]; best_e = e; }
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ob = __shfl_xor(best, o, 64);
            const int oe = __shfl_xor(best_e, o, 64);
            if (ob > best || (ob == best && oe < best_e)) { best = ob; best_e = oe; }
        }
        if (best_e < E && (best_e & 63) == lane) chosen |= 1u << (best_e >> 6);
        kept += best * inv;
    }
    const float f = (renorm ? inv / (kept + how.eps) : inv) * how.scale;
#pragma unroll
    for (int j = 0; j < MOE_EPL; ++j) {
        const int e = lane + 64 * j;
        if (e < E) wr[e] = (chosen >> j & 1u) ? s[j] * f : 0.f;
    }
}

__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ logits, int l_stride, float* __restrict__ weights,
                                                       int T, int E, int top, RouteHow how) {
    const int lane = threadIdx.x & 63, t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= T) return;
    route_token(logits + (size_t)t * l_stride, weights + (size_t)t * E, E, top, how, lane);
}

enum { ACT_SILU = 0, ACT_CLIPPED = 1, ACT_RELU2 = 2 };

// What an expert does with its gate and up values, and where its weight goes.
struct ActHow {
    int form;                 // ACT_SILU: silu(g) u;  ACT_CLIPPED: the clipped form;  ACT_RELU2: relu(u)^2, no gate
    float limit, shared_limit, slope, shift;
    int weigh_input;          // the weight multiplies g and u (the expert's input), not the result
    __device__ __forceinline__ int cols() const { return form == ACT_RELU2 ? 1 : 2; }      // columns of gu a column of act
};

__device__ __forceinline__ float gated_pair(float g, float u, const ActHow& how, float limit) {
    if (how.form == ACT_RELU2) { u = fmaxf(u, 0.f); return u * u; }
    if (how.form == ACT_SILU) return (g / (1.f + expf(-g))) * u;
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return (g / (1.f + expf(-how.slope * g))) * (u + how.shift);
}

__device__ __forceinline__ float weighted_pair(float wgt, float g, float u, const ActHow& how) {
    return how.weigh_input ? gated_pair(wgt * g, wgt * u, how, how.limit) : wgt * gated_pair(g, u, how, how.limit);
}

// column i of the shared expert's activation from its gate and up columns [gate Fs | up Fs] (or [up Fs]); 0 beyond Fs.
// gate: the logit of its own gate, or null
template <typename T>
__device__ __forceinline__ float shared_column(const T* __restrict__ row, int i, int Fs, const ActHow& how, const float* __restrict__ gate) {
    if (i >= Fs) return 0.f;
    const float y = gated_pair(ld_f32(row + i), ld_f32(row + (how.cols() - 1) * Fs + i), how, how.shared_limit);
    return gate ? y / (1.f + expf(-*gate)) : y;
}

// moe_swiglu_weighted with the routing done on the way: the block's first wave makes the token's weights
// from its logits into LDS (every block of a token the same ones), then all threads use them.
template <typename T>
__global__ __launch_bounds__(256) void moe_swiglu_routed_kernel(const T* __restrict__ gu, int gu_stride, const float* __restrict__ logits,
                                                               int l_stride, T* __restrict__ act, int act_stride, int E, int F,
                                                               int top, RouteHow how, int Fs, int width, ActHow ah,
                                                               const float* __restrict__ sg, int sg_stride) {
    __shared__ float wts[64 * MOE_EPL];
    const int t = blockIdx.y;
    if (threadIdx.x < 64) route_token(logits + (size_t)t * l_stride, wts, E, top, how, threadIdx.x);
    __syncthreads();
    const int idx = blockIdx.x * 256 + threadIdx.x;
    if (idx >= width) return;
    if (idx >= E * F) { st_f32(act + (size_t)t * act_stride + idx, shared_column(gu + (size_t)t * gu_stride + (size_t)E * ah.cols() * F, idx - E * F, Fs, ah, sg ? sg + (size_t)t * sg_stride : nullptr)); return; }
    const int e = idx / F, i = idx - e * F;
    const float wgt = wts[e];
    float y = 0.f;
    if (wgt != 0.f) {
        const T* row = gu + (size_t)t * gu_stride + (size_t)e * ah.cols() * F;
        const float g = ld_f32(row + i), u = ld_f32(row + (ah.cols() - 1) * F + i);
        y = weighted_pair(wgt, g, u, ah);
    }
    st_f32(act + (size_t)t * act_stride + idx, y);
}

template <typename T>
__global__ __launch_bounds__(256) void moe_swiglu_weighted_kernel(const T* __restrict__ gu, int gu_stride, const float* __restrict__ weights,
                                                                 T* __restrict__ act, int act_stride, int E, int F, int Fs, int width, ActHow ah,
                                                                 const float* __restrict__ sg, int sg_stride) {
    const int t = blockIdx.y;
    const int idx = blockIdx.x * 256 + threadIdx.x;
    if (idx >= width) return;
    if (idx >= E * F) { st_f32(act + (size_t)t * act_stride + idx, shared_column(gu + (size_t)t * gu_stride + (size_t)E * ah.cols() * F, idx - E * F, Fs, ah, sg ? sg + (size_t)t * sg_stride : nullptr)); return; }
    const int e = idx / F, i = idx - e * F;
    const float wgt = weights[(size_t)t * E + e];
    float y = 0.f;
    if (wgt != 0.f) {
        const T* row = gu + (size_t)t * gu_stride + (size_t)e * ah.cols() * F;
        const float g = ld_f32(row + i), u = ld_f32(row + (ah.cols() - 1) * F + i);
        y = weighted_pair(wgt, g, u, ah);
    }
    st_f32(act + (size_t)t * act_stride + idx, y);
}

// moe_swiglu_weighted, eight columns a thread (16 bytes of bfloat16 a load): E F, Fs, the width and the strides
// multiples of eight, F a multiple of eight so that a thread's columns belong to one expert.  The columns of experts
// that a token did not choose are written without anything being read.
template <typename T>
__global__ __launch_bounds__(256) void moe_swiglu_weighted_vec_kernel(const T* __restrict__ gu, int gu_stride, const float* __restrict__ weights,
                                                                     T* __restrict__ act, int act_stride, int E, int F, int Fs, int width, ActHow ah,
                                                                     const float* __restrict__ sg, int sg_stride) {
    const int t = blockIdx.y;
    const int idx = (blockIdx.x * 256 + threadIdx.x) * 8;
    if (idx >= width) return;
    float y[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) y[u] = 0.f;
    const bool shared = idx >= E * F;
    const int e = shared ? E : idx / F, i = shared ? idx - E * F : idx - e * F, n = shared ? Fs : F;
    const float wgt = shared ? (i < Fs ? 1.f : 0.f) : weights[(size_t)t * E + e];
    if (wgt != 0.f) {
        const T* row = gu + (size_t)t * gu_stride + (size_t)e * ah.cols() * F + i;
        float g[8] = {}, up[8];
#pragma unroll
        for (int u = 0; u < 8; u += 4) {
            VecLoad<4>::ld(row + (ah.cols() - 1) * n + u, up + u);
            if (ah.form != ACT_RELU2) VecLoad<4>::ld(row + u, g + u);
        }
        if (shared) {
            const float f = sg ? 1.f + expf(-sg[(size_t)t * sg_stride]) : 1.f;
#pragma unroll
            for (int u = 0; u < 8; ++u) y[u] = gated_pair(g[u], up[u], ah, ah.shared_limit) / f;
        } else {
#pragma unroll
            for (int u = 0; u < 8; ++u) y[u] = weighted_pair(wgt, g[u], up[u], ah);
        }
    }
    T* dst = act + (size_t)t * act_stride + idx;
#pragma unroll
    for (int u = 0; u < 8; u += 4) VecLoad<4>::st(dst + u, y + u);
}

}  // namespace

extern "C" int ri_moe_route_as(const float* logits, int l_stride, float* weights, int T, int E, int top, int renorm,
                               int score, float eps, float scale, const float* bias, hipStream_t stream) {
    RI_REQUIRE(T >= 0 && E > 0 && top > 0 && top <= E && l_stride >= E, "ri_moe_route: bad sizes T=%d E=%d top=%d", T, E, top);
    RI_REQUIRE(score >= ROUTE_SOFTMAX && score <= ROUTE_CHOSEN, "ri_moe_route: unknown score %d", score);
    RI_REQUIRE(E <= 64 * MOE_EPL, "ri_moe_route: %d experts, the kernel takes up to %d", E, 64 * MOE_EPL);
    if (T == 0) return 0;
    RI_REQUIRE(logits && weights, "ri_moe_route: null pointer");
    const RouteHow how{score, renorm, eps, scale, bias};
    moe_route_kernel<<<(T + 3) / 4, 256, 0, stream>>>(logits, l_stride, weights, T, E, top, how);
    RI_LAUNCHED("ri_moe_route");
    return 0;
}

extern "C" int ri_moe_route(const float* logits, int l_stride, float* weights, int T, int E, int top, int renorm, hipStream_t stream) {
    return ri_moe_route_as(logits, l_stride, weights, T, E, top, renorm, ROUTE_SOFTMAX, 0.f, 1.f, nullptr, stream);
}

// Fs: columns of a shared expert behind the experts' (0: none); width: columns of act that are written
// (E F + Fs of activations, zeros beyond).  form, limit, shared_limit, slope, shift, weigh_input: see ActHow.
// sg (null: none): 32-bit logits of the shared expert's gate, token t's at sg[t * sg_stride].
extern "C" int ri_moe_act_weighted(const void* gu, int gu_stride, const float* weights, void* act, int act_stride, int dtype,
                                   int T, int E, int F, int Fs, int width, int form, float limit, float shared_limit,
                                   float slope, float shift, int weigh_input, const float* sg, int sg_stride, hipStream_t stream) {
    RI_REQUIRE(T >= 0 && E > 0 && F > 0 && Fs >= 0 && width >= E * F + Fs && form >= ACT_SILU && form <= ACT_RELU2 && gu_stride >= (form == ACT_RELU2 ? 1 : 2) * (E * F + Fs) && act_stride >= width,
               "ri_moe_act_weighted: bad sizes");
    RI_REQUIRE(!sg || sg_stride > 0, "ri_moe_act_weighted: the shared gate's logits need a stride");
    if (T == 0) return 0;
    RI_REQUIRE(gu && weights && act, "ri_moe_act_weighted: null pointer");
    RI_REQUIRE(T <= 65535, "ri_moe_act_weighted: too many rows for the grid");
    const dim3 grid((width + 255) / 256, T);
    const ActHow ah{form, limit, shared_limit, slope, shift, weigh_input};
    if (F % 8 == 0 && Fs % 8 == 0 && width % 8 == 0 && gu_stride % 8 == 0 && act_stride % 8 == 0 && (uintptr_t)gu % 16 == 0 && (uintptr_t)act % 16 == 0) {
        const dim3 few((width / 8 + 255) / 256, T);
        if (dtype == RI_F32) moe_swiglu_weighted_vec_kernel<float><<<few, 256, 0, stream>>>((const float*)gu, gu_stride, weights, (float*)act, act_stride, E, F, Fs, width, ah, sg, sg_stride);
        else if (dtype == RI_BF16) moe_swiglu_weighted_vec_kernel<bf16_t><<<few, 256, 0, stream>>>((const bf16_t*)gu, gu_stride, weights, (bf16_t*)act, act_stride, E, F, Fs, width, ah, sg, sg_stride);
        else return ri_fail("ri_moe_act_weighted: unknown dtype %d", dtype);
        RI_LAUNCHED("ri_moe_act_weighted");
        return 0;
    }
    if (dtype == RI_F32) moe_swiglu_weighted_kernel<float><<<grid, 256, 0, stream>>>((const float*)gu, gu_stride, weights, (float*)act, act_stride, E, F, Fs, width, ah, sg, sg_stride);
    else if (dtype == RI_BF16) moe_swiglu_weighted_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)gu, gu_stride, weights, (bf16_t*)act, act_stride, E, F, Fs, width, ah, sg, sg_stride);
    else return ri_fail("ri_moe_act_weighted: unknown dtype %d", dtype);
    RI_LAUNCHED("ri_moe_act_weighted");
    return 0;
}

// The two in one launch: act from gate_up and the router's 32-bit logits [T][>= E].
extern "C" int ri_moe_act_routed(const void* gu, int gu_stride, const float* logits, int l_stride, void* act, int act_stride,
                                 int dtype, int T, int E, int F, int top, int renorm, int score, float eps, float scale,
                                 const float* bias, int Fs, int width, int form, float limit, float shared_limit, float slope, float shift,
                                 int weigh_input, const float* sg, int sg_stride, hipStream_t stream) {
    RI_REQUIRE(T >= 0 && E > 0 && F > 0 && Fs >= 0 && width >= E * F + Fs && form >= ACT_SILU && form <= ACT_RELU2 && gu_stride >= (form == ACT_RELU2 ? 1 : 2) * (E * F + Fs) && act_stride >= width && l_stride >= E,
               "ri_moe_act_routed: bad sizes");
    RI_REQUIRE(score >= ROUTE_SOFTMAX && score <= ROUTE_CHOSEN, "ri_moe_act_routed: unknown score %d", score);
    RI_REQUIRE(top > 0 && top <= E && E <= 64 * MOE_EPL, "ri_moe_act_routed: top %d of %d experts (up to %d)", top, E, 64 * MOE_EPL);
    RI_REQUIRE(!sg || sg_stride > 0, "ri_moe_act_routed: the shared gate's logits need a stride");
    if (T == 0) return 0;
    RI_REQUIRE(gu && logits && act, "ri_moe_act_routed: null pointer");
    RI_REQUIRE(T <= 65535, "ri_moe_act_routed: too many rows for the grid");
    const dim3 grid((width + 255) / 256, T);
    const RouteHow how{score, renorm, eps, scale, bias};
    const ActHow ah{form, limit, shared_limit, slope, shift, weigh_input};
    if (dtype == RI_F32) moe_swiglu_routed_kernel<float><<<grid, 256, 0, stream>>>((const float*)gu, gu_stride, logits, l_stride, (float*)act, act_stride, E, F, top, how, Fs, width, ah, sg, sg_stride);
    else if (dtype == RI_BF16) moe_swiglu_routed_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)gu, gu_stride, logits, l_stride, (bf16_t*)act, act_stride, E, F, top, how, Fs, width, ah, sg, sg_stride);
    else return ri_fail("ri_moe_act_routed: unknown dtype %d", dtype);
    RI_LAUNCHED("ri_moe_act_routed");
    return 0;
}
