// A residual stream of several rows a token (hyper-connections): what happens between two sub-layers, in one pass.
//
//   new_t = sum_s mix[s][t] x_s + out[t] * delta        for every stream t, from the old streams (delta: what the
//                                                       sub-layer returned, possibly in partial sums)
//   u     = sum_t in[t] * new_t                         what the next sub-layer's norm reads
//   act   = norm(u)                                     layer norm ((u - mean) / sqrt(var + eps) * w (+ b)) or RMS norm
//
// Without a delta the streams are taken as they are (the first sub-layer); streams that are all equal to one row are
// read from that row (stream stride 0).  The new streams are written back only where somebody reads them again: after
// the last sub-layer `in` is all ones and nothing but act leaves.  All arithmetic 32-bit, streams 32-bit.
//
// One block a row.  A row's u stays in registers, what does not fit there in LDS.
#include "common.h"
#include <math.h>

namespace {

constexpr int HS_MAX = 8;         // streams
constexpr int HS_CACHE = 4;       // u: so many loads of VEC values a thread stay in registers

// S: the number of streams, or 0: `streams` of them (up to HS_MAX).
template <typename TD, typename TO, int S, int BLOCK, int VEC>
__global__ __launch_bounds__(BLOCK) void hyper_streams_kernel(
        const float* x, size_t x_row, size_t x_stream, const int* __restrict__ rows, int streams,
        const TD* __restrict__ delta, int parts, size_t part_stride, const float* __restrict__ mix, const float* __restrict__ out_w,
        const float* __restrict__ in_w, float* y, const float* __restrict__ w, const float* __restrict__ b, float eps, int centered,
        TO* __restrict__ act, int d) {
    extern __shared__ __align__(16) float rest[];      // u beyond the registers
    __shared__ float red[16];
    using L = VecLoad<VEC>;
    constexpr int N = S > 0 ? S : HS_MAX;
    const int n = S > 0 ? S : streams;
    const int t = blockIdx.x, src = rows ? rows[t] : t;
    const float* xr = x + (size_t)src * x_row;
    const TD* dr = delta ? delta + (size_t)src * d : nullptr;
    float* yr = y ? y + (size_t)t * n * d : nullptr;
    // one piece of VEC values: mixes, writes the new streams, leaves u
    auto piece = [&](int i, float (&u)[VEC]) {
        float xs[N][VEC];
#pragma unroll
        for (int s = 0; s < N; ++s)
            if (s < n) L::ld(xr + s * x_stream + i, xs[s]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] = 0.f;
        if (dr == nullptr) {
#pragma unroll
            for (int s = 0; s < N; ++s)
                if (s < n) {
                    const float a = in_w[s];
#pragma unroll
                    for (int e = 0; e < VEC; ++e) u[e] = fmaf(a, xs[s][e], u[e]);
                    if (yr) L::st(yr + (size_t)s * d + i, xs[s]);
                }
            return;
        }
        float v[VEC];
        L::ld(dr + i, v);
        for (int k0 = 1; k0 < parts; k0 += 4) {        // four partial sums are asked for at once
            float p[4][VEC];
#pragma unroll
            for (int k = 0; k < 4; ++k)
                if (k0 + k < parts) L::ld(dr + (size_t)(k0 + k) * part_stride + i, p[k]);
#pragma unroll
            for (int k = 0; k < 4; ++k)
                if (k0 + k < parts) {
#pragma unroll
                    for (int e = 0; e < VEC; ++e) v[e] += p[k][e];
                }
        }
#pragma unroll
        for (int to = 0; to < N; ++to)
            if (to < n) {
                float z[VEC];
                const float o = out_w[to], a = in_w[to];
#pragma unroll
                for (int e = 0; e < VEC; ++e) z[e] = o * v[e];
#pragma unroll
                for (int s = 0; s < N; ++s)
                    if (s < n) {
                        const float m = mix[s * n + to];
#pragma unroll
                        for (int e = 0; e < VEC; ++e) z[e] = fmaf(m, xs[s][e], z[e]);
                    }
#pragma unroll
                for (int e = 0; e < VEC; ++e) u[e] = fmaf(a, z[e], u[e]);
                if (yr) L::st(yr + (size_t)to * d + i, z);
            }
    };
    float u[HS_CACHE][VEC];
    float sum = 0.f;
#pragma unroll
    for (int k = 0; k < HS_CACHE; ++k) {
        const int i = (threadIdx.x + k * BLOCK) * VEC;
        if (i < d) {
            piece(i, u[k]);
#pragma unroll
            for (int e = 0; e < VEC; ++e) sum += u[k][e];
        }
    }
    constexpr int HELD = HS_CACHE * BLOCK * VEC;
    // (a thread reads back from LDS only what it wrote there itself)
    for (int i = HELD + threadIdx.x * VEC; i < d; i += BLOCK * VEC) {
        float v[VEC];
        piece(i, v);
        L::st(rest + i - HELD, v);
#pragma unroll
        for (int e = 0; e < VEC; ++e) sum += v[e];
    }
    const float mean = centered ? block_sum(sum, red) / (float)d : 0.f;
    float q = 0.f;
#pragma unroll
    for (int k = 0; k < HS_CACHE; ++k)
        if ((int)(threadIdx.x + k * BLOCK) * VEC < d) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) { const float c = u[k][e] - mean; q = fmaf(c, c, q); }
        }
    for (int i = HELD + threadIdx.x * VEC; i < d; i += BLOCK * VEC) {
        float v[VEC];
        L::ld(rest + i - HELD, v);
#pragma unroll
        for (int e = 0; e < VEC; ++e) { const float c = v[e] - mean; q = fmaf(c, c, q); }
    }
    const float rstd = 1.f / sqrtf(block_sum(q, red) / (float)d + eps);
    TO* o = act + (size_t)t * d;
    auto finish = [&](int i, const float* v) {
        float wv[VEC], r[VEC];
        L::ld(w + i, wv);
#pragma unroll
        for (int e = 0; e < VEC; ++e) r[e] = (v[e] - mean) * rstd * wv[e];
        if (b) {
            float bv[VEC];
            L::ld(b + i, bv);
#pragma unroll
            for (int e = 0; e < VEC; ++e) r[e] += bv[e];
        }
        L::st(o + i, r);
    };
#pragma unroll
    for (int k = 0; k < HS_CACHE; ++k) {
        const int i = (threadIdx.x + k * BLOCK) * VEC;
        if (i < d) finish(i, u[k]);
    }
    for (int i = HELD + threadIdx.x * VEC; i < d; i += BLOCK * VEC) {
        float v[VEC];
        L::ld(rest + i - HELD, v);
        finish(i, v);
    }
}

constexpr int HS_FEW_ROWS = 256;                   // up to this many rows, 1,024 threads a row
bool hs_aligned(const void* p, size_t n) { return ((uintptr_t)p & (n - 1)) == 0; }

}  // namespace

// x: row r's stream s begins at x + r * x_row + s * x_stream (x_stream 0: all streams are that row).  rows (or null): the
// rows taken, n_out of them.  delta [parts][rows of x][d] (or null) of delta_dtype, partial sums 32-bit and part_stride
// apart.  mix [streams][streams] (from, to), out_w and in_w [streams], w and b (or null) [d]: 32-bit.  y (or null): the new
// streams [n_out][streams][d], may be x itself where rows is null and x is laid out like that.  act [n_out][d].
extern "C" int ri_hyper_streams(const float* x, long long x_row, long long x_stream, const int* rows, int streams, const void* delta,
                                int delta_dtype, int parts, long long part_stride, const float* mix, const float* out_w, const float* in_w,
                                float* y, const float* w, const float* b, float eps, int centered, void* act, int act_dtype,
                                int n_out, int d, hipStream_t stream) {
    RI_REQUIRE(n_out >= 0 && d > 0 && eps > 0.f && streams > 0 && streams <= HS_MAX && x_row >= 0 && x_stream >= 0,
               "ri_hyper_streams: bad sizes rows=%d d=%d streams=%d", n_out, d, streams);
    RI_REQUIRE(d <= 16384, "ri_hyper_streams: rows of %d values, the kernel takes up to 16384", d);
    if (n_out == 0) return 0;
    RI_REQUIRE(x && in_w && w && act, "ri_hyper_streams: null pointer");
    RI_REQUIRE(!delta || (mix && out_w && parts >= 1 && part_stride >= 0 && (parts == 1 || delta_dtype == RI_F32)),
               "ri_hyper_streams: a delta needs its weights, and partial sums are 32-bit");
    RI_REQUIRE(!y || y != x || (!rows && x_stream == d && x_row == (long long)streams * d), "ri_hyper_streams: streams change in place only as [rows][streams][d]");
    const bool v4 = d % 4 == 0 && x_row % 4 == 0 && x_stream % 4 == 0 && hs_aligned(x, 16) && hs_aligned(y, 16) && hs_aligned(w, 16) && hs_aligned(b, 16)
        && hs_aligned(delta, delta_dtype == RI_F32 ? 16 : 8) && (parts == 1 || part_stride % 4 == 0) && hs_aligned(act, act_dtype == RI_F32 ? 16 : 8);
    const bool wide = n_out <= HS_FEW_ROWS && d >= 1024;
    const int held = HS_CACHE * (v4 ? 4 : 1) * (v4 && wide ? 1024 : 256);
    const size_t lds = d > held ? sizeof(float) * (size_t)(d - held) : 0;
    if (!delta) delta_dtype = RI_F32;
#define RI_HS_L(TD, TO, SS, BLOCK, VEC) hyper_streams_kernel<TD, TO, SS, BLOCK, VEC><<<n_out, BLOCK, lds, stream>>>( \
        x, (size_t)x_row, (size_t)x_stream, rows, streams, (const TD*)delta, parts, (size_t)part_stride, mix, out_w, in_w, y, w, b, eps, centered, (TO*)act, d)
#define RI_HS_S(TD, TO, BLOCK, VEC) do { if (streams == 1) RI_HS_L(TD, TO, 1, BLOCK, VEC); else if (streams == 2) RI_HS_L(TD, TO, 2, BLOCK, VEC); \
        else if (streams == 4) RI_HS_L(TD, TO, 4, BLOCK, VEC); else RI_HS_L(TD, TO, 0, BLOCK, VEC); } while (0)
#define RI_HS(DD, TD, AD, TO) if (delta_dtype == DD && act_dtype == AD) { \
        if (!v4) RI_HS_S(TD, TO, 256, 1); else if (wide) RI_HS_S(TD, TO, 1024, 4); else RI_HS_S(TD, TO, 256, 4); \
        RI_LAUNCHED("ri_hyper_streams"); return 0; }
    RI_HS(RI_F32, float, RI_F32, float)
    RI_HS(RI_F32, float, RI_BF16, bf16_t)
    RI_HS(RI_BF16, bf16_t, RI_BF16, bf16_t)
#undef RI_HS
#undef RI_HS_S
#undef RI_HS_L
    return ri_fail("ri_hyper_streams: dtypes delta=%d activations=%d not taken", delta_dtype, act_dtype);
}
