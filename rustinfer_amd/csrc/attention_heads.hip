// What some attention mixers do to their projected rows, head by head, before the attention
// kernels see them (all arithmetic 32-bit, storage 32-bit or bfloat16):
//
//   head_norm_kv_write   queries and keys divided by their root mean square over the head, times a
//                        weight of the head's size shared by all heads, the query times a
//                        temperature that grows with the logarithm of its position, both turned by
//                        their position over their first features; the query in
//                        place, the normed key and the value into the token's page (a head may hold
//                        several queries or keys side by side, each normed on its own);
//   latent_kv_write      attention through one latent vector a token: the first R features of the
//                        down projection are normed (c), the last r are one rotated key part for all
//                        heads; the page takes the key [c, rotated part] and the value c; the
//                        rotated part of every head's query goes to the tail of that head's
//                        absorbed query [R + r]; where the queries come from a latent of their own,
//                        that latent is normed in the same pass (its product with the heads' matrix
//                        comes after, and head_linear makes the tails);
//   head_linear          out[t, h, :] = W_h x[t, h, :] for every head: the product that turns a
//                        head's unrotated query into the latent space (W_uk,h^T q) and the weighted
//                        sum of latents back into the head's value space (W_uv,h o), there times a
//                        sigmoid a feature if the mixer has an output gate.
//
// Cache layout as everywhere: keys [pages][Hkv][page][dk], values [pages][Hkv][dv][page].
#include "common.h"
#include <math.h>

namespace {

// ---------------------------------------------------------------------------
// Blocks (token, four heads): one wave a head (queries first, then keys); the blocks of a token's
// first heads also copy its values.
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void head_norm_kv_write_kernel(
        T* __restrict__ q, int q_stride, const T* __restrict__ k, int k_stride, const T* __restrict__ v, int v_stride,
        int H, int Hkv, int dk, int dv, const float* __restrict__ qw, const float* __restrict__ kw, int do_norm, float eps,
        float temp_coef, int temp_every, const int* __restrict__ positions, const int* __restrict__ row_of_token,
        T* __restrict__ kc, T* __restrict__ vc, const int* __restrict__ table, int max_blocks, int page, int write_kv, int maps,
        int rot, const float* __restrict__ cos_t, const float* __restrict__ sin_t) {
    const int t = blockIdx.x;
    const int b = row_of_token[t];
    if (b < 0) return;                       // padding token
    const int pos = positions[t];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int Hq = H * maps, Hk = Hkv * maps;          // what is normed: every map of every head
    int blk = -1;
    if (write_kv) blk = table[(size_t)b * max_blocks + pos / page];
    const int slot = pos % page;
    const float temp = temp_every > 0 ? 1.f + temp_coef * logf((float)((pos + 1) / temp_every) + 1.f) : 1.f;
    const int units = Hq + (blk >= 0 ? Hk : 0);
    for (int u = blockIdx.y * 4 + wave; u < units; u += 4 * gridDim.y) {
        const bool is_q = u < Hq;
        const int g = is_q ? 0 : u - Hq;
        const T* src = is_q ? q + (size_t)t * q_stride + u * dk : k + (size_t)t * k_stride + g * dk;
        T* dst = is_q ? q + (size_t)t * q_stride + u * dk : kc + (((size_t)blk * Hkv + g / maps) * page + slot) * (maps * dk) + g % maps * dk;
        const float* w = is_q ? qw : kw;
        float f = is_q ? temp : 1.f;
        if (do_norm) {
            float ss = 0.f;
            for (int i = lane; i < dk; i += 64) { const float x = ld_f32(src + i); ss = fmaf(x, x, ss); }
            ss = wave_sum(ss);
            f *= 1.f / sqrtf(ss / (float)dk + eps);
        }
        const int half = rot >> 1;
        for (int i = lane; i < half; i += 64) {            // a pair a lane: nobody else reads or writes its two features
            const float a = ld_f32(src + i) * f * (w ? w[i] : 1.f), bb = ld_f32(src + i + half) * f * (w ? w[i + half] : 1.f);
            const float c = cos_t[(size_t)pos * half + i], s = sin_t[(size_t)pos * half + i];
            st_f32(dst + i, a * c - bb * s);
            st_f32(dst + i + half, bb * c + a * s);
        }
        for (int i = rot + lane; i < dk; i += 64) {
            const float x = ld_f32(src + i);
            st_f32(dst + i, x * f * (w ? w[i] : 1.f));
        }
    }
    if (blk < 0) return;
    const T* vrow = v + (size_t)t * v_stride;
    for (int idx = blockIdx.y * 256 + threadIdx.x; idx < Hkv * dv; idx += 256 * gridDim.y) {
        const int g = idx / dv, dd = idx - g * dv;
        vc[(((size_t)blk * Hkv + g) * dv + dd) * page + slot] = vrow[idx];
    }
}

// The same with eight features a lane (16 bytes of bfloat16 a load): dk, the turned half and every row stride multiples of
// eight.  LPH lanes, a power of two that holds dk / 8, share a head; a block's 256 / LPH heads go side by side, so a token's
// heads are read at once instead of one behind the other.
template <typename T, int LPH>
__global__ __launch_bounds__(256) void head_norm_kv_write_vec_kernel(
        T* __restrict__ q, int q_stride, const T* __restrict__ k, int k_stride, const T* __restrict__ v, int v_stride,
        int H, int Hkv, int dk, int dv, const float* __restrict__ qw, const float* __restrict__ kw, int do_norm, float eps,
        float temp_coef, int temp_every, const int* __restrict__ positions, const int* __restrict__ row_of_token,
        T* __restrict__ kc, T* __restrict__ vc, const int* __restrict__ table, int max_blocks, int page, int write_kv, int maps,
        int rot, const float* __restrict__ cos_t, const float* __restrict__ sin_t) {
    using L = VecLoad<4>;
    const int t = blockIdx.x;
    const int b = row_of_token[t];
    if (b < 0) return;                       // padding token
    const int pos = positions[t];
    const int Hq = H * maps, Hk = Hkv * maps;
    int blk = -1;
    if (write_kv) blk = table[(size_t)b * max_blocks + pos / page];
    const int slot = pos % page;
    const float temp = temp_every > 0 ? 1.f + temp_coef * logf((float)((pos + 1) / temp_every) + 1.f) : 1.f;
    const int units = Hq + (blk >= 0 ? Hk : 0);
    const int l = threadIdx.x % LPH, i = 8 * l, half = rot >> 1;
    const bool mine = i < dk, low = i < half;
    const int partner = low ? l + half / 8 : l - half / 8;         // (used where i < rot)
    float c[8], s[8];
    if (mine && i < rot) {
        const size_t at = (size_t)pos * half + (low ? i : i - half);
#pragma unroll
        for (int e = 0; e < 8; e += 4) { L::ld(cos_t + at + e, c + e); L::ld(sin_t + at + e, s + e); }
    }
    constexpr int HPB = 256 / LPH;
    // (every lane of a wave goes round equally often: the shuffles below are met by all)
    for (int u0 = blockIdx.y * HPB; u0 < units; u0 += HPB * gridDim.y) {
        const int u = u0 + threadIdx.x / LPH;
        const bool on = mine && u < units, is_q = u < Hq;
        const int g = is_q ? 0 : u - Hq;
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = 0.f;
        if (on) {
            const T* src = is_q ? q + (size_t)t * q_stride + u * dk + i : k + (size_t)t * k_stride + g * dk + i;
#pragma unroll
            for (int e = 0; e < 8; e += 4) L::ld(src + e, x + e);
        }
        float f = is_q ? temp : 1.f;
        if (do_norm) {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss = fmaf(x[e], x[e], ss);
#pragma unroll
            for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, LPH);
            f *= 1.f / sqrtf(ss / (float)dk + eps);
        }
        const float* w = is_q ? qw : kw;
        float wv[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) wv[e] = 1.f;
        if (on && w) {
#pragma unroll
            for (int e = 0; e < 8; e += 4) L::ld(w + i + e, wv + e);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = x[e] * f * wv[e];
        if (rot > 0) {                       // (uniform)
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float y = __shfl(x[e], partner & (LPH - 1), LPH);
                if (i < rot) x[e] = low ? x[e] * c[e] - y * s[e] : x[e] * c[e] + y * s[e];
            }
        }
        if (on) {
            T* dst = is_q ? q + (size_t)t * q_stride + u * dk + i : kc + (((size_t)blk * Hkv + g / maps) * page + slot) * (maps * dk) + g % maps * dk + i;
#pragma unroll
            for (int e = 0; e < 8; e += 4) L::st(dst + e, x + e);
        }
    }
    if (blk < 0) return;
    const T* vrow = v + (size_t)t * v_stride;
    for (int idx = blockIdx.y * 256 + threadIdx.x; idx < Hkv * dv; idx += 256 * gridDim.y) {
        const int g = idx / dv, dd = idx - g * dv;
        vc[(((size_t)blk * Hkv + g) * dv + dd) * page + slot] = vrow[idx];
    }
}

// ---------------------------------------------------------------------------
// One block a token.  q [T][H (d + r)]: a head's unrotated features, then its r rotated ones, of which
// the first `rot` are turned (feature i with i + rot/2).  down [T][R + r].  q_abs [T][H (R + r)].
// q null: the heads' queries are not there yet.  ql [T][Rq] (or null): the queries' latent, normed into ql_out [T][Rq] by a
// second block a token (blockIdx.y = 1).
// ---------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void latent_kv_write_kernel(
        const T* __restrict__ q, int q_stride, const T* __restrict__ down, int down_stride, T* __restrict__ q_abs, int qa_stride,
        int H, int d, int r, int R, int rot, const float* __restrict__ cw, float eps,
        const float* __restrict__ cos_t, const float* __restrict__ sin_t,
        const int* __restrict__ positions, const int* __restrict__ row_of_token,
        T* __restrict__ kc, T* __restrict__ vc, const int* __restrict__ table, int max_blocks, int page, int write_kv,
        const T* __restrict__ ql, int ql_stride, int Rq, const float* __restrict__ qlw, T* __restrict__ ql_out, int qo_stride) {
    __shared__ float red[16];
    const int t = blockIdx.x;
    const int b = row_of_token[t];
    if (b < 0) return;                       // padding token
    const int pos = positions[t];
    const int half = rot >> 1;
    const bool rotate = cos_t != nullptr && half > 0;
    const float* cs = rotate ? cos_t + (size_t)pos * half : nullptr;
    const float* sn = rotate ? sin_t + (size_t)pos * half : nullptr;
    auto turned = [&](const T* part, int j) -> float {      // feature j of a rotated part after the turn
        if (rotate && j < half) return ld_f32(part + j) * cs[j] - ld_f32(part + j + half) * sn[j];
        if (rotate && j < rot) return ld_f32(part + j) * cs[j - half] + ld_f32(part + j - half) * sn[j - half];
        return ld_f32(part + j);
    };
    if (blockIdx.y == 1) {
        const T* row = ql + (size_t)t * ql_stride;
        float ss = 0.f;
        for (int i = threadIdx.x; i < Rq; i += 256) { const float x = ld_f32(row + i); ss = fmaf(x, x, ss); }
        ss = block_sum(ss, red);
        const float rs = 1.f / sqrtf(ss / (float)Rq + eps);
        for (int i = threadIdx.x; i < Rq; i += 256) st_f32(ql_out + (size_t)t * qo_stride + i, ld_f32(row + i) * rs * (qlw ? qlw[i] : 1.f));
        return;
    }
    if (q) {
        const T* qrow = q + (size_t)t * q_stride;
        T* qa = q_abs + (size_t)t * qa_stride;
        for (int idx = threadIdx.x; idx < H * r; idx += 256) {
            const int h = idx / r, j = idx - h * r;
            st_f32(qa + h * (R + r) + R + j, turned(qrow + h * (d + r) + d, j));
        }
    }
    if (!write_kv) return;
    const int blk = table[(size_t)b * max_blocks + pos / page];
    if (blk < 0) return;                     // (uniform over the block)
    const int slot = pos % page;
    const T* drow = down + (size_t)t * down_stride;
    float ss = 0.f;
    for (int i = threadIdx.x; i < R; i += 256) { const float x = ld_f32(drow + i); ss = fmaf(x, x, ss); }
    ss = block_sum(ss, red);
    const float rs = 1.f / sqrtf(ss / (float)R + eps);
    T* krow = kc + ((size_t)blk * page + slot) * (R + r);
    for (int i = threadIdx.x; i < R; i += 256) {
        const float c = ld_f32(drow + i) * rs * (cw ? cw[i] : 1.f);
        st_f32(krow + i, c);
        st_f32(vc + ((size_t)blk * R + i) * page + slot, c);
    }
    for (int j = threadIdx.x; j < r; j += 256) st_f32(krow + R + j, turned(drow + R, j));
}

// ---------------------------------------------------------------------------
// out[t][h * out_head + n] = sum_k x[t][h * x_head + k] * w[(h * N + n) * K + k],  n < N, k < K.
// A block of 256 threads owns 64 tokens x 64 outputs of one head; K goes by in steps of 16 through
// LDS; a thread sums a 4 x 4 patch in 32-bit, in the order of k.
// ---------------------------------------------------------------------------
constexpr int HL_T = 64, HL_N = 64, HL_K = 16;

// What else a head's product may do.  tail > 0: the `tail` features behind the K that are multiplied go, turned by
// the token's position (the first `rot` of them, feature i with i + rot/2), behind the N outputs.  gate (or null): output n of
// head h is multiplied by sigmoid(gate[t * gate_stride + h * N + n]).
template <typename T>
struct HeadExtra {
    int tail, rot, table_rows;
    const float *cos_t, *sin_t;
    const int* positions;
    const T* gate;
    int gate_stride;
    __device__ __forceinline__ float gated(float v, int t, int at) const {
        return gate ? v / (1.f + expf(-ld_f32(gate + (size_t)t * gate_stride + at))) : v;
    }
    // feature j of the tail that starts at `part`, for token t
    __device__ __forceinline__ float turned(const T* part, int t, int j) const {
        const int half = rot >> 1;
        if (j >= 2 * half) return ld_f32(part + j);
        const size_t at = (size_t)min(max(positions[t], 0), table_rows - 1) * half;
        if (j < half) return ld_f32(part + j) * cos_t[at + j] - ld_f32(part + j + half) * sin_t[at + j];
        return ld_f32(part + j) * cos_t[at + j - half] + ld_f32(part + j - half) * sin_t[at + j - half];
    }
};

template <typename T>
__global__ __launch_bounds__(256) void head_linear_kernel(
        const T* __restrict__ x, int x_stride, int x_head, const T* __restrict__ w, T* __restrict__ out, int out_stride,
        int out_head, int Tn, int N, int K, HeadExtra<T> extra) {
    __shared__ float xs[HL_K][HL_T + 4];
    __shared__ float ws[HL_K][HL_N + 4];
    const int h = blockIdx.z, t0 = blockIdx.x * HL_T, n0 = blockIdx.y * HL_N;
    if (n0 >= N) {                                     // the blocks of the tail (there are none without one)
        for (int e = threadIdx.x; e < HL_T * extra.tail; e += 256) {
            const int t = t0 + e / extra.tail, j = e % extra.tail;
            if (t < Tn) st_f32(out + (size_t)t * out_stride + h * out_head + N + j, extra.turned(x + (size_t)t * x_stride + h * x_head + K, t, j));
        }
        return;
    }
    const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;           // outputs 4 tx.., tokens 4 ty..
    const T* wh = w + (size_t)h * N * K;
    float acc[4][4] = {};
    for (int k0 = 0; k0 < K; k0 += HL_K) {
        for (int e = threadIdx.x; e < HL_T * HL_K; e += 256) {
            const int kk = e % HL_K, tt = e / HL_K;
            const int t = t0 + tt, k = k0 + kk;
            xs[kk][tt] = (t < Tn && k < K) ? ld_f32(x + (size_t)t * x_stride + h * x_head + k) : 0.f;
        }
        for (int e = threadIdx.x; e < HL_N * HL_K; e += 256) {
            const int kk = e % HL_K, nn = e / HL_K;
            const int n = n0 + nn, k = k0 + kk;
            ws[kk][nn] = (n < N && k < K) ? ld_f32(wh + (size_t)n * K + k) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < HL_K; ++kk) {
            const float4 xv = *reinterpret_cast<const float4*>(&xs[kk][4 * ty]);
            const float4 wv = *reinterpret_cast<const float4*>(&ws[kk][4 * tx]);
            const float xa[4] = {xv.x, xv.y, xv.z, xv.w}, wa[4] = {wv.x, wv.y, wv.z, wv.w};
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xa[i], wa[j], acc[i][j]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = t0 + 4 * ty + i;
        if (t >= Tn) continue;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = n0 + 4 * tx + j;
            if (n < N) st_f32(out + (size_t)t * out_stride + h * out_head + n, extra.gated(acc[i][j], t, h * N + n));
        }
    }
}

// The same product for a step of few tokens (up to HLF_T): no staging.  Eight lanes share an output
// and divide K between them in pieces of 16 bytes (VEC: operands aligned for that; else element by
// element), each summing all tokens' terms of its pieces; a block owns 32 outputs of one head.  The
// sums of a token are added in a fixed order whatever else the step holds.
constexpr int HLF_T = 16;

__device__ __forceinline__ void hl_ld16(const float* p, float* f) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
}
__device__ __forceinline__ void hl_ld16(const bf16_t* p, float* f) {
    const uint4 v = *reinterpret_cast<const uint4*>(p);
    f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
    f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
    f[4] = __uint_as_float(v.z << 16); f[5] = __uint_as_float(v.z & 0xffff0000u);
    f[6] = __uint_as_float(v.w << 16); f[7] = __uint_as_float(v.w & 0xffff0000u);
}

// TT: the tokens a lane asks for at once (a step of fewer repeats its last one and drops the result): with a
// bound in the loop instead every load would wait for the one before it.
template <typename T, bool VEC, int TT>
__global__ __launch_bounds__(256) void head_linear_few_kernel(
        const T* __restrict__ x, int x_stride, int x_head, const T* __restrict__ w, T* __restrict__ out, int out_stride,
        int out_head, int Tn, int N, int K, HeadExtra<T> extra) {
    constexpr int VL = VEC ? 16 / (int)sizeof(T) : 1;
    if ((int)blockIdx.x * 32 >= N) {                   // the block of the tail (there is none without one)
        const int h = blockIdx.y;
        for (int e = threadIdx.x; e < Tn * extra.tail; e += 256) {
            const int t = e / extra.tail, j = e % extra.tail;
            st_f32(out + (size_t)t * out_stride + h * out_head + N + j, extra.turned(x + (size_t)t * x_stride + h * x_head + K, t, j));
        }
        return;
    }
    const int h = blockIdx.y, part = threadIdx.x & 7, n = blockIdx.x * 32 + (threadIdx.x >> 3);
    const bool live = n < N;
    const T* wr = w + ((size_t)h * N + (live ? n : 0)) * K;
    const T* xh = x + (size_t)h * x_head;
    float acc[TT];
#pragma unroll
    for (int t = 0; t < TT; ++t) acc[t] = 0.f;
    for (int k = part * VL; k < K; k += 8 * VL) {
        float wv[VL], xv[TT][VL];
        if (VEC) hl_ld16(wr + k, wv); else wv[0] = ld_f32(wr + k);
#pragma unroll
        for (int t = 0; t < TT; ++t) {
            const T* row = xh + (size_t)min(t, Tn - 1) * x_stride + k;
            if (VEC) hl_ld16(row, xv[t]); else xv[t][0] = ld_f32(row);
        }
#pragma unroll
        for (int t = 0; t < TT; ++t)
#pragma unroll
            for (int u = 0; u < VL; ++u) acc[t] = fmaf(xv[t][u], wv[u], acc[t]);
    }
    // all eight lanes have every token's sum; lane `part` writes the tokens part, part + 8
    float keep[(TT + 7) / 8];
#pragma unroll
    for (int t = 0; t < TT; ++t) {
        float v = acc[t];
#pragma unroll
        for (int o = 4; o > 0; o >>= 1) v += __shfl_xor(v, o, 8);
        if ((t & 7) == part) keep[t >> 3] = v;
    }
#pragma unroll
    for (int j = 0; j < (TT + 7) / 8; ++j) {
        const int t = part + 8 * j;
        if (t < TT && t < Tn && live) st_f32(out + (size_t)t * out_stride + h * out_head + n, extra.gated(keep[j], t, h * N + n));
    }
}

// The same product of many bfloat16 tokens on the matrix instructions (v_mfma_f32_32x32x16_bf16, 32-bit sums): a wave owns
// 32 tokens and 64 outputs of one head, both operands straight from memory, 16 bytes a lane.  K and the row strides
// multiples of eight; wide: the outputs may be written four at a time.
typedef __bf16 hl_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float hl_f32x16_t __attribute__((ext_vector_type(16)));

__global__ __launch_bounds__(256) void head_linear_mfma_kernel(
        const bf16_t* __restrict__ x, int x_stride, int x_head, const bf16_t* __restrict__ w, bf16_t* __restrict__ out, int out_stride,
        int out_head, int Tn, int N, int K, int wide, HeadExtra<bf16_t> extra) {
    const int h = blockIdx.z, n0 = blockIdx.y * 64, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int t0 = blockIdx.x * 128 + wave * 32;
    if (n0 >= N) {                                     // the blocks of the tail (there are none without one)
        for (int e = threadIdx.x; e < 128 * extra.tail; e += 256) {
            const int t = blockIdx.x * 128 + e / extra.tail, j = e % extra.tail;
            if (t < Tn) st_f32(out + (size_t)t * out_stride + h * out_head + N + j, extra.turned(x + (size_t)t * x_stride + h * x_head + K, t, j));
        }
        return;
    }
    if (t0 >= Tn) return;
    const int lr = lane & 31, lh = lane >> 5;
    const int t = t0 + lr;
    const bf16_t* xr = x + (size_t)min(t, Tn - 1) * x_stride + (size_t)h * x_head;
    const bf16_t* w0 = w + ((size_t)h * N + min(n0 + lr, N - 1)) * K, *w1 = w + ((size_t)h * N + min(n0 + 32 + lr, N - 1)) * K;
    hl_f32x16_t a0, a1;
#pragma unroll
    for (int i = 0; i < 16; ++i) a0[i] = a1[i] = 0.f;
    const hl_bf16x8_t zero = __builtin_bit_cast(hl_bf16x8_t, ri_u32x4_t{0u, 0u, 0u, 0u});
#pragma unroll 4
    for (int k0 = 0; k0 < K; k0 += 16) {
        const int k = k0 + 8 * lh, kk = min(k, K - 8);
        hl_bf16x8_t xv = *reinterpret_cast<const hl_bf16x8_t*>(xr + kk);
        hl_bf16x8_t wa = *reinterpret_cast<const hl_bf16x8_t*>(w0 + kk), wb = *reinterpret_cast<const hl_bf16x8_t*>(w1 + kk);
        if (k >= K) xv = wa = wb = zero;               // the upper half of a last step of eight
        a0 = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wa, xv, a0, 0, 0, 0);
        a1 = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wb, xv, a1, 0, 0, 0);
    }
    if (t >= Tn) return;
    bf16_t* o = out + (size_t)t * out_stride + h * out_head;
#pragma unroll
    for (int tile = 0; tile < 2; ++tile)
#pragma unroll
        for (int i = 0; i < 16; i += 4) {              // registers i .. i + 3: outputs 8 (i / 4) + 4 lh + 0..3 of the tile
            const int n = n0 + 32 * tile + 2 * i + 4 * lh;
            float v[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = n + e < N ? extra.gated(tile == 0 ? a0[i + e] : a1[i + e], t, h * N + n + e) : 0.f;
            if (wide && n + 4 <= N) VecLoad<4>::st(o + n, v);
            else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e < N) st_f32(o + n + e, v[e]);
            }
        }
}

}  // namespace

// q [T][>= H dk] is normed in place; k [T][>= Hkv dk], v [T][>= Hkv dv] go to the token's page
// (write_kv; a layer that reads another layer's cache has none).  qw, kw: 32-bit weights of dk
// entries or null; do_norm 0: no division by the root mean square (weights and temperature only).
// temp_every > 0: the query at position p is multiplied by 1 + temp_coef ln(floor((p + 1) / temp_every) + 1).
// maps: queries a query head and keys a key head hold, side by side (q [T][>= H maps dk], k [T][>= Hkv maps dk]);
// each is normed on its own with the same weight, and the cached key row has maps dk features.
// rot > 0: behind the norm the first rot features of every query and key are turned by the token's position (feature i
// with i + rot/2; tables [table_rows][rot / 2]).
extern "C" int ri_head_norm_kv_write(
        void* q, int q_stride, const void* k, int k_stride, const void* v, int v_stride, int dtype, int T,
        int H, int Hkv, int dk, int dv, const float* qw, const float* kw, int do_norm, float eps,
        float temp_coef, int temp_every, const int* positions, const int* row_of_token,
        void* kc, void* vc, int num_pages, const int* table, int max_blocks, int page, int write_kv, int maps,
        int rot, const float* cos_t, const float* sin_t, int table_rows, hipStream_t stream) {
    RI_REQUIRE(T >= 0 && H > 0 && Hkv > 0 && dk > 0 && dv > 0 && page > 0 && maps > 0, "ri_head_norm_kv_write: bad sizes");
    RI_REQUIRE(q_stride >= H * maps * dk, "ri_head_norm_kv_write: query row stride %d too small", q_stride);
    RI_REQUIRE(!do_norm || eps > 0.f, "ri_head_norm_kv_write: eps must be > 0");
    RI_REQUIRE(rot == 0 || (rot > 0 && rot % 2 == 0 && rot <= dk && cos_t && sin_t && table_rows > 0), "ri_head_norm_kv_write: rot %d must be even and within the key size %d, with tables", rot, dk);
    if (write_kv) RI_REQUIRE(k && v && kc && vc && table && max_blocks > 0 && num_pages > 0 && k_stride >= Hkv * maps * dk && v_stride >= Hkv * dv,
                             "ri_head_norm_kv_write: no keys, values or cache given, or their row strides too small");
    if (T == 0) return 0;
    RI_REQUIRE(q && positions && row_of_token, "ri_head_norm_kv_write: null pointer");
#define RI_HN(KERNEL, TT, GRID) KERNEL<<<GRID, 256, 0, stream>>>((TT*)q, q_stride, (const TT*)k, k_stride, (const TT*)v, v_stride, H, Hkv, dk, dv, qw, kw, do_norm, eps, \
        temp_coef, temp_every, positions, row_of_token, (TT*)kc, (TT*)vc, table, max_blocks, page, write_kv, maps, rot, cos_t, sin_t)
    if (dk % 8 == 0 && dk <= 256 && rot % 16 == 0 && q_stride % 8 == 0 && (!write_kv || k_stride % 8 == 0) && (uintptr_t)q % 16 == 0 &&
        (!write_kv || ((uintptr_t)k % 16 == 0 && (uintptr_t)kc % 16 == 0)) && (uintptr_t)qw % 16 == 0 && (uintptr_t)kw % 16 == 0 &&
        (uintptr_t)cos_t % 16 == 0 && (uintptr_t)sin_t % 16 == 0 && (dtype == RI_F32 || dtype == RI_BF16)) {
        int lph = 1;
        while (8 * lph < dk) lph *= 2;
        const int hpb = 256 / lph;
        const dim3 vgrid(T, T <= 256 ? min(((H + Hkv) * maps + hpb - 1) / hpb, 64) : 1);
#define RI_HN_L(TT) do { if (lph == 1) RI_HN((head_norm_kv_write_vec_kernel<TT, 1>), TT, vgrid); else if (lph == 2) RI_HN((head_norm_kv_write_vec_kernel<TT, 2>), TT, vgrid); \
        else if (lph == 4) RI_HN((head_norm_kv_write_vec_kernel<TT, 4>), TT, vgrid); else if (lph == 8) RI_HN((head_norm_kv_write_vec_kernel<TT, 8>), TT, vgrid); \
        else if (lph == 16) RI_HN((head_norm_kv_write_vec_kernel<TT, 16>), TT, vgrid); else RI_HN((head_norm_kv_write_vec_kernel<TT, 32>), TT, vgrid); } while (0)
        if (dtype == RI_F32) RI_HN_L(float);
        else RI_HN_L(bf16_t);
#undef RI_HN_L
        RI_LAUNCHED("ri_head_norm_kv_write");
        return 0;
    }
    // a step of few tokens: a block for every four heads, so that no wave walks a chain of heads
    const int by = T <= 256 ? min(((H + Hkv) * maps + 3) / 4, 64) : 1;
    const dim3 grid(T, by);
    if (dtype == RI_F32) RI_HN(head_norm_kv_write_kernel<float>, float, grid);
    else if (dtype == RI_BF16) RI_HN(head_norm_kv_write_kernel<bf16_t>, bf16_t, grid);
    else
        return ri_fail("ri_head_norm_kv_write: unknown dtype %d", dtype);
#undef RI_HN
    RI_LAUNCHED("ri_head_norm_kv_write");
    return 0;
}

// The cache belongs to one key/value head with keys of R + r features and values of R.  q null: no queries' tails.
// ql [T][>= Rq] (null: none): rows that are divided by their root mean square and multiplied by qlw into ql_out.
extern "C" int ri_latent_kv_write(
        const void* q, int q_stride, const void* down, int down_stride, void* q_abs, int qa_stride, int dtype, int T,
        int H, int d, int r, int R, int rot, const float* cw, float eps, const float* cos_t, const float* sin_t, int table_rows,
        const int* positions, const int* row_of_token, void* kc, void* vc, int num_pages,
        const int* table, int max_blocks, int page, int write_kv,
        const void* ql, int ql_stride, int Rq, const float* qlw, void* ql_out, int qo_stride, hipStream_t stream) {
    RI_REQUIRE(T >= 0 && H > 0 && d >= 0 && r >= 0 && R > 0 && page > 0, "ri_latent_kv_write: bad sizes");
    RI_REQUIRE((!q || (q_stride >= H * (d + r) && qa_stride >= H * (R + r))) && down_stride >= R + r, "ri_latent_kv_write: row strides too small");
    RI_REQUIRE(eps > 0.f, "ri_latent_kv_write: eps must be > 0");
    if (cos_t) RI_REQUIRE(rot > 0 && rot % 2 == 0 && rot <= r && sin_t && table_rows > 0, "ri_latent_kv_write: rot %d must be even and within the rotated part %d", rot, r);
    if (write_kv) RI_REQUIRE(kc && vc && table && max_blocks > 0 && num_pages > 0, "ri_latent_kv_write: no cache given");
    if (T == 0) return 0;
    RI_REQUIRE((!q || q_abs) && down && positions && row_of_token, "ri_latent_kv_write: null pointer");
    RI_REQUIRE(!ql || (ql_out && Rq > 0 && ql_stride >= Rq && qo_stride >= Rq), "ri_latent_kv_write: the queries' latent needs a place and row strides of at least its size");
    if (dtype == RI_F32)
        latent_kv_write_kernel<float><<<dim3(T, ql ? 2 : 1), 256, 0, stream>>>((const float*)q, q_stride, (const float*)down, down_stride, (float*)q_abs, qa_stride, H, d, r, R, rot, cw, eps, cos_t, sin_t, positions, row_of_token, (float*)kc, (float*)vc, table, max_blocks, page, write_kv, (const float*)ql, ql_stride, Rq, qlw, (float*)ql_out, qo_stride);
    else if (dtype == RI_BF16)
        latent_kv_write_kernel<bf16_t><<<dim3(T, ql ? 2 : 1), 256, 0, stream>>>((const bf16_t*)q, q_stride, (const bf16_t*)down, down_stride, (bf16_t*)q_abs, qa_stride, H, d, r, R, rot, cw, eps, cos_t, sin_t, positions, row_of_token, (bf16_t*)kc, (bf16_t*)vc, table, max_blocks, page, write_kv, (const bf16_t*)ql, ql_stride, Rq, qlw, (bf16_t*)ql_out, qo_stride);
    else
        return ri_fail("ri_latent_kv_write: unknown dtype %d", dtype);
    RI_LAUNCHED("ri_latent_kv_write");
    return 0;
}

// x [T][x_stride], head h at column h * x_head; w [H][N][K] contiguous; out [T][out_stride], head h
// at column h * out_head.  tail, rot, the tables and the gate: see HeadExtra.
extern "C" int ri_head_linear(const void* x, int x_stride, int x_head, const void* w, void* out, int out_stride, int out_head,
                              int dtype, int T, int H, int N, int K, int tail, int rot, const float* cos_t, const float* sin_t, int table_rows,
                              const int* positions, const void* gate, int gate_stride, hipStream_t stream) {
    RI_REQUIRE(T >= 0 && H > 0 && N > 0 && K > 0, "ri_head_linear: bad sizes T=%d H=%d N=%d K=%d", T, H, N, K);
    RI_REQUIRE(tail >= 0 && rot >= 0 && rot % 2 == 0 && rot <= tail && (rot == 0 || (cos_t && sin_t && table_rows > 0 && positions)), "ri_head_linear: a tail of %d with %d turned features", tail, rot);
    RI_REQUIRE(!gate || gate_stride >= H * N, "ri_head_linear: the gate's row stride is too small");
    RI_REQUIRE(x_head >= 0 && out_head >= 0 && x_stride >= (H - 1) * x_head + K + tail && out_stride >= (H - 1) * out_head + N + tail,
               "ri_head_linear: row strides too small");
    if (T == 0) return 0;
    RI_REQUIRE(x && w && out, "ri_head_linear: null pointer");
    RI_REQUIRE(H <= 65535 && (N + HL_N - 1) / HL_N <= 65535, "ri_head_linear: too many heads or outputs for the grid");
    if (T <= HLF_T) {
        const dim3 few((N + 31) / 32 + (tail > 0), H);
        const int vl = dtype == RI_F32 ? 4 : 8;
        const bool vec = K % vl == 0 && x_stride % vl == 0 && x_head % vl == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0;
#define RI_HLF(TY, VV, TT) head_linear_few_kernel<TY, VV, TT><<<few, 256, 0, stream>>>((const TY*)x, x_stride, x_head, (const TY*)w, (TY*)out, out_stride, out_head, T, N, K, \
                                          HeadExtra<TY>{tail, rot, table_rows, cos_t, sin_t, positions, (const TY*)gate, gate_stride})
#define RI_HLF_T(TY, VV) do { if (T <= 1) RI_HLF(TY, VV, 1); else if (T <= 2) RI_HLF(TY, VV, 2); else if (T <= 4) RI_HLF(TY, VV, 4); \
                              else if (T <= 8) RI_HLF(TY, VV, 8); else RI_HLF(TY, VV, 16); } while (0)
        if (dtype == RI_F32) { if (vec) RI_HLF_T(float, true); else RI_HLF_T(float, false); }
        else if (dtype == RI_BF16) { if (vec) RI_HLF_T(bf16_t, true); else RI_HLF_T(bf16_t, false); }
        else
            return ri_fail("ri_head_linear: unknown dtype %d", dtype);
#undef RI_HLF_T
#undef RI_HLF
        RI_LAUNCHED("ri_head_linear");
        return 0;
    }
    if (dtype == RI_BF16 && K % 8 == 0 && x_stride % 8 == 0 && x_head % 8 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0) {
        const int wide = out_stride % 4 == 0 && out_head % 4 == 0 && (uintptr_t)out % 8 == 0;
        head_linear_mfma_kernel<<<dim3((T + 127) / 128, (N + 63) / 64 + (tail > 0), H), 256, 0, stream>>>((const bf16_t*)x, x_stride, x_head, (const bf16_t*)w,
            (bf16_t*)out, out_stride, out_head, T, N, K, wide, HeadExtra<bf16_t>{tail, rot, table_rows, cos_t, sin_t, positions, (const bf16_t*)gate, gate_stride});
        RI_LAUNCHED("ri_head_linear");
        return 0;
    }
    const dim3 grid((T + HL_T - 1) / HL_T, (N + HL_N - 1) / HL_N + (tail > 0), H);
    if (dtype == RI_F32)
        head_linear_kernel<float><<<grid, 256, 0, stream>>>((const float*)x, x_stride, x_head, (const float*)w, (float*)out, out_stride, out_head, T, N, K,
            HeadExtra<float>{tail, rot, table_rows, cos_t, sin_t, positions, (const float*)gate, gate_stride});
    else if (dtype == RI_BF16)
        head_linear_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)x, x_stride, x_head, (const bf16_t*)w, (bf16_t*)out, out_stride, out_head, T, N, K,
            HeadExtra<bf16_t>{tail, rot, table_rows, cos_t, sin_t, positions, (const bf16_t*)gate, gate_stride});
    else
        return ri_fail("ri_head_linear: unknown dtype %d", dtype);
    RI_LAUNCHED("ri_head_linear");
    return 0;
}
