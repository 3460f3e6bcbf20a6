// bfloat16 attention over the paged cache whose softmax weights keep their 32 bits on the bfloat16
// matrix instructions (gfx950).
//
// The scores of bfloat16 queries and keys are exact products with 32-bit sums.  A weight is the sum of
// three bfloat16 numbers, its leading, middle and last eight bits (parts3): three products with the
// bfloat16 values into one 32-bit accumulator give the weighted sum that a 32-bit product would.  The
// bfloat16 instructions do sixteen times the work of the 32-bit ones, so three of them are a fifth of one.
//
// Keys in sight, heads of two maps and their difference: attention_masks.h, attention_window.hip (which
// takes what these kernels do not: 32-bit storage, turned values, kept first positions, sigmoid
// weights, other page sizes).  A sink joins the denominator at the end.  Scores may be soft-capped, c tanh(s / c), and
// a head's output may be multiplied by a sigmoid (HeadGate).
// Cache layout: keys [pages][Hkv][page][maps dk], values [pages][Hkv][dv][page]; pages of a multiple of 16.
//
// Nothing but the final outputs passes through LDS.  The accumulator of S^T = K Q^T holds one query a
// lane and, with the keys of a stretch of 16 dealt to the tile's rows for it, eight CONSECUTIVE keys in
// the eight registers that are the operand of the second product: a lane's values are one 16-byte load
// from the position-contiguous cache.
//   attn_parts_prefill   steps with prompt portions: a wave owns 32 queries of one map of one head
//                        (v_mfma_f32_32x32x16_bf16), a block four waves;
//   attn_parts_decode    steps of single tokens: a wave owns stretches of 64 keys of a row and all maps of
//                        all heads of a key/value head as the columns of v_mfma_f32_16x16x32_bf16;
//   attn_parts_combine   merges the decode kernel's partial results.
#include "common.h"
#include "attention_masks.h"
#include <math.h>

namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef float f32x16_t __attribute__((ext_vector_type(16)));

constexpr float LOG2E = 1.4426950408889634f;

// x = p[0] + p[1] + p[2] for 32-bit x: eight bits of the mantissa each
__device__ __forceinline__ void parts3(const float (&x)[8], bf16x8_t (&p)[3]) {
    float r[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) r[i] = x[i];
#pragma unroll
    for (int k = 0; k < 3; ++k) {
        ri_u32x4_t w;
#pragma unroll
        for (int j = 0; j < 4; ++j) w[j] = __builtin_amdgcn_perm(__float_as_uint(r[2 * j + 1]), __float_as_uint(r[2 * j]), 0x07060302u);
        p[k] = __builtin_bit_cast(bf16x8_t, w);
        if (k < 2) {
#pragma unroll
            for (int i = 0; i < 8; ++i) r[i] -= __uint_as_float(__float_as_uint(r[i]) & 0xffff0000u);
        }
    }
}

__device__ __forceinline__ bf16x8_t zero8() {
    return __builtin_bit_cast(bf16x8_t, ri_u32x4_t{0u, 0u, 0u, 0u});
}

// Scores from the products of queries and keys, in the log2 domain: scale, or the soft cap c tanh(s / c) as
// c (1 - 2 / (1 + exp(2 s / c))).
struct ScoreHow {
    float scale_log2e;      // what a product is multiplied by (1 behind a cap, which leaves log2 units)
    float cap_log2e, cap_k; // c log2(e) (0: no cap), and 2 scale log2(e) / c
    __device__ __forceinline__ float cap(float s) const {
        return cap_log2e * fmaf(-2.f, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s * cap_k)), 1.f);
    }
};

// 1 / denominator of a map from its reference m (log2 domain) and sum l, a sink (natural domain) joining
__device__ __forceinline__ float ap_final(float m, float l, const float* __restrict__ sink, int vh) {
    if (!(l > 0.f)) return 0.f;
    if (sink == nullptr) return 1.f / l;
    const float s = sink[vh] * LOG2E, M = fmaxf(m, s), a = __builtin_amdgcn_exp2f(m - M);
    return a / (l * a + __builtin_amdgcn_exp2f(s - M));
}

// ---------------------------------------------------------------------------
// Prompt portions.  DU: 16-feature units of a map's (padded) queries and keys; FT: 32-feature tiles of the
// values.  Heads here are maps of heads: G = maps H / Hkv of them on a key/value head; the four waves of
// a block are HB = min(G, 4) of them on 4 / HB consecutive tiles of 32 queries.
// ---------------------------------------------------------------------------
size_t ap_lds_bytes(int dv) { return sizeof(float) * 4 * 32 * (size_t)(dv + 4); }

template <int DU, int FT>
__global__ __launch_bounds__(256, FT <= 4 && DU <= 8 ? 2 : 1) void attn_parts_prefill_kernel(
        const bf16_t* __restrict__ q, int q_stride, bf16_t* __restrict__ out, int out_stride,
        const bf16_t* __restrict__ kc, const bf16_t* __restrict__ vc, const int* __restrict__ table, int max_blocks,
        const int* __restrict__ cu_q, const int* __restrict__ q_start, const int* __restrict__ kv_lens,
        int num_rows, int H, int Hkv, int dk, int dv, int page, ScoreHow how, int window, int chunk, int maps, DiffHow diff,
        const float* __restrict__ sink, HeadGate<bf16_t> hgate, int tiles) {
    const float scale_log2e = how.scale_log2e;
    extern __shared__ __align__(16) float lds[];       // [4 waves][32][dv + 4]: the outputs, after the last keys
    const int G = H / Hkv, HB = G < 4 ? G : 4, SB = 4 / HB, TQB = 32 * SB;
    // Blocks of one key/value head are Hkv apart (with eight heads: an XCD's L2 each).  A late tile sees many keys, an
    // early one few: the first half of the blocks take tiles from the end, the second half from the start.
    const int bx = (int)blockIdx.x, g = bx % Hkv, hgroup = blockIdx.y;
    const int at = bx / Hkv, first_half = (tiles + 1) / 2;
    const int tile = at < first_half ? tiles - 1 - at : at - first_half;
    int b = -1, t0 = 0, nt = 0, before = 0;
    for (int r = 0; r < num_rows; ++r) {
        const int lo = cu_q[r], ql = cu_q[r + 1] - lo, n = (ql + TQB - 1) / TQB;
        if (tile < before + n) {
            b = r;
            t0 = lo + (tile - before) * TQB;
            nt = min(TQB, lo + ql - t0);
            break;
        }
        before += n;
    }
    if (b < 0) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int lq = lane & 31, lh = lane >> 5;          // the lane's query (or key row, or value feature), and its half
    const int sub = wave / HB, hh = hgroup * 4 + wave % HB;
    const bool wave_on = sub < SB && hh < G && nt - 32 * sub > 0;
    const int t0w = t0 + 32 * sub, ntw = wave_on ? min(32, nt - 32 * sub) : 0;
    const int p0w = q_start[b] + (t0w - cu_q[b]), kv_len = kv_lens[b];
    const int vh = g * G + (hh < G ? hh : 0), map = maps == 2 ? vh & 1 : 0;
    const int pq = p0w + lq, q_first = aw_first_key(pq, window, chunk);
    const int w_last = wave_on ? min(kv_len, p0w + ntw) : 0;
    const int w_first = aw_first_key(p0w, window, chunk);
    const int* trow = table + (size_t)b * max_blocks;
    const int dkr = maps * dk;
    // row lq of a key tile holds key 16 (lq / 16) + 8 (bit 2 of lq) + 4 (bit 3) + lq % 4 of its 32
    const int krow = ((lq >> 2) & 1) * 8 + ((lq >> 3) & 1) * 4 + (lq & 3);

    bf16x8_t qf[DU];
#pragma unroll
    for (int u = 0; u < DU; ++u) {
        const int d = 16 * u + 8 * lh;
        qf[u] = zero8();                               // beyond dk: zeros, whatever the key operand holds there
        if (lq < ntw && d < dk) qf[u] = *reinterpret_cast<const bf16x8_t*>(q + (size_t)(t0w + lq) * q_stride + (size_t)vh * dk + d);
    }
    f32x16_t o[FT];
#pragma unroll
    for (int ft = 0; ft < FT; ++ft)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[ft][i] = 0.f;
    float m = -INFINITY, l = 0.f;

    auto pages_of = [&](int key0, int& pa, int& pb) {
        pa = trow[min(key0 / page, max_blocks - 1)];
        pb = trow[min((key0 + 16) / page, max_blocks - 1)];
        if (key0 >= kv_len) pa = -1;
        if (key0 + 16 >= kv_len) pb = -1;
    };
    auto load_keys = [&](int key0, int pa, int pb, bf16x8_t (&kf)[DU]) {
        const int pid = max(lq < 16 ? pa : pb, 0);     // a page that is not held: any, its keys are masked
        const int slot = (lq < 16 ? key0 % page : (key0 + 16) % page) + krow;
        const bf16_t* src = kc + (((size_t)pid * Hkv + g) * page + slot) * dkr + map * dk;
#pragma unroll
        for (int u = 0; u < DU; ++u) kf[u] = *reinterpret_cast<const bf16x8_t*>(src + min(16 * u + 8 * lh, dk - 8));
    };
    auto load_values = [&](int key0, int pa, int pb, bf16x8_t (&vf)[FT][2]) {
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const int pid = max(s == 0 ? pa : pb, 0), slot = (key0 + 16 * s) % page + 8 * lh;
            const bf16_t* src = vc + ((size_t)pid * Hkv + g) * dv * page + slot;
#pragma unroll
            for (int ft = 0; ft < FT; ++ft) vf[ft][s] = *reinterpret_cast<const bf16x8_t*>(src + (size_t)min(32 * ft + lq, dv - 1) * page);
        }
    };
    // tiles of 32 keys aligned to absolute positions; those in [hot_lo, hot_hi) need no masks
    const int k_begin = w_first / 32 * 32;
    const int hot_lo = (aw_first_key(p0w + (ntw > 0 ? ntw - 1 : 0), window, chunk) + 31) / 32 * 32, hot_hi = (p0w + 1) / 32 * 32;
    bf16x8_t kf[DU];
    int pa = -1, pb = -1;
    if (k_begin < w_last) {
        pages_of(k_begin, pa, pb);
        load_keys(k_begin, pa, pb, kf);
    }
    for (int key0 = k_begin; key0 < w_last; key0 += 32) {
        bf16x8_t vf[FT][2];
        load_values(key0, pa, pb, vf);
        f32x16_t s;
#pragma unroll
        for (int i = 0; i < 16; ++i) s[i] = 0.f;
#pragma unroll
        for (int u = 0; u < DU; ++u) s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[u], qf[u], s, 0, 0, 0);
        int na = -1, nb = -1;
        if (key0 + 32 < w_last) {                      // the next tile's keys, while this one is worked on
            pages_of(key0 + 32, na, nb);
            load_keys(key0 + 32, na, nb, kf);
        }
        if (how.cap_log2e > 0.f) {
#pragma unroll
            for (int i = 0; i < 16; ++i) s[i] = how.cap(s[i]);
        }
        // register i: key key0 + 16 (i / 8) + 8 lh + i % 8, for the lane's query
        if (key0 < hot_lo || key0 >= hot_hi) {
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const int key = key0 + 16 * (i >> 3) + 8 * lh + (i & 7);
                if (!(key <= pq && key >= q_first && key < kv_len)) s[i] = -INFINITY;
            }
            // positions that no token has written, or of a page that is not held, may be anything
            if (key0 + 32 > kv_len || pa < 0 || pb < 0) {
#pragma unroll
                for (int st = 0; st < 2; ++st) {
                    const int n = (st == 0 ? pa : pb) < 0 ? 0 : kv_len - (key0 + 16 * st + 8 * lh);
#pragma unroll
                    for (int ft = 0; ft < FT; ++ft)
#pragma unroll
                        for (int x = 0; x < 8; ++x)
                            if (x >= n) vf[ft][st][x] = (__bf16)0.f;
                }
            }
        }
        float mx = s[0];
#pragma unroll
        for (int i = 1; i < 16; ++i) mx = fmaxf(mx, s[i]);
        // The reference subtracted before exp2 need not be the maximum, only within 2^24 of it: it moves (and the
        // sums so far are rescaled) when some query of the wave needs it, rarely after a query's first tile.
        if (__any(mx * scale_log2e > m + 24.f)) {
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            const float m_new = fmaxf(m, mx * scale_log2e);
            const float alpha = m_new == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m - m_new);
            l *= alpha;
#pragma unroll
            for (int ft = 0; ft < FT; ++ft)
#pragma unroll
                for (int i = 0; i < 16; ++i) o[ft][i] *= alpha;
            m = m_new;
        }
        const float m_ref = m == -INFINITY ? 0.f : m;  // a query that has seen no key yet
#pragma unroll
        for (int st = 0; st < 2; ++st) {
            float e[8];
#pragma unroll
            for (int x = 0; x < 8; ++x) e[x] = __builtin_amdgcn_exp2f(fmaf(s[8 * st + x], scale_log2e, -m_ref));
            l += ((e[0] + e[1]) + (e[2] + e[3])) + ((e[4] + e[5]) + (e[6] + e[7]));
            bf16x8_t pf[3];
            parts3(e, pf);
#pragma unroll
            for (int ft = 0; ft < FT; ++ft) {
                o[ft] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[ft][st], pf[2], o[ft], 0, 0, 0);
                o[ft] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[ft][st], pf[1], o[ft], 0, 0, 0);
                o[ft] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[ft][st], pf[0], o[ft], 0, 0, 0);
            }
        }
        pa = na;
        pb = nb;
    }
    l += __shfl_xor(l, 32, 64);
    float inv = ap_final(m, l, sink, vh);
    if (lq < ntw) inv *= hgate.at(t0w + lq, vh);           // (one map a head)
    const int os = dv + 4;
    float* ow = lds + (size_t)wave * 32 * os;
    if (wave_on) {
#pragma unroll
        for (int ft = 0; ft < FT; ++ft)
#pragma unroll
            for (int i = 0; i < 16; i += 4) {
                const int f = 32 * ft + 2 * i + 4 * lh;      // rows 8 (i / 4) + 4 lh + 0..3
                if (f < dv) *reinterpret_cast<float4*>(ow + lq * os + f) = make_float4(o[ft][i] * inv, o[ft][i + 1] * inv, o[ft][i + 2] * inv, o[ft][i + 3] * inv);
            }
    }
    __syncthreads();
    if (!wave_on) return;
    constexpr int NC = (FT + 1) / 2;
    if (maps == 2) {
        // the wave and its neighbour hold the two maps of one head for the same 32 tokens: each writes every other token
        const float* o1 = lds + (size_t)(wave & ~1) * 32 * os, *o2 = o1 + (size_t)32 * os;
        for (int r = wave & 1; r < ntw; r += 2) {
            float a[NC], bb[NC];
#pragma unroll
            for (int c = 0; c < NC; ++c) {
                const int f = lane + 64 * c;
                a[c] = f < dv ? o1[r * os + f] : 0.f;
                bb[c] = f < dv ? o2[r * os + f] : 0.f;
            }
            aw_write_difference<bf16_t, NC>(out + (size_t)(t0w + r) * out_stride + vh / 2 * dv, a, bb, dv, lane, diff);
        }
        return;
    }
    for (int r = 0; r < ntw; ++r)
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int f = lane + 64 * c;
            if (f < dv) st_f32(out + (size_t)(t0w + r) * out_stride + vh * dv + f, ow[r * os + f]);
        }
}

// ---------------------------------------------------------------------------
// Single tokens.  KU: 32-feature units of a whole (padded) key row, all maps of it; VU: 16-feature tiles of the
// values.  Column c of the products is map c of the heads of a key/value head (16 a block; CG blocks deal
// the columns); a column's query is zero outside its own map's part of the key row.
// ---------------------------------------------------------------------------
constexpr int AP_KEYS = 64;          // keys a stretch
constexpr int AP_SLOTS = 64;         // most partial results a (token, map of a head): longer rows loop

template <int KU, int VU>
__global__ __launch_bounds__(64) void attn_parts_decode_kernel(
        const bf16_t* __restrict__ q, int q_stride, const bf16_t* __restrict__ kc, const bf16_t* __restrict__ vc,
        const int* __restrict__ table, int max_blocks, const int* __restrict__ cu_q, const int* __restrict__ q_start,
        const int* __restrict__ kv_lens, int H, int Hkv, int dk, int dv, int page, ScoreHow how, int window, int chunk, int maps,
        int slots, int CG, float* __restrict__ part_ml, float* __restrict__ part_o) {
    const int G = H / Hkv, b = blockIdx.z, g = blockIdx.y / CG, c0 = (blockIdx.y % CG) * 16;
    const int lane = threadIdx.x, col = lane & 15, grp = lane >> 4;
    const int t = cu_q[b];
    const bool has_token = cu_q[b + 1] > t;
    const int p = q_start[b], visible = min(kv_lens[b], p + 1);
    const int j0 = aw_first_key(p, window, chunk);
    const int base = j0 / AP_KEYS, slot = blockIdx.x;
    int c = base + slot;
    if (!has_token || c * AP_KEYS >= visible) return;
    const int* trow = table + (size_t)b * max_blocks;
    const int dkr = maps * dk, vh = c0 + col, map = maps == 2 ? vh & 1 : 0;
    bf16x8_t qf[KU];
#pragma unroll
    for (int u = 0; u < KU; ++u) {
        const int d = 32 * u + 8 * grp - map * dk;     // feature of the column's own map (dk is a multiple of 8)
        qf[u] = zero8();
        if (vh < G && d >= 0 && d < dk) qf[u] = *reinterpret_cast<const bf16x8_t*>(q + (size_t)t * q_stride + (size_t)(g * G + vh) * dk + d);
    }
    f32x4_t o[VU];
#pragma unroll
    for (int f = 0; f < VU; ++f) o[f] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    for (; c * AP_KEYS < visible; c += slots) {
        const int c_lo = c * AP_KEYS;
        // all keys and values of the stretch are asked for before anything is computed.  Span sp = keys
        // c_lo + 32 sp .. + 31; its tile e holds, in row r, key 8 (r / 4) + 4 e + r % 4, so that a lane's four scores of
        // either tile are eight consecutive keys
        int pid[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int j = c_lo + 16 * i;
            pid[i] = j < visible && j + 16 > j0 ? trow[min(j / page, max_blocks - 1)] : -1;
        }
        bf16x8_t kf[4][KU], vf[2][VU];
#pragma unroll
        for (int sp = 0; sp < 2; ++sp) {
            const int span0 = c_lo + 32 * sp;
            const int kp = max(col < 8 ? pid[2 * sp] : pid[2 * sp + 1], 0);
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const int key = span0 + (col >> 2) * 8 + 4 * e + (col & 3);
                const bf16_t* src = kc + (((size_t)kp * Hkv + g) * page + key % page) * dkr;
#pragma unroll
                for (int u = 0; u < KU; ++u) kf[2 * sp + e][u] = ld_stream16<bf16x8_t>(src + min(32 * u + 8 * grp, dkr - 8));
            }
            const int vp = max(grp < 2 ? pid[2 * sp] : pid[2 * sp + 1], 0);
            const bf16_t* src = vc + ((size_t)vp * Hkv + g) * dv * page + (span0 + 8 * grp) % page;
#pragma unroll
            for (int f = 0; f < VU; ++f) vf[sp][f] = ld_stream16<bf16x8_t>(src + (size_t)min(16 * f + col, dv - 1) * page);
        }
        // S^T: register i of tile 2 sp + e is key c_lo + 32 sp + 8 grp + 4 e + i, for the lane's column
        f32x4_t s[4];
#pragma unroll
        for (int tl = 0; tl < 4; ++tl) {
            s[tl] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int u = 0; u < KU; ++u) s[tl] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[tl][u], qf[u], s[tl], 0, 0, 0);
        }
        float m_new = m;
#pragma unroll
        for (int tl = 0; tl < 4; ++tl)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int key = c_lo + 32 * (tl >> 1) + 8 * grp + 4 * (tl & 1) + i;
                s[tl][i] = key >= j0 && key < visible ? (how.cap_log2e > 0.f ? how.cap(s[tl][i]) : s[tl][i] * how.scale_log2e) : -INFINITY;
                m_new = fmaxf(m_new, s[tl][i]);
            }
        m_new = fmaxf(m_new, __shfl_xor(m_new, 16, 64));
        m_new = fmaxf(m_new, __shfl_xor(m_new, 32, 64));         // finite: a stretch of the row holds a visible key
        const float alpha = __builtin_amdgcn_exp2f(m - m_new);
        l *= alpha;
#pragma unroll
        for (int i = 0; i < 4; ++i) {                            // sums' rows are the columns 4 grp + i
            const float ai = __shfl(alpha, grp * 4 + i, 64);
#pragma unroll
            for (int f = 0; f < VU; ++f) o[f][i] *= ai;
        }
        m = m_new;
#pragma unroll
        for (int sp = 0; sp < 2; ++sp) {
            const int key0 = c_lo + 32 * sp + 8 * grp;
            // positions that no token has written, or of a page that is not held, may be anything
            const int n = (grp < 2 ? pid[2 * sp] : pid[2 * sp + 1]) < 0 ? 0 : visible - key0;
            if (__any(n < 8)) {
#pragma unroll
                for (int f = 0; f < VU; ++f)
#pragma unroll
                    for (int x = 0; x < 8; ++x)
                        if (x >= n) vf[sp][f][x] = (__bf16)0.f;
            }
            float e[8];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                e[i] = __builtin_amdgcn_exp2f(s[2 * sp][i] - m);
                e[4 + i] = __builtin_amdgcn_exp2f(s[2 * sp + 1][i] - m);
            }
            l += ((e[0] + e[1]) + (e[2] + e[3])) + ((e[4] + e[5]) + (e[6] + e[7]));
            bf16x8_t pf[3];
            parts3(e, pf);
#pragma unroll
            for (int f = 0; f < VU; ++f) {
                o[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[2], vf[sp][f], o[f], 0, 0, 0);
                o[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[1], vf[sp][f], o[f], 0, 0, 0);
                o[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[0], vf[sp][f], o[f], 0, 0, 0);
            }
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (grp == 0 && vh < G) {
        float* dst = part_ml + (((size_t)t * H + g * G + vh) * slots + slot) * 2;
        dst[0] = m;
        dst[1] = l;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int v = c0 + 4 * grp + i;
        if (v >= G) continue;
        float* dst = part_o + (((size_t)t * H + g * G + v) * slots + slot) * dv;
#pragma unroll
        for (int f = 0; f < VU; ++f)
            if (16 * f + col < dv) dst[16 * f + col] = o[f][i];
    }
}

// One block of four waves a (token, head): every wave takes the factors of all partial results of the head's
// maps, the waves divide the results between them, and the first wave adds up, takes the difference, writes.
template <int NC, int MAPS>
__global__ __launch_bounds__(256) void attn_parts_combine_kernel(
        const float* __restrict__ part_ml, const float* __restrict__ part_o, bf16_t* __restrict__ out, int out_stride,
        const int* __restrict__ cu_q, const int* __restrict__ q_start, const int* __restrict__ kv_lens,
        int H, int dv, int window, int chunk, int slots, DiffHow diff, const float* __restrict__ sink,
        HeadGate<bf16_t> hgate) {
    __shared__ float wts[MAPS][AP_SLOTS];
    __shared__ float acc_s[4][MAPS][64 * NC];
    const int b = blockIdx.y, ho = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int t = cu_q[b];
    const int p = q_start[b], visible = min(kv_lens[b], p + 1);
    if (cu_q[b + 1] <= t) return;
    const int n = min(slots, (visible + AP_KEYS - 1) / AP_KEYS - aw_first_key(p, window, chunk) / AP_KEYS);
    float fin[MAPS];
#pragma unroll
    for (int k = 0; k < MAPS; ++k) {
        const size_t at = ((size_t)t * H + ho * MAPS + k) * slots;
        const float m = lane < n ? part_ml[(at + lane) * 2] : -INFINITY, l = lane < n ? part_ml[(at + lane) * 2 + 1] : 0.f;
        const float M = wave_max(m), w = lane < n ? __builtin_amdgcn_exp2f(m - M) : 0.f;
        fin[k] = ap_final(M, wave_sum(w * l), sink, ho * MAPS + k);
        if (MAPS == 1) fin[k] *= hgate.at(t, ho);
        if (wave == 0 && lane < AP_SLOTS) wts[k][lane] = w;
    }
    __syncthreads();
    float acc[MAPS][NC];
#pragma unroll
    for (int k = 0; k < MAPS; ++k)
#pragma unroll
        for (int c = 0; c < NC; ++c) acc[k][c] = 0.f;
#pragma unroll 4
    for (int s = wave; s < n; s += 4)
#pragma unroll
        for (int k = 0; k < MAPS; ++k) {
            const float* src = part_o + (((size_t)t * H + ho * MAPS + k) * slots + s) * dv;
#pragma unroll
            for (int c = 0; c < NC; ++c) acc[k][c] = fmaf(wts[k][s], lane + 64 * c < dv ? src[lane + 64 * c] : 0.f, acc[k][c]);
        }
#pragma unroll
    for (int k = 0; k < MAPS; ++k)
#pragma unroll
        for (int c = 0; c < NC; ++c) acc_s[wave][k][lane + 64 * c] = acc[k][c];
    __syncthreads();
    if (wave != 0) return;
#pragma unroll
    for (int k = 0; k < MAPS; ++k)
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int i = lane + 64 * c;
            acc[k][c] = ((acc_s[0][k][i] + acc_s[1][k][i]) + (acc_s[2][k][i] + acc_s[3][k][i])) * fin[k];
        }
    bf16_t* o = out + (size_t)t * out_stride + ho * dv;
    if constexpr (MAPS == 2) {
        aw_write_difference<bf16_t, NC>(o, acc[0], acc[1], dv, lane, diff);
    } else {
#pragma unroll
        for (int c = 0; c < NC; ++c)
            if (lane + 64 * c < dv) st_f32(o + lane + 64 * c, acc[0][c]);
    }
}

int ap_slots(int window, int chunk, int max_kv_len) {
    int span = max_kv_len;
    if (window > 0) span = min(window, span);
    if (chunk > 0) span = min(chunk, span);
    const int n = (span + AP_KEYS - 1) / AP_KEYS + (window > 0 || chunk > 0 ? 1 : 0);    // a window or chunk may begin inside a stretch
    return min(max(n, 1), AP_SLOTS);
}

}  // namespace

extern "C" int ri_attention_parts_supported(int H, int Hkv, int dk, int dv, int maps, int page) {
    return H > 0 && Hkv > 0 && H % Hkv == 0 && (maps == 1 || maps == 2) && H / Hkv * maps <= 256 && dk > 0 && dk % 8 == 0
        && maps * dk <= 256 && dv > 0 && dv % 8 == 0 && dv <= 256 && page > 0 && page % 16 == 0;
}

// Floats of workspace for a step of T single tokens whose longest request has max_kv_len keys.
extern "C" size_t ri_attention_parts_workspace(int T, int H, int dv, int maps, int window, int chunk, int max_kv_len) {
    return (size_t)T * H * maps * ap_slots(window, chunk, max_kv_len) * (dv + 2);
}

// bfloat16 attention of the step's tokens over the cache; arguments as ri_attention_window's.
// single_tokens != 0: every row has at most one token, row b's is token cu_q[b] (workspace needed).
// softcap > 0: a score s becomes softcap tanh(s / softcap).  gate [T][>= H] (null: none) with a row stride: a head's
// output is multiplied by the sigmoid of its number there (maps = 1).
extern "C" int ri_attention_parts(
        const void* q, int q_stride, void* out, int out_stride, const void* kc, const void* vc, int num_pages, int page,
        int H, int Hkv, int dk, int dv, const int* table, int max_blocks, const int* cu_q, const int* q_start, const int* kv_lens,
        int num_rows, int T, float scale, int window, int chunk, int maps, float diff_lam, float diff_gain, float diff_eps,
        const float* sink, float softcap, const void* gate, int gate_stride, int single_tokens, int max_kv_len, float* workspace,
        size_t workspace_floats, hipStream_t stream) {
    RI_REQUIRE(ri_attention_parts_supported(H, Hkv, dk, dv, maps, page), "ri_attention_parts: sizes not taken (H=%d Hkv=%d dk=%d dv=%d maps=%d page=%d)", H, Hkv, dk, dv, maps, page);
    RI_REQUIRE(T >= 0 && num_rows >= 0 && max_blocks > 0 && num_pages > 0 && window >= 0 && chunk >= 0, "ri_attention_parts: bad sizes");
    RI_REQUIRE(maps == 1 || diff_eps > 0.f, "ri_attention_parts: the difference of two maps takes an eps > 0");
    RI_REQUIRE(q_stride >= H * maps * dk && out_stride >= H * dv && q_stride % 8 == 0, "ri_attention_parts: row strides too small, or a query stride that is no multiple of 8");
    RI_REQUIRE(softcap >= 0.f && (!gate || (maps == 1 && gate_stride >= H)), "ri_attention_parts: softcap must be >= 0; a gate goes with one map a head and a row stride of at least the heads");
    if (T == 0 || num_rows == 0) return 0;
    RI_REQUIRE(q && out && kc && vc && table && cu_q && q_start && kv_lens, "ri_attention_parts: null pointer");
    RI_REQUIRE((uintptr_t)q % 16 == 0 && (uintptr_t)kc % 16 == 0 && (uintptr_t)vc % 16 == 0, "ri_attention_parts: operands must be aligned to 16 bytes");
    const DiffHow diff{diff_lam, diff_gain, diff_eps};
    const int Hm = H * maps, G = Hm / Hkv;
    const bf16_t* qb = (const bf16_t*)q;
    const bf16_t* kb = (const bf16_t*)kc;
    const bf16_t* vb = (const bf16_t*)vc;
    bf16_t* ob = (bf16_t*)out;
    const ScoreHow how{softcap > 0.f ? 1.f : scale * LOG2E, softcap * LOG2E, softcap > 0.f ? 2.f * scale * LOG2E / softcap : 0.f};
    const HeadGate<bf16_t> hgate{(const bf16_t*)gate, gate_stride};
    if (single_tokens) {
        const int slots = ap_slots(window, chunk, max_kv_len), CG = (G + 15) / 16;
        RI_REQUIRE(workspace && max_kv_len > 0 && workspace_floats >= (size_t)T * Hm * slots * (dv + 2), "ri_attention_parts: workspace of %zu floats for %d slots", workspace_floats, slots);
        RI_REQUIRE(num_rows <= 65535 && (long)Hkv * CG <= 65535, "ri_attention_parts: too many rows or heads for the grid");
        float* part_ml = workspace;
        float* part_o = workspace + (size_t)T * Hm * slots * 2;
        const int KU = (maps * dk + 31) / 32, VU = (dv + 15) / 16;
        auto part = KU <= 2 ? (VU <= 4 ? attn_parts_decode_kernel<2, 4> : VU <= 8 ? attn_parts_decode_kernel<2, 8> : attn_parts_decode_kernel<2, 16>)
                  : KU <= 4 ? (VU <= 4 ? attn_parts_decode_kernel<4, 4> : VU <= 8 ? attn_parts_decode_kernel<4, 8> : attn_parts_decode_kernel<4, 16>)
                            : (VU <= 4 ? attn_parts_decode_kernel<8, 4> : VU <= 8 ? attn_parts_decode_kernel<8, 8> : attn_parts_decode_kernel<8, 16>);
        part<<<dim3(slots, Hkv * CG, num_rows), 64, 0, stream>>>(qb, q_stride, kb, vb, table, max_blocks, cu_q, q_start, kv_lens, Hm, Hkv, dk, dv, page, how,
                                                                 window, chunk, maps, slots, CG, part_ml, part_o);
        const int NC = (dv + 63) / 64;
#define RI_AP_COMBINE(MM) (NC == 1 ? attn_parts_combine_kernel<1, MM> : NC == 2 ? attn_parts_combine_kernel<2, MM> \
                         : NC == 3 ? attn_parts_combine_kernel<3, MM> : attn_parts_combine_kernel<4, MM>)
        auto combine = maps == 2 ? RI_AP_COMBINE(2) : RI_AP_COMBINE(1);
#undef RI_AP_COMBINE
        combine<<<dim3(H, num_rows), 256, 0, stream>>>(part_ml, part_o, ob, out_stride, cu_q, q_start, kv_lens, Hm, dv, window, chunk, slots, diff, sink, hgate);
        RI_LAUNCHED("ri_attention_parts");
        return 0;
    }
    const int HB = G < 4 ? G : 4, TQB = 32 * (4 / HB);
    const int tiles = (T + TQB - 1) / TQB + num_rows;      // at most: every request may end in a short tile
    const size_t lds = ap_lds_bytes(dv);
    const int DU = (dk + 15) / 16, FT = (dv + 31) / 32;
#define RI_AP(D, F) do { auto kernel = attn_parts_prefill_kernel<D, F>; \
        if (lds > 64 * 1024) { \
            static bool asked = false; \
            if (!asked) { \
                hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); \
                RI_REQUIRE(e == hipSuccess, "ri_attention_parts: %zu bytes of LDS refused: %s", lds, hipGetErrorString(e)); \
                asked = true; \
            } \
        } \
        kernel<<<dim3(tiles * Hkv, (G + 3) / 4), 256, lds, stream>>>(qb, q_stride, ob, out_stride, kb, vb, table, max_blocks, cu_q, q_start, kv_lens, num_rows, \
            Hm, Hkv, dk, dv, page, how, window, chunk, maps, diff, sink, hgate, tiles); } while (0)
#define RI_AP_F(D) do { if (FT <= 2) RI_AP(D, 2); else if (FT <= 4) RI_AP(D, 4); else RI_AP(D, 8); } while (0)
    if (DU <= 4) RI_AP_F(4);
    else if (DU <= 8) RI_AP_F(8);
    else RI_AP_F(16);
#undef RI_AP_F
#undef RI_AP
    RI_LAUNCHED("ri_attention_parts");
    return 0;
}
