// rope_kv.hip — rotary positions fused with the paged KV store, and what attention heads need after the softmax when they are
// gated or combined.
//
// Rotation: inside a head, for i < rot_dims / 2, dimension 2i is paired with dimension 2i + 1 (interleaved pairs) or dimension i
// with dimension i + rot_dims / 2 (halves: the kernels that take `half`); the pair (u, v) of a token at position p becomes
// (u cos a - v sin a, v cos a + u sin a), a = p * freq[i]. The frequencies come from the host as a float64 table (evaluated once
// per model, any interpolation included); the angle and its sine and cosine are evaluated in float64 per (token, i) into LDS —
// times a constant, where the kernel takes one — and used in fp32 by every head of the token: exact to fp32 rounding at any
// position. Dimensions from rot_dims on pass unchanged.
//
//   swl_rope_store_kv         rows [q: nq heads of d | k: nk heads of d | v: nv heads of dv]: q rotated in place, k rotated
//                             into the K pool, v copied into the V pool.
//   swl_qk_norm_rope_store_kv rows [q | k (| v)] of a projection whose biases are still to be added: per head bias, weighted RMS norm,
//                             rotation; q times a factor per head into a buffer of its own, k into the K pool, and into the V
//                             pool either the value columns or the KEYS AS PROJECTED (bias added, neither normed nor rotated).
//   swl_qkv_conv_rope_store_kv  rows [q | k | v] of a projection whose biases are still to be added, each step optional: bias, causal
//                             convolution over time per channel (inputs of earlier steps carried as projected, conv_tail.h),
//                             weighted RMS norm of the q / k heads, rotation; q into a buffer of its own, k into the K pool, v
//                             times a constant into the V pool. The row passes through LDS in fp32 and is rounded once.
//   swl_latent_rope_store_kv  latent attention. Rows hold H query heads [d unrotated | dr rotated] and (optionally) the
//                             compressed key/value row [r latent | dr shared rotated key part]. The rotated query parts go
//                             to qa[t][h][r : r + dr] (the caller fills qa[t][h][0 : r] with the queries folded through
//                             the key up-projection); the latent is RMS-normed (fp32 statistics, weight) and stored
//                             together with the rotated key part as ONE key head of r + dr, and once more, transposed, as
//                             the value head of r: attention over the pool then IS the latent attention with the
//                             up-projections applied outside (queries before, outputs after).
//   swl_diff_head_combine     out = unit_rms(a1 - lambda a2) * mult * sigmoid(gate) per head, a1 / a2 the fp32 results of two
//                             score maps over the same values.
//   swl_head_gate             y[t][h][:] *= sigmoid(gate[t][h]).
//
// Pool layout as in qknorm_kv.hip: keys of a page [heads, 16, d], values transposed [heads, dv, 16]. The two kernels in the
// middle may lay heads out wider than they are (k_dim, v_dim: the row sizes that a compiled attention kernel serves); the
// columns beyond the head are written as zeros, which neither scores nor outputs see.
#include "swl_common.h"
#include "conv_tail.h"

namespace swl {

constexpr int kRkThreads = 256;
constexpr int kRkBlock = 16;        // tokens per KV block
constexpr int kRkMaxPairs = 256;    // rot_dims <= 512

__device__ __forceinline__ void rk_angles(float *cs, float *sn, const double *freq, int pos, int pairs, double mult = 1.0) {
    for (int i = threadIdx.x; i < pairs; i += kRkThreads) {
        const double a = static_cast<double>(pos) * freq[i];
        cs[i] = static_cast<float>(cos(a) * mult);
        sn[i] = static_cast<float>(sin(a) * mult);
    }
}

__device__ __forceinline__ float rk_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

template <typename T>
__global__ __launch_bounds__(kRkThreads) void rope_store_kv_kernel(
    T *qkv, const double *freq, T *k_cache, T *v_cache, const int32_t *block_table, const int32_t *tok_seq,
    const int32_t *tok_pos, int nq, int nk, int nv, int d, int dv, int rot_dims, int64_t tok_stride, int max_blocks_per_seq,
    int64_t block_stride) {
    __shared__ float cs[kRkMaxPairs], sn[kRkMaxPairs];
    const int64_t t = blockIdx.x;
    const int pos = tok_pos[t];
    const int pairs = rot_dims >> 1;
    rk_angles(cs, sn, freq, pos, pairs);
    __syncthreads();
    T *row = qkv + t * tok_stride;
    const bool store = k_cache != nullptr;
    int64_t blk = 0;
    if (store) blk = block_table[static_cast<int64_t>(tok_seq[t]) * max_blocks_per_seq + pos / kRkBlock];
    const int off = pos % kRkBlock;
    // queries: only the rotated pairs change
    for (int i = threadIdx.x; i < nq * pairs; i += kRkThreads) {
        const int h = i / pairs, j = i - h * pairs;
        T *p = row + static_cast<int64_t>(h) * d + 2 * j;
        const float u = to_f(p[0]), v = to_f(p[1]);
        p[0] = to_t<T>(u * cs[j] - v * sn[j]);
        p[1] = to_t<T>(v * cs[j] + u * sn[j]);
    }
    if (!store) return;
    // keys: every element goes to the pool, the first rot_dims of each head rotated
    const T *krow = row + static_cast<int64_t>(nq) * d;
    for (int i = threadIdx.x; i < nk * d; i += kRkThreads) {
        const int g = i / d, e = i - g * d;
        float x = to_f(krow[i]);
        if (e < rot_dims) {
            const int j = e >> 1;
            const float other = to_f(krow[i ^ 1]);      // (d is even: the partner is inside the head)
            x = (e & 1) ? x * cs[j] + other * sn[j] : x * cs[j] - other * sn[j];
        }
        k_cache[blk * block_stride + (static_cast<int64_t>(g) * kRkBlock + off) * d + e] = to_t<T>(x);
    }
    const T *vrow = krow + static_cast<int64_t>(nk) * d;
    for (int i = threadIdx.x; i < nv * dv; i += kRkThreads)
        v_cache[blk * block_stride + static_cast<int64_t>(i) * kRkBlock + off] = vrow[i];       // transposed page
}

template <typename T>
__global__ __launch_bounds__(kRkThreads) void qk_norm_rope_store_kv_kernel(
    const T *rows, T *q_out, const float *q_b, const float *k_b, const float *q_w, const float *k_w, const float *q_mult,
    const double *freq, T *k_cache, T *v_cache, const int32_t *block_table, const int32_t *tok_seq, const int32_t *tok_pos, int nq,
    int nk, int nv, int d, int dv, int rot_dims, int half, double rot_mult, int64_t tok_stride, int64_t q_out_stride, int k_dim,
    int v_dim, int keys_as_values, int max_blocks_per_seq, int64_t block_stride, float eps) {
    __shared__ float cs[kRkMaxPairs], sn[kRkMaxPairs];
    const int64_t t = blockIdx.x;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int pos = tok_pos[t];
    const int pairs = rot_dims >> 1;
    const T *row = rows + t * tok_stride;
    T *qrow = q_out + t * q_out_stride;
    const bool store = k_cache != nullptr;
    int64_t blk = 0;
    if (store) blk = block_table[static_cast<int64_t>(tok_seq[t]) * max_blocks_per_seq + pos / kRkBlock];
    const int off = pos % kRkBlock;
    T *kpage = k_cache + blk * block_stride, *vpage = v_cache + blk * block_stride;
    const int heads = store ? nq + nk : nq;
    bool wide = false;
    if constexpr (sizeof(T) == 2) {
        // 16-bit heads of a multiple of 8 elements up to 128 on 16-byte-aligned rows: a power-of-two group of lanes per head,
        // 8 elements per lane; a rotated lane's partner elements are 8 neighbours too (or, interleaved, its own)
        wide = d % 8 == 0 && d <= 128 && (tok_stride & 7) == 0 && (q_out_stride & 7) == 0 && (k_dim & 7) == 0 &&
               (half ? (pairs & 7) == 0 : (rot_dims & 7) == 0) && (block_stride & 7) == 0 &&
               ((reinterpret_cast<uintptr_t>(rows) | reinterpret_cast<uintptr_t>(q_out) | reinterpret_cast<uintptr_t>(k_cache) |
                 reinterpret_cast<uintptr_t>(q_b) | reinterpret_cast<uintptr_t>(k_b) | reinterpret_cast<uintptr_t>(q_w) |
                 reinterpret_cast<uintptr_t>(k_w)) & 15) == 0;
        if (wide) {
            const int lph = d <= 8 ? 1 : d <= 16 ? 2 : d <= 32 ? 4 : d <= 64 ? 8 : 16;      // lanes per head
            const int hpw = 64 / lph;
            const int slot = lane / lph, el = lane - slot * lph, e0 = el * 8;
            const bool turns = e0 < rot_dims, first = e0 < pairs;
            // (half) the partner elements of this lane's, and the pair index of its first element
            const int p0 = half && turns ? (first ? e0 + pairs : e0 - pairs) : e0;
            const int a0 = half ? (first ? e0 : p0) : e0 >> 1;
            // everything a head needs from memory is requested together, the first head's before the angles are evaluated
            vec8_t<T> own, other;
            float4_t bo[2], bp[2], wo[2], wp[2];
            float mult;
            auto fetch = [&](int hb) {
                const int h = hb + slot;
                const bool live = h < heads && e0 < d, is_q = h < nq;
                own = other = vec8_t<T>{};
                mult = 1.0f;
#pragma unroll
                for (int k = 0; k < 2; ++k) {
                    bo[k] = bp[k] = float4_t{0.f, 0.f, 0.f, 0.f};
                    wo[k] = wp[k] = float4_t{1.f, 1.f, 1.f, 1.f};
                }
                if (!live) return;
                const T *src = row + static_cast<int64_t>(h) * d;
                const float *bias = is_q ? q_b : k_b, *wn = is_q ? q_w : k_w;
                own = load8(src + e0);
                other = load8(src + p0);
                if (bias) {
                    bias += static_cast<int64_t>(is_q ? h : h - nq) * d;
#pragma unroll
                    for (int k = 0; k < 2; ++k) {
                        bo[k] = *reinterpret_cast<const float4_t *>(bias + e0 + 4 * k);
                        bp[k] = *reinterpret_cast<const float4_t *>(bias + p0 + 4 * k);
                    }
                }
                if (wn) {
#pragma unroll
                    for (int k = 0; k < 2; ++k) {
                        wo[k] = *reinterpret_cast<const float4_t *>(wn + e0 + 4 * k);
                        wp[k] = *reinterpret_cast<const float4_t *>(wn + p0 + 4 * k);
                    }
                }
                if (is_q && q_mult) mult = q_mult[h];
            };
            fetch(wave * hpw);
            rk_angles(cs, sn, freq, pos, pairs, rot_mult);
            __syncthreads();
            for (int hb = wave * hpw; hb < heads; hb += (kRkThreads / 64) * hpw) {
                if (hb != wave * hpw) fetch(hb);
                const int h = hb + slot;
                const bool live = h < heads && e0 < d, is_q = h < nq;
                float v[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) v[j] = to_f(own[j]) + bo[j >> 2][j & 3];
                float ss = 0.f;
#pragma unroll
                for (int j = 0; j < 8; ++j) ss += v[j] * v[j];
                ss = lph == 1 ? ss : lph == 2 ? group_allreduce_sum<2>(ss) : lph == 4 ? group_allreduce_sum<4>(ss)
                   : lph == 8 ? group_allreduce_sum<8>(ss) : group_allreduce_sum<16>(ss);
                if (!live) continue;
                const float r = (is_q ? q_w : k_w) ? 1.0f / sqrtf(ss / static_cast<float>(d) + eps) : 1.0f;
                if (!is_q && keys_as_values) {
                    T *dst = vpage + (static_cast<int64_t>(h - nq) * v_dim + e0) * kRkBlock + off;
#pragma unroll
                    for (int j = 0; j < 8; ++j) dst[j * kRkBlock] = to_t<T>(v[j]);
                }
                float n[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) n[j] = v[j] * r * wo[j >> 2][j & 3];
                if (turns && half) {
#pragma unroll
                    for (int j = 0; j < 8; ++j) {
                        const float w = (to_f(other[j]) + bp[j >> 2][j & 3]) * r * wp[j >> 2][j & 3];
                        n[j] = first ? n[j] * cs[a0 + j] - w * sn[a0 + j] : n[j] * cs[a0 + j] + w * sn[a0 + j];
                    }
                } else if (turns) {
#pragma unroll
                    for (int j = 0; j < 8; j += 2) {
                        const float c = cs[a0 + (j >> 1)], sv = sn[a0 + (j >> 1)], u = n[j], w = n[j + 1];
                        n[j] = u * c - w * sv;
                        n[j + 1] = w * c + u * sv;
                    }
                }
                vec8_t<T> o;
#pragma unroll
                for (int j = 0; j < 8; ++j) o[j] = to_t<T>(n[j] * mult);
                store8(is_q ? qrow + static_cast<int64_t>(h) * k_dim + e0
                            : kpage + (static_cast<int64_t>(h - nq) * kRkBlock + off) * k_dim + e0, o);
            }
        }
    }
    if (!wide) {
        rk_angles(cs, sn, freq, pos, pairs, rot_mult);
        __syncthreads();
    }
    for (int h = wave; h < heads && !wide; h += kRkThreads / 64) {
        const bool is_q = h < nq;
        const T *src = row + static_cast<int64_t>(h) * d;
        const float *bias = is_q ? q_b : k_b, *wn = is_q ? q_w : k_w;
        if (bias) bias += static_cast<int64_t>(is_q ? h : h - nq) * d;
        auto biased = [&](int e) { return to_f(src[e]) + (bias ? bias[e] : 0.f); };
        float ss = 0.f;
        for (int e = lane; e < d; e += 64) {
            const float v = biased(e);
            ss += v * v;
            if (!is_q && keys_as_values) vpage[(static_cast<int64_t>(h - nq) * v_dim + e) * kRkBlock + off] = to_t<T>(v);
        }
        ss = wave_allreduce_sum(ss);
        const float r = wn ? 1.0f / sqrtf(ss / static_cast<float>(d) + eps) : 1.0f;
        auto normed = [&](int e) { return wn ? biased(e) * r * wn[e] : biased(e); };
        const float mult = is_q && q_mult ? q_mult[h] : 1.0f;
        T *dst = is_q ? qrow + static_cast<int64_t>(h) * k_dim : kpage + (static_cast<int64_t>(h - nq) * kRkBlock + off) * k_dim;
        for (int e = lane; e < d; e += 64) {
            float n = normed(e);
            if (e < rot_dims) {
                const bool first = half ? e < pairs : (e & 1) == 0;
                const int p = half ? (first ? e + pairs : e - pairs) : e ^ 1, a = half ? (first ? e : p) : e >> 1;
                const float w = normed(p);
                n = first ? n * cs[a] - w * sn[a] : n * cs[a] + w * sn[a];
            }
            dst[e] = to_t<T>(n * mult);
        }
    }
    // zero the columns beyond the head
    const int kpad = k_dim - d;
    for (int i = threadIdx.x; i < heads * kpad; i += kRkThreads) {
        const int h = i / kpad, e = d + i - h * kpad;
        if (h < nq) qrow[static_cast<int64_t>(h) * k_dim + e] = to_t<T>(0.f);
        else kpage[(static_cast<int64_t>(h - nq) * kRkBlock + off) * k_dim + e] = to_t<T>(0.f);
    }
    if (!store) return;
    const int nval = keys_as_values ? nk : nv, dval = keys_as_values ? d : dv, vpad = v_dim - dval;
    if (!keys_as_values) {
        const T *vrow = row + static_cast<int64_t>(nq + nk) * d;
        for (int i = threadIdx.x; i < nv * dv; i += kRkThreads) {
            const int g = i / dv, c = i - g * dv;
            vpage[(static_cast<int64_t>(g) * v_dim + c) * kRkBlock + off] = vrow[i];
        }
    }
    for (int i = threadIdx.x; i < nval * vpad; i += kRkThreads) {
        const int g = i / vpad, c = dval + i - g * vpad;
        vpage[(static_cast<int64_t>(g) * v_dim + c) * kRkBlock + off] = to_t<T>(0.f);
    }
}

template <typename T>
__global__ __launch_bounds__(kRkThreads) void qkv_conv_rope_store_kv_kernel(
    const T *rows, int64_t tok_stride, T *q_out, int64_t q_out_stride, const float *bias, const float *conv_w, int taps,
    const float *q_w, const float *k_w, const double *freq, int rot_dims, int half, double rot_mult, float v_mult, T *k_cache,
    T *v_cache, const int32_t *block_table, int max_blocks_per_seq, int64_t block_stride, float *state, int64_t slot_stride,
    int64_t tail_off, const int32_t *tok_pos, const int32_t *tok_start, const int32_t *tok_state, const int32_t *tok_seq,
    int64_t num_tokens, int nq, int nk, int d, int dv, int k_dim, int v_dim, float eps) {
    extern __shared__ float act[];      // [(nq + nk) d + nk dv] biased, convolved channels; then [nq + nk] the heads' 1 / rms
    __shared__ float cs[kRkMaxPairs], sn[kRkMaxPairs];
    const int64_t t = blockIdx.x;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int pos = tok_pos[t];
    const int pairs = rot_dims >> 1, heads = nq + nk, C = heads * d + nk * dv;
    float *rinv = act + C;
    const T *row = rows + t * tok_stride;
    if (conv_w) {
        const ConvTail tail(state, slot_stride, tail_off, tok_pos, tok_start, tok_state, tok_seq, num_tokens, C, taps, t);
        bool wide = false;
        if constexpr (sizeof(T) == 2) {
            wide = ConvTail::wide_ok(rows, tok_stride, conv_w, state, slot_stride, tail_off, C) &&
                   (reinterpret_cast<uintptr_t>(bias) & 15) == 0;
            if (wide) {
                for (int c = threadIdx.x * 8; c < C; c += kRkThreads * 8) {
                    const vec8_t<T> x = load8(row + c);
                    float cur[8], b[8], a[8];
#pragma unroll
                    for (int j = 0; j < 8; ++j) {
                        cur[j] = to_f(x[j]);
                        b[j] = bias ? bias[c + j] : 0.f;
                        a[j] = 0.f;
                    }
                    for (int k = taps - 1; k >= 1; --k) {       // inputs before the sequence are zero, biases included
                        if (pos - k < 0) continue;
                        float v[8];
                        tail.at8(rows, tok_stride, c, pos - k, v);
                        const float *wk = conv_w + static_cast<int64_t>(taps - 1 - k) * C + c;
#pragma unroll
                        for (int j = 0; j < 8; ++j) a[j] += wk[j] * (v[j] + b[j]);
                    }
                    const float *wl = conv_w + static_cast<int64_t>(taps - 1) * C + c;
#pragma unroll
                    for (int j = 0; j < 8; ++j) act[c + j] = a[j] + wl[j] * (cur[j] + b[j]);
                    tail.save8(rows, tok_stride, c, cur);
                }
            }
        }
        for (int c = threadIdx.x; c < C && !wide; c += kRkThreads) {
            const float cur = to_f(row[c]), b = bias ? bias[c] : 0.f;
            float a = 0.f;
            for (int k = taps - 1; k >= 1; --k)
                if (pos - k >= 0)
                    a += conv_w[static_cast<int64_t>(taps - 1 - k) * C + c] * (tail.at(rows, tok_stride, c, pos - k) + b);
            act[c] = a + conv_w[static_cast<int64_t>(taps - 1) * C + c] * (cur + b);
            tail.save(rows, tok_stride, c, cur);
        }
    } else {
        bool wide = false;
        if constexpr (sizeof(T) == 2) {
            wide = (C & 7) == 0 && (tok_stride & 7) == 0 && (reinterpret_cast<uintptr_t>(rows) & 15) == 0;
            if (wide) {
                for (int c = threadIdx.x * 8; c < C; c += kRkThreads * 8) {
                    const vec8_t<T> x = load8(row + c);
#pragma unroll
                    for (int j = 0; j < 8; ++j) act[c + j] = to_f(x[j]) + (bias ? bias[c + j] : 0.f);
                }
            }
        }
        for (int c = threadIdx.x; c < C && !wide; c += kRkThreads) act[c] = to_f(row[c]) + (bias ? bias[c] : 0.f);
    }
    rk_angles(cs, sn, freq, pos, pairs, rot_mult);
    __syncthreads();
    if (q_w) {
        for (int h = wave; h < heads; h += kRkThreads / 64) {
            float ss = 0.f;
            for (int e = lane; e < d; e += 64) ss += act[h * d + e] * act[h * d + e];
            ss = wave_allreduce_sum(ss);
            if (lane == 0) rinv[h] = 1.0f / sqrtf(ss / static_cast<float>(d) + eps);
        }
        __syncthreads();
    }
    auto element = [&](int h, int e) {      // element e of head h: normed and rotated
        const float *a = act + h * d, *w = h < nq ? q_w : k_w;
        const float r = q_w ? rinv[h] : 1.f;
        float n = q_w ? a[e] * r * w[e] : a[e];
        if (e < rot_dims) {
            const bool first = half ? e < pairs : (e & 1) == 0;
            const int p = half ? (first ? e + pairs : e - pairs) : e ^ 1, i = half ? (first ? e : p) : e >> 1;
            const float o = q_w ? a[p] * r * w[p] : a[p];
            n = first ? n * cs[i] - o * sn[i] : n * cs[i] + o * sn[i];
        }
        return n;
    };
    const bool store = k_cache != nullptr;
    int64_t blk = 0;
    if (store) blk = block_table[static_cast<int64_t>(tok_seq[t]) * max_blocks_per_seq + pos / kRkBlock];
    const int off = pos % kRkBlock;
    T *qrow = q_out + t * q_out_stride;
    T *kpage = k_cache + blk * block_stride, *vpage = v_cache + blk * block_stride;
    const int outs = store ? heads : nq;
    if (sizeof(T) == 2 && (k_dim & 7) == 0 && (q_out_stride & 7) == 0 && (block_stride & 7) == 0 &&
        ((reinterpret_cast<uintptr_t>(q_out) | reinterpret_cast<uintptr_t>(k_cache)) & 15) == 0) {
        const int per = k_dim >> 3;
        for (int i = threadIdx.x; i < outs * per; i += kRkThreads) {
            const int h = i / per, e0 = (i - h * per) * 8;
            vec8_t<T> o;
#pragma unroll
            for (int j = 0; j < 8; ++j) o[j] = to_t<T>(e0 + j < d ? element(h, e0 + j) : 0.f);
            store8(h < nq ? qrow + static_cast<int64_t>(h) * k_dim + e0
                          : kpage + (static_cast<int64_t>(h - nq) * kRkBlock + off) * k_dim + e0, o);
        }
    } else {
        for (int i = threadIdx.x; i < outs * k_dim; i += kRkThreads) {
            const int h = i / k_dim, e = i - h * k_dim;
            T *dst = h < nq ? qrow + static_cast<int64_t>(h) * k_dim : kpage + (static_cast<int64_t>(h - nq) * kRkBlock + off) * k_dim;
            dst[e] = to_t<T>(e < d ? element(h, e) : 0.f);
        }
    }
    if (!store) return;
    for (int i = threadIdx.x; i < nk * v_dim; i += kRkThreads) {        // (the transposed page: 16 tokens of a column together)
        const int g = i / v_dim, c = i - g * v_dim;
        vpage[static_cast<int64_t>(i) * kRkBlock + off] = to_t<T>(c < dv ? act[heads * d + g * dv + c] * v_mult : 0.f);
    }
}

template <typename T>
__global__ __launch_bounds__(kRkThreads) void latent_rope_store_kv_kernel(
    const T *proj, T *qa, const double *freq, const float *c_w, T *k_cache, T *v_cache, const int32_t *block_table,
    const int32_t *tok_seq, const int32_t *tok_pos, int H, int d, int dr, int r, int64_t proj_stride, int64_t dkv_col,
    int64_t qa_stride, int max_blocks_per_seq, int64_t block_stride, float eps, int half, double rot_mult, int k_dim,
    int v_dim) {
    __shared__ float cs[kRkMaxPairs], sn[kRkMaxPairs];
    __shared__ float red[kRkThreads / 64];
    const int64_t t = blockIdx.x;
    const int pos = tok_pos[t];
    const int pairs = dr >> 1;
    rk_angles(cs, sn, freq, pos, pairs, rot_mult);
    __syncthreads();
    const T *row = proj + t * proj_stride;
    T *qrow = qa + t * qa_stride;
    // pair j of a rotated part: elements (2j, 2j + 1), or (j, j + pairs)
    const int step = half ? 1 : 2, gap = half ? pairs : 1;
    for (int i = threadIdx.x; i < H * pairs; i += kRkThreads) {
        const int h = i / pairs, j = i - h * pairs;
        const T *p = row + static_cast<int64_t>(h) * (d + dr) + d + step * j;
        T *o = qrow + static_cast<int64_t>(h) * k_dim + r + step * j;
        const float u = to_f(p[0]), v = to_f(p[gap]);
        o[0] = to_t<T>(u * cs[j] - v * sn[j]);
        o[gap] = to_t<T>(v * cs[j] + u * sn[j]);
    }
    const int kpad = k_dim - r - dr, vpad = v_dim - r;
    for (int i = threadIdx.x; i < H * kpad; i += kRkThreads) {
        const int h = i / kpad;
        qrow[static_cast<int64_t>(h) * k_dim + r + dr + i - h * kpad] = to_t<T>(0.f);
    }
    if (dkv_col < 0 || k_cache == nullptr) return;
    const T *z = row + dkv_col;
    float ss = 0.f;
    for (int i = threadIdx.x; i < r; i += kRkThreads) {
        const float x = to_f(z[i]);
        ss += x * x;
    }
    ss = wave_allreduce_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < kRkThreads / 64; ++w) ss += red[w];
    const float rinv = 1.0f / sqrtf(ss / static_cast<float>(r) + eps);
    const int64_t blk = block_table[static_cast<int64_t>(tok_seq[t]) * max_blocks_per_seq + pos / kRkBlock];
    const int off = pos % kRkBlock;
    T *kdst = k_cache + blk * block_stride + static_cast<int64_t>(off) * k_dim;
    T *vdst = v_cache + blk * block_stride + off;
    for (int i = threadIdx.x; i < r; i += kRkThreads) {
        const T c = to_t<T>(to_f(z[i]) * rinv * c_w[i]);
        kdst[i] = c;
        vdst[static_cast<int64_t>(i) * kRkBlock] = c;
    }
    for (int j = threadIdx.x; j < pairs; j += kRkThreads) {
        const float u = to_f(z[r + step * j]), v = to_f(z[r + step * j + gap]);
        kdst[r + step * j] = to_t<T>(u * cs[j] - v * sn[j]);
        kdst[r + step * j + gap] = to_t<T>(v * cs[j] + u * sn[j]);
    }
    for (int i = threadIdx.x; i < kpad; i += kRkThreads) kdst[r + dr + i] = to_t<T>(0.f);
    for (int i = threadIdx.x; i < vpad; i += kRkThreads) vdst[static_cast<int64_t>(r + i) * kRkBlock] = to_t<T>(0.f);
}

template <typename T>
__global__ __launch_bounds__(256) void diff_head_combine_kernel(T *out, const float *a, const T *gate, int64_t gate_stride,
                                                                float lambda, float mult, float eps, int H, int dv) {
    const int64_t t = blockIdx.x;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    for (int h = wave; h < H; h += 4) {
        const float *a1 = a + ((t * 2) * H + h) * dv, *a2 = a + ((t * 2 + 1) * H + h) * dv;
        float ss = 0.f;
        for (int e = lane; e < dv; e += 64) {
            const float o = a1[e] - lambda * a2[e];
            ss += o * o;
        }
        ss = wave_allreduce_sum(ss);
        const float g = gate ? rk_sigmoid(to_f(gate[t * gate_stride + h])) : 1.0f;
        const float f = mult * g / sqrtf(ss / static_cast<float>(dv) + eps);
        for (int e = lane; e < dv; e += 64) out[(t * H + h) * dv + e] = to_t<T>((a1[e] - lambda * a2[e]) * f);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void head_gate_kernel(T *y, const T *gate, int64_t gate_stride, int H, int dv) {
    const int64_t t = blockIdx.x;
    if constexpr (sizeof(T) == 2) {
        if ((dv & 7) == 0 && (reinterpret_cast<uintptr_t>(y) & 15) == 0) {      // 8 columns of one head per lane
            for (int i = threadIdx.x * 8; i < H * dv; i += 256 * 8) {
                const float g = rk_sigmoid(to_f(gate[t * gate_stride + i / dv]));
                vec8_t<T> v = load8(y + t * H * dv + i);
#pragma unroll
                for (int j = 0; j < 8; ++j) v[j] = to_t<T>(to_f(v[j]) * g);
                store8(y + t * H * dv + i, v);
            }
            return;
        }
    }
    for (int i = threadIdx.x; i < H * dv; i += 256) {
        const float g = rk_sigmoid(to_f(gate[t * gate_stride + i / dv]));
        y[t * H * dv + i] = to_t<T>(to_f(y[t * H * dv + i]) * g);
    }
}

} // namespace swl

extern "C" int swl_rope_store_kv(void *qkv, const double *freq, void *k_cache, void *v_cache, const int32_t *block_table,
                                 const int32_t *tok_seq, const int32_t *tok_pos, int64_t num_tokens, int32_t num_q_heads,
                                 int32_t num_k_heads, int32_t num_v_heads, int32_t dim, int32_t vdim, int32_t rot_dims,
                                 int64_t tok_stride, int32_t max_blocks_per_seq, int64_t block_stride, int32_t dtype,
                                 swl_stream_t stream) {
    if (num_tokens < 0 || num_q_heads <= 0 || num_k_heads < 0 || num_v_heads < 0 || dim <= 0 || vdim <= 0) return SWL_ERR_BAD_ARG;
    if (rot_dims < 0 || (rot_dims & 1) || rot_dims > dim || (dim & 1)) return SWL_ERR_BAD_ARG;
    if (tok_stride < static_cast<int64_t>(num_q_heads + num_k_heads) * dim + static_cast<int64_t>(num_v_heads) * vdim)
        return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!qkv || !tok_pos || (rot_dims > 0 && !freq)) return SWL_ERR_BAD_ARG;
    if (k_cache && (!v_cache || !block_table || !tok_seq || max_blocks_per_seq <= 0)) return SWL_ERR_BAD_ARG;
    if (num_tokens > 0x7fffffffLL || rot_dims > 2 * swl::kRkMaxPairs) return SWL_ERR_UNSUPPORTED;
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::rope_store_kv_kernel<T>), dim3(static_cast<unsigned>(num_tokens)), dim3(swl::kRkThreads), 0,
                           static_cast<hipStream_t>(stream), static_cast<T *>(qkv), freq, static_cast<T *>(k_cache),
                           static_cast<T *>(v_cache), block_table, tok_seq, tok_pos, num_q_heads, num_k_heads, num_v_heads,
                           dim, vdim, rot_dims, tok_stride, max_blocks_per_seq, block_stride);
    });
    return swl::check_launch();
}

extern "C" int swl_qk_norm_rope_store_kv(const void *rows, void *q_out, const float *q_b, const float *k_b, const float *q_w,
                                         const float *k_w, const float *q_mult, const double *freq, void *k_cache, void *v_cache,
                                         const int32_t *block_table, const int32_t *tok_seq, const int32_t *tok_pos,
                                         int64_t num_tokens, int32_t num_q_heads, int32_t num_k_heads, int32_t num_v_heads,
                                         int32_t dim, int32_t vdim, int32_t rot_dims, int32_t half, double rot_mult,
                                         int64_t tok_stride, int64_t q_out_stride, int32_t k_dim, int32_t v_dim,
                                         int32_t keys_as_values, int32_t max_blocks_per_seq, int64_t block_stride, float eps,
                                         int32_t dtype, swl_stream_t stream) {
    if (num_tokens < 0 || num_q_heads <= 0 || num_k_heads < 0 || num_v_heads < 0 || dim <= 0 || vdim <= 0) return SWL_ERR_BAD_ARG;
    if (rot_dims < 0 || (rot_dims & 1) || rot_dims > dim || (!half && (dim & 1))) return SWL_ERR_BAD_ARG;
    if (keys_as_values && (num_v_heads != 0 || vdim != dim)) return SWL_ERR_BAD_ARG;
    if (k_dim < dim || v_dim < vdim || q_out_stride < static_cast<int64_t>(num_q_heads) * k_dim) return SWL_ERR_BAD_ARG;
    if (tok_stride < static_cast<int64_t>(num_q_heads + num_k_heads) * dim + static_cast<int64_t>(num_v_heads) * vdim)
        return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!rows || !q_out || rows == q_out || !tok_pos || (rot_dims > 0 && !freq)) return SWL_ERR_BAD_ARG;
    if (k_cache && (!v_cache || !block_table || !tok_seq || max_blocks_per_seq <= 0)) return SWL_ERR_BAD_ARG;
    if (num_tokens > 0x7fffffffLL || rot_dims > 2 * swl::kRkMaxPairs) return SWL_ERR_UNSUPPORTED;
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::qk_norm_rope_store_kv_kernel<T>), dim3(static_cast<unsigned>(num_tokens)), dim3(swl::kRkThreads),
                           0, static_cast<hipStream_t>(stream), static_cast<const T *>(rows), static_cast<T *>(q_out), q_b, k_b,
                           q_w, k_w, q_mult, freq, static_cast<T *>(k_cache), static_cast<T *>(v_cache), block_table, tok_seq,
                           tok_pos, num_q_heads, num_k_heads, num_v_heads, dim, vdim, rot_dims, half, rot_mult, tok_stride,
                           q_out_stride, k_dim, v_dim, keys_as_values, max_blocks_per_seq, block_stride, eps);
    });
    return swl::check_launch();
}

extern "C" int swl_qkv_conv_rope_store_kv(
    const void *rows, int64_t tok_stride, void *q_out, int64_t q_out_stride, const float *bias, const float *conv_w, int32_t taps,
    const float *q_w, const float *k_w, const double *freq, int32_t rot_dims, int32_t half, double rot_mult, float v_mult,
    void *k_cache, void *v_cache, const int32_t *block_table, int32_t max_blocks_per_seq, int64_t block_stride, float *state,
    int64_t slot_stride, int64_t tail_off, const int32_t *tok_pos, const int32_t *tok_start, const int32_t *tok_state,
    const int32_t *tok_seq, int64_t num_tokens, int32_t num_q_heads, int32_t num_kv_heads, int32_t dim, int32_t vdim, int32_t k_dim,
    int32_t v_dim, float eps, int32_t dtype, swl_stream_t stream) {
    if (num_tokens < 0 || num_q_heads <= 0 || num_kv_heads <= 0 || dim <= 0 || vdim <= 0) return SWL_ERR_BAD_ARG;
    if (rot_dims < 0 || (rot_dims & 1) || rot_dims > dim || (!half && (dim & 1))) return SWL_ERR_BAD_ARG;
    if (k_dim < dim || v_dim < vdim || q_out_stride < static_cast<int64_t>(num_q_heads) * k_dim) return SWL_ERR_BAD_ARG;
    const int64_t C = static_cast<int64_t>(num_q_heads + num_kv_heads) * dim + static_cast<int64_t>(num_kv_heads) * vdim;
    if (tok_stride < C || (conv_w && taps < 1) || (!q_w) != (!k_w)) return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!rows || !q_out || rows == q_out || !tok_pos || !tok_seq || (rot_dims > 0 && !freq)) return SWL_ERR_BAD_ARG;
    if (conv_w && (!tok_start || (taps > 1 && (!state || !tok_state)))) return SWL_ERR_BAD_ARG;
    if (k_cache && (!v_cache || !block_table || max_blocks_per_seq <= 0)) return SWL_ERR_BAD_ARG;
    const size_t lds = (static_cast<size_t>(C) + num_q_heads + num_kv_heads) * sizeof(float);
    if (num_tokens > 0x7fffffffLL || rot_dims > 2 * swl::kRkMaxPairs || lds > 60 * 1024) return SWL_ERR_UNSUPPORTED;
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::qkv_conv_rope_store_kv_kernel<T>), dim3(static_cast<unsigned>(num_tokens)), dim3(swl::kRkThreads),
                           lds, static_cast<hipStream_t>(stream), static_cast<const T *>(rows), tok_stride, static_cast<T *>(q_out),
                           q_out_stride, bias, conv_w, taps, q_w, k_w, freq, rot_dims, half, rot_mult, v_mult,
                           static_cast<T *>(k_cache), static_cast<T *>(v_cache), block_table, max_blocks_per_seq, block_stride,
                           state, slot_stride, tail_off, tok_pos, tok_start, tok_state, tok_seq, num_tokens, num_q_heads,
                           num_kv_heads, dim, vdim, k_dim, v_dim, eps);
    });
    return swl::check_launch();
}

extern "C" int swl_latent_rope_store_kv(const void *proj, void *qa, const double *freq, const float *c_norm, void *k_cache,
                                        void *v_cache, const int32_t *block_table, const int32_t *tok_seq,
                                        const int32_t *tok_pos, int64_t num_tokens, int32_t num_heads, int32_t dim,
                                        int32_t rot_dim, int32_t kv_rank, int64_t proj_stride, int64_t dkv_col,
                                        int64_t qa_stride, int32_t max_blocks_per_seq, int64_t block_stride, float eps,
                                        int32_t half, double rot_mult, int32_t k_dim, int32_t v_dim, int32_t dtype,
                                        swl_stream_t stream) {
    if (num_tokens < 0 || num_heads <= 0 || dim <= 0 || rot_dim <= 0 || (rot_dim & 1) || kv_rank <= 0) return SWL_ERR_BAD_ARG;
    if (k_dim < kv_rank + rot_dim || v_dim < kv_rank) return SWL_ERR_BAD_ARG;
    if (proj_stride < static_cast<int64_t>(num_heads) * (dim + rot_dim) || qa_stride < static_cast<int64_t>(num_heads) * k_dim)
        return SWL_ERR_BAD_ARG;
    if (dkv_col >= 0 && dkv_col + kv_rank + rot_dim > proj_stride) return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!proj || !qa || !freq || !tok_pos) return SWL_ERR_BAD_ARG;
    if (dkv_col >= 0 && k_cache && (!v_cache || !c_norm || !block_table || !tok_seq || max_blocks_per_seq <= 0))
        return SWL_ERR_BAD_ARG;
    if (num_tokens > 0x7fffffffLL || rot_dim > 2 * swl::kRkMaxPairs) return SWL_ERR_UNSUPPORTED;
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::latent_rope_store_kv_kernel<T>), dim3(static_cast<unsigned>(num_tokens)),
                           dim3(swl::kRkThreads), 0, static_cast<hipStream_t>(stream), static_cast<const T *>(proj),
                           static_cast<T *>(qa), freq, c_norm, static_cast<T *>(k_cache), static_cast<T *>(v_cache),
                           block_table, tok_seq, tok_pos, num_heads, dim, rot_dim, kv_rank, proj_stride, dkv_col, qa_stride,
                           max_blocks_per_seq, block_stride, eps, half, rot_mult, k_dim, v_dim);
    });
    return swl::check_launch();
}

extern "C" int swl_diff_head_combine(void *out, const float *maps, const void *gate, int64_t gate_stride, float lambda,
                                     float mult, float eps, int64_t num_tokens, int32_t num_heads, int32_t vdim,
                                     int32_t dtype, swl_stream_t stream) {
    if (num_tokens < 0 || num_heads <= 0 || vdim <= 0 || (gate && gate_stride < num_heads)) return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!out || !maps) return SWL_ERR_BAD_ARG;
    if (num_tokens > 0x7fffffffLL) return SWL_ERR_UNSUPPORTED;
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::diff_head_combine_kernel<T>), dim3(static_cast<unsigned>(num_tokens)), dim3(256), 0,
                           static_cast<hipStream_t>(stream), static_cast<T *>(out), maps, static_cast<const T *>(gate),
                           gate_stride, lambda, mult, eps, num_heads, vdim);
    });
    return swl::check_launch();
}

extern "C" int swl_head_gate(void *y, const void *gate, int64_t gate_stride, int64_t num_tokens, int32_t num_heads,
                             int32_t vdim, int32_t dtype, swl_stream_t stream) {
    if (num_tokens < 0 || num_heads <= 0 || vdim <= 0 || gate_stride < num_heads) return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!y || !gate) return SWL_ERR_BAD_ARG;
    if (num_tokens > 0x7fffffffLL) return SWL_ERR_UNSUPPORTED;
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::head_gate_kernel<T>), dim3(static_cast<unsigned>(num_tokens)), dim3(256), 0,
                           static_cast<hipStream_t>(stream), static_cast<T *>(y), static_cast<const T *>(gate), gate_stride,
                           num_heads, vdim);
    });
    return swl::check_launch();
}
