// linear_scan.hip — recurrences that are linear in a matrix state, with a decay per key channel (or one per head), for any mixture
// of prompt portions and decoded tokens. Per head, with S [dim, vdim] fp32 in the sequence's state slot:
//     plain:   S <- diag(a) S + k v^T;   o = S^T q                       (gated linear attention; state-space duality: a scalar a)
//     bonus u: o = (S + diag(u) k v^T)^T q;   S <- diag(a) S + k v^T      (time mixing: the decay acts after the read-out)
//   optionally k times a factor per (token, head), and o + D v with D per head.
//
// Prompts run in tiles of 16 tokens (the plan's tiles: runs of up to 16 consecutive tokens of one portion). Inside a tile the
// recurrence unrolls into products whose decays are all products of factors in [0, 1], so nothing is divided and nothing overflows,
// however strong the decay:
//     o_t = (q_t * A_(0..t])^T S0 + sum_(s <= t) M[t][s] v_s,     M[t][s] = sum_i q_t[i] k_s[i] prod_(s < m <= t) a_m[i]
//     S   = diag(A_(0..n]) S0 + sum_s (k_s * A_(s..n]) v_s^T
//   (with the bonus the products end at t - 1 and M[t][t] = sum_i q_t[i] u[i] k_t[i]).
//   swl_linear_chunks: one workgroup per (tile, head), all tiles at once: decayed queries and keys, the tile's total decay and M.
//                      Running products over the tokens; nothing here depends on the state.
//   swl_linear_scan:   one workgroup (4 waves) per (portion, head, 16 state columns): walks the portion's tiles. The state lives in
//                      the accumulators of the fp32 matrix core (16x16x4: exact fp32 operands): the rows are shared out over the
//                      waves, and an accumulator tile is, register by register, the B operand of the read-out when the reduction
//                      index is taken in the order 4 (lane / 16) + r — so the state never moves. The waves' partial outputs meet
//                      in LDS, one barrier per tile; the next tile's operands are requested a tile ahead.
//   swl_linear_step:   steps whose portions are single tokens (decode): one workgroup per (sequence, head) streams the state once
//                      and finishes the head — read-out, RMS norm over the head, weight, gate — in the same launch.
// Everything after the loads of q, k, v is fp32.
#include "swl_common.h"

namespace swl {

constexpr int kLsTile = 16;
constexpr int kLsThreads = 256;
constexpr int kLsWaves = kLsThreads / 64;
constexpr int kLsMaxDim = 320;          // padded key channels: 3 * 16 * 320 floats of LDS

__device__ __forceinline__ float ls_silu(float z) { return z / (1.0f + expf(-z)); }

template <typename T, bool BONUS>
__global__ __launch_bounds__(kLsThreads) void linear_chunks_kernel(
    float *qd, float *kd, float *total, float *intra, const T *q, int64_t q_stride, const T *k, int64_t k_stride, const float *decay,
    int64_t decay_stride, int per_channel, const float *k_scale, const float *bonus, float q_scale, const int32_t *tile_row0,
    const int32_t *tile_cnt, int H, int rep, int d, int dp) {
    extern __shared__ float lds[];
    float *qs = lds, *ks = qs + kLsTile * dp, *as = ks + kLsTile * dp;      // [16][dp] each
    const int tile = blockIdx.x, h = blockIdx.y;
    const int row0 = tile_row0[tile], cnt = tile_cnt[tile];
    const int64_t at = static_cast<int64_t>(tile) * H + h;
    const int qk0 = (h / rep) * d;
    // tokens beyond the tile's and channels beyond the head: q = k = 0, decay 1
    for (int i = threadIdx.x; i < kLsTile * dp; i += kLsThreads) {
        const int t = i / dp, e = i - t * dp;
        float qv = 0.f, kv = 0.f, av = 1.f;
        if (t < cnt && e < d) {
            const int64_t row = row0 + t;
            qv = to_f(q[row * q_stride + qk0 + e]) * q_scale;
            kv = to_f(k[row * k_stride + qk0 + e]);
            if (k_scale) kv *= k_scale[row * H + h];
            av = decay[row * decay_stride + (per_channel ? h * d + e : h)];
        }
        qs[i] = qv;
        ks[i] = kv;
        as[i] = av;
    }
    __syncthreads();
    for (int e = threadIdx.x; e < dp; e += kLsThreads) {
        float p = 1.f;
        float *qo = qd + at * kLsTile * dp + e;
#pragma unroll
        for (int t = 0; t < kLsTile; ++t) {
            const float a = as[t * dp + e];
            if constexpr (BONUS) {
                qo[t * dp] = qs[t * dp + e] * p;
                p *= a;
            } else {
                p *= a;
                qo[t * dp] = qs[t * dp + e] * p;
            }
        }
        total[at * dp + e] = p;
        float kk[kLsTile];
        p = 1.f;
#pragma unroll
        for (int t = kLsTile - 1; t >= 0; --t) {
            kk[t] = ks[t * dp + e] * p;
            p *= as[t * dp + e];
        }
        float *ko = kd + (at * dp + e) * kLsTile;
#pragma unroll
        for (int t = 0; t < kLsTile; t += 4) *reinterpret_cast<float4_t *>(ko + t) = float4_t{kk[t], kk[t + 1], kk[t + 2], kk[t + 3]};
    }
    // M: thread (s, g) takes key token s and the channels g, g + 16, ...; sixteen neighbouring lanes share an s
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int s = threadIdx.x >> 4, g = threadIdx.x & 15;
    float acc[kLsTile];
#pragma unroll
    for (int t = 0; t < kLsTile; ++t) acc[t] = 0.f;
    for (int e = g; e < d; e += 16) {
        float p = ks[s * dp + e];
        float diag = 0.f;
        if constexpr (BONUS) diag = p * bonus[h * d + e];
#pragma unroll
        for (int t = 0; t < kLsTile; ++t) {
            if (t >= 4 * wave) {        // (wave-uniform: the wave's key tokens are 4 wave .. 4 wave + 3)
                const float a = as[t * dp + e], qv = qs[t * dp + e];
                if constexpr (BONUS) {
                    acc[t] = fmaf(qv, t > s ? p : t == s ? diag : 0.f, acc[t]);
                    if (t > s) p *= a;
                } else {
                    if (t > s) p *= a;
                    acc[t] = fmaf(qv, t >= s ? p : 0.f, acc[t]);
                }
            }
        }
    }
    float mine = 0.f;
#pragma unroll
    for (int t = 0; t < kLsTile; ++t) {
        const float v = group_allreduce_sum<16>(acc[t]);
        if (g == t) mine = v;
    }
    intra[at * 256 + g * kLsTile + s] = mine;       // [t][s]
}

__device__ __forceinline__ float4_t mfma_f32_16x16x4(float a, float b, float4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// What a wave needs of one tile. Loaded without predicates (addresses are clamped, what does not count is masked at its use): a
// predicated load would be waited for on the spot, and the point is to have a tile's loads in flight while others are computed.
template <typename T, int TW>
struct LsOperands {
    float4_t q[TW], k[TW], a[TW];
    float m;
    T v[4];
};

// TW: 16-row state tiles per wave; AHEAD: tiles requested ahead of the one being computed
template <typename T, int TW, int AHEAD>
__global__ __launch_bounds__(kLsThreads) void linear_scan_kernel(
    float *o, int64_t o_stride, const float *qd, const float *kd, const float *total, const float *intra, const T *v,
    int64_t v_stride, const float *dskip, float *state, int64_t slot_stride, int64_t s_off, const int32_t *seq_row0,
    const int32_t *seq_cnt, const int32_t *seq_tile0, const int32_t *tok_pos, const int32_t *tok_state, int H, int d, int dp,
    int dv) {
    __shared__ float red[2][kLsWaves][256];
    const int seq = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * 16;
    const int row0 = seq_row0[seq], cnt = seq_cnt[seq], tile0 = seq_tile0[seq];
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int li = lane & 15, lq = lane >> 4;
    const int col = col0 + li;
    const bool okc = col < dv;
    const int ntiles = dp >> 4;
    float *S = state + static_cast<int64_t>(tok_state[row0] >> 1) * slot_stride + s_off + static_cast<int64_t>(h) * d * dv;
    const bool fresh = tok_pos[row0] == 0;      // a sequence starts from the zero state whatever the slot held
    float4_t st[TW];        // st[j][r] = S[16 (wave TW + j) + 4 lq + r][col]
#pragma unroll
    for (int j = 0; j < TW; ++j) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * (wave * TW + j) + 4 * lq + r;
            st[j][r] = (!fresh && okc && row < d) ? S[static_cast<int64_t>(row) * dv + col] : 0.f;
        }
    }
    const float dh = dskip ? dskip[h] : 0.f;
    const int nt = (cnt + kLsTile - 1) / kLsTile;
    const T *vcol = v + static_cast<int64_t>(row0) * v_stride + static_cast<int64_t>(h) * dv + (okc ? col : dv - 1);
    auto load = [&](int i, LsOperands<T, TW> &f) {
        i = min(i, nt - 1);
        const int64_t at = static_cast<int64_t>(tile0 + i) * H + h;
#pragma unroll
        for (int j = 0; j < TW; ++j) {
            const int tl = min(wave * TW + j, ntiles - 1);
            f.q[j] = *reinterpret_cast<const float4_t *>(qd + (at * kLsTile + li) * dp + 16 * tl + 4 * lq);
            f.k[j] = *reinterpret_cast<const float4_t *>(kd + (at * dp + 16 * tl + li) * kLsTile + 4 * lq);
            f.a[j] = *reinterpret_cast<const float4_t *>(total + at * dp + 16 * tl + 4 * lq);
        }
        f.m = intra[at * 256 + li * kLsTile + 4 * lq + wave];
#pragma unroll
        for (int r = 0; r < 4; ++r) f.v[r] = vcol[static_cast<int64_t>(min(i * kLsTile + 4 * lq + r, cnt - 1)) * v_stride];
    };
    auto compute = [&](int i, const LsOperands<T, TW> &f) {
        float vv[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) vv[r] = (i * kLsTile + 4 * lq + r < cnt && okc) ? to_f(f.v[r]) : 0.f;
        // this wave's share of the outputs: its state rows, and the in-tile keys 4 lq + wave
        float4_t part[TW + 1];
        part[TW] = mfma_f32_16x16x4(f.m, wave == 0 ? vv[0] : wave == 1 ? vv[1] : wave == 2 ? vv[2] : vv[3],
                                    float4_t{0.f, 0.f, 0.f, 0.f});
#pragma unroll
        for (int j = 0; j < TW; ++j) part[j] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
#pragma unroll
            for (int j = 0; j < TW; ++j) part[j] = mfma_f32_16x16x4(f.q[j][r], st[j][r], part[j]);
        }
#pragma unroll
        for (int j = 0; j < TW; ++j) {
            mfma_results_ready<8>(st[j]);
            st[j] *= f.a[j];
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
#pragma unroll
            for (int j = 0; j < TW; ++j) st[j] = mfma_f32_16x16x4(f.k[j][r], vv[r], st[j]);
        }
        float4_t out = part[TW];
        mfma_results_ready<8>(out);
#pragma unroll
        for (int j = 0; j < TW; ++j) {
            mfma_results_ready<8>(part[j]);
            if (wave * TW + j < ntiles) out += part[j];     // (wave-uniform; a row tile beyond the state repeats the last one)
        }
        if (dskip && wave == 0) {       // (v of this lane: token 4 lq + r, column li — the layout of the result)
#pragma unroll
            for (int r = 0; r < 4; ++r) out[r] = fmaf(dh, vv[r], out[r]);
        }
        float *rb = &red[i & 1][0][0];
        *reinterpret_cast<float4_t *>(rb + wave * 256 + lane * 4) = out;
        __syncthreads();        // (two buffers: the next tile's partials go to the other one)
        const int t = threadIdx.x >> 4, c = threadIdx.x & 15;
        const int from = ((t >> 2) * 16 + c) * 4 + (t & 3);
        float sum = 0.f;
#pragma unroll
        for (int w = 0; w < kLsWaves; ++w) sum += rb[w * 256 + from];
        const int tok = i * kLsTile + t;
        if (tok < cnt && col0 + c < dv) o[(row0 + tok) * o_stride + static_cast<int64_t>(h) * dv + col0 + c] = sum;
    };
    LsOperands<T, TW> f[AHEAD + 1];
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) load(a, f[a]);
    int i = 0;
    for (; i + AHEAD < nt; i += AHEAD + 1) {
#pragma unroll
        for (int a = 0; a <= AHEAD; ++a) {
            load(i + a + AHEAD, f[(a + AHEAD) % (AHEAD + 1)]);
            compute(i + a, f[a]);
        }
    }
#pragma unroll
    for (int a = 0; a < AHEAD; ++a)
        if (i + a < nt) compute(i + a, f[a]);       // (uniform)
#pragma unroll
    for (int j = 0; j < TW; ++j) {
        float4_t s = st[j];
        mfma_results_ready<8>(s);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * (wave * TW + j) + 4 * lq + r;
            if (okc && row < d) S[static_cast<int64_t>(row) * dv + col] = s[r];
        }
    }
}

// One token per sequence. Thread (rg, cg) owns columns V cg .. V cg + V - 1 and the state rows rg, rg + R, ...
constexpr int kLsBatch = 8;     // state rows in flight per thread

template <typename T, int V, bool BONUS>
__global__ __launch_bounds__(kLsThreads) void linear_step_kernel(
    T *out, int64_t out_stride, float *y, int64_t y_stride, const T *q, int64_t q_stride, const T *k, int64_t k_stride, const T *v,
    int64_t v_stride, const float *decay, int64_t decay_stride, int per_channel, const float *k_scale, const float *bonus,
    float q_scale, const float *dskip, float *state, int64_t slot_stride, int64_t s_off, const int32_t *seq_row0,
    const int32_t *tok_pos, const int32_t *tok_state, int H, int rep, int d, int dv, const float *norm_w, int norm_head_stride,
    const T *gate, int64_t gate_stride, float eps, float mult) {
    extern __shared__ float lds[];
    const int ncg = (dv + V - 1) / V, R = kLsThreads / ncg;
    float *qs = lds, *ks = qs + d, *as = ks + d, *us = as + d, *os = us + d;     // [d] x 4, then [R][ncg * V]
    __shared__ float red[kLsWaves];
    const int seq = blockIdx.x, h = blockIdx.y;
    const int64_t row = seq_row0[seq];
    const int cg = threadIdx.x % ncg, rg = threadIdx.x / ncg;
    const bool live = rg < R;
    float *S = state + static_cast<int64_t>(tok_state[row] >> 1) * slot_stride + s_off + static_cast<int64_t>(h) * d * dv;
    const bool fresh = tok_pos[row] == 0;
    // the first rows of the state are requested before anything else
    float sv[kLsBatch][V];
    auto fetch = [&](int b) {
#pragma unroll
        for (int j = 0; j < kLsBatch; ++j) {
            const int e = b + rg + j * R;
#pragma unroll
            for (int c = 0; c < V; ++c) sv[j][c] = 0.f;
            if (live && !fresh && e < d) {
                const float *p = S + static_cast<int64_t>(e) * dv + cg * V;
                if constexpr (V == 4) {
                    const float4_t x = *reinterpret_cast<const float4_t *>(p);
#pragma unroll
                    for (int c = 0; c < 4; ++c) sv[j][c] = x[c];
                } else {
                    sv[j][0] = p[0];
                }
            }
        }
    };
    fetch(0);
    for (int e = threadIdx.x; e < d; e += kLsThreads) {
        qs[e] = to_f(q[row * q_stride + static_cast<int64_t>(h / rep) * d + e]) * q_scale;
        const float kv = to_f(k[row * k_stride + static_cast<int64_t>(h / rep) * d + e]);
        ks[e] = k_scale ? kv * k_scale[row * H + h] : kv;
        as[e] = decay[row * decay_stride + (per_channel ? h * d + e : h)];
        if constexpr (BONUS) us[e] = bonus[h * d + e];
    }
    float vv[V], acc[V];
#pragma unroll
    for (int c = 0; c < V; ++c) {
        vv[c] = live ? to_f(v[row * v_stride + static_cast<int64_t>(h) * dv + cg * V + c]) : 0.f;
        acc[c] = 0.f;
    }
    __syncthreads();
    for (int b = 0; b < d; b += kLsBatch * R) {
        if (b) fetch(b);
#pragma unroll
        for (int j = 0; j < kLsBatch; ++j) {
            const int e = b + rg + j * R;
            if (live && e < d) {
                const float qe = qs[e], ke = ks[e], ae = as[e];
                float x[V];
#pragma unroll
                for (int c = 0; c < V; ++c) {
                    const float kv = ke * vv[c];
                    if constexpr (BONUS) {
                        acc[c] = fmaf(qe, fmaf(us[e], kv, sv[j][c]), acc[c]);
                        x[c] = fmaf(ae, sv[j][c], kv);
                    } else {
                        x[c] = fmaf(ae, sv[j][c], kv);
                        acc[c] = fmaf(qe, x[c], acc[c]);
                    }
                }
                float *p = S + static_cast<int64_t>(e) * dv + cg * V;
                if constexpr (V == 4) *reinterpret_cast<float4_t *>(p) = float4_t{x[0], x[1], x[2], x[3]};
                else p[0] = x[0];
            }
        }
    }
    const int cols = ncg * V;       // (V divides dv: cols == dv)
    if (live) {
#pragma unroll
        for (int c = 0; c < V; ++c) os[rg * cols + cg * V + c] = acc[c];
    }
    __syncthreads();
    float ss = 0.f;
    for (int c = threadIdx.x; c < dv; c += kLsThreads) {
        float a = 0.f;
        for (int r = 0; r < R; ++r) a += os[r * cols + c];
        if (dskip) a = fmaf(dskip[h], to_f(v[row * v_stride + static_cast<int64_t>(h) * dv + c]), a);
        if (y) y[row * y_stride + static_cast<int64_t>(h) * dv + c] = a;
        os[c] = a;          // (column c is read and written by this thread only)
        ss += a * a;
    }
    if (!out) return;
    ss = wave_allreduce_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < kLsWaves; ++w) ss += red[w];
    const float r = mult / sqrtf(ss / static_cast<float>(dv) + eps);
    for (int c = threadIdx.x; c < dv; c += kLsThreads) {
        const int64_t hc = static_cast<int64_t>(h) * dv + c;
        out[row * out_stride + hc] = to_t<T>(os[c] * r * norm_w[static_cast<int64_t>(h) * norm_head_stride + c] *
                                             ls_silu(to_f(gate[row * gate_stride + hc])));
    }
}

} // namespace swl

extern "C" int swl_linear_chunks(float *qd, float *kd, float *total, float *intra, const void *q, int64_t q_stride, const void *k,
                                 int64_t k_stride, const float *decay, int64_t decay_stride, int32_t per_channel,
                                 const float *k_scale, const float *bonus, float q_scale, const int32_t *tile_row0,
                                 const int32_t *tile_cnt, int32_t num_tiles, int32_t num_heads, int32_t num_qk_heads, int32_t dim,
                                 int32_t dtype, swl_stream_t stream) {
    if (num_tiles < 0 || num_heads <= 0 || num_qk_heads <= 0 || num_heads % num_qk_heads || dim <= 0) return SWL_ERR_BAD_ARG;
    const int64_t width = static_cast<int64_t>(num_qk_heads) * dim;
    if (q_stride < width || k_stride < width || decay_stride < (per_channel ? static_cast<int64_t>(num_heads) * dim : num_heads))
        return SWL_ERR_BAD_ARG;
    if (num_tiles == 0) return SWL_OK;
    if (!qd || !kd || !total || !intra || !q || !k || !decay || !tile_row0 || !tile_cnt || !swl::aligned16(kd))
        return SWL_ERR_BAD_ARG;
    const int dp = (dim + 15) / 16 * 16;
    if (dp > swl::kLsMaxDim || num_heads > 65535) return SWL_ERR_UNSUPPORTED;
    const size_t lds = 3ull * swl::kLsTile * dp * sizeof(float);
    const dim3 grid(static_cast<unsigned>(num_tiles), static_cast<unsigned>(num_heads));
    SWL_DISPATCH_DTYPE3(dtype, T, {
        auto kernel = bonus ? swl::linear_chunks_kernel<T, true> : swl::linear_chunks_kernel<T, false>;
        hipLaunchKernelGGL(kernel, grid, dim3(swl::kLsThreads), lds, static_cast<hipStream_t>(stream), qd, kd, total, intra,
                           static_cast<const T *>(q), q_stride, static_cast<const T *>(k), k_stride, decay, decay_stride,
                           per_channel, k_scale, bonus, q_scale, tile_row0, tile_cnt, num_heads, num_heads / num_qk_heads, dim, dp);
    });
    return swl::check_launch();
}

extern "C" int swl_linear_scan(float *o, int64_t o_stride, const float *qd, const float *kd, const float *total, const float *intra,
                               const void *v, int64_t v_stride, const float *dskip, float *state, int64_t slot_stride,
                               int64_t s_off, const int32_t *seq_row0, const int32_t *seq_cnt, const int32_t *seq_tile0,
                               const int32_t *tok_pos, const int32_t *tok_state, int32_t num_seqs, int32_t num_heads, int32_t dim,
                               int32_t vdim, int32_t dtype, swl_stream_t stream) {
    if (num_seqs < 0 || num_heads <= 0 || dim <= 0 || vdim <= 0) return SWL_ERR_BAD_ARG;
    const int64_t width = static_cast<int64_t>(num_heads) * vdim;
    if (o_stride < width || v_stride < width) return SWL_ERR_BAD_ARG;
    if (num_seqs == 0) return SWL_OK;
    if (!o || !qd || !kd || !total || !intra || !v || !state || !seq_row0 || !seq_cnt || !seq_tile0 || !tok_pos || !tok_state)
        return SWL_ERR_BAD_ARG;
    if (!swl::aligned16(qd) || !swl::aligned16(kd) || !swl::aligned16(total)) return SWL_ERR_BAD_ARG;
    const int dp = (dim + 15) / 16 * 16, shares = (vdim + 15) / 16;
    if (dp > swl::kLsMaxDim || num_heads > 65535 || shares > 65535) return SWL_ERR_UNSUPPORTED;
    const int tw = (dp / 16 + swl::kLsWaves - 1) / swl::kLsWaves;       // 1 .. 5
    const dim3 grid(static_cast<unsigned>(num_seqs), static_cast<unsigned>(num_heads), static_cast<unsigned>(shares));
#define SWL_LS(N)                                                                                                             \
    case N:                                                                                                                   \
        hipLaunchKernelGGL((swl::linear_scan_kernel<T, N, (N <= 2 ? 2 : 1)>), grid, dim3(swl::kLsThreads), 0,                 \
                           static_cast<hipStream_t>(stream), o, o_stride, qd, kd, total, intra,                         \
                           static_cast<const T *>(v), v_stride, dskip, state, slot_stride, s_off,                             \
                           seq_row0, seq_cnt, seq_tile0, tok_pos, tok_state, num_heads, dim, dp, vdim);                       \
        break
    SWL_DISPATCH_DTYPE3(dtype, T, {
        switch (tw) {
            SWL_LS(1);
            SWL_LS(2);
            SWL_LS(3);
            SWL_LS(4);
            SWL_LS(5);
        default: return SWL_ERR_UNSUPPORTED;
        }
    });
#undef SWL_LS
    return swl::check_launch();
}

extern "C" int swl_linear_step(void *out, int64_t out_stride, float *y, int64_t y_stride, const void *q, int64_t q_stride,
                               const void *k, int64_t k_stride, const void *v, int64_t v_stride, const float *decay,
                               int64_t decay_stride, int32_t per_channel, const float *k_scale, const float *bonus, float q_scale,
                               const float *dskip, float *state, int64_t slot_stride, int64_t s_off, const int32_t *seq_row0,
                               const int32_t *tok_pos, const int32_t *tok_state, int32_t num_seqs, int32_t num_heads,
                               int32_t num_qk_heads, int32_t dim, int32_t vdim, const float *norm_w, int32_t norm_head_stride,
                               const void *gate, int64_t gate_stride, float eps, float mult, int32_t dtype, swl_stream_t stream) {
    if (num_seqs < 0 || num_heads <= 0 || num_qk_heads <= 0 || num_heads % num_qk_heads || dim <= 0 || vdim <= 0)
        return SWL_ERR_BAD_ARG;
    const int64_t wq = static_cast<int64_t>(num_qk_heads) * dim, wv = static_cast<int64_t>(num_heads) * vdim;
    if (q_stride < wq || k_stride < wq || v_stride < wv) return SWL_ERR_BAD_ARG;
    if (decay_stride < (per_channel ? static_cast<int64_t>(num_heads) * dim : num_heads)) return SWL_ERR_BAD_ARG;
    if (num_seqs == 0) return SWL_OK;
    if ((!out && !y) || !q || !k || !v || !decay || !state || !seq_row0 || !tok_pos || !tok_state) return SWL_ERR_BAD_ARG;
    if (out && (!norm_w || !gate || out_stride < wv || gate_stride < wv)) return SWL_ERR_BAD_ARG;
    if (y && y_stride < wv) return SWL_ERR_BAD_ARG;
    const bool quads = vdim % 4 == 0 && swl::aligned16(state) && slot_stride % 4 == 0 && s_off % 4 == 0;
    const int ncg = quads ? vdim / 4 : vdim;
    if (ncg > swl::kLsThreads || num_heads > 65535) return SWL_ERR_UNSUPPORTED;
    const int R = swl::kLsThreads / ncg;
    const size_t lds = (4ull * dim + static_cast<size_t>(R) * vdim) * sizeof(float);
    if (lds > 60 * 1024) return SWL_ERR_UNSUPPORTED;
    const dim3 grid(static_cast<unsigned>(num_seqs), static_cast<unsigned>(num_heads));
    SWL_DISPATCH_DTYPE3(dtype, T, {
        auto kernel = quads ? (bonus ? swl::linear_step_kernel<T, 4, true> : swl::linear_step_kernel<T, 4, false>)
                            : (bonus ? swl::linear_step_kernel<T, 1, true> : swl::linear_step_kernel<T, 1, false>);
        hipLaunchKernelGGL(kernel, grid, dim3(swl::kLsThreads), lds, static_cast<hipStream_t>(stream), static_cast<T *>(out),
                           out_stride, y, y_stride, static_cast<const T *>(q), q_stride, static_cast<const T *>(k), k_stride,
                           static_cast<const T *>(v), v_stride, decay, decay_stride, per_channel, k_scale, bonus, q_scale, dskip,
                           state, slot_stride, s_off, seq_row0, tok_pos, tok_state, num_heads, num_heads / num_qk_heads, dim, vdim,
                           norm_w, norm_head_stride, static_cast<const T *>(gate), gate_stride, eps, mult);
    });
    return swl::check_launch();
}
