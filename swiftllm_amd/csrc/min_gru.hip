// min_gru.hip — minGRU: an element-wise gated recurrence whose gates read only the current token, as a recurrent mixer with
// per-sequence state slots, for any mixture of prompt portions and decoded tokens.
//
// Per channel, fp32:  a = sigmoid(z + z_b),  c = g(u + u_b) with g(v) = v + 1/2 for v >= 0 and sigmoid(v) below,
//                     S <- (1 - a) S + a c,  out = S * silu(gate)
// from projection rows [z | u | gate] of `width` columns each.
//
// The recurrence is linear in S, so a portion longer than one chunk (a run of tokens of one sequence) is evaluated in parallel
// over its chunks:
//   swl_min_gru_chunks:  every chunk's composed step S -> P S + Q (P = product of 1 - a, Q = the chunk walked from zero),
//   swl_min_gru_carry:   one thread per (sequence, channel) walks the chunks: each chunk's start state, the slot's new state,
//   swl_min_gru_apply:   every chunk is walked from its start state and the gated outputs are written.
// When no portion of a step is longer than a chunk (decode steps among them), swl_min_gru_apply alone does the step: it reads
// and writes the slots itself.
#include "swl_common.h"

namespace swl {

constexpr int kMgThreads = 256;
constexpr int kMgAhead = 8;         // tokens whose loads are in flight together

__device__ __forceinline__ float mg_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }
__device__ __forceinline__ float mg_candidate(float v) { return v >= 0.f ? v + 0.5f : mg_sigmoid(v); }

template <typename T, int V>
struct MgVec {
    typedef T type __attribute__((ext_vector_type(V)));
};
template <typename T>
struct MgVec<T, 1> {
    typedef T type;
};
template <typename T, int V>
__device__ __forceinline__ void mg_load(float *dst, const T *p) {
    if constexpr (V == 1) {
        dst[0] = to_f(p[0]);
    } else {
        const typename MgVec<T, V>::type v = *reinterpret_cast<const typename MgVec<T, V>::type *>(p);
#pragma unroll
        for (int j = 0; j < V; ++j) dst[j] = to_f(v[j]);
    }
}

// part [chunks][2][width]: P then Q of every chunk
template <typename T, int V>
__global__ __launch_bounds__(kMgThreads) void min_gru_chunks_kernel(float *part, const T *proj, int64_t proj_stride,
                                                                    const float *z_b, const float *u_b,
                                                                    const int32_t *chunk_row0, const int32_t *chunk_cnt,
                                                                    int width) {
    const int64_t chunk = blockIdx.x;
    const int c = (blockIdx.y * kMgThreads + threadIdx.x) * V;
    if (c >= width) return;
    const int row0 = chunk_row0[chunk], cnt = chunk_cnt[chunk];
    const T *src = proj + static_cast<int64_t>(row0) * proj_stride + c;
    float zb[V], ub[V], P[V], Q[V];
#pragma unroll
    for (int j = 0; j < V; ++j) {
        zb[j] = z_b ? z_b[c + j] : 0.f;
        ub[j] = u_b ? u_b[c + j] : 0.f;
        P[j] = 1.f;
        Q[j] = 0.f;
    }
    for (int t0 = 0; t0 < cnt; t0 += kMgAhead) {
        float z[kMgAhead][V], u[kMgAhead][V];
#pragma unroll
        for (int k = 0; k < kMgAhead; ++k) {        // (rows past the end re-read the last one: never used)
            const T *p = src + static_cast<int64_t>(min(t0 + k, cnt - 1)) * proj_stride;
            mg_load<T, V>(z[k], p);
            mg_load<T, V>(u[k], p + width);
        }
#pragma unroll
        for (int k = 0; k < kMgAhead; ++k) {
            if (t0 + k < cnt) {
#pragma unroll
                for (int j = 0; j < V; ++j) {
                    const float a = mg_sigmoid(z[k][j] + zb[j]);
                    P[j] *= 1.f - a;
                    Q[j] = fmaf(1.f - a, Q[j], a * mg_candidate(u[k][j] + ub[j]));
                }
            }
        }
    }
    float *dst = part + chunk * 2 * width + c;
#pragma unroll
    for (int j = 0; j < V; ++j) {
        dst[j] = P[j];
        dst[width + j] = Q[j];
    }
}

// Leaves every chunk's start state where its P was.
__global__ __launch_bounds__(kMgThreads) void min_gru_carry_kernel(float *part, float *state, int64_t slot_stride,
                                                                   int64_t s_off, const int32_t *seq_row0,
                                                                   const int32_t *seq_cnt, const int32_t *seq_chunk0,
                                                                   const int32_t *tok_pos, const int32_t *tok_state,
                                                                   int chunk_tokens, int width) {
    const int seq = blockIdx.x;
    const int c = blockIdx.y * kMgThreads + threadIdx.x;
    if (c >= width) return;
    const int row0 = seq_row0[seq], n = (seq_cnt[seq] + chunk_tokens - 1) / chunk_tokens;
    float *slot = state + static_cast<int64_t>(tok_state[row0] >> 1) * slot_stride + s_off + c;
    float S = tok_pos[row0] == 0 ? 0.f : *slot;     // a sequence starts from the zero state whatever the slot held
    float *p = part + static_cast<int64_t>(seq_chunk0[seq]) * 2 * width + c;
    for (int k0 = 0; k0 < n; k0 += kMgAhead) {
        float P[kMgAhead], Q[kMgAhead];
#pragma unroll
        for (int k = 0; k < kMgAhead; ++k) {
            const int64_t at = static_cast<int64_t>(min(k0 + k, n - 1)) * 2 * width;
            P[k] = p[at];
            Q[k] = p[at + width];
        }
#pragma unroll
        for (int k = 0; k < kMgAhead; ++k) {
            if (k0 + k < n) {
                p[static_cast<int64_t>(k0 + k) * 2 * width] = S;
                S = fmaf(P[k], S, Q[k]);
            }
        }
    }
    *slot = S;
}

// start (may be NULL: the slots, which then also receive the end states) [chunks][2][width]: the chunks' start states
template <typename T, int V>
__global__ __launch_bounds__(kMgThreads) void min_gru_apply_kernel(T *out, const T *proj, int64_t proj_stride,
                                                                   const float *z_b, const float *u_b, const float *start,
                                                                   float *state, int64_t slot_stride, int64_t s_off,
                                                                   const int32_t *chunk_row0, const int32_t *chunk_cnt,
                                                                   const int32_t *tok_pos, const int32_t *tok_state,
                                                                   int width) {
    const int64_t chunk = blockIdx.x;
    const int c = (blockIdx.y * kMgThreads + threadIdx.x) * V;
    if (c >= width) return;
    const int row0 = chunk_row0[chunk], cnt = chunk_cnt[chunk];
    const T *src = proj + static_cast<int64_t>(row0) * proj_stride + c;
    float *slot = start ? nullptr : state + static_cast<int64_t>(tok_state[row0] >> 1) * slot_stride + s_off + c;
    const bool fresh = !start && tok_pos[row0] == 0;
    float zb[V], ub[V], S[V];
#pragma unroll
    for (int j = 0; j < V; ++j) {
        zb[j] = z_b ? z_b[c + j] : 0.f;
        ub[j] = u_b ? u_b[c + j] : 0.f;
        S[j] = start ? start[chunk * 2 * width + c + j] : fresh ? 0.f : slot[j];
    }
    for (int t0 = 0; t0 < cnt; t0 += kMgAhead) {
        float z[kMgAhead][V], u[kMgAhead][V], g[kMgAhead][V];
#pragma unroll
        for (int k = 0; k < kMgAhead; ++k) {
            const T *p = src + static_cast<int64_t>(min(t0 + k, cnt - 1)) * proj_stride;
            mg_load<T, V>(z[k], p);
            mg_load<T, V>(u[k], p + width);
            mg_load<T, V>(g[k], p + 2 * static_cast<int64_t>(width));
        }
#pragma unroll
        for (int k = 0; k < kMgAhead; ++k) {
            if (t0 + k < cnt) {
                T *dst = out + static_cast<int64_t>(row0 + t0 + k) * width + c;
                typename MgVec<T, V>::type o;
#pragma unroll
                for (int j = 0; j < V; ++j) {
                    const float a = mg_sigmoid(z[k][j] + zb[j]);
                    S[j] = fmaf(1.f - a, S[j], a * mg_candidate(u[k][j] + ub[j]));
                    const T v = to_t<T>(S[j] * (g[k][j] * mg_sigmoid(g[k][j])));
                    if constexpr (V == 1) o = v;
                    else o[j] = v;
                }
                *reinterpret_cast<typename MgVec<T, V>::type *>(dst) = o;
            }
        }
    }
    if (!start) {
#pragma unroll
        for (int j = 0; j < V; ++j) slot[j] = S[j];
    }
}

// two columns per thread when every row starts on a two-element boundary
inline bool mg_pairs(int width, int64_t stride, const void *a, const void *b) {
    return width % 2 == 0 && stride % 2 == 0 && ((reinterpret_cast<uintptr_t>(a) | reinterpret_cast<uintptr_t>(b)) & 7) == 0;
}

} // namespace swl

extern "C" int swl_min_gru_chunks(float *part, const void *proj, int64_t proj_stride, const float *z_b, const float *u_b,
                                  const int32_t *chunk_row0, const int32_t *chunk_cnt, int32_t num_chunks, int32_t width,
                                  int32_t dtype, swl_stream_t stream) {
    if (num_chunks < 0 || width <= 0 || proj_stride < 3LL * width) return SWL_ERR_BAD_ARG;
    if (num_chunks == 0) return SWL_OK;
    if (!part || !proj || !chunk_row0 || !chunk_cnt) return SWL_ERR_BAD_ARG;
    const bool pairs = swl::mg_pairs(width, proj_stride, proj, proj);
    const int per = swl::kMgThreads * (pairs ? 2 : 1);
    const dim3 grid(static_cast<unsigned>(num_chunks), static_cast<unsigned>((width + per - 1) / per));
    if (grid.y > 65535) return SWL_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    SWL_DISPATCH_DTYPE3(dtype, T, {
        if (pairs)
            hipLaunchKernelGGL((swl::min_gru_chunks_kernel<T, 2>), grid, dim3(swl::kMgThreads), 0, s, part,
                               static_cast<const T *>(proj), proj_stride, z_b, u_b, chunk_row0, chunk_cnt, width);
        else
            hipLaunchKernelGGL((swl::min_gru_chunks_kernel<T, 1>), grid, dim3(swl::kMgThreads), 0, s, part,
                               static_cast<const T *>(proj), proj_stride, z_b, u_b, chunk_row0, chunk_cnt, width);
    });
    return swl::check_launch();
}

extern "C" int swl_min_gru_carry(float *part, float *state, int64_t slot_stride, int64_t s_off, const int32_t *seq_row0,
                                 const int32_t *seq_cnt, const int32_t *seq_chunk0, const int32_t *tok_pos,
                                 const int32_t *tok_state, int32_t num_seqs, int32_t chunk_tokens, int32_t width,
                                 swl_stream_t stream) {
    if (num_seqs < 0 || width <= 0 || chunk_tokens <= 0) return SWL_ERR_BAD_ARG;
    if (num_seqs == 0) return SWL_OK;
    if (!part || !state || !seq_row0 || !seq_cnt || !seq_chunk0 || !tok_pos || !tok_state) return SWL_ERR_BAD_ARG;
    const dim3 grid(static_cast<unsigned>(num_seqs), static_cast<unsigned>((width + swl::kMgThreads - 1) / swl::kMgThreads));
    if (grid.y > 65535) return SWL_ERR_UNSUPPORTED;
    hipLaunchKernelGGL(swl::min_gru_carry_kernel, grid, dim3(swl::kMgThreads), 0, static_cast<hipStream_t>(stream), part, state,
                       slot_stride, s_off, seq_row0, seq_cnt, seq_chunk0, tok_pos, tok_state, chunk_tokens, width);
    return swl::check_launch();
}

extern "C" int swl_min_gru_apply(void *out, const void *proj, int64_t proj_stride, const float *z_b, const float *u_b,
                                 const float *start, float *state, int64_t slot_stride, int64_t s_off,
                                 const int32_t *chunk_row0, const int32_t *chunk_cnt, const int32_t *tok_pos,
                                 const int32_t *tok_state, int32_t num_chunks, int32_t width, int32_t dtype,
                                 swl_stream_t stream) {
    if (num_chunks < 0 || width <= 0 || proj_stride < 3LL * width) return SWL_ERR_BAD_ARG;
    if (num_chunks == 0) return SWL_OK;
    if (!out || !proj || !chunk_row0 || !chunk_cnt) return SWL_ERR_BAD_ARG;
    if (!start && (!state || !tok_pos || !tok_state)) return SWL_ERR_BAD_ARG;
    const bool pairs = swl::mg_pairs(width, proj_stride, proj, out);
    const int per = swl::kMgThreads * (pairs ? 2 : 1);
    const dim3 grid(static_cast<unsigned>(num_chunks), static_cast<unsigned>((width + per - 1) / per));
    if (grid.y > 65535) return SWL_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    SWL_DISPATCH_DTYPE3(dtype, T, {
        if (pairs)
            hipLaunchKernelGGL((swl::min_gru_apply_kernel<T, 2>), grid, dim3(swl::kMgThreads), 0, s, static_cast<T *>(out),
                               static_cast<const T *>(proj), proj_stride, z_b, u_b, start, state, slot_stride, s_off,
                               chunk_row0, chunk_cnt, tok_pos, tok_state, width);
        else
            hipLaunchKernelGGL((swl::min_gru_apply_kernel<T, 1>), grid, dim3(swl::kMgThreads), 0, s, static_cast<T *>(out),
                               static_cast<const T *>(proj), proj_stride, z_b, u_b, start, state, slot_stride, s_off,
                               chunk_row0, chunk_cnt, tok_pos, tok_state, width);
    });
    return swl::check_launch();
}
