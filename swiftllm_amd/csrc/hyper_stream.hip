// hyper_stream.hip — the fp32 residual of models with hyper-connections: S parallel streams per token instead of one.
//
//   swl_embed_streams: x[t][s] = embed[token[t]] for every stream s.
//   swl_hyper_step:    the step between two sublayers in one launch, one workgroup per token. With the previous sublayer's result
//                      y (the sum of y_parts rows per token: the results of a token's experts, or of fp32 slabs: the K shares of
//                      the product that makes it; + y2: a second addend, + y_bias: a
//                      bias of its output projection)
//       X_t <- sum_s mix[s][t] X_s + out[t] * y        all streams at once from the old ones
//       u    = sum_s in[s] X_s                         what the next sublayer reads
//       h    = u / rms(u over each of `groups` equal parts) * w
//     Any half may be absent: no y = norm only (of rows row_idx, when given), no h = update only. Streams, statistics and sums are
//     fp32; y, y2 and h are the compute dtype. S = 1 with mix = in = out = 1 is the ordinary pre-norm residual.
//
// A thread owns the same columns of every stream, so the update and the weighted sum happen in its registers; only the norm's
// statistics cross threads. Layout: x [tokens, S, width].
#include "swl_common.h"

namespace swl {

constexpr int kHsThreads = 256;
constexpr int kHsMaxStreams = 16;
constexpr int kHsQuickGroups = 4;       // norm parts whose sums are kept in registers

template <typename T>
__global__ __launch_bounds__(kHsThreads) void embed_streams_kernel(float *x, const T *embed, const int32_t *tokens, int width,
                                                                   int streams) {
    const int64_t t = blockIdx.x;
    const T *e = embed + static_cast<int64_t>(tokens[t]) * width;
    float *xr = x + t * streams * width;
    for (int i = threadIdx.x; i < width; i += kHsThreads) {
        const float v = to_f(e[i]);
        for (int s = 0; s < streams; ++s) xr[static_cast<int64_t>(s) * width + i] = v;
    }
}

template <typename T, int V>
__device__ __forceinline__ void hs_load(float *dst, const T *p) {
    if constexpr (V == 4) {
        const vec4_t<T> v = *reinterpret_cast<const vec4_t<T> *>(p);
#pragma unroll
        for (int j = 0; j < 4; ++j) dst[j] = to_f(v[j]);
    } else {
        dst[0] = to_f(p[0]);
    }
}
template <typename T, int V>
__device__ __forceinline__ void hs_store(T *p, const float *src) {
    if constexpr (V == 4) {
        vec4_t<T> v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = to_t<T>(src[j]);
        *reinterpret_cast<vec4_t<T> *>(p) = v;
    } else {
        p[0] = to_t<T>(src[0]);
    }
}

// S: streams held in registers (S == streams when EXACT, else S >= streams). V: columns per access (4 when width % 4 == 0).
template <typename T, int S, int V, bool EXACT>
__global__ __launch_bounds__(kHsThreads) void hyper_step_kernel(
    float *x, const T *y, int y_parts, const float *slabs, int64_t slab_stride, const T *y2, const float *y_bias,
    const float *__restrict__ mix, const float *__restrict__ outw,
    const float *__restrict__ inw, const float *__restrict__ norm_w, T *h, const int32_t *row_idx, int width, int streams,
    int groups, float eps) {
    extern __shared__ float lds[];
    float *row = lds;                           // [width] u
    float *rstd = row + width;                  // [groups]
    float *red = rstd + groups;                 // [waves][kHsQuickGroups]
    const int64_t o = blockIdx.x;
    const int64_t t = row_idx ? row_idx[o] : o;
    float *xr = x + t * streams * width;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int part = width / groups;
    // the parts' sums of squares in registers when there are few of them and an access never straddles two
    const bool quick = groups <= kHsQuickGroups && part % V == 0;
    float ss[kHsQuickGroups];
#pragma unroll
    for (int g = 0; g < kHsQuickGroups; ++g) ss[g] = 0.f;

    for (int c = threadIdx.x * V; c < width; c += kHsThreads * V) {
        float xs[S][V];
#pragma unroll
        for (int s = 0; s < S; ++s) {
            if (EXACT || s < streams) hs_load<float, V>(xs[s], xr + static_cast<int64_t>(s) * width + c);
            else
#pragma unroll
                for (int j = 0; j < V; ++j) xs[s][j] = 0.f;
        }
        float u[V];
#pragma unroll
        for (int j = 0; j < V; ++j) u[j] = 0.f;
        if (y || slabs) {
            float yv[V];
            if (slabs) {        // (four at a time: requested before the first sum)
                const float *p = slabs + t * width + c;
                hs_load<float, V>(yv, p);
                for (int k = 1; k < y_parts; k += 4) {
                    float b[4][V];
#pragma unroll
                    for (int u = 0; u < 4; ++u) hs_load<float, V>(b[u], p + min(k + u, y_parts - 1) * slab_stride);
#pragma unroll
                    for (int u = 0; u < 4; ++u) {
                        if (k + u < y_parts) {
#pragma unroll
                            for (int j = 0; j < V; ++j) yv[j] += b[u][j];
                        }
                    }
                }
            } else {
                hs_load<T, V>(yv, y + t * y_parts * width + c);
                for (int k = 1; k < y_parts; ++k) {
                    float b[V];
                    hs_load<T, V>(b, y + (t * y_parts + k) * width + c);
#pragma unroll
                    for (int j = 0; j < V; ++j) yv[j] += b[j];
                }
            }
            if (y2) {
                float b[V];
                hs_load<T, V>(b, y2 + t * width + c);
#pragma unroll
                for (int j = 0; j < V; ++j) yv[j] += b[j];
            }
            if (y_bias) {
                float b[V];
                hs_load<float, V>(b, y_bias + c);
#pragma unroll
                for (int j = 0; j < V; ++j) yv[j] += b[j];
            }
#pragma unroll
            for (int d = 0; d < S; ++d) {
                if (EXACT || d < streams) {
                    float nx[V];
                    const float ow = outw[d];
#pragma unroll
                    for (int j = 0; j < V; ++j) nx[j] = ow * yv[j];
#pragma unroll
                    for (int s = 0; s < S; ++s) {
                        if (EXACT || s < streams) {
                            const float m = mix[s * streams + d];
#pragma unroll
                            for (int j = 0; j < V; ++j) nx[j] = fmaf(m, xs[s][j], nx[j]);
                        }
                    }
                    hs_store<float, V>(xr + static_cast<int64_t>(d) * width + c, nx);
                    const float iw = inw ? inw[d] : 1.f;
#pragma unroll
                    for (int j = 0; j < V; ++j) u[j] = fmaf(iw, nx[j], u[j]);
                }
            }
        } else {
#pragma unroll
            for (int s = 0; s < S; ++s) {
                if (EXACT || s < streams) {
                    const float iw = inw ? inw[s] : 1.f;
#pragma unroll
                    for (int j = 0; j < V; ++j) u[j] = fmaf(iw, xs[s][j], u[j]);
                }
            }
        }
        if (!h) continue;
        float sq = 0.f;
#pragma unroll
        for (int j = 0; j < V; ++j) {
            row[c + j] = u[j];
            sq += u[j] * u[j];
        }
        if (quick) {
            const int g = groups > 1 ? c / part : 0;
#pragma unroll
            for (int k = 0; k < kHsQuickGroups; ++k) ss[k] += g == k ? sq : 0.f;
        }
    }
    if (!h) return;
    if (quick) {
#pragma unroll
        for (int k = 0; k < kHsQuickGroups; ++k) {
            if (k < groups) {
                const float v = wave_allreduce_sum(ss[k]);
                if (lane == 0) red[wave * kHsQuickGroups + k] = v;
            }
        }
        __syncthreads();
        if (threadIdx.x < static_cast<unsigned>(groups)) {
            float v = 0.f;
#pragma unroll
            for (int w = 0; w < kHsThreads / 64; ++w) v += red[w * kHsQuickGroups + threadIdx.x];
            rstd[threadIdx.x] = 1.0f / sqrtf(v / static_cast<float>(part) + eps);
        }
    } else {
        __syncthreads();
        for (int g = wave; g < groups; g += kHsThreads / 64) {
            float v = 0.f;
            for (int i = lane; i < part; i += 64) {
                const float a = row[g * part + i];
                v += a * a;
            }
            v = wave_allreduce_sum(v);
            if (lane == 0) rstd[g] = 1.0f / sqrtf(v / static_cast<float>(part) + eps);
        }
    }
    __syncthreads();
    for (int c = threadIdx.x * V; c < width; c += kHsThreads * V) {     // (each thread reads back its own columns of row[])
        float v[V], w[V];
        hs_load<float, V>(w, norm_w + c);
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] = row[c + j] * rstd[groups > 1 ? (c + j) / part : 0] * w[j];
        hs_store<T, V>(h + o * width + c, v);
    }
}

inline size_t hs_lds_bytes(int width, int groups) {
    return (static_cast<size_t>(width) + groups + (kHsThreads / 64) * kHsQuickGroups) * sizeof(float);
}

template <typename T, int V>
void launch_hs(dim3 grid, size_t lds, hipStream_t s, float *x, const T *y, int yp, const float *sl, int64_t ss, const T *y2,
               const float *yb, const float *mix,
               const float *ow, const float *iw, const float *nw, T *h, const int32_t *ri, int width, int streams, int groups,
               float eps) {
#define SWL_HS(S, X)                                                                                                          \
    hipLaunchKernelGGL((hyper_step_kernel<T, S, V, X>), grid, dim3(kHsThreads), lds, s, x, y, yp, sl, ss, y2, yb, mix, ow, iw, nw, h, ri, \
                       width, streams, groups, eps)
    switch (streams) {
    case 1: SWL_HS(1, true); break;
    case 2: SWL_HS(2, true); break;
    case 3: SWL_HS(3, true); break;
    case 4: SWL_HS(4, true); break;
    default:
        if (streams <= 8) SWL_HS(8, false);
        else SWL_HS(kHsMaxStreams, false);
        break;
    }
#undef SWL_HS
}

} // namespace swl

extern "C" int swl_embed_streams(float *x, const void *embed, const int32_t *tokens, int64_t num_tokens, int32_t width,
                                 int32_t streams, int32_t dtype, swl_stream_t stream) {
    if (num_tokens < 0 || width <= 0 || streams <= 0) return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!x || !embed || !tokens) return SWL_ERR_BAD_ARG;
    if (num_tokens > 0x7fffffffLL) return SWL_ERR_UNSUPPORTED;
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::embed_streams_kernel<T>), dim3(static_cast<unsigned>(num_tokens)), dim3(swl::kHsThreads), 0,
                           static_cast<hipStream_t>(stream), x, static_cast<const T *>(embed), tokens, width, streams);
    });
    return swl::check_launch();
}

extern "C" int swl_hyper_step(float *x, const void *y, int32_t y_parts, const float *slabs, int64_t slab_stride, const void *y2,
                              const float *y_bias, const float *mix, const float *outw, const float *inw, const float *norm_w, void *h,
                              const int32_t *row_idx,
                              int64_t num_rows, int32_t width, int32_t streams, int32_t groups, float eps, int32_t dtype,
                              swl_stream_t stream) {
    const bool has_y = y || slabs;
    if ((y && slabs) || (has_y && y_parts < 1)) return SWL_ERR_BAD_ARG;
    if (num_rows < 0 || width <= 0 || streams <= 0 || groups <= 0 || width % groups) return SWL_ERR_BAD_ARG;
    if (num_rows == 0) return SWL_OK;
    if (!x || (has_y && (!mix || !outw)) || (!has_y && (y2 || y_bias)) || (h && !norm_w) || (row_idx && has_y))
        return SWL_ERR_BAD_ARG;
    if (!has_y && !h) return SWL_OK;
    const size_t lds = swl::hs_lds_bytes(width, groups);
    if (num_rows > 0x7fffffffLL || streams > swl::kHsMaxStreams || lds > 64 * 1024) return SWL_ERR_UNSUPPORTED;
    const bool wide = width % 4 == 0 && swl::aligned16(x) && swl::aligned16(y) && swl::aligned16(slabs) &&
                      slab_stride % 4 == 0 && swl::aligned16(y2) && swl::aligned16(y_bias) &&
                      swl::aligned16(norm_w) && swl::aligned16(h);
    const dim3 grid(static_cast<unsigned>(num_rows));
    hipStream_t s = static_cast<hipStream_t>(stream);
    SWL_DISPATCH_DTYPE3(dtype, T, {
        if (wide)
            swl::launch_hs<T, 4>(grid, lds, s, x, static_cast<const T *>(y), y_parts, slabs, slab_stride, static_cast<const T *>(y2),
                                 y_bias, mix, outw, inw,
                                 norm_w, static_cast<T *>(h), row_idx, width, streams, groups, eps);
        else
            swl::launch_hs<T, 1>(grid, lds, s, x, static_cast<const T *>(y), y_parts, slabs, slab_stride, static_cast<const T *>(y2),
                                 y_bias, mix, outw, inw,
                                 norm_w, static_cast<T *>(h), row_idx, width, streams, groups, eps);
    });
    return swl::check_launch();
}
