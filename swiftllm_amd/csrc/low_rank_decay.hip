// low_rank_decay.hip — per-channel decays of a recurrence from a low-rank projection, in one launch:
//     z   = act(W1 x)            (optional: without W1 the rows of x are z already)       act: 0 identity, 1 tanh
//     y   = W2 z + b
//     out = sigmoid(y)^p         (kind 0)      or      exp(-exp(y))     (kind 1)          fp32 [T, channels]
// W1 [rank, width] and W2 [channels, rank] are the compute dtype, the bias, the activations and the decays fp32.
//
//   16-bit, width a multiple of 32, rank and channels of 16: one workgroup per (16 tokens, share of the channels) on the matrix
//   cores. The waves share the reduction over the width (their partial z meet in LDS, where the activation is applied and z becomes a
//   16-bit operand again), then the channel tiles, a tile's weights requested while the one before is computed.
//   otherwise: one workgroup per token, a wave per rank row, then a thread per channel.
#include "swl_common.h"

namespace swl {

constexpr int kLdThreads = 256;
constexpr int kLdWaves = kLdThreads / 64;
constexpr int kLdMaxRank = 256;

__device__ __forceinline__ float ld_decay(float y, int kind, float power) {
    // sigmoid(y)^p = exp(p ln sigmoid(y)), ln sigmoid(y) = min(y, 0) - ln(1 + e^-|y|)
    if (kind == 0) return expf(power * (fminf(y, 0.f) - log1pf(expf(-fabsf(y)))));
    return expf(-expf(y));
}

// The same on the exp2 / log2 units, for 16-bit models: absolute error of a rounding of the decay.
__device__ __forceinline__ float ld_decay_fast(float y, int kind, float power) {
    constexpr float kLog2e = 1.4426950408889634f;
    if (kind == 0) {
        const float x = fast_exp2(-kLog2e * fabsf(y));
        const float l = x < 1e-4f ? kLog2e * x : __log2f(1.0f + x);      // log2(1 + x)
        return fast_exp2(power * (kLog2e * fminf(y, 0.f) - l));
    }
    return fast_exp2(-kLog2e * fast_exp2(kLog2e * y));
}

__device__ __forceinline__ float4_t mfma32(vec8_t<bf16> a, vec8_t<bf16> b, float4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ float4_t mfma32(vec8_t<f16> a, vec8_t<f16> b, float4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(a, b, c, 0, 0, 0);
}

template <typename T>
__global__ __launch_bounds__(kLdThreads) void low_rank_decay_kernel(float *out, const T *x, int64_t x_stride, const T *w1, const T *w2,
                                                                    const float *bias, int width, int rank, int channels,
                                                                    int act, int kind, float power) {
    __shared__ float z[kLdMaxRank];
    const int64_t t = blockIdx.x;
    const T *row = x + t * x_stride;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    if (w1) {
        for (int r = wave; r < rank; r += kLdWaves) {
            const T *w = w1 + static_cast<int64_t>(r) * width;
            float a = 0.f;
            for (int i = lane; i < width; i += 64) a += to_f(row[i]) * to_f(w[i]);
            a = wave_allreduce_sum(a);
            if (lane == 0) z[r] = act ? tanhf(a) : a;
        }
    } else {
        for (int r = threadIdx.x; r < rank; r += kLdThreads) z[r] = act ? tanhf(to_f(row[r])) : to_f(row[r]);
    }
    __syncthreads();
    for (int c = threadIdx.x; c < channels; c += kLdThreads) {
        const T *w = w2 + static_cast<int64_t>(c) * rank;
        float a = bias[c];
        for (int r = 0; r < rank; ++r) a += to_f(w[r]) * z[r];
        out[t * channels + c] = ld_decay(a, kind, power);
    }
}

// RT: rank tiles of 16; NW: waves
template <typename T, int RT, int NW>
__global__ __launch_bounds__(NW * 64) void low_rank_decay_mfma_kernel(float *out, const T *x, int64_t x_stride, const T *w1,
                                                                         const T *w2, const float *bias, int64_t num_tokens, int width,
                                                                         int channels, int act, int kind, float power) {
    constexpr int R = RT * 16;
    constexpr int ZS = R + 4;       // (16-bit elements per row of z: 8-byte operand loads, rows 8 bytes apart in the banks)
    __shared__ float part[NW][16][R + 1];
    __shared__ alignas(16) T z[16][ZS];
    const int64_t t0 = static_cast<int64_t>(blockIdx.x) * 16;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int li = lane & 15, lq = lane >> 4;
    const int64_t last = num_tokens - 1;
    if (w1) {
        // D[token][rank row] = sum_i x[token][i] w1[rank row][i]: A lane = token li, B lane = rank row li, both at i = 8 lq ..
        float4_t acc[RT];
#pragma unroll
        for (int j = 0; j < RT; ++j) acc[j] = float4_t{0.f, 0.f, 0.f, 0.f};
        const T *xr = x + (t0 + li < num_tokens ? t0 + li : last) * x_stride + 8 * lq;
        const T *wr = w1 + static_cast<int64_t>(li) * width + 8 * lq;
        for (int i = wave * 32; i < width; i += NW * 32 * 4) {       // four steps' operands are requested together
            vec8_t<T> a[4], b[4][RT];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int iu = min(i + u * NW * 32, width - 32);
                a[u] = load8(xr + iu);
#pragma unroll
                for (int j = 0; j < RT; ++j) b[u][j] = load8(wr + static_cast<int64_t>(j) * 16 * width + iu);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                if (i + u * NW * 32 < width) {        // (wave-uniform)
#pragma unroll
                    for (int j = 0; j < RT; ++j) acc[j] = mfma32(a[u], b[u][j], acc[j]);
                }
            }
        }
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            mfma_results_ready<4>(acc[j]);
#pragma unroll
            for (int r = 0; r < 4; ++r) part[wave][4 * lq + r][16 * j + li] = acc[j][r];
        }
        __syncthreads();
        for (int i = threadIdx.x; i < 16 * R; i += NW * 64) {
            const int t = i / R, c = i - t * R;
            float a = 0.f;
#pragma unroll
            for (int w = 0; w < NW; ++w) a += part[w][t][c];
            z[t][c] = to_t<T>(act ? tanhf(a) : a);
        }
    } else {
        for (int i = threadIdx.x; i < 16 * R; i += NW * 64) {
            const int t = i / R, c = i - t * R;
            const float a = to_f(x[(t0 + t < num_tokens ? t0 + t : last) * x_stride + c]);
            z[t][c] = to_t<T>(act ? tanhf(a) : a);
        }
    }
    __syncthreads();
    vec4_t<T> za[RT];
#pragma unroll
    for (int j = 0; j < RT; ++j) load4(za[j], &z[li][16 * j + 4 * lq]);
    const int tiles = channels >> 4, step = NW * static_cast<int>(gridDim.y);
    int ct = static_cast<int>(blockIdx.y) * NW + wave;
    if (ct >= tiles) return;
    vec4_t<T> b[RT];
    float bc;
    auto fetch = [&](int tile) {
        const int c = tile * 16 + li;
#pragma unroll
        for (int j = 0; j < RT; ++j) load4(b[j], w2 + static_cast<int64_t>(c) * R + 4 * lq + 16 * j);
        bc = bias[c];
    };
    fetch(ct);
    for (; ct < tiles; ct += step) {
        float4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < RT; ++j) acc = mfma16(za[j], b[j], acc);
        const float add = bc;
        fetch(min(ct + step, tiles - 1));
        mfma_results_ready<4>(acc);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int64_t t = t0 + 4 * lq + r;
            if (t < num_tokens) out[t * channels + ct * 16 + li] = ld_decay_fast(acc[r] + add, kind, power);
        }
    }
}

} // namespace swl

extern "C" int swl_low_rank_decay(float *out, const void *x, int64_t x_stride, const void *w1, const void *w2, const float *bias,
                                  int64_t num_tokens, int32_t width, int32_t rank, int32_t channels, int32_t act, int32_t kind,
                                  float power, int32_t dtype, swl_stream_t stream) {
    if (num_tokens < 0 || rank <= 0 || channels <= 0 || act < 0 || act > 1 || kind < 0 || kind > 1) return SWL_ERR_BAD_ARG;
    if (w1 && width <= 0) return SWL_ERR_BAD_ARG;
    if (x_stride < (w1 ? width : rank)) return SWL_ERR_BAD_ARG;
    if (num_tokens == 0) return SWL_OK;
    if (!out || !x || !w2 || !bias) return SWL_ERR_BAD_ARG;
    if (num_tokens > 0x7fffffffLL || rank > swl::kLdMaxRank) return SWL_ERR_UNSUPPORTED;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const auto eight = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 7) == 0; };
    const int rt = rank / 16;
    if (dtype != SWL_F32 && rank % 16 == 0 && (rt == 1 || rt == 2 || rt == 4 || rt == 8) && channels % 16 == 0 &&
        (!w1 || (width % 32 == 0 && x_stride % 8 == 0 && swl::aligned16(x) && swl::aligned16(w1))) && eight(w2)) {
        const int64_t tiles = (num_tokens + 15) / 16;
        // few tokens: the channels are shared out over workgroups (each makes the small z again)
        const int waves = rt <= 4 ? 8 : 4;      // (a wave's partial z is 16 x rank floats of LDS)
        int shares = 1;
        while (tiles * shares < 128 && shares < 8 && channels / 16 >= 2 * shares * waves) shares *= 2;
        const dim3 grid(static_cast<unsigned>(tiles), static_cast<unsigned>(shares));
#define SWL_LD(N)                                                                                                             \
    case N:                                                                                                                   \
        hipLaunchKernelGGL((swl::low_rank_decay_mfma_kernel<T, N, (N <= 4 ? 8 : 4)>), grid, dim3(waves * 64), 0, s, out,       \
                           static_cast<const T *>(x),                                                                        \
                           x_stride, static_cast<const T *>(w1), static_cast<const T *>(w2), bias, num_tokens, width, channels, act, \
                           kind, power);                                                                                      \
        break
        SWL_DISPATCH_DTYPE(dtype, T, {
            switch (rt) {
                SWL_LD(1);
                SWL_LD(2);
                SWL_LD(4);
                SWL_LD(8);
            }
        });
#undef SWL_LD
        return swl::check_launch();
    }
    SWL_DISPATCH_DTYPE3(dtype, T, {
        hipLaunchKernelGGL((swl::low_rank_decay_kernel<T>), dim3(static_cast<unsigned>(num_tokens)), dim3(swl::kLdThreads), 0, s, out,
                           static_cast<const T *>(x), x_stride, static_cast<const T *>(w1), static_cast<const T *>(w2), bias, width,
                           rank, channels, act, kind, power);
    });
    return swl::check_launch();
}
