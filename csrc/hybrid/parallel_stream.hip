// parallel_stream.hip — the float32 residual stream of hybrid decoders whose layers have ONE layer norm that the mixer
// and the feed-forward both read, and the RMS norm of a few columns of a wider projection.
//
//   layer_norm_join   x <- x + y (+ y2);  h = (x - mean) / sqrt(var + eps) * w + b, var the mean of the squared
//                     deviations.  Everything in float; y, y2 and h in the activation type.  A row of up to 16 values per
//                     thread stays in registers between the sum, the two statistics (mean first, then the deviations)
//                     and the output: one pass over memory.  Rows up to 1024 wide take one wave each, wider ones a
//                     workgroup of 4, 8 or 16 waves.
//   norm_cols         columns off .. off + n of a row divided by their root mean square, times w: a latent that the
//                     next projection reads.  One wave per row.
#include "hybrid_common.h"

namespace chronos {
namespace hy {

template <typename T, int V> __device__ __forceinline__ void ps_ld(const T* p, float* v) {
    if constexpr (V == 4 && sizeof(T) == 4) {
        const f32x4 q = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = q[i];
    } else if constexpr (V == 4) {
        const u16x4 q = *reinterpret_cast<const u16x4*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = bf2f(q[i]);
    } else {
        v[0] = ld<T>(p);
    }
}
template <typename T, int V> __device__ __forceinline__ void ps_st(T* p, const float* v) {
    if constexpr (V == 4 && sizeof(T) == 4) *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    else if constexpr (V == 4) *reinterpret_cast<u16x4*>(p) = u16x4{f2bf(v[0]), f2bf(v[1]), f2bf(v[2]), f2bf(v[3])};
    else st<T>(p, v[0]);
}

// sum over the NT threads of a row; `red` holds one float per wave
template <int NT> __device__ __forceinline__ float row_sum(float v, float* red) {
    v = wave_sum(v);
    if constexpr (NT > 64) {
        __syncthreads();   // the previous sum has been read by everyone
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
        __syncthreads();
        v = 0.f;
#pragma unroll
        for (int w = 0; w < NT / 64; ++w) v += red[w];
    }
    return v;
}

// NT threads per row; a workgroup of max(NT, 256) threads takes one row, or with NT = 64 one row per wave
template <typename T, int V, int NT>
__global__ void __launch_bounds__(NT < 256 ? 256 : NT) layer_norm_join_kernel(
        const T* __restrict__ y, const T* __restrict__ y2, float* __restrict__ x, const float* __restrict__ wb,
        T* __restrict__ h, int rows, int d, float eps) {
    constexpr int NC = 4;
    __shared__ float red[NT / 64];
    const int tid = NT == 64 ? threadIdx.x & 63 : threadIdx.x;
    const int64_t row = NT == 64 ? (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6) : blockIdx.x;
    if (row >= rows) return;   // (whole waves; with NT = 64 nothing below is shared between them)
    float* xr = x + row * d;
    float c[NC][V];
    float sum = 0.f;
    auto joined = [&](int i, float* v) {   // the stream's new values at columns i .. i + V, written back
        ps_ld<float, V>(xr + i, v);
        if (y != nullptr) {
            float a[V];
            ps_ld<T, V>(y + row * d + i, a);
            if (y2 != nullptr) {
                float b[V];
                ps_ld<T, V>(y2 + row * d + i, b);
#pragma unroll
                for (int u = 0; u < V; ++u) a[u] += b[u];
            }
#pragma unroll
            for (int u = 0; u < V; ++u) v[u] += a[u];
            ps_st<float, V>(xr + i, v);
        }
#pragma unroll
        for (int u = 0; u < V; ++u) sum += v[u];
    };
#pragma unroll
    for (int j = 0; j < NC; ++j) {
        const int i = (tid + NT * j) * V;
        if (i < d) joined(i, c[j]);
    }
    for (int i = (tid + NT * NC) * V; i < d; i += NT * V) {
        float v[V];
        joined(i, v);
    }
    if (h == nullptr) return;
    const float mean = row_sum<NT>(sum, red) / (float)d;
    float sq = 0.f;
    auto deviate = [&](float* v) {
#pragma unroll
        for (int u = 0; u < V; ++u) {
            v[u] -= mean;
            sq += v[u] * v[u];
        }
    };
#pragma unroll
    for (int j = 0; j < NC; ++j)
        if ((tid + NT * j) * V < d) deviate(c[j]);
    for (int i = (tid + NT * NC) * V; i < d; i += NT * V) {   // (a thread re-reads what it has written)
        float v[V];
        ps_ld<float, V>(xr + i, v);
        deviate(v);
    }
    const float rstd = 1.f / sqrtf(row_sum<NT>(sq, red) / (float)d + eps);
    auto put = [&](int i, float* v) {      // v: deviations from the mean
        float w[V], b[V];
        ps_ld<float, V>(wb + i, w);
        ps_ld<float, V>(wb + d + i, b);
#pragma unroll
        for (int u = 0; u < V; ++u) v[u] = v[u] * rstd * w[u] + b[u];
        ps_st<T, V>(h + row * d + i, v);
    };
#pragma unroll
    for (int j = 0; j < NC; ++j) {
        const int i = (tid + NT * j) * V;
        if (i < d) put(i, c[j]);
    }
    for (int i = (tid + NT * NC) * V; i < d; i += NT * V) {
        float v[V];
        ps_ld<float, V>(xr + i, v);
#pragma unroll
        for (int u = 0; u < V; ++u) v[u] -= mean;
        put(i, v);
    }
}

template <typename T, int V>
__global__ void __launch_bounds__(256) norm_cols_kernel(const T* __restrict__ src, int64_t lds, const float* __restrict__ w,
                                                        T* __restrict__ out, int rows, int n, float eps) {
    constexpr int NC = 8;
    const int lane = threadIdx.x & 63;
    const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= rows) return;
    const T* s = src + row * lds;
    T* o = out + row * n;
    float c[NC][V];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NC; ++j) {
        const int i = (lane + 64 * j) * V;
        if (i < n) {
            ps_ld<T, V>(s + i, c[j]);
#pragma unroll
            for (int u = 0; u < V; ++u) ss += c[j][u] * c[j][u];
        }
    }
    for (int i = (lane + 64 * NC) * V; i < n; i += 64 * V) {
        float v[V];
        ps_ld<T, V>(s + i, v);
#pragma unroll
        for (int u = 0; u < V; ++u) ss += v[u] * v[u];
    }
    const float inv = 1.f / sqrtf(wave_sum(ss) / (float)n + eps);
    auto put = [&](int i, float* v) {
        float wv[V];
        ps_ld<float, V>(w + i, wv);
#pragma unroll
        for (int u = 0; u < V; ++u) v[u] = v[u] * inv * wv[u];
        ps_st<T, V>(o + i, v);
    };
#pragma unroll
    for (int j = 0; j < NC; ++j) {
        const int i = (lane + 64 * j) * V;
        if (i < n) put(i, c[j]);
    }
    for (int i = (lane + 64 * NC) * V; i < n; i += 64 * V) {
        float v[V];
        ps_ld<T, V>(s + i, v);
        put(i, v);
    }
}

}  // namespace hy

// y == nullptr: the stream stays as it is; y2 == nullptr: one summand; h == nullptr: nothing is emitted.
void launch_hy_layer_norm_join(const void* y, const void* y2, float* x, const float* wb, void* h, int rows, int d,
                               float eps, bool f32, hipStream_t s) {
    if (rows == 0 || (y == nullptr && h == nullptr)) return;
#define HY_LJ(T, V, NT) hy::layer_norm_join_kernel<T, V, NT><<<NT == 64 ? (rows + 3) / 4 : rows, NT < 256 ? 256 : NT, 0, s>>>((const T*)y, (const T*)y2, x, wb, (T*)h, rows, d, eps)
#define HY_LJ_T(T)                                  \
    do {                                            \
        if (d % 4) HY_LJ(T, 1, 256);                \
        else if (d <= 1024) HY_LJ(T, 4, 64);        \
        else if (d <= 4096) HY_LJ(T, 4, 256);       \
        else if (d <= 8192) HY_LJ(T, 4, 512);       \
        else HY_LJ(T, 4, 1024);                     \
    } while (0)
    if (f32) HY_LJ_T(float);
    else HY_LJ_T(uint16_t);
#undef HY_LJ_T
#undef HY_LJ
}

// src: the first column of row 0 (row stride lds)
void launch_hy_norm_cols(const void* src, int64_t lds, const float* w, void* out, int rows, int n, float eps, bool f32,
                         hipStream_t s) {
    if (rows == 0) return;
    const bool vec = n % 4 == 0 && lds % 4 == 0 && reinterpret_cast<uintptr_t>(src) % (f32 ? 16 : 8) == 0;
    const unsigned grid = (unsigned)((rows + 3) / 4);
#define HY_NC(T, V) hy::norm_cols_kernel<T, V><<<grid, 256, 0, s>>>((const T*)src, lds, w, (T*)out, rows, n, eps)
    if (f32) { if (vec) HY_NC(float, 4); else HY_NC(float, 1); }
    else { if (vec) HY_NC(uint16_t, 4); else HY_NC(uint16_t, 1); }
#undef HY_NC
}

}  // namespace chronos
