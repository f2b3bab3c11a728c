// gated_stream.hip — the float32 residual stream of pre-norm hybrid decoders whose norms are Dynamic Tanh, whose
// sublayers are gated element by element and whose layers hand on weighted sums of all earlier results, and the PolyNorm
// activation.
//
//   dyn_tanh     h = tanh(alpha x) w + b                                   (no statistic: element-wise)
//   gated_join   X = x + mult * sigmoid(g + gb) * y;   x <- X, or with depth weights
//                x <- sum_{j <= run} dwa[j] hist[j] + dwa[run + 1] X  and  hist[run + 1] <- X;   h = dyn_tanh(x)
//                One pass: a thread owns 4 (or 1) neighbouring columns of a row; every operand is read once, the older
//                results' loads are independent of each other and of the gate's math.  All arithmetic in float; the
//                gate's columns are read where the sublayer's own first projection left them.
//   poly_norm    a N(z) + b N(z^2) + c N(z^3) + e, N(v) = v / sqrt(mean(v^2) + eps): one workgroup per row, the three
//                means in one reduction, rows up to 16384 wide are read once.
#include "hybrid_common.h"

namespace chronos {
namespace hy {

template <typename T, int V> struct Vec { float v[V]; };
template <typename T, int V> __device__ __forceinline__ Vec<T, V> gs_ld(const T* p) {
    Vec<T, V> r;
    if constexpr (V == 4 && sizeof(T) == 4) {
        const f32x4 q = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) r.v[i] = q[i];
    } else if constexpr (V == 4) {
        const u16x4 q = *reinterpret_cast<const u16x4*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) r.v[i] = bf2f(q[i]);
    } else {
        r.v[0] = ld<T>(p);
    }
    return r;
}
template <typename T, int V> __device__ __forceinline__ void gs_st(T* p, const float* v) {
    if constexpr (V == 4 && sizeof(T) == 4) *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    else if constexpr (V == 4) *reinterpret_cast<u16x4*>(p) = u16x4{f2bf(v[0]), f2bf(v[1]), f2bf(v[2]), f2bf(v[3])};
    else st<T>(p, v[0]);
}

// sigmoid and tanh on the hardware's exp2 and reciprocal (about one unit in the last place each); tanh near zero by
// its Taylor polynomial, where 1 - 2 / (exp(2t) + 1) would cancel
__device__ __forceinline__ float gs_sigmoid(float z) {
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}
__device__ __forceinline__ float gs_tanh(float t) {
    const float a = fabsf(t), s = t * t;
    const float small = t * (1.f + s * (-1.f / 3.f + s * (2.f / 15.f + s * (-17.f / 315.f + s * (62.f / 2835.f)))));
    const float big = 1.f - 2.f * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(2.8853900817779268f * a) + 1.f);
    return a < 0.25f ? small : copysignf(big, t);
}

template <typename T, int V>
__global__ void __launch_bounds__(256) dyn_tanh_kernel(const float* __restrict__ x, const float* __restrict__ wba,
                                                       T* __restrict__ h, int n, int d) {
    const int e = blockIdx.x * 256 + threadIdx.x;
    if (e >= n) return;
    const int c = e % (d / V) * V;
    const float alpha = wba[2 * d];
    auto xv = gs_ld<float, V>(x + (int64_t)e * V);
    const auto wv = gs_ld<float, V>(wba + c), bv = gs_ld<float, V>(wba + d + c);
#pragma unroll
    for (int i = 0; i < V; ++i) xv.v[i] = gs_tanh(alpha * xv.v[i]) * wv.v[i] + bv.v[i];
    gs_st<T, V>(h + (int64_t)e * V, xv.v);
}

// VG: the gate's columns may be read 4 at a time
template <typename T, int V, bool VG>
__global__ void __launch_bounds__(256) gated_join_kernel(const T* __restrict__ y, float* __restrict__ x,
                                                         const T* __restrict__ gsrc, int64_t ldg,
                                                         const float* __restrict__ gb, float mult,
                                                         const float* __restrict__ wba, T* __restrict__ h,
                                                         float* __restrict__ hist, const float* __restrict__ dwa, int run,
                                                         int keep, int n, int d) {
    const int e = blockIdx.x * 256 + threadIdx.x;
    if (e >= n) return;
    const int row = e / (d / V), c = (e - row * (d / V)) * V;
    const int64_t off = (int64_t)e * V;
    const auto yv = gs_ld<T, V>(y + off);
    auto xv = gs_ld<float, V>(x + off);
    float acc[V];
#pragma unroll
    for (int i = 0; i < V; ++i) acc[i] = 0.f;
    const int64_t plane = (int64_t)n * V;
    if (dwa != nullptr) {
#pragma unroll 4
        for (int j = 0; j <= run; ++j) {
            const auto p = gs_ld<float, V>(hist + j * plane + off);
            const float wj = dwa[j];
#pragma unroll
            for (int i = 0; i < V; ++i) acc[i] += wj * p.v[i];
        }
    }
    float f[V];
#pragma unroll
    for (int i = 0; i < V; ++i) f[i] = mult;
    if (gsrc != nullptr) {
        const T* gp = gsrc + row * ldg + c;
        float g[V];
        if constexpr (VG) {
            const auto q = gs_ld<T, V>(gp);
#pragma unroll
            for (int i = 0; i < V; ++i) g[i] = q.v[i];
        } else {
#pragma unroll
            for (int i = 0; i < V; ++i) g[i] = ld<T>(gp + i);
        }
        if (gb != nullptr) {
            const auto q = gs_ld<float, V>(gb + c);
#pragma unroll
            for (int i = 0; i < V; ++i) g[i] += q.v[i];
        }
#pragma unroll
        for (int i = 0; i < V; ++i) f[i] *= gs_sigmoid(g[i]);
    }
#pragma unroll
    for (int i = 0; i < V; ++i) xv.v[i] += f[i] * yv.v[i];
    if (dwa != nullptr) {
        if (keep) gs_st<float, V>(hist + (run + 1) * plane + off, xv.v);
        const float wl = dwa[run + 1];
#pragma unroll
        for (int i = 0; i < V; ++i) xv.v[i] = acc[i] + wl * xv.v[i];
    }
    gs_st<float, V>(x + off, xv.v);
    if (h == nullptr) return;
    const float alpha = wba[2 * d];
    const auto wv = gs_ld<float, V>(wba + c), bv = gs_ld<float, V>(wba + d + c);
#pragma unroll
    for (int i = 0; i < V; ++i) xv.v[i] = gs_tanh(alpha * xv.v[i]) * wv.v[i] + bv.v[i];
    gs_st<T, V>(h + off, xv.v);
}

// NT threads per row; the first 16 NT values (V = 4) or 4 NT values (V = 1) of a row stay in registers
template <typename T, int V, int NT>
__global__ void __launch_bounds__(NT) poly_norm_kernel(const T* __restrict__ z, int64_t ldz, const float* __restrict__ abce,
                                                       T* __restrict__ out, int F, float eps) {
    constexpr int NW = NT / 64;
    __shared__ float red[3][NW];
    const T* zr = z + (int64_t)blockIdx.x * ldz;
    T* orow = out + (int64_t)blockIdx.x * F;
    Vec<T, V> c[4];
    float s2 = 0.f, s4 = 0.f, s6 = 0.f;
    auto add = [&](const Vec<T, V>& q) {
#pragma unroll
        for (int i = 0; i < V; ++i) {
            const float v2 = q.v[i] * q.v[i], v4 = v2 * v2;
            s2 += v2;
            s4 += v4;
            s6 += v4 * v2;
        }
    };
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int i = (threadIdx.x + NT * j) * V;
        if (i < F) {
            c[j] = gs_ld<T, V>(zr + i);
            add(c[j]);
        }
    }
    for (int i = (threadIdx.x + 4 * NT) * V; i < F; i += NT * V) add(gs_ld<T, V>(zr + i));
    s2 = wave_sum(s2);
    s4 = wave_sum(s4);
    s6 = wave_sum(s6);
    if constexpr (NW > 1) {
        if ((threadIdx.x & 63) == 0) {
            red[0][threadIdx.x >> 6] = s2;
            red[1][threadIdx.x >> 6] = s4;
            red[2][threadIdx.x >> 6] = s6;
        }
        __syncthreads();
        s2 = s4 = s6 = 0.f;
#pragma unroll
        for (int w = 0; w < NW; ++w) {
            s2 += red[0][w];
            s4 += red[1][w];
            s6 += red[2][w];
        }
    }
    const float k1 = abce[0] / sqrtf(s2 / (float)F + eps), k2 = abce[1] / sqrtf(s4 / (float)F + eps),
                k3 = abce[2] / sqrtf(s6 / (float)F + eps), k0 = abce[3];
    auto put = [&](int i, Vec<T, V> q) {
#pragma unroll
        for (int u = 0; u < V; ++u) q.v[u] = q.v[u] * (k1 + q.v[u] * (k2 + q.v[u] * k3)) + k0;
        gs_st<T, V>(orow + i, q.v);
    };
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int i = (threadIdx.x + NT * j) * V;
        if (i < F) put(i, c[j]);
    }
    for (int i = (threadIdx.x + 4 * NT) * V; i < F; i += NT * V) put(i, gs_ld<T, V>(zr + i));
}

}  // namespace hy

void launch_hy_dyn_tanh(const float* x, const float* wba, void* h, int rows, int d, bool f32, hipStream_t s) {
    if (rows == 0) return;
    const bool vec = d % 4 == 0;
    const int n = (int)((int64_t)rows * d / (vec ? 4 : 1));
    const unsigned grid = (unsigned)((n + 255) / 256);
#define HY_DT(T, V) hy::dyn_tanh_kernel<T, V><<<grid, 256, 0, s>>>(x, wba, (T*)h, n, d)
    if (f32) { if (vec) HY_DT(float, 4); else HY_DT(float, 1); }
    else { if (vec) HY_DT(uint16_t, 4); else HY_DT(uint16_t, 1); }
#undef HY_DT
}

// gsrc: the gate's first column of row 0 (row stride ldg), or nullptr.  dwa == nullptr: no depth average.  keep: hist
// has a plane for this run's own result.  h == nullptr: nothing is emitted.
void launch_hy_gated_join(const void* y, float* x, const void* gsrc, int64_t ldg, const float* gb, float mult,
                          const float* wba, void* h, float* hist, const float* dwa, int run, bool keep, int rows, int d,
                          bool f32, hipStream_t s) {
    if (rows == 0) return;
    const bool vec = d % 4 == 0;
    const int n = (int)((int64_t)rows * d / (vec ? 4 : 1));
    const unsigned grid = (unsigned)((n + 255) / 256);
    const bool vg = vec && ldg % 4 == 0 && (reinterpret_cast<uintptr_t>(gsrc) % (f32 ? 16 : 8)) == 0;
#define HY_GJ(T, V, VG) hy::gated_join_kernel<T, V, VG><<<grid, 256, 0, s>>>((const T*)y, x, (const T*)gsrc, ldg, gb, mult, wba, (T*)h, hist, dwa, run, keep, n, d)
    if (f32) { if (vg) HY_GJ(float, 4, true); else if (vec) HY_GJ(float, 4, false); else HY_GJ(float, 1, false); }
    else { if (vg) HY_GJ(uint16_t, 4, true); else if (vec) HY_GJ(uint16_t, 4, false); else HY_GJ(uint16_t, 1, false); }
#undef HY_GJ
}

void launch_hy_poly_norm(const void* z, int64_t ldz, const float* abce, void* out, int rows, int F, float eps, bool f32,
                         hipStream_t s) {
    if (rows == 0 || F == 0) return;
    const bool vec = F % 4 == 0 && ldz % 4 == 0;
#define HY_PN(T, V, NT) hy::poly_norm_kernel<T, V, NT><<<rows, NT, 0, s>>>((const T*)z, ldz, abce, (T*)out, F, eps)
#define HY_PN_T(T)                                                                             \
    do {                                                                                       \
        if (!vec) HY_PN(T, 1, 256);                                                            \
        else if (F <= 1024) HY_PN(T, 4, 64);                                                   \
        else if (F <= 4096) HY_PN(T, 4, 256);                                                  \
        else if (F <= 8192) HY_PN(T, 4, 512);                                                  \
        else HY_PN(T, 4, 1024);                                                                \
    } while (0)
    if (f32) HY_PN_T(float);
    else HY_PN_T(uint16_t);
#undef HY_PN_T
#undef HY_PN
}

}  // namespace chronos
