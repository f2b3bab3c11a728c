// head_matmul.hip — every head's own small matrix product of the latent attention:
//
//     out[t, h, n] = sum_k a[t, h, k] w[h, n, k]   (times sigmoid(g[t, h N + n]) when gate columns are given)
//
// used to carry queries into the latent space (N = latent size, K = head size) and the attention's latent-space output
// back (N = value size, K = latent size).  Rows of a and out are column ranges of wider rows (a projection's, the
// latent query's), so nothing is copied before or after.
//
//   head_matmul_mfma   bfloat16: a workgroup of 4 waves takes 64 MT tokens and 16 NTL output columns of one head.  W
//                      tiles of 64 k-columns are staged in LDS (all waves read them), a wave's own token rows go from
//                      memory straight into registers as B operands; both for the next step while the current one
//                      multiplies.  C^T = W A^T in 16x16x32 MFMAs: a lane ends up with 4 neighbouring output columns
//                      of one token (8-byte stores), which the gate multiplies in float.
//   head_matmul        any sizes and types: 64 x 64 tiles on the vector ALUs, float accumulation.
#include "hybrid_common.h"

namespace chronos {
namespace hy {

constexpr int HKS = 64;               // k-columns per step
constexpr int HLS = HKS * 2 + 16;     // LDS bytes per W row

template <int MT, int NTL>
__global__ void __launch_bounds__(256) head_matmul_mfma_kernel(
        const uint16_t* __restrict__ a, int64_t lda, int64_t ha, const uint16_t* __restrict__ w,
        uint16_t* __restrict__ out, int64_t ldo, int64_t ho, const uint16_t* __restrict__ gsrc, int64_t ldg, int T, int N,
        int K, int vst) {
    constexpr int WCH = NTL * 16 * (HKS / 8) / 256;   // 16-byte W chunks per thread and step
    __shared__ __attribute__((aligned(16))) unsigned char wl[NTL * 16 * HLS];
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, g = lane >> 4, r = lane & 15;
    const int h = blockIdx.z, n0 = blockIdx.y * NTL * 16;
    const int t0 = blockIdx.x * 64 * MT + wv * 16 * MT;
    const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
    const uint16_t* wh = w + (int64_t)h * N * K;
    const uint16_t* ar[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) ar[m] = a + (int64_t)min(t0 + 16 * m + r, T - 1) * lda + h * ha;
    u16x8 wreg[WCH], areg[MT][2];
    auto fetch = [&](int k0) {
#pragma unroll
        for (int u = 0; u < WCH; ++u) {
            const int it = threadIdx.x + 256 * u, row = it / (HKS / 8), kc = k0 + it % (HKS / 8) * 8;
            wreg[u] = (n0 + row < N && kc < K) ? *reinterpret_cast<const u16x8*>(wh + (int64_t)(n0 + row) * K + kc) : zero;
        }
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                const int kc = k0 + 32 * s + 8 * g;
                areg[m][s] = kc < K ? *reinterpret_cast<const u16x8*>(ar[m] + kc) : zero;
            }
    };
    f32x4 acc[MT][NTL];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NTL; ++n) acc[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    fetch(0);
    for (int k0 = 0; k0 < K; k0 += HKS) {
        __syncthreads();   // everyone has read the previous step's W tile
#pragma unroll
        for (int u = 0; u < WCH; ++u) {
            const int it = threadIdx.x + 256 * u;
            *reinterpret_cast<u16x8*>(wl + it / (HKS / 8) * HLS + it % (HKS / 8) * 16) = wreg[u];
        }
        bf16x8 bf[MT][2];
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int s = 0; s < 2; ++s) bf[m][s] = __builtin_bit_cast(bf16x8, areg[m][s]);
        __syncthreads();
        if (k0 + HKS < K) fetch(k0 + HKS);
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int n = 0; n < NTL; ++n) {
                const bf16x8 af = *reinterpret_cast<const bf16x8*>(wl + (16 * n + r) * HLS + s * 64 + g * 16);
#pragma unroll
                for (int m = 0; m < MT; ++m)
                    acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af, bf[m][s], acc[m][n], 0, 0, 0);
            }
    }
    // lane holds out[token r of tile m][column 16 n + 4 g + i]
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int t = t0 + 16 * m + r;
        if (t >= T) continue;
        uint16_t* orow = out + (int64_t)t * ldo + h * ho;
        const uint16_t* grow = gsrc != nullptr ? gsrc + (int64_t)t * ldg + (int64_t)h * N : nullptr;
#pragma unroll
        for (int n = 0; n < NTL; ++n) {
            const int c = n0 + 16 * n + 4 * g;
            if (c >= N) continue;
            f32x4 v = acc[m][n];
            if (vst && c + 3 < N) {
                if (grow != nullptr) {
                    const u16x4 q = *reinterpret_cast<const u16x4*>(grow + c);
#pragma unroll
                    for (int i = 0; i < 4; ++i) v[i] *= sigmoidf_(bf2f(q[i]));
                }
                *reinterpret_cast<u16x4*>(orow + c) = u16x4{f2bf(v[0]), f2bf(v[1]), f2bf(v[2]), f2bf(v[3])};
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (c + i < N) orow[c + i] = f2bf(grow != nullptr ? v[i] * sigmoidf_(bf2f(grow[c + i])) : v[i]);
            }
        }
    }
}

template <typename T>
__global__ void __launch_bounds__(256) head_matmul_kernel(const T* __restrict__ a, int64_t lda, int64_t ha,
                                                          const T* __restrict__ w, T* __restrict__ out, int64_t ldo,
                                                          int64_t ho, const T* __restrict__ gsrc, int64_t ldg, int TT, int N,
                                                          int K) {
    constexpr int KS = 16;
    __shared__ float as[KS][65], ws[KS][65];   // [k][row], odd stride
    const int h = blockIdx.z, n0 = blockIdx.y * 64, t0 = blockIdx.x * 64;
    const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
    const T* wh = w + (int64_t)h * N * K;
    float acc[4][4] = {};
    for (int k0 = 0; k0 < K; k0 += KS) {
        __syncthreads();
        for (int it = threadIdx.x; it < 64 * KS; it += 256) {
            const int row = it / KS, k = it % KS;
            as[k][row] = (t0 + row < TT && k0 + k < K) ? ld<T>(a + (int64_t)(t0 + row) * lda + h * ha + k0 + k) : 0.f;
            ws[k][row] = (n0 + row < N && k0 + k < K) ? ld<T>(wh + (int64_t)(n0 + row) * K + k0 + k) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < KS; ++k)
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] += as[k][ty + 16 * i] * ws[k][tx + 16 * j];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int t = t0 + ty + 16 * i, n = n0 + tx + 16 * j;
            if (t < TT && n < N) {
                float v = acc[i][j];
                if (gsrc != nullptr) v *= sigmoidf_(ld<T>(gsrc + (int64_t)t * ldg + (int64_t)h * N + n));
                st<T>(out + (int64_t)t * ldo + h * ho + n, v);
            }
        }
}

}  // namespace hy

// a: row t, head h at a + t lda + h ha (K columns); out likewise with ldo / ho (N columns); w [H, N, K] contiguous; gsrc
// (first gate column of row 0, row stride ldg) or nullptr.
void launch_hy_head_matmul(const void* a, int64_t lda, int64_t ha, const void* w, void* out, int64_t ldo, int64_t ho,
                           const void* gsrc, int64_t ldg, int T, int H, int N, int K, bool f32, hipStream_t s) {
    if (T == 0 || H == 0 || N == 0) return;
    auto al = [](const void* p, uintptr_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; };
    if (!f32 && K % 8 == 0 && lda % 8 == 0 && ha % 8 == 0 && al(a, 16) && al(w, 16)) {
        const bool vst = ldo % 4 == 0 && ho % 4 == 0 && al(out, 8) && (gsrc == nullptr || (ldg % 4 == 0 && N % 4 == 0 && al(gsrc, 8)));
#define HY_HM(MT, NTL) hy::head_matmul_mfma_kernel<MT, NTL><<<dim3((T + 64 * MT - 1) / (64 * MT), (N + 16 * NTL - 1) / (16 * NTL), H), 256, 0, s>>>((const uint16_t*)a, lda, ha, (const uint16_t*)w, (uint16_t*)out, ldo, ho, (const uint16_t*)gsrc, ldg, T, N, K, vst)
        if (T <= 256) HY_HM(1, 4);
        else if (N <= 64) HY_HM(2, 4);
        else HY_HM(2, 8);
#undef HY_HM
        return;
    }
    const dim3 grid((T + 63) / 64, (N + 63) / 64, H);
    if (f32) hy::head_matmul_kernel<float><<<grid, 256, 0, s>>>((const float*)a, lda, ha, (const float*)w, (float*)out, ldo, ho, (const float*)gsrc, ldg, T, N, K);
    else hy::head_matmul_kernel<uint16_t><<<grid, 256, 0, s>>>((const uint16_t*)a, lda, ha, (const uint16_t*)w, (uint16_t*)out, ldo, ho, (const uint16_t*)gsrc, ldg, T, N, K);
}

}  // namespace chronos
