// conv_prep.hip — what an attention layer needs of its projection when queries and keys pass a short causal
// convolution and the keys are the values divided by their root mean square.  Per token and head, in one pass:
//
//   y = sum_i w[:, i] u_(t - (K-1) + i)     u: the projected columns; inputs before the step's first token come from the
//                                           sequence's history row, or are zero when the step starts at position 0
//   query heads:  q = y / rms(y) * temperature[position]                  -> q [T, H D]
//   key heads:    v = y as the cache holds it -> the token's page and slot; 1 / rms(v) -> the key's factor beside it
//   gate columns: their float copy                                        -> gate [T, H]
//
//   conv_prep_vec   up to 4 taps, D = 32, 64, 128 or 256: a thread owns 8 neighbouring columns of one head (16-byte
//                   loads), D / 8 lanes share a head (the mean of squares is a few shuffles), and walks several
//                   consecutive tokens with its taps and the last K-1 inputs in registers, so that a projected value is
//                   loaded once.
//   conv_prep       any other sizes (D <= 256): one wave per head and token.
//
// With one token per sequence (decode) the history is rewritten in the same pass: a thread is the only reader and writer of
// its columns of the sequence's row.  Otherwise a second launch follows (linear_scan.hip).
#include "hybrid_common.h"

namespace chronos {
namespace hy {

template <typename T> __device__ __forceinline__ void cp_ld8(const T* p, float* v) {
    if constexpr (sizeof(T) == 4) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            v[i] = a[i];
            v[4 + i] = b[i];
        }
    } else {
        const u16x8 a = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = bf2f(a[i]);
    }
}
template <typename T> __device__ __forceinline__ void cp_st8(T* p, const float* v) {
    if constexpr (sizeof(T) == 4) {
        *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
        *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
    } else {
        u16x8 a;
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] = f2bf(v[i]);
        *reinterpret_cast<u16x8*>(p) = a;
    }
}

struct ConvPrepArgs {
    int64_t ldp;                 // row stride of the projection
    const float* taps;           // [C, K]
    const int32_t *tok_seq, *q_start, *pos0, *slots, *pos, *block_table;
    int max_blocks, T, H, G, D, BS;
    float eps;
    const float* temp;           // [P] or nullptr
    float* ks;                   // [NB, BS, G]
    float* gate;                 // [T, H] or nullptr
    int g_off;
};

template <typename T, int K>
__global__ void __launch_bounds__(256) conv_prep_vec_kernel(const T* __restrict__ proj, T* hist, T* __restrict__ q,
                                                            T* __restrict__ vc, const ConvPrepArgs a, int TT, int rewrite) {
    const int lph = a.D / 8;                               // lanes per head, a power of two up to 32
    const int jr = blockIdx.y * (256 / lph) + threadIdx.x / lph;
    const bool on = jr < a.H + a.G;
    const int j = on ? jr : a.H + a.G - 1;                 // (idle lanes follow along for the shuffles)
    const int c0 = threadIdx.x % lph * 8, col = j * a.D + c0, C = (a.H + a.G) * a.D;
    float w[8][K];
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
        for (int k = 0; k < K; ++k) w[i][k] = a.taps[(int64_t)(col + i) * K + k];
    float u[K][8];
    int pb = -1;
    const int tb = blockIdx.x * TT, te = min(a.T, tb + TT);
    for (int t = tb; t < te; ++t) {
        const int b = a.tok_seq[t];
        T* hrow = hist + (int64_t)a.slots[b] * (K - 1) * C + col;
        if (b != pb) {
            pb = b;
            const int t0 = a.q_start[b];
            const bool past = a.pos0[b] > 0;
#pragma unroll
            for (int i = 0; i < K - 1; ++i) {
                const int s = t - (K - 1) + i;
                if (s >= t0) cp_ld8<T>(proj + s * a.ldp + col, u[i]);
                else if (past) cp_ld8<T>(hrow + (int64_t)((K - 1) + (s - t0)) * C, u[i]);
                else {
#pragma unroll
                    for (int e = 0; e < 8; ++e) u[i][e] = 0.f;
                }
            }
        }
        cp_ld8<T>(proj + t * a.ldp + col, u[K - 1]);
        float y[8];
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float v = 0.f;
#pragma unroll
            for (int i = 0; i < K; ++i) v += w[e][i] * u[i][e];
            y[e] = j < a.H ? v : rnd<T>(v);
            ss += y[e] * y[e];
        }
        for (int m = 1; m < lph; m <<= 1) ss += __shfl_xor(ss, m, 64);
        const float inv = 1.f / sqrtf(ss / (float)a.D + a.eps);
        const int p = a.pos[t];
        if (on && j < a.H) {
            const float f = a.temp != nullptr ? inv * a.temp[p] : inv;
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] *= f;
            cp_st8<T>(q + (int64_t)t * a.H * a.D + col, y);
        } else if (on) {
            const int64_t slot = ((int64_t)a.block_table[(int64_t)b * a.max_blocks + p / a.BS] * a.BS + p % a.BS) * a.G + (j - a.H);
            cp_st8<T>(vc + slot * a.D + c0, y);
            if (c0 == 0) a.ks[slot] = inv;
        }
        if (rewrite && on) {
#pragma unroll
            for (int i = 0; i < K - 1; ++i) cp_st8<T>(hrow + (int64_t)i * C, u[i + 1]);
        }
#pragma unroll
        for (int i = 0; i < K - 1; ++i)
#pragma unroll
            for (int e = 0; e < 8; ++e) u[i][e] = u[i + 1][e];
        if (a.gate != nullptr && blockIdx.y == 0)
            for (int h = threadIdx.x; h < a.H; h += 256) a.gate[(int64_t)t * a.H + h] = ld<T>(proj + t * a.ldp + a.g_off + h);
    }
}

// grid (T, ceil((H + G) / 4)): a wave takes one head of one token, a lane every 64th column
template <typename T>
__global__ void __launch_bounds__(256) conv_prep_kernel(const T* __restrict__ proj, T* hist, T* __restrict__ q,
                                                        T* __restrict__ vc, const ConvPrepArgs a, int K, int rewrite) {
    const int64_t t = blockIdx.x;
    const int lane = threadIdx.x & 63, j = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (a.gate != nullptr && blockIdx.y == 0)
        for (int h = threadIdx.x; h < a.H; h += 256) a.gate[t * a.H + h] = ld<T>(proj + t * a.ldp + a.g_off + h);
    if (j >= a.H + a.G) return;
    const int b = a.tok_seq[t], t0 = a.q_start[b], p = a.pos[t], C = (a.H + a.G) * a.D;
    const bool past = a.pos0[b] > 0;
    T* hrow = hist + (int64_t)a.slots[b] * (K - 1) * C;
    float y[4];
    float ss = 0.f;
#pragma unroll
    for (int m = 0; m < 4; ++m) {
        const int c = lane + 64 * m, col = j * a.D + c;
        y[m] = 0.f;
        if (c >= a.D) continue;
        for (int i = 0; i < K; ++i) {
            const int64_t s = t - (K - 1) + i;
            float v = 0.f;
            if (s >= t0) v = ld<T>(proj + s * a.ldp + col);
            else if (past) v = ld<T>(hrow + (int64_t)((K - 1) + (s - t0)) * C + col);
            y[m] += a.taps[(int64_t)col * K + i] * v;
        }
        if (j >= a.H) y[m] = rnd<T>(y[m]);
        ss += y[m] * y[m];
        if (rewrite) {   // this token is its sequence's only one: entry i takes entry i + 1, the last one the token
            for (int i = 0; i < K - 1; ++i) {
                float v = 0.f;
                if (i == K - 2) v = ld<T>(proj + t * a.ldp + col);
                else if (past) v = ld<T>(hrow + (int64_t)(i + 1) * C + col);
                st<T>(hrow + (int64_t)i * C + col, v);
            }
        }
    }
    const float inv = 1.f / sqrtf(wave_sum(ss) / (float)a.D + a.eps);
    const float f = a.temp != nullptr ? inv * a.temp[p] : inv;
    const int64_t slot = ((int64_t)a.block_table[(int64_t)b * a.max_blocks + p / a.BS] * a.BS + p % a.BS) * a.G + (j - a.H);
#pragma unroll
    for (int m = 0; m < 4; ++m) {
        const int c = lane + 64 * m;
        if (c >= a.D) continue;
        if (j < a.H) st<T>(q + t * a.H * a.D + j * a.D + c, y[m] * f);
        else st<T>(vc + slot * a.D + c, y[m]);
    }
    if (j >= a.H && lane == 0) a.ks[slot] = inv;
}

}  // namespace hy

template <typename T>
static void conv_prep_t(const T* proj, T* hist, T* q, T* vc, const hy::ConvPrepArgs& a, int K, bool one_each, hipStream_t s) {
    const int lph = a.D / 8;
    const bool pow2 = a.D % 8 == 0 && (lph & (lph - 1)) == 0 && lph >= 4 && lph <= 32;
    auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
    if (pow2 && K <= 4 && a.ldp % 8 == 0 && al(proj) && al(hist) && al(q) && al(vc)) {
        const int hpb = 256 / lph, TT = one_each || a.T < 2048 ? 1 : 8;
        const dim3 grid((a.T + TT - 1) / TT, (a.H + a.G + hpb - 1) / hpb);
#define HY_CP(KK) hy::conv_prep_vec_kernel<T, KK><<<grid, 256, 0, s>>>(proj, hist, q, vc, a, TT, one_each)
        if (K == 1) HY_CP(1);
        else if (K == 2) HY_CP(2);
        else if (K == 3) HY_CP(3);
        else HY_CP(4);
#undef HY_CP
        return;
    }
    hy::conv_prep_kernel<T><<<dim3(a.T, (a.H + a.G + 3) / 4), 256, 0, s>>>(proj, hist, q, vc, a, K, one_each);
}

void launch_hy_conv_hist(const void* x, int ldx, const int32_t* q_start, const int32_t* pos0, const int32_t* slots,
                         void* hist, int B, int C, int K, bool f32, hipStream_t s);

// one_each: no sequence brings more than one token (the history is then rewritten in the same pass)
void launch_hy_conv_prep(const void* proj, int64_t ldp, const float* taps, int K, const int32_t* tok_seq,
                         const int32_t* q_start, const int32_t* pos0, const int32_t* slots, void* hist, const int32_t* pos,
                         const int32_t* block_table, int max_blocks, int T, int B, int H, int G, int D, float eps,
                         const float* temp, float* ks, void* vc, int BS, void* q, float* gate, int g_off, bool one_each,
                         bool f32, hipStream_t s) {
    if (T == 0) return;
    const hy::ConvPrepArgs a{ldp, taps, tok_seq, q_start, pos0, slots, pos, block_table, max_blocks, T, H, G, D, BS, eps,
                             temp, ks, gate, g_off};
    if (f32) conv_prep_t<float>((const float*)proj, (float*)hist, (float*)q, (float*)vc, a, K, one_each, s);
    else conv_prep_t<uint16_t>((const uint16_t*)proj, (uint16_t*)hist, (uint16_t*)q, (uint16_t*)vc, a, K, one_each, s);
    if (!one_each && K > 1) launch_hy_conv_hist(proj, (int)ldp, q_start, pos0, slots, hist, B, (H + G) * D, K, f32, s);
}

}  // namespace chronos
