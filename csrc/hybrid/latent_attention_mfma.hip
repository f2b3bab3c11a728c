// latent_attention_mfma.hip — the bfloat16 latent attention on the matrix cores (see latent_attention.hip for the
// math: one cached row per token, key = the whole row, value = its first `rank` columns, shared by all heads).
//
// One workgroup takes up to 128 (token, head) rows of one sequence — 16 per wave, rows are (token * H + head), so any
// head count tiles the same way — and walks the sequence's keys 64 at a time:
//   * the key tile goes from memory straight into LDS (no staging registers), row-major [64][DK], two tiles deep: the
//     next tile is on its way while the current one is computed, one barrier per tile.  Both MFMA operands want 8
//     k-values per lane — dims for the scores, KEYS for the weighted sum: the scores read rows as they lie, the sum
//     reads the same image through gfx950's transposing LDS reads (4 keys of 16 columns each).
//   * scores  S^T = K Q^T : 16x16x32 MFMAs with the key rows as A operand and the wave's 16 query rows (held in
//     registers for the whole kernel) as B operand, so a lane ends up with 4 keys x 1 query row per 16-key tile;
//   * softmax in float per query row (lane & 15): causal mask by the row's own position, running maximum and sum,
//     reductions over the 4 lane groups by two shuffles;
//   * sum  O^T = V^T P^T : the lane's 8 weights of two neighbouring 16-key tiles ARE a B operand (the k index is a
//     fixed permutation of the 32 keys, the same one the value columns are read with), so the weights never
//     leave registers.  Accumulators: rank / 16 tiles x 4 registers.  Optionally each weight enters as two
//     bfloat16 terms (rounded value + remainder), which keeps the float softmax weights nearly exact.
// After the last key a sink per head may join the denominator.
// With a window a row sees only its last `window` positions: the walk starts at the tile of the first row's first
// visible key and every row masks by its own position.
// Sizes: DK % 8 == 0 (the scores' steps past it are zero), rank % 16 == 0, DK <= 576, rank <= 512.
// Everything else takes latent_attention.hip.
#include "hybrid_common.h"

namespace chronos {
namespace hy {

constexpr int MKT = 64;  // keys per tile
constexpr float kLog2e = 1.4426950408889634f;

// NS: k-steps of the scores (DK / 32) at most; NCT: 16-column tiles of the output (rank / 16) at most.  All of them are
// computed whatever the sizes (a run-time test in front of every product would serialise the loop); the surplus is zero
// times a real number or never stored.
// NW: waves per workgroup, 4 or 8 (16 query rows each): with 8 a staged key tile serves 128 rows and every SIMD holds two
// waves, so one wave's softmax and staging run beside the other's MFMAs.
// TT: weights as two bfloat16 terms.
// KS: waves that share 16 query rows.  With few rows (decode) a tile's keys are dealt to 2 or 4 waves, each with a softmax
// of its own over its keys (16 keys per wave: 16x16x16 products in the sum), and merged through LDS at the end.
template <int NS, int NCT, int NW, int KS, bool TT>
__global__ void __launch_bounds__(64 * NW) latent_attention_mfma_kernel(
        const uint16_t* __restrict__ qa, const uint16_t* __restrict__ cache, const int32_t* __restrict__ block_table,
        int max_blocks, const int32_t* __restrict__ q_start, const int32_t* __restrict__ pos,
        const float* __restrict__ gate, uint16_t* __restrict__ out, int H, int DK, int rank, int BS, float scale,
        int window, int nsplit, float* __restrict__ part_o, float* __restrict__ part_ml, int bs_shift,
        const float* __restrict__ sink) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int b = blockIdx.x;
    const int t0 = q_start[b], t1 = q_start[b + 1];
    const int rows_total = (t1 - t0) * H;
    constexpr int KT = MKT, RPB = 16 * NW / KS;  // query rows per workgroup
    const int rb0 = blockIdx.y * RPB;
    if (rb0 >= rows_total) return;
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, g = lane >> 4, qi = lane & 15;
    const int nct = rank / 16;
    constexpr int CPR = NS * 4 + 1, krs = CPR * 16;   // key row in LDS: 16-byte chunks, bytes
    __shared__ int krow[2][KT];  // cache row (page * page size + slot) of each key of a tile
    // this lane's query row (for the B operand and for the softmax): row r of the sequence, token t0 + r / H
    const int kpart = wv % KS;   // which part of a tile's keys this wave takes
    const int r = rb0 + wv / KS * 16 + qi;
    const bool rok = r < rows_total;
    const int rc = rok ? r : rows_total - 1;
    const int64_t grow = (int64_t)t0 * H + rc;              // row of qa / out / gate
    const int prow = rok ? pos[t0 + rc / H] : -1;
    const int last_row = min(rows_total, rb0 + RPB) - 1;
    const int pmax = pos[t0 + last_row / H];                // positions grow along the sequence
    const int k_lo = window > 0 ? max(0, pos[t0 + rb0 / H] - window + 1) / KT * KT : 0;
    const int row_lo = window > 0 ? prow - window + 1 : 0;  // the first key this lane's row sees
    bf16x8 qf[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) {   // columns past the row's end are zero here (and real numbers in the key image)
        const u16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
        qf[s] = 32 * s + 8 * g < DK ? *reinterpret_cast<const bf16x8*>(qa + grow * DK + 32 * s + 8 * g)
                                    : __builtin_bit_cast(bf16x8, z);
    }
    f32x4 O[NCT];
#pragma unroll
    for (int c = 0; c < NCT; ++c) O[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    float mrow = -INFINITY, lrow = 0.f;
    const float scale2 = scale * kLog2e;   // scores, maxima and sums live in the base-2 domain
    const int32_t* bt = block_table + (int64_t)b * max_blocks;
    const int chunks = DK / 8;
    const uint32_t lds0 = lds_offset(smem);
    // key tiles are dealt round-robin to the nsplit workgroups of this row block (blockIdx.z): the context length is
    // only known on the device, and a split that gets no tile contributes an empty partial
    const int kfirst = k_lo + blockIdx.z * KT, kstep = KT * nsplit;
    auto row_of = [&](int k0) {
        const int key = min(k0 + (int)threadIdx.x, pmax);  // past the end: a real row, masked below
        return bs_shift >= 0 ? ((bt[key >> bs_shift] << bs_shift) + (key & (BS - 1))) : (bt[key / BS] * BS + key % BS);
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int j = wv; j < CPR; j += NW) dma_rows<CPR>(cache, krow[buf], DK, chunks, j, lds0 + buf * KT * krs, lane);
    };
    if (threadIdx.x < KT) krow[0][threadIdx.x] = row_of(kfirst);
    __syncthreads();
    if (kfirst <= pmax) stage(0);
    if (threadIdx.x < KT) krow[1][threadIdx.x] = row_of(kfirst + kstep);
    const bool wave_on = rb0 + wv / KS * 16 < rows_total;   // (a wave without rows only helps to stage)
    int buf = 0;
    for (int k0 = kfirst; k0 <= pmax; k0 += kstep, buf ^= 1) {
        dma_wait();        // this wave's pieces of the tile have landed
        __syncthreads();   // ... everyone's; the other buffer's tile has been read by all; its next rows are known
        if (k0 + kstep <= pmax) stage(buf ^ 1);
        const int nrow = threadIdx.x < KT ? row_of(k0 + 2 * kstep) : 0;
        const unsigned char* kimg = smem + buf * KT * krs;
        if (wave_on) {
        // ---- scores: KT / 16 key tiles of 16; lane gets keys 16 kt + 4 g + i of query row qi
        constexpr int NKT = KT / 16 / KS;
        const int key0 = kpart * (KT / KS);
        f32x4 S[NKT];
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt) {
            S[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
            const unsigned char* arow = kimg + (key0 + 16 * kt + qi) * krs + g * 16;
#pragma unroll
            for (int s = 0; s < NS; ++s)
                S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(arow + s * 64), qf[s],
                                                                S[kt], 0, 0, 0);
        }
        // ---- softmax over the tile for query row qi (this lane and the 3 other lane groups hold its keys)
        float mx = -INFINITY;
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int key = k0 + key0 + 16 * kt + 4 * g + i;
                const float sv = key <= prow && key >= row_lo ? S[kt][i] * scale2 : -INFINITY;
                S[kt][i] = sv;
                mx = fmaxf(mx, sv);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float mn = fmaxf(mrow, mx);
        const float corr = (mn == -INFINITY) ? 1.f : __builtin_amdgcn_exp2f(mrow - mn);
        const float mref = (mn == -INFINITY) ? 0.f : mn;   // (all masked: every exponent is -inf, every weight 0)
        float sum = 0.f;
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float p = __builtin_amdgcn_exp2f(S[kt][i] - mref);
                S[kt][i] = p;
                sum += p;
            }
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        lrow = lrow * corr + sum;
        mrow = mn;
        // ---- weighted sum of the value columns: k index of step u = [tile 2u keys 4g..4g+3 | tile 2u+1 keys 4g..4g+3]
        constexpr int NU = NKT / 2;
        if (__builtin_amdgcn_ballot_w64(corr != 1.f) != 0) {   // (rarely, once the maxima have settled)
#pragma unroll
            for (int c = 0; c < NCT; ++c) O[c] *= corr;
        }
        const unsigned char* vt = kimg + (key0 + 4 * g + (qi >> 2)) * krs + (qi & 3) * 8;
        if constexpr (NKT == 1) {
            bf16x4 pf, pl;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                pf[e] = (__bf16)S[0][e];
                if constexpr (TT) pl[e] = (__bf16)(S[0][e] - (float)pf[e]);
            }
#pragma unroll
            for (int c = 0; c < NCT; ++c) {
                const bf16x4 vf = lds_read_tr4(vt + c * 32);
                O[c] = mfma_16x16x16(vf, pf, O[c]);
                if constexpr (TT) O[c] = mfma_16x16x16(vf, pl, O[c]);
            }
        }
#pragma unroll
        for (int u = 0; u < NU; ++u) {
            bf16x8 pf, pl;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float w = S[2 * u + (e >> 2)][e & 3];
                pf[e] = (__bf16)w;
                if constexpr (TT) pl[e] = (__bf16)(w - (float)pf[e]);
            }
#pragma unroll
            for (int c = 0; c < NCT; ++c) {
                const bf16x4 lo = lds_read_tr4(vt + 32 * u * krs + c * 32);
                const bf16x4 hi = lds_read_tr4(vt + (32 * u + 16) * krs + c * 32);
                const bf16x8 vf = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
                O[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf, O[c], 0, 0, 0);
                if constexpr (TT) O[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl, O[c], 0, 0, 0);
            }
        }
        }
        if (threadIdx.x < KT) krow[buf][threadIdx.x] = nrow;
    }
    if constexpr (KS > 1) {   // the waves that share these rows merge their partial results; the first one goes on
        constexpr int MS = NCT * 16 + 4;    // floats per row (padded)
        float* mb = reinterpret_cast<float*>(smem);
        static_assert(NW * 16 * MS * 4 <= 2 * KT * krs, "the partial rows fit the key tiles' LDS");
        __shared__ float ml[NW][16][2];
        __syncthreads();                    // everyone is done with the key tiles
#pragma unroll
        for (int c = 0; c < NCT; ++c) *reinterpret_cast<f32x4*>(mb + (wv * 16 + qi) * MS + 16 * c + 4 * g) = O[c];
        if (g == 0) {
            ml[wv][qi][0] = mrow;
            ml[wv][qi][1] = lrow;
        }
        __syncthreads();
        if (kpart != 0) return;
        float mn = mrow, e[KS];
#pragma unroll
        for (int k = 1; k < KS; ++k) mn = fmaxf(mn, ml[wv + k][qi][0]);
        const float mref = mn == -INFINITY ? 0.f : mn;
        e[0] = exp2f(mrow - mref);
        lrow *= e[0];
#pragma unroll
        for (int k = 1; k < KS; ++k) {
            e[k] = exp2f(ml[wv + k][qi][0] - mref);
            lrow += e[k] * ml[wv + k][qi][1];
        }
        mrow = mn;
#pragma unroll
        for (int c = 0; c < NCT; ++c) {
            O[c] *= e[0];
#pragma unroll
            for (int k = 1; k < KS; ++k)
                O[c] += e[k] * *reinterpret_cast<const f32x4*>(mb + ((wv + k) * 16 + qi) * MS + 16 * c + 4 * g);
        }
    }
    if (!rok) return;
    if (nsplit > 1) {  // unnormalised partial: the combine kernel merges the splits
        const int64_t pr = grow * nsplit + blockIdx.z;
        if (g == 0) {
            part_ml[pr * 2] = mrow;
            part_ml[pr * 2 + 1] = lrow;
        }
#pragma unroll
        for (int c = 0; c < NCT; ++c)
            if (c < nct) *reinterpret_cast<f32x4*>(part_o + pr * rank + 16 * c + 4 * g) = O[c];
        return;
    }
    float f = 1.f / lrow;
    if (sink != nullptr) {   // exp(sink) joins the denominator, without a value
        const float sk = sink[rc % H] * kLog2e, mn = fmaxf(mrow, sk), c = exp2f(mrow - mn);
        f = c / (lrow * c + exp2f(sk - mn));
    }
    if (gate != nullptr) f *= sigmoidf_(gate[grow]);
    // lane holds O^T[col = 16 c + 4 g + i][query row qi]
#pragma unroll
    for (int c = 0; c < NCT; ++c)
        if (c < nct) {
            const u16x4 o = u16x4{f2bf(O[c][0] * f), f2bf(O[c][1] * f), f2bf(O[c][2] * f), f2bf(O[c][3] * f)};
            *reinterpret_cast<u16x4*>(out + grow * rank + 16 * c + 4 * g) = o;
        }
}

// one wave per (token, head) row: out = sum_z 2^(m_z - m) O_z / (sum_z 2^(m_z - m) l_z + 2^(sink log2 e - m)) * sigmoid(gate)
// (the partial maxima are in the base-2 domain: score * scale * log2 e).  Lane z holds
// split z's maximum and sum (nsplit <= 16); a lane then sums 4 neighbouring columns over the splits, whose loads do not
// depend on each other.
__global__ void __launch_bounds__(256) latent_combine_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                                             const float* __restrict__ gate, uint16_t* __restrict__ out,
                                                             int64_t rows, int rank, int nsplit,
                                                             const float* __restrict__ sink, int H) {
    const int lane = threadIdx.x & 63;
    const int64_t r = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (r >= rows) return;
    const float mz = lane < nsplit ? part_ml[(r * nsplit + lane) * 2] : -INFINITY;
    const float lz = lane < nsplit ? part_ml[(r * nsplit + lane) * 2 + 1] : 0.f;
    const float sk = sink != nullptr ? sink[r % H] * kLog2e : -INFINITY;
    const float m = fmaxf(wave_max(mz), sk);
    float e = mz == -INFINITY ? 0.f : exp2f(mz - m);   // (a split without a visible key adds nothing)
    const float l = wave_sum(e * lz) + (sink != nullptr ? exp2f(sk - m) : 0.f);
    e *= (gate != nullptr ? sigmoidf_(gate[r]) : 1.f) / l;
    for (int c = lane * 4; c < rank; c += 256) {      // (rank is a multiple of 16)
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int z = 0; z < nsplit; ++z) {
            const float w = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(e), z));
            acc += w * *reinterpret_cast<const f32x4*>(part_o + (r * nsplit + z) * rank + c);
        }
        *reinterpret_cast<u16x4*>(out + r * rank + c) = u16x4{f2bf(acc[0]), f2bf(acc[1]), f2bf(acc[2]), f2bf(acc[3])};
    }
}

}  // namespace hy

template <int NS, int NCT, int NW, int KS, bool TT>
static void la_mfma_launch(const uint16_t* qa, const uint16_t* cache, const int32_t* bt, int max_blocks,
                           const int32_t* q_start, const int32_t* pos, const float* gate, uint16_t* out, int B, int H,
                           int DK, int rank, int BS, int max_q, float scale, int window, int nsplit, float* part_o,
                           float* part_ml, const float* sink, hipStream_t s) {
    auto kern = hy::latent_attention_mfma_kernel<NS, NCT, NW, KS, TT>;
    constexpr int bytes = 2 * hy::MKT * (NS * 64 + 16);
    static int set_bytes = 0;
    if (bytes > set_bytes) {
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
        set_bytes = bytes;
    }
    const dim3 grid(B, (max_q * H + 16 * NW / KS - 1) / (16 * NW / KS), nsplit);
    const int bs_shift = (BS & (BS - 1)) == 0 ? __builtin_ctz(BS) : -1;
    kern<<<grid, 64 * NW, bytes, s>>>(qa, cache, bt, max_blocks, q_start, pos, gate, out, H, DK, rank, BS, scale, window,
                                  nsplit, part_o, part_ml, bs_shift, sink);
}

bool hy_latent_mfma_ok(int DK, int rank) { return !(DK % 8 || rank % 16 || DK > 576 || rank > 512 || rank > DK); }

// Splits of the key range (flash-decoding) for a launch of `wgs` workgroups over contexts of at most max_ctx keys:
// enough workgroups to cover the chip, at least 4 key tiles per split (2 behind a window, whose few tiles are all of the
// walk), at most 16.
int hy_latent_nsplit(int wgs, int max_ctx, bool windowed) {
    if (wgs >= 128) return 1;
    int want = (256 + wgs - 1) / wgs, cap = max_ctx / ((windowed ? 2 : 4) * hy::MKT);
    if (want > 16) want = 16;
    if (want > cap) want = cap;
    return want < 1 ? 1 : want;
}

// false: these sizes are not served here (the caller takes the general kernel).  nsplit > 1: part_o float
// [T * H * nsplit, rank] and part_ml float [T * H * nsplit, 2] scratch.
bool launch_hy_latent_attention_mfma(const uint16_t* qa, const uint16_t* cache, const int32_t* bt, int max_blocks,
                                     const int32_t* q_start, const int32_t* pos, const float* gate, uint16_t* out, int B,
                                     int H, int DK, int rank, int BS, int max_q, float scale, int window, bool two_term,
                                     int nsplit, float* part_o, float* part_ml, int64_t total_rows, const float* sink,
                                     hipStream_t s) {
    if (!hy_latent_mfma_ok(DK, rank)) return false;
    if (B == 0 || max_q == 0) return true;
#define HY_LAM(NS, NCT, NW, KS, TT) la_mfma_launch<NS, NCT, NW, KS, TT>(qa, cache, bt, max_blocks, q_start, pos, gate, out, B, H, DK, rank, BS, max_q, scale, window, nsplit, part_o, part_ml, sink, s)
    // 8 waves per workgroup when a sequence brings more than 64 rows; up to 32 or 16 rows 2 or 4 waves share them
    const int rows = max_q * H;
#define HY_LAM_R(NS, NCT, TT)                             \
    do {                                                  \
        if (rows > 64) HY_LAM(NS, NCT, 8, 1, TT);         \
        else if (rows > 32) HY_LAM(NS, NCT, 4, 1, TT);    \
        else if (rows > 16) HY_LAM(NS, NCT, 4, 2, TT);    \
        else HY_LAM(NS, NCT, 4, 4, TT);                   \
    } while (0)
#define HY_LAM_T(NS, NCT)                                                                       \
    do {                                                                                        \
        if (two_term) HY_LAM_R(NS, NCT, true); else HY_LAM_R(NS, NCT, false);                   \
    } while (0)
    if (DK <= 128 && rank <= 64) HY_LAM_T(4, 4);
    else if (DK <= 192 && rank <= 128) HY_LAM_T(6, 8);
    else if (DK <= 320 && rank <= 256) HY_LAM_T(10, 16);
    else HY_LAM_T(18, 32);
#undef HY_LAM_T
#undef HY_LAM_R
#undef HY_LAM
    if (nsplit > 1)
        hy::latent_combine_kernel<<<(unsigned)((total_rows + 3) / 4), 256, 0, s>>>(part_o, part_ml, gate, out, total_rows, rank, nsplit, sink, H);
    return true;
}

}  // namespace chronos
