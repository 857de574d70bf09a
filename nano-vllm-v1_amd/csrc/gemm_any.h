// The any-shape product as device functions, shared by the plain entry point (one weight matrix, rows as they lie) and
// the grouped one (a weight matrix per tile, rows gathered through an index): a tile of the grid is handed the rows it
// covers through `RowMap`, everything else is the same code, so a row's result never depends on which entry point, tile
// or batch it travelled in.
#pragma once
#include "common.h"

namespace nvh_any {

// Which rows a 64-row tile covers: row r of the tile (r < rows) is read from x row `src(r)` and written to y row `dst(r)`.
struct RowMap {
    const int32_t* gather;     // source row per destination row (null: the destination row itself)
    int row0;                  // first destination row of the tile
    int rows;                  // real rows of the tile (<= 64)
    __device__ __forceinline__ int64_t dst(int r) const { return row0 + r; }
    __device__ __forceinline__ int64_t src(int r) const { return gather ? gather[row0 + r] : row0 + r; }
};

__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// ---------------------------------------------------------------------------------------------------------------
// y[M, N] = x[M, K] w[N, K]^T (+ bias[N]) (times sigmoid(gate[m, n]) when a gate is given; squared relu with `relu2`) for ANY M, N, K (ragged
// edges are zero-filled on the way into LDS and masked on the way out).  The order in which an output element sums over k depends on
// (N, K) only, never on M or on the row's place in the batch.  bf16: 64 x 64 tile per workgroup, four waves of 2 x 2 MFMA 16x16x32
// tiles, fp32 accumulation.  fp32: the same tile with 4 x 4 outputs per lane on the vector ALU (true fp32 products and sums).
constexpr int GT = 64, GK = 64, GLD = GK + 8;

// What happens to a sum on its way out.
struct Epilogue {
    const bf16* bias;
    const bf16* gate;
    int64_t ldg;
    int relu2;
    __device__ __forceinline__ float operator()(float v, int64_t m, int n) const {
        if (bias) v += (float)bias[n];
        if (gate) v *= sigmoid((float)gate[m * ldg + n]);
        if (relu2) {
            v = fmaxf(v, 0.f);
            v *= v;
        }
        return v;
    }
};

template <bool OUT_F32, bool VEC>
__device__ __forceinline__ void gemm_any_bf16_tile_body(const bf16* __restrict__ x, int64_t ldx, const bf16* __restrict__ w, int64_t ldw, void* __restrict__ yv,
                                                        int64_t ldy, const RowMap rm, int n0, int N, int K, const Epilogue epi, bf16* lds) {
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, fr = lane & 15, fq = lane >> 4;
    const int wm = (wave >> 1) * 32, wn = (wave & 1) * 32;
    f32x4 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int lr = tid >> 2, lc = (tid & 3) * 16;            // this thread's row and first column of the 64 x 64 tile
    // (VEC: rows beyond the tile's or the matrix's repeat a real one - their sums are not written; columns beyond K are zeroed on the way into LDS)
    const bf16* xrow = x + rm.src(min(lr, rm.rows - 1)) * ldx;
    const bf16* wrow = w + (int64_t)min(n0 + lr, N - 1) * ldw;
    // This thread's four 16-byte pieces of a k-step's tiles (x: 0, 1; w: 2, 3) are loaded two steps ahead: two register sets, two LDS
    // buffers, one barrier a step.  A load is issued on every path (past the end: the last columns once more), so the waits leave the
    // younger set in flight.
    bf16x8 pre_a[4], pre_b[4];
    auto gload = [&](int k0, bf16x8 (&pre)[4]) {
#pragma unroll
        for (int which = 0; which < 2; ++which)
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                const bf16* src = which ? wrow : xrow;
                const int kc = k0 + lc + half * 8;
                if constexpr (VEC) {
                    pre[which * 2 + half] = *reinterpret_cast<const bf16x8*>(src + min(kc, K - 8));
                } else {
                    bf16x8 v;
#pragma unroll
                    for (int e = 0; e < 8; ++e) v[e] = kc + e < K ? src[kc + e] : (bf16)0.f;
                    pre[which * 2 + half] = v;
                }
            }
    };
    auto step = [&](int k0, bf16* buf, bf16x8 (&pre)[4]) {
        bf16 *xs = buf, *ws = buf + GT * GLD;
#pragma unroll
        for (int which = 0; which < 2; ++which)
#pragma unroll
            for (int half = 0; half < 2; ++half)
                *reinterpret_cast<bf16x8*>((which ? ws : xs) + lr * GLD + lc + half * 8) = !VEC || k0 + lc + half * 8 < K ? pre[which * 2 + half] : bf16x8{};
        __syncthreads();
        gload(k0 + 2 * GK, pre);
#pragma unroll
        for (int ks = 0; ks < GK / 32; ++ks) {
            bf16x8 wf[2], xf[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                wf[i] = *reinterpret_cast<const bf16x8*>(ws + (wn + i * 16 + fr) * GLD + ks * 32 + fq * 8);
                xf[i] = *reinterpret_cast<const bf16x8*>(xs + (wm + i * 16 + fr) * GLD + ks * 32 + fq * 8);
            }
#pragma unroll
            for (int i = 0; i < 2; ++i)
#pragma unroll
                for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[i], xf[j], acc[i][j], 0, 0, 0);
        }
    };
    gload(0, pre_a);
    gload(GK, pre_b);
    int k0 = 0;
    for (; k0 + GK < K; k0 += 2 * GK) {
        step(k0, lds, pre_a);
        step(k0 + GK, lds + 2 * GT * GLD, pre_b);
    }
    if (k0 < K) step(k0, lds, pre_a);
    // lane holds, for weight tile i and row tile j: row m = wm + 16 j + fr, columns n = wn + 16 i + 4 fq + e
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int r = wm + j * 16 + fr;
            if (r >= rm.rows) continue;
            const int64_t m = rm.dst(r);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = n0 + wn + i * 16 + fq * 4 + e;
                if (n >= N) continue;
                const float v = epi(acc[i][j][e], m, n);
                if constexpr (OUT_F32) ((float*)yv)[m * ldy + n] = v;
                else ((bf16*)yv)[m * ldy + n] = (bf16)v;
            }
        }
}

template <bool OUT_F32>
__device__ __forceinline__ void gemm_any_bf16_tile(const bf16* __restrict__ x, int64_t ldx, const bf16* __restrict__ w, int64_t ldw,
                                                   const bf16* __restrict__ bias, void* __restrict__ yv, int64_t ldy, const RowMap rm, int n0, int N, int K,
                                                   int vec_ok, const bf16* __restrict__ gate = nullptr, int64_t ldg = 0, int relu2 = 0) {
    __shared__ __attribute__((aligned(16))) bf16 lds[4 * GT * GLD];
    const Epilogue epi{bias, gate, ldg, relu2};
    if (vec_ok) gemm_any_bf16_tile_body<OUT_F32, true>(x, ldx, w, ldw, yv, ldy, rm, n0, N, K, epi, lds);
    else gemm_any_bf16_tile_body<OUT_F32, false>(x, ldx, w, ldw, yv, ldy, rm, n0, N, K, epi, lds);
}

// The same tile when few of its rows are real (at most 16 NR; K a multiple of 32, 16-byte rows): a wave takes 16 columns and all rows, the
// operands go from memory to the matrix cores without LDS, U products of 32 ahead, so what a wave waits for is the weights' stream and
// not a barrier a step.  Sums in the same order as above: bit for bit the same results.
template <bool OUT_F32, int NR>
__device__ __forceinline__ void gemm_any_bf16_few_rows(const bf16* __restrict__ x, int64_t ldx, const bf16* __restrict__ w, int64_t ldw, void* __restrict__ yv,
                                                       int64_t ldy, const RowMap rm, int n0, int N, int K, const Epilogue epi) {
    constexpr int U = NR == 1 ? 8 : 4;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, fr = lane & 15, fq = lane >> 4;
    const int nw = n0 + wave * 16;
    if (nw >= N) return;
    const bf16* wp = w + (int64_t)min(nw + fr, N - 1) * ldw + fq * 8;
    const bf16* xp[NR];
    f32x4 acc[NR];
#pragma unroll
    for (int j = 0; j < NR; ++j) {
        xp[j] = x + rm.src(min(16 * j + fr, rm.rows - 1)) * ldx + fq * 8;
        acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    bf16x8 wa[U], xa[U][NR], wb[U], xb[U][NR];
    auto load = [&](int k0, bf16x8 (&wf)[U], bf16x8 (&xf)[U][NR]) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = min(k0 + 32 * u, K - 32);
            wf[u] = *reinterpret_cast<const bf16x8*>(wp + k);
#pragma unroll
            for (int j = 0; j < NR; ++j) xf[u][j] = *reinterpret_cast<const bf16x8*>(xp[j] + k);
        }
    };
    auto multiply = [&](int k0, bf16x8 (&wf)[U], bf16x8 (&xf)[U][NR]) {
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (k0 + 32 * u < K)
#pragma unroll
                for (int j = 0; j < NR; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[u], xf[u][j], acc[j], 0, 0, 0);
    };
    load(0, wa, xa);
    for (int k0 = 0; k0 < K; k0 += 64 * U) {
        load(k0 + 32 * U, wb, xb);
        multiply(k0, wa, xa);
        load(k0 + 64 * U, wa, xa);
        multiply(k0 + 32 * U, wb, xb);
    }
#pragma unroll
    for (int j = 0; j < NR; ++j) {
        const int r = 16 * j + fr;
        if (r >= rm.rows) continue;
        const int64_t m = rm.dst(r);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = nw + fq * 4 + e;
            if (n >= N) continue;
            const float v = epi(acc[j][e], m, n);
            if constexpr (OUT_F32) ((float*)yv)[m * ldy + n] = v;
            else ((bf16*)yv)[m * ldy + n] = (bf16)v;
        }
    }
}

__device__ __forceinline__ void gemm_any_f32_tile(const float* __restrict__ x, int64_t ldx, const float* __restrict__ w, int64_t ldw,
                                                  const float* __restrict__ bias, float* __restrict__ y, int64_t ldy, const RowMap rm, int n0, int N, int K,
                                                  const float* __restrict__ gate = nullptr, int64_t ldg = 0, int relu2 = 0) {
    constexpr int BK = 16;
    __shared__ float xs[BK][GT + 4];
    __shared__ float ws[BK][GT + 4];
    const int tid = threadIdx.x;
    const int tm = (tid >> 4) * 4, tn = (tid & 15) * 4;
    float acc[4][4] = {};
    const int lr = tid >> 2, lc = (tid & 3) * 4;             // 64 rows x 16 columns per stage: 4 consecutive k per thread
    const int64_t xrow = lr < rm.rows ? rm.src(lr) : 0;
    for (int k0 = 0; k0 < K; k0 += BK) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int k = k0 + lc + e;
            xs[lc + e][lr] = (lr < rm.rows && k < K) ? x[xrow * ldx + k] : 0.f;
            ws[lc + e][lr] = (n0 + lr < N && k < K) ? w[(int64_t)(n0 + lr) * ldw + k] : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < BK; ++k) {
            float a[4], b[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                a[e] = xs[k][tm + e];
                b[e] = ws[k][tn + e];
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_fmaf(a[i], b[j], acc[i][j]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = n0 + tn + j;
            if (tm + i < rm.rows && n < N) {
                const int64_t m = rm.dst(tm + i);
                float v = acc[i][j] + (bias ? bias[n] : 0.f);
                if (gate) v *= sigmoid(gate[m * ldg + n]);
                if (relu2) {
                    v = fmaxf(v, 0.f);
                    v *= v;
                }
                y[m * ldy + n] = v;
            }
        }
}

}  // namespace nvh_any
