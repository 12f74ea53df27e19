// One row times a dense matrix: the body that the matrix-vector kernels share.  A wave works 4 consecutive matrix rows; KS waves
// split the depth of the same 4 rows (small matrices: enough loads in flight on every compute unit).  The first weights are
// requested before the prologue prepares the vector in LDS.
#pragma once

#include "dense.h"

namespace fh {

constexpr uint32_t GEMV_THREADS = 256;
template <int KS> constexpr uint32_t gemv_rows() { return 4 * (GEMV_THREADS / 64) / KS; }    // matrix rows of a workgroup

// xs: LDS, K floats, filled by `prologue`; red: LDS, 16 floats.
template <typename T, int KS, DenseEpi MODE, typename Prologue>
__device__ __forceinline__ void gemv_body(const T* __restrict__ w, uint32_t N, uint32_t K, uint32_t row0, float* xs, float* red,
                                          const DenseEpiArgs& e, Prologue prologue) {
    typedef typename Vec<T>::x8 x8;
    constexpr int U = sizeof(T) == 2 ? 2 : 1;
    constexpr uint32_t STEP = KS * 512;
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const uint32_t part = wave % KS, n0 = row0 + (wave / KS) * 4;
    const T* rows[4];
#pragma unroll
    for (int i = 0; i < 4; i++) rows[i] = w + (size_t)min(n0 + i, N - 1) * K;
    const uint32_t k_lane = (part * 64 + lane) * 8;
    auto fetch = [&](x8 (&v)[U][4], uint32_t k) {
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int i = 0; i < 4; i++) v[u][i] = k + u * STEP < K ? load8(rows[i] + k + u * STEP) : zero8<T>();
    };
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    auto add = [&](const x8 (&v)[U][4], uint32_t k) {
#pragma unroll
        for (int u = 0; u < U; u++) {
            if (k + u * STEP >= K) break;
            const v4f xa = *reinterpret_cast<const v4f*>(xs + k + u * STEP), xb = *reinterpret_cast<const v4f*>(xs + k + u * STEP + 4);
#pragma unroll
            for (int i = 0; i < 4; i++) {
#pragma unroll
                for (int j = 0; j < 4; j++) acc[i] = fmaf((float)v[u][i][j], xa[j], acc[i]);
#pragma unroll
                for (int j = 0; j < 4; j++) acc[i] = fmaf((float)v[u][i][4 + j], xb[j], acc[i]);
            }
        }
    };
    x8 cur[U][4], nxt[U][4];
    fetch(cur, k_lane);
    prologue();
    __syncthreads();
    for (uint32_t k = 0; k < K; k += U * STEP) {
        const bool more = k + U * STEP < K;
        if (more) fetch(nxt, k_lane + k + U * STEP);
        add(cur, k_lane + k);
        if (more) {
#pragma unroll
            for (int u = 0; u < U; u++)
#pragma unroll
                for (int i = 0; i < 4; i++) cur[u][i] = nxt[u][i];
        }
    }
#pragma unroll
    for (int i = 0; i < 4; i++) acc[i] = wave_sum(acc[i]);
    if (KS > 1) {
        if (lane == 0) {
#pragma unroll
            for (int i = 0; i < 4; i++) red[wave * 4 + i] = acc[i];
        }
        __syncthreads();
#pragma unroll
        for (int p = 1; p < KS; p++)
#pragma unroll
            for (int i = 0; i < 4; i++)
                if (part == 0) acc[i] += red[(wave + p) * 4 + i];
    }
    if (part == 0 && lane == 0 && n0 < N) dense_epilogue<T, MODE>(e, 0, n0, N, acc);
}

// Depth split of an N-row matrix: as many waves per row group as it takes to have a few workgroups on every compute unit.
inline int gemv_depth_split(uint32_t N, uint32_t K) {
    if (N / 16 >= 768 || K <= 512) return 1;
    if (N / 8 >= 768 || K <= 1024) return 2;
    return 4;
}

}  // namespace fh
