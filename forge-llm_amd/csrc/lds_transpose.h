// A wave's "8 elements per lane" fragment of 16 rows, laid down transposed in LDS.
#pragma once

#include "dense.h"

namespace fh {

// f: row r0 + l16, columns c0 + 8 lg .. + 7  ->  dst[c0 + 8 lg + e][r0 + l16], rows of STRIDE elements.
template <typename T, uint32_t STRIDE>
__device__ __forceinline__ void lay_down_transposed(T* dst, const typename Vec<T>::x8& f, uint32_t c0, uint32_t r0, uint32_t l16, uint32_t lg) {
    if constexpr (sizeof(T) == 2) {
        // pairs of rows: the even lane writes elements 0..3 of both rows, the odd lane 4..7
        const uint4 b = __builtin_bit_cast(uint4, f);
        const bool odd = l16 & 1;
        const uint32_t give0 = odd ? b.x : b.z, give1 = odd ? b.y : b.w;
        const uint32_t got0 = lane_xor<1>(give0), got1 = lane_xor<1>(give1);
        const uint32_t mine0 = odd ? b.z : b.x, mine1 = odd ? b.w : b.y;
        const uint32_t e0 = odd ? got0 : mine0, e1 = odd ? got1 : mine1;      // even row
        const uint32_t d0 = odd ? mine0 : got0, d1 = odd ? mine1 : got1;      // odd row
        uint32_t* at = reinterpret_cast<uint32_t*>(dst + (c0 + 8 * lg + (odd ? 4 : 0)) * STRIDE + r0 + (l16 & ~1u));
        at[0 * (STRIDE / 2)] = __builtin_amdgcn_perm(d0, e0, 0x05040100u);
        at[1 * (STRIDE / 2)] = __builtin_amdgcn_perm(d0, e0, 0x07060302u);
        at[2 * (STRIDE / 2)] = __builtin_amdgcn_perm(d1, e1, 0x05040100u);
        at[3 * (STRIDE / 2)] = __builtin_amdgcn_perm(d1, e1, 0x07060302u);
    } else {
#pragma unroll
        for (int e = 0; e < 8; e++) dst[(c0 + 8 * lg + e) * STRIDE + r0 + l16] = f[e];
    }
}

}  // namespace fh
