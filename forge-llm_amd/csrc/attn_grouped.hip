// Grouped-query attention whose query and key heads are RMS-normed and rotated: norms, the cache and the decode step.  (A prompt's
// rows attend in attn_prompt.hip.)  The raw projections come in 32-bit; norms, rotation, scores and softmax are 32-bit, q and the
// cache are T.
#include <hip/hip_runtime.h>

#include "common.h"
#include "dense.h"
#include "device_utils.h"
#include "lds_transpose.h"

namespace fh {

constexpr float LOG2E = 1.4426950408889634f;
constexpr float NO_KEYS = -3.0e38f;          // maximum of a part without keys: weight 0
constexpr uint32_t GA_NW = 4, GA_KT = 16 * GA_NW, GA_SPLITS_MAX = 64;

// Sum over groups of LANES lanes.
template <int LANES> __device__ __forceinline__ float group_sum(float v) {
    static_assert(LANES == 16 || LANES == 32 || LANES == 64, "power of two up to the wave");
    if (LANES >= 64) v = lane_xor_add<32>(v);
    if (LANES >= 32) v = lane_xor_add<16>(v);
    return lane_xor_add<1>(lane_xor_add<2>(lane_xor_add<4>(lane_xor_add<8>(v))));
}

// One head of `dim` raw elements by a group of LANES >= dim / 4 lanes, of which this one is number `sub`: norm, rotation of the pairs
// (2 i, 2 i + 1), i < pairs, store as T.
template <typename T, int LANES>
__device__ __forceinline__ void norm_rotate_head(const float* __restrict__ raw, const float* __restrict__ w, uint32_t dim, uint32_t dim_n, float eps,
                                                 const float* __restrict__ ct, const float* __restrict__ st, uint32_t pairs, T* out, uint32_t sub) {
    const bool in = 4 * sub < dim;
    v4f v = (v4f){0.f, 0.f, 0.f, 0.f}, nw = v;
    float c[2] = {1.f, 1.f}, s[2] = {0.f, 0.f};
    if (in) {
        v = *reinterpret_cast<const v4f*>(raw + 4 * sub);                // zero past dim_n
        nw = *reinterpret_cast<const v4f*>(w + 4 * sub);
#pragma unroll
        for (uint32_t i = 0; i < 2; i++)
            if (2 * sub + i < pairs) { c[i] = ct[2 * sub + i]; s[i] = st[2 * sub + i]; }
    }
    const float inv = 1.0f / sqrtf(group_sum<LANES>((v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3])) / (float)dim_n + eps);
    if (!in) return;
    v *= inv;
    v *= nw;
    store4<T>(out + 4 * sub, v[0] * c[0] - v[1] * s[0], v[1] * c[0] + v[0] * s[0], v[2] * c[1] - v[3] * s[1], v[3] * c[1] + v[2] * s[1]);
}

// One workgroup per row: 256 / LANES heads at a time.
template <typename T, int LANES>
__global__ __launch_bounds__(256) void grouped_norm_store_kernel(GroupedShape sh, const float* __restrict__ raw, const float* __restrict__ q_norm,
                                                                 const float* __restrict__ k_norm, const float* __restrict__ cos_t,
                                                                 const float* __restrict__ sin_t, uint32_t base_pos, T* __restrict__ q,
                                                                 T* __restrict__ kc, T* __restrict__ vc) {
    const uint32_t m = blockIdx.x, tid = threadIdx.x, sub = tid % LANES, pos = base_pos + m;
    const float* row = raw + (size_t)m * sh.raw_row();
    const float* ct = cos_t + (size_t)pos * sh.rot_pairs;
    const float* st = sin_t + (size_t)pos * sh.rot_pairs;
    // the keys' heads follow the queries'
    for (uint32_t h = tid / LANES; h < sh.heads + sh.kv_heads; h += 256 / LANES) {
        const bool query = h < sh.heads;
        T* out = query ? q + ((size_t)m * sh.heads + h) * sh.dim : kc + (size_t)pos * sh.k_row() + (h - sh.heads) * sh.dim;
        norm_rotate_head<T, LANES>(row + h * sh.dim, query ? q_norm : k_norm, sh.dim, sh.dim_n, sh.eps, ct, st, sh.rot_pairs, out, sub);
    }
    const float* vr = row + (sh.heads + sh.kv_heads) * sh.dim;
    for (uint32_t i = tid * 4; i < sh.v_row(); i += 1024) {
        const float4 v = *reinterpret_cast<const float4*>(vr + i);
        store4<T>(vc + (size_t)pos * sh.v_row() + i, v.x, v.y, v.z, v.w);
    }
}

// Attention of one row: part blockIdx.x of the keys for up to 16 query heads of one key / value head.  A tile is 64 keys; wave w
// computes the scores of 16 of them straight from the cache rows and lays their values down transposed in LDS, then weighs its share
// of the value columns.  The part that holds the row's own position writes its cache row first (every part norms its queries).
// parts[part][head][vdim + 4]: sums, maximum (base 2), weight sum.  DK, DV: pieces of 32 of a key and of a value row, at least.
template <typename T, int DK, int DV>
__global__ __launch_bounds__(GA_NW * 64) void grouped_decode_kernel(GroupedShape sh, const float* __restrict__ raw, const float* __restrict__ q_norm,
                                                                    const float* __restrict__ k_norm, const float* __restrict__ cos_t,
                                                                    const float* __restrict__ sin_t, T* kc, T* vc, float* __restrict__ parts,
                                                                    uint32_t base_pos, const uint32_t* __restrict__ pos_dev) {
    typedef typename Vec<T>::x8 x8;
    constexpr uint32_t NW = GA_NW, KT = GA_KT, PAD = 16 / sizeof(T), VS = KT + PAD, MAXT = (2 * DV + NW - 1) / NW;
    constexpr uint32_t LANES = 8 * DK;                      // that norm one head
    extern __shared__ __attribute__((aligned(16))) uint8_t ga_lds[];
    const uint32_t QS = sh.dim + PAD;
    T* Vt = reinterpret_cast<T*>(ga_lds);                   // [vdim][VS]
    T* P = Vt + sh.vdim * VS;                               // [16][VS]
    T* Q = P + 16 * VS;                                     // [16][QS]
    float* smax = reinterpret_cast<float*>(Q + 16 * QS);    // [NW][16]
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const uint32_t pos = pos_dev ? *pos_dev : base_pos;
    const uint32_t ntiles = pos / KT + 1, per = (ntiles + gridDim.x - 1) / gridDim.x;
    const uint32_t t0 = blockIdx.x * per, t1 = min(t0 + per, ntiles);
    const uint32_t group = sh.group(), hb = (group + 15) / 16;
    const uint32_t kvh = blockIdx.y / hb, h0 = kvh * group + blockIdx.y % hb * 16, nh = min(16u, (kvh + 1) * group - h0);
    float* rec0 = parts + ((size_t)blockIdx.x * sh.heads + h0) * (sh.vdim + 4);
    if (t0 >= t1) {
        if (tid < nh) {
            rec0[tid * (sh.vdim + 4) + sh.vdim] = NO_KEYS;
            rec0[tid * (sh.vdim + 4) + sh.vdim + 1] = 0.f;
        }
        return;
    }
    const uint32_t nk = sh.dim / 32, nv = sh.vdim / 32;
    const T* krow0 = kc + kvh * sh.dim + 8 * lg;
    const T* vrow0 = vc + kvh * sh.vdim + 8 * lg;
    const bool fresh = t1 == ntiles;                        // this part holds the row's own position
    // rows other than the fresh one are there already: the first tile is requested ahead of the norms
    x8 kf[DK], vf[DV];
    auto fetch = [&](uint32_t tile) {
        const size_t row = min(tile * KT + wave * 16 + l16, pos);
#pragma unroll
        for (uint32_t s = 0; s < DK; s++) kf[s] = s < nk ? load8(krow0 + row * sh.k_row() + 32 * s) : zero8<T>();
#pragma unroll
        for (uint32_t s = 0; s < DV; s++) vf[s] = s < nv ? load8(vrow0 + row * sh.v_row() + 32 * s) : zero8<T>();
    };
    const bool early = t0 + 1 < ntiles;                     // the first tile is not the one with the fresh row
    if (early) fetch(t0);
    const float* ct = cos_t + (size_t)pos * sh.rot_pairs;
    const float* st = sin_t + (size_t)pos * sh.rot_pairs;
    if (fresh) {
        const float* kr = raw + sh.heads * sh.dim;
        if (wave == NW - 1 && lane < LANES)
            norm_rotate_head<T, LANES>(kr + kvh * sh.dim, k_norm, sh.dim, sh.dim_n, sh.eps, ct, st, sh.rot_pairs, kc + (size_t)pos * sh.k_row() + kvh * sh.dim, lane);
        const float* vr = kr + sh.k_row() + kvh * sh.vdim;
        if (wave == NW - 2)
            for (uint32_t i = lane; i < sh.vdim; i += 64) vc[(size_t)pos * sh.v_row() + kvh * sh.vdim + i] = (T)vr[i];
    }
#pragma unroll
    for (uint32_t i = 0; i < 16 * LANES / (NW * 64); i++) {
        const uint32_t h = tid / LANES + i * (NW * 64 / LANES), sub = tid % LANES;
        if (h < nh) norm_rotate_head<T, LANES>(raw + (h0 + h) * sh.dim, q_norm, sh.dim, sh.dim_n, sh.eps, ct, st, sh.rot_pairs, Q + h * QS, sub);
        else if (4 * sub < sh.dim) store4<T>(Q + h * QS + 4 * sub, 0.f, 0.f, 0.f, 0.f);
    }
    __syncthreads();
    if (!early) fetch(t0);
    const float c2 = sh.scale * LOG2E;
    const uint32_t rtiles = sh.vdim / 16;
    v4f o[MAXT];
#pragma unroll
    for (uint32_t i = 0; i < MAXT; i++) o[i] = (v4f){0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;

    for (uint32_t tile = t0; tile < t1; tile++) {
        const uint32_t tk = tile * KT + wave * 16;          // the wave's first key
        v4f sacc = (v4f){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (uint32_t s = 0; s < DK; s++)
            if (s < nk) sacc = mma16(kf[s], load8(Q + l16 * QS + 32 * s + 8 * lg), sacc);
#pragma unroll
        for (uint32_t s = 0; s < DV; s++)
            if (s < nv) lay_down_transposed<T, VS>(Vt, vf[s], 32 * s, 16 * wave, l16, lg);
        if (tile + 1 < t1) fetch(tile + 1);
        // register r: key tk + 4 lg + r, column l16: head h0 + l16
        float mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            sacc[r] = tk + 4 * lg + r <= pos ? sacc[r] * c2 : -INFINITY;
            mx = fmaxf(mx, sacc[r]);
        }
        mx = lane_xor_max<32>(lane_xor_max<16>(mx));
        if (lane < 16) smax[wave * 16 + l16] = mx;
        __syncthreads();
        float m_new = m_run;
#pragma unroll
        for (uint32_t w = 0; w < NW; w++) m_new = fmaxf(m_new, smax[w * 16 + l16]);
        // finite: the tile's first key is visible
        const float alpha = m_run == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m_run - m_new);
        m_run = m_new;
        float p[4];
        l_run *= alpha;
#pragma unroll
        for (int r = 0; r < 4; r++) { p[r] = __builtin_amdgcn_exp2f(sacc[r] - m_new); l_run += p[r]; }
        store4<T>(P + l16 * VS + 16 * wave + 4 * lg, p[0], p[1], p[2], p[3]);
        __syncthreads();
#pragma unroll
        for (uint32_t i = 0; i < MAXT; i++) {
            const uint32_t rt = wave + i * NW;
            if (rt < rtiles) {
                o[i] *= alpha;
#pragma unroll
                for (uint32_t k = 0; k < KT / 32; k++)
                    o[i] = mma16(load8(Vt + (rt * 16 + l16) * VS + 32 * k + 8 * lg), load8(P + l16 * VS + 32 * k + 8 * lg), o[i]);
            }
        }
        __syncthreads();
    }
    l_run = lane_xor_add<32>(lane_xor_add<16>(l_run));
    if (lane < 16) smax[wave * 16 + l16] = l_run;
    __syncthreads();
    if (l16 < nh) {
        float* rec = rec0 + l16 * (sh.vdim + 4);
#pragma unroll
        for (uint32_t i = 0; i < MAXT; i++) {
            const uint32_t rt = wave + i * NW;
            if (rt < rtiles) *reinterpret_cast<v4f*>(rec + rt * 16 + 4 * lg) = o[i];
        }
        if (tid < 16) {
            float l = 0.f;
            for (uint32_t w = 0; w < NW; w++) l += smax[w * 16 + l16];
            rec[sh.vdim] = m_run;
            rec[sh.vdim + 1] = l;
        }
    }
}

// [merge of the parts | gate], one workgroup (64 threads) per head and 64 value columns.  Sums of parts without keys are whatever an
// earlier step left there: finite, and weighted with 0.
template <typename T>
__global__ __launch_bounds__(64) void grouped_merge_kernel(const float* __restrict__ parts, uint32_t nparts, uint32_t heads, uint32_t vdim, const T* __restrict__ gate, T* __restrict__ out) {
    __shared__ float wt[GA_SPLITS_MAX];
    static_assert(GA_SPLITS_MAX == 64, "the parts' weights are made by one wave");
    const uint32_t lane = threadIdx.x, head = blockIdx.x, c = blockIdx.y * 64 + lane;
    const size_t step = (size_t)heads * (vdim + 4);
    const float* rec = parts + (size_t)head * (vdim + 4);
    const bool in = c < vdim;
    constexpr uint32_t B = 32;
    float r[B];
    auto fetch = [&](uint32_t p0) {
#pragma unroll
        for (uint32_t p = 0; p < B; p++) r[p] = in ? rec[min(p0 + p, nparts - 1) * step + c] : 0.f;
    };
    fetch(0);
    {
        const float m = lane < nparts ? rec[lane * step + vdim] : -INFINITY;
        const float ls = lane < nparts ? rec[lane * step + vdim + 1] : 0.f;
        const float w = __builtin_amdgcn_exp2f(m - wave_max(m));         // the maximum is finite: some part holds keys
        wt[lane] = w / wave_sum(w * ls);                                 // 0 past the last part
    }
    __syncthreads();
    float v = 0.f;
    for (uint32_t p0 = 0; p0 < nparts; p0 += B) {
        if (p0) fetch(p0);
#pragma unroll
        for (uint32_t p = 0; p < B; p++) v = fmaf(wt[p0 + p], r[p], v);
    }
    if (in) out[head * vdim + c] = (T)(v * (float)gate[head * vdim + c]);
}

namespace {

template <typename T, int DK, int DV>
void go(const GroupedShape& sh, const GroupedIo& io, float* parts, hipStream_t s) {
    constexpr uint32_t PAD = 16 / sizeof(T), VS = GA_KT + PAD;
    static const hipError_t ok = hipFuncSetAttribute((const void*)grouped_decode_kernel<T, DK, DV>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    (void)ok;
    const uint32_t lds = ((sh.vdim + 16) * VS + 16 * (sh.dim + PAD)) * sizeof(T) + GA_NW * 16 * 4;
    fh::launch(grouped_decode_kernel<T, DK, DV>, dim3(grouped_splits(sh, io.max_seq), sh.kv_heads * ((sh.group() + 15) / 16)), GA_NW * 64, lds, s, sh, io.raw,
               io.q_norm, io.k_norm, io.cos_t, io.sin_t, (T*)io.k_cache, (T*)io.v_cache, parts, io.base_pos, io.pos_dev);
}

template <typename T>
void decode(const GroupedShape& sh, const GroupedIo& io, float* parts, const void* gate, void* out, hipStream_t s) {
    const uint32_t d = std::max(sh.dim, sh.vdim);
    if (d <= 64) go<T, 2, 2>(sh, io, parts, s);
    else if (d <= 128) go<T, 4, 4>(sh, io, parts, s);
    else go<T, 8, 8>(sh, io, parts, s);
    fh::launch(grouped_merge_kernel<T>, dim3(sh.heads, (sh.vdim + 63) / 64), 64, 0, s, parts, grouped_splits(sh, io.max_seq), sh.heads, sh.vdim, (const T*)gate, (T*)out);
}

template <typename T>
void norm_store(const GroupedShape& sh, const GroupedIo& io, uint32_t M, void* q, hipStream_t s) {
    auto go = [&](auto kernel) {
        fh::launch(kernel, dim3(M), 256, 0, s, sh, io.raw, io.q_norm, io.k_norm, io.cos_t, io.sin_t, io.base_pos, (T*)q, (T*)io.k_cache, (T*)io.v_cache);
    };
    if (sh.dim <= 64) go(grouped_norm_store_kernel<T, 16>);
    else if (sh.dim <= 128) go(grouped_norm_store_kernel<T, 32>);
    else go(grouped_norm_store_kernel<T, 64>);
}

}  // namespace

uint32_t grouped_splits(const GroupedShape&, uint32_t max_seq) { return std::max(1u, std::min(GA_SPLITS_MAX, (max_seq + GA_KT - 1) / GA_KT)); }

size_t grouped_parts_bytes(const GroupedShape& sh, uint32_t max_seq) { return (size_t)grouped_splits(sh, max_seq) * sh.heads * (sh.vdim + 4) * 4; }

void launch_grouped_norm_store(DType t, const GroupedShape& sh, const GroupedIo& io, uint32_t M, void* q, hipStream_t s) {
    if (t == DType::BF16) norm_store<__bf16>(sh, io, M, q, s);
    else norm_store<float>(sh, io, M, q, s);
}

void launch_grouped_decode(DType t, const GroupedShape& sh, const GroupedIo& io, float* parts, const void* gate, void* out, hipStream_t s) {
    if (t == DType::BF16) decode<__bf16>(sh, io, parts, gate, out, s);
    else decode<float>(sh, io, parts, gate, out, s);
}

}  // namespace fh
