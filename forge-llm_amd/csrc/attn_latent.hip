// Latent attention: per position the cache holds one latent vector c (RMS-normed) and one rotated key part that all heads share;
// a head's unrotated key and its value are W_uk c and W_uv c.  An optional window keeps the last `window` positions visible.
//
// Prompt rows work on expanded keys and values (a product of the cached latents with [W_uk; W_uv] ahead of attn_prompt.hip): per
// (query, key) pair that is dim + rot + vdim multiply-adds against 2 rank + rot on the latents.  Decode works on the latents
// themselves: the query goes through W_uk^T once, every head then attends to the same cached row, which is read once for 16
// heads, and the weighted latents go through W_uv once.
//
// T: __bf16 or float (dense.h); scores, softmax and sums are 32-bit in both.
#include <hip/hip_runtime.h>

#include "common.h"
#include "dense.h"
#include "dense_gemv.h"
#include "device_utils.h"
#include "lds_transpose.h"

namespace fh {

constexpr float LOG2E = 1.4426950408889634f;
constexpr float NO_KEYS = -3.0e38f;          // maximum of a part without keys: weight 0, and finite where another layer's records overlap it
constexpr uint32_t RANK_MAX = 1024, SPLITS_MAX = 64;

// ---- the new cache row and the normed query latent of one position; `tid` of `nt` threads, red: LDS, nt / 64 floats -----------------
template <typename T>
__device__ __forceinline__ void store_cache_row(const LatentShape& sh, const float* raw, const float* kv_norm, const float* cos_t, const float* sin_t,
                                                uint32_t pos, T* cache, float* red, uint32_t tid, uint32_t nt) {
    const float* c = raw + sh.q_rank;
    const float* kr = c + sh.rank;
    float ss = 0.f;
    for (uint32_t i = tid; i < sh.rank; i += nt) ss = fmaf(c[i], c[i], ss);      // padding is zero
    const float inv = 1.0f / sqrtf(block_sum(ss, red, tid, nt) / (float)sh.rank_n + sh.eps);
    T* row = cache + (size_t)pos * sh.cache_row();
    for (uint32_t i = tid; i < sh.rank; i += nt) row[i] = (T)(c[i] * inv * kv_norm[i]);
    for (uint32_t i = tid; i < sh.rot / 2; i += nt) {
        float u = kr[2 * i], v = kr[2 * i + 1];
        if (i < sh.rot_pairs) {
            const float cs = cos_t[(size_t)pos * sh.rot_pairs + i], sn = sin_t[(size_t)pos * sh.rot_pairs + i];
            const float u2 = u * cs - v * sn;
            v = v * cs + u * sn;
            u = u2;
        }
        row[sh.rank + 2 * i] = (T)u;
        row[sh.rank + 2 * i + 1] = (T)v;
    }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_norm_store_kernel(LatentShape sh, const float* __restrict__ raw, const float* __restrict__ q_norm,
                                                                const float* __restrict__ kv_norm, const float* __restrict__ cos_t,
                                                                const float* __restrict__ sin_t, uint32_t base_pos, T* __restrict__ cq, T* __restrict__ cache) {
    __shared__ float red[4];
    const uint32_t m = blockIdx.x, tid = threadIdx.x;
    const float* row = raw + (size_t)m * sh.raw_row();
    float ss = 0.f;
    for (uint32_t i = tid; i < sh.q_rank; i += 256) ss = fmaf(row[i], row[i], ss);
    const float inv = 1.0f / sqrtf(block_sum(ss, red, tid, 256) / (float)sh.q_rank_n + sh.eps);
    for (uint32_t i = tid; i < sh.q_rank; i += 256) cq[(size_t)m * sh.q_rank + i] = (T)(row[i] * inv * q_norm[i]);
    store_cache_row<T>(sh, row, kv_norm, cos_t, sin_t, base_pos + m, cache, red, tid, 256);
}

// ---- decode ----------------------------------------------------------------------------------------------------------------
// [RMS norm of the query latent | W_uq | rotation]; the last workgroup writes the position's cache row instead.
template <typename T, int KS>
__global__ __launch_bounds__(GEMV_THREADS) void latent_query_kernel(LatentShape sh, const float* __restrict__ raw, const float* __restrict__ q_norm,
                                                                    const float* __restrict__ kv_norm, const T* __restrict__ uq, DenseEpiArgs e,
                                                                    T* __restrict__ cache) {
    extern __shared__ __attribute__((aligned(16))) float lq_lds[];
    const uint32_t tid = threadIdx.x, K = sh.q_rank;
    float* xs = lq_lds;
    float* red = lq_lds + K;
    if (blockIdx.x == gridDim.x - 1) {
        store_cache_row<T>(sh, raw, kv_norm, e.cos_t, e.sin_t, e.pos_dev ? *e.pos_dev : e.base_pos, cache, red, tid, GEMV_THREADS);
        return;
    }
    gemv_body<T, KS, DenseEpi::Rope>(uq, sh.q_row(), K, blockIdx.x * gemv_rows<KS>(), xs, red, e, [&]() {
        float ss = 0.f;
        for (uint32_t i = tid; i < K; i += GEMV_THREADS) ss = fmaf(raw[i], raw[i], ss);
        const float inv = 1.0f / sqrtf(block_sum(ss, red, tid, GEMV_THREADS) / (float)sh.q_rank_n + sh.eps);
        for (uint32_t i = tid; i < K; i += GEMV_THREADS) xs[i] = raw[i] * inv * q_norm[i];
    });
}

// ql[head][r] = sum_d q[head][d] W_uk[head dim + d][r].  Workgroup = (64 columns, head): a wave reads 8 rows of 64 columns at a time.
template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentShape sh, const T* __restrict__ q, const T* __restrict__ uk, T* __restrict__ ql) {
    __shared__ float part[32][64];
    const uint32_t tid = threadIdx.x, lane8 = tid & 7, drow = tid >> 3, head = blockIdx.y, r0 = blockIdx.x * 64;
    const T* qh = q + head * (sh.dim + sh.rot);
    const T* w = uk + (size_t)head * sh.dim * sh.rank + r0 + lane8 * 8;
    float acc[8];
#pragma unroll
    for (int j = 0; j < 8; j++) acc[j] = 0.f;
    for (uint32_t d = drow; d < sh.dim; d += 32) {
        const typename Vec<T>::x8 v = load8(w + (size_t)d * sh.rank);
        const float x = (float)qh[d];
#pragma unroll
        for (int j = 0; j < 8; j++) acc[j] = fmaf((float)v[j], x, acc[j]);
    }
#pragma unroll
    for (int j = 0; j < 8; j++) part[drow][lane8 * 8 + j] = acc[j];
    __syncthreads();
    if (tid < 64) {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < 32; i++) s += part[i][tid];
        ql[(size_t)head * sh.rank + r0 + tid] = (T)s;
    }
}

// Attention of one row over the cached latents, 16 heads per workgroup: part blockIdx.x of the visible keys, heads 16 blockIdx.y...
// A tile is 16 NW keys; wave w computes the scores of 16 of them (straight from the cache rows in registers, which it also lays
// down transposed in LDS), and then the weighted latents of its share of the rank.  parts[part][head][rank + 2]: sums, maximum
// (base 2), weight sum.
template <typename T, int NW, int MAXT>
__global__ __launch_bounds__(NW * 64) void latent_attn_decode_kernel(LatentShape sh, const T* __restrict__ q, const T* __restrict__ ql, const T* __restrict__ cache,
                                                                     float* __restrict__ parts, uint32_t base_pos, const uint32_t* __restrict__ pos_dev) {
    typedef typename Vec<T>::x8 x8;
    constexpr uint32_t KT = 16 * NW, PAD = 16 / sizeof(T), VS = KT + PAD;
    constexpr uint32_t KSTEPS = KT / 32;
    static_assert(KT % 32 == 0, "the second product works 32 keys at a time");
    static_assert(SPLITS_MAX == 64, "the parts' weights are made by one wave");
    extern __shared__ __attribute__((aligned(16))) uint8_t ld_lds[];
    T* Ct = reinterpret_cast<T*>(ld_lds);                   // [rank][VS]
    T* P = Ct + sh.rank * VS;                               // [16][VS]
    float* smax = reinterpret_cast<float*>(P + 16 * VS);    // [NW][16]
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const uint32_t pos = pos_dev ? *pos_dev : base_pos;
    const uint32_t lo = sh.window && pos >= sh.window ? pos - sh.window + 1 : 0;
    const uint32_t nk = pos + 1 - lo, ntiles = (nk + KT - 1) / KT, per = (ntiles + gridDim.x - 1) / gridDim.x;
    const uint32_t t0 = blockIdx.x * per, t1 = min(t0 + per, ntiles);
    const uint32_t head = blockIdx.y * 16 + l16, hq = min(head, sh.heads - 1);
    const uint32_t NS = sh.cache_row() / 32, NSR = sh.rank / 32;
    const T* qn = ql + (size_t)hq * sh.rank + 8 * lg;
    const T* qr = q + (size_t)hq * (sh.dim + sh.rot) + sh.dim + 8 * lg;
    const float c2 = sh.scale * LOG2E;
    const uint32_t rtiles = sh.rank / 16;

    v4f o[MAXT];
#pragma unroll
    for (int i = 0; i < MAXT; i++) o[i] = (v4f){0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;

    for (uint32_t tile = t0; tile < t1; tile++) {
        const uint32_t tk = lo + tile * KT + wave * 16;          // the wave's first key
        const T* row = cache + (size_t)min(tk + l16, pos) * sh.cache_row() + 8 * lg;
        v4f sacc = (v4f){0.f, 0.f, 0.f, 0.f};
        auto lay_down = [&](uint32_t s, const x8& f) { lay_down_transposed<T, VS>(Ct, f, 32 * s, 16 * wave, l16, lg); };
        // bfloat16: a whole row of up to 512 latents is requested at once, with the first rotated dimensions
        constexpr uint32_t U = sizeof(T) == 2 ? (MAXT * NW / 2 < 16 ? MAXT * NW / 2 : 16) : 2;
        constexpr uint32_t UR = 2;
        x8 fr[UR], gr[UR];
#pragma unroll
        for (uint32_t u = 0; u < UR; u++) {
            const bool in = NSR + u < NS;
            fr[u] = in ? load8(row + 32 * (NSR + u)) : zero8<T>();
            gr[u] = in ? load8(qr + 32 * u) : zero8<T>();
        }
        for (uint32_t s = 0; s < NSR; s += U) {
            x8 f[U], g[U];
#pragma unroll
            for (uint32_t u = 0; u < U; u++)
                if (s + u < NSR) { f[u] = load8(row + 32 * (s + u)); g[u] = load8(qn + 32 * (s + u)); }
#pragma unroll
            for (uint32_t u = 0; u < U; u++)
                if (s + u < NSR) { sacc = mma16(f[u], g[u], sacc); lay_down(s + u, f[u]); }
        }
#pragma unroll
        for (uint32_t u = 0; u < UR; u++) sacc = mma16(fr[u], gr[u], sacc);
        for (uint32_t s = NSR + UR; s < NS; s++) sacc = mma16(load8(row + 32 * s), load8(qr + 32 * (s - NSR)), sacc);
        // register r: key tk + 4 lg + r, this lane's head
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
        for (int w = 0; w < NW; w++) m_new = fmaxf(m_new, smax[w * 16 + l16]);
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
        for (int i = 0; i < MAXT; i++) {
            const uint32_t rt = wave + i * NW;
            if (rt < rtiles) {
                o[i] *= alpha;
#pragma unroll
                for (uint32_t k = 0; k < KSTEPS; k++)
                    o[i] = mma16(load8(Ct + (rt * 16 + l16) * VS + 32 * k + 8 * lg), load8(P + l16 * VS + 32 * k + 8 * lg), o[i]);
            }
        }
        __syncthreads();
    }
    float* rec = parts + ((size_t)blockIdx.x * sh.heads + hq) * (sh.rank + 4);
    l_run = lane_xor_add<32>(lane_xor_add<16>(l_run));
    if (lane < 16) smax[wave * 16 + l16] = l_run;
    __syncthreads();
    if (head < sh.heads) {
        if (t0 < t1) {
#pragma unroll
            for (int i = 0; i < MAXT; i++) {
                const uint32_t rt = wave + i * NW;
                if (rt < rtiles) *reinterpret_cast<v4f*>(rec + rt * 16 + 4 * lg) = o[i];
            }
        }
        if (tid < 16) {
            float l = 0.f;
            for (int w = 0; w < NW; w++) l += smax[w * 16 + l16];
            rec[sh.rank] = t0 < t1 ? m_run : NO_KEYS;
            rec[sh.rank + 1] = l;
        }
    }
}

// [merge of the parts | W_uv | gate]: a workgroup's rows belong to one head.
template <typename T>
__global__ __launch_bounds__(GEMV_THREADS) void latent_value_kernel(LatentShape sh, const float* __restrict__ parts, uint32_t nparts, const T* __restrict__ uv, DenseEpiArgs e) {
    extern __shared__ __attribute__((aligned(16))) float lv_lds[];
    // the workgroups of a head are `heads` apart: with a multiple of 8 heads they sit on one XCD and share the parts in its L2
    const uint32_t tid = threadIdx.x, K = sh.rank, head = blockIdx.x % sh.heads;
    const uint32_t row0 = head * sh.vdim + blockIdx.x / sh.heads * gemv_rows<1>();
    float* xs = lv_lds;
    float* red = lv_lds + K;
    float* wt = red + 16;           // [SPLITS_MAX]
    gemv_body<T, 1, DenseEpi::GateMul>(uv, sh.heads * sh.vdim, K, row0, xs, red, e, [&]() {
        const size_t step = (size_t)sh.heads * (sh.rank + 4);
        const float* rec = parts + (size_t)head * (sh.rank + 4);
        // the first sums are requested ahead of the statistics they are weighted with
        constexpr uint32_t B = 32;
        float2 r[B];
        auto fetch = [&](uint32_t p0, uint32_t i) {
#pragma unroll
            for (uint32_t p = 0; p < B; p++) r[p] = *reinterpret_cast<const float2*>(rec + min(p0 + p, nparts - 1) * step + i);
        };
        if (tid * 2 < K) fetch(0, tid * 2);
        if (tid < 64) {
            const float m = tid < nparts ? rec[tid * step + sh.rank] : -INFINITY;
            const float ls = tid < nparts ? rec[tid * step + sh.rank + 1] : 0.f;
            const float mx = wave_max(m);
            const float w = __builtin_amdgcn_exp2f(m - mx);          // mx is finite: some part holds keys
            const float l = wave_sum(w * ls);
            wt[tid] = w / l;                                         // 0 past the last part
        }
        __syncthreads();
        for (uint32_t i = tid * 2; i < K; i += GEMV_THREADS * 2) {
            float v0 = 0.f, v1 = 0.f;
            for (uint32_t p0 = 0; p0 < nparts; p0 += B) {
                if (p0 || i != tid * 2) fetch(p0, i);
#pragma unroll
                for (uint32_t p = 0; p < B; p++) {
                    v0 = fmaf(wt[p0 + p], r[p].x, v0);
                    v1 = fmaf(wt[p0 + p], r[p].y, v1);
                }
            }
            xs[i] = v0;
            xs[i + 1] = v1;
        }
    });
}

namespace {

template <typename T, int NW, int MAXT>
void go_decode(const LatentShape& sh, const LatentDecodeIo& io, hipStream_t s) {
    constexpr uint32_t VS = 16 * NW + 16 / sizeof(T);
    static const hipError_t ok = hipFuncSetAttribute((const void*)latent_attn_decode_kernel<T, NW, MAXT>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    (void)ok;
    const uint32_t lds = (sh.rank + 16) * VS * sizeof(T) + NW * 16 * 4;
    fh::launch(latent_attn_decode_kernel<T, NW, MAXT>, dim3(latent_splits(sh, io.max_seq), (sh.heads + 15) / 16), NW * 64, lds, s, sh, (const T*)io.q,
               (const T*)io.ql, (const T*)io.cache, io.parts, io.base_pos, io.pos_dev);
}

template <typename T, int KS>
void go_query(const LatentShape& sh, const LatentDecodeIo& io, const DenseEpiArgs& e, hipStream_t s) {
    static const hipError_t ok = hipFuncSetAttribute((const void*)latent_query_kernel<T, KS>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    (void)ok;
    fh::launch(latent_query_kernel<T, KS>, dim3((sh.q_row() + gemv_rows<KS>() - 1) / gemv_rows<KS>() + 1), GEMV_THREADS, (sh.q_rank + 16) * 4, s, sh, io.raw,
               io.q_norm, io.kv_norm, (const T*)io.uq.p, e, (T*)io.cache);
}

template <typename T>
void query(const LatentShape& sh, const LatentDecodeIo& io, hipStream_t s) {
    DenseEpiArgs e;
    e.out = io.q;
    e.ld_out = sh.q_row();
    e.cos_t = io.cos_t;
    e.sin_t = io.sin_t;
    e.base_pos = io.base_pos;
    e.pos_dev = io.pos_dev;
    e.head_stride = sh.dim + sh.rot;
    e.rot_off = sh.dim;
    e.rot_pairs = sh.rot_pairs;
    switch (gemv_depth_split(sh.q_row(), sh.q_rank)) {
        case 1: go_query<T, 1>(sh, io, e, s); break;
        case 2: go_query<T, 2>(sh, io, e, s); break;
        default: go_query<T, 4>(sh, io, e, s); break;
    }
}

template <typename T>
void decode(const LatentShape& sh, const LatentDecodeIo& io, hipStream_t s) {
    fh::launch(latent_absorb_kernel<T>, dim3(sh.rank / 64, sh.heads), 256, 0, s, sh, (const T*)io.q, (const T*)io.ukv.p, (T*)io.ql);
    if constexpr (sizeof(T) == 2) {
        if (sh.rank <= 128) go_decode<T, 4, 2>(sh, io, s);
        else if (sh.rank <= 512) go_decode<T, 4, 8>(sh, io, s);
        else go_decode<T, 4, 16>(sh, io, s);
    } else {
        if (sh.rank <= 128) go_decode<T, 4, 2>(sh, io, s);
        else if (sh.rank <= 512) go_decode<T, 4, 8>(sh, io, s);
        else go_decode<T, 2, 32>(sh, io, s);
    }
    DenseEpiArgs e;
    e.out = io.out;
    e.gate = io.gate;
    // the 16 rows of a workgroup lie in one head (vdim is a multiple of 32); every workgroup merges its head's parts, so few of them
    const T* uv = (const T*)io.ukv.p + (size_t)sh.heads * sh.dim * sh.rank;
    const uint32_t N = sh.heads * sh.vdim, lds = (sh.rank + 16 + SPLITS_MAX) * 4, np = latent_splits(sh, io.max_seq);
    fh::launch(latent_value_kernel<T>, dim3(N / gemv_rows<1>()), GEMV_THREADS, lds, s, sh, io.parts, np, uv, e);
}

}  // namespace

bool latent_shape_supported(DType, const LatentShape& sh) {
    return sh.dim + sh.rot <= DENSE_HEAD_MAX && sh.vdim <= DENSE_HEAD_MAX && sh.rank <= RANK_MAX && sh.q_rank <= dense_k_max();
}

uint32_t latent_splits(const LatentShape& sh, uint32_t max_seq) {
    const uint32_t keys = sh.window && sh.window < max_seq ? sh.window : max_seq;
    return std::max(1u, std::min(SPLITS_MAX, (keys + 63) / 64));
}

size_t latent_parts_bytes(const LatentShape& sh, uint32_t max_seq) {
    return (size_t)latent_splits(sh, max_seq) * sh.heads * (sh.rank + 4) * 4;
}

void launch_latent_norm_store(DType t, const LatentShape& sh, const float* raw, const float* q_norm, const float* kv_norm, const float* cos_t,
                              const float* sin_t, uint32_t M, uint32_t base_pos, void* cq, void* cache, hipStream_t s) {
    if (t == DType::BF16)
        fh::launch(latent_norm_store_kernel<__bf16>, dim3(M), 256, 0, s, sh, raw, q_norm, kv_norm, cos_t, sin_t, base_pos, (__bf16*)cq, (__bf16*)cache);
    else
        fh::launch(latent_norm_store_kernel<float>, dim3(M), 256, 0, s, sh, raw, q_norm, kv_norm, cos_t, sin_t, base_pos, (float*)cq, (float*)cache);
}

void launch_latent_query(DType t, const LatentShape& sh, const LatentDecodeIo& io, hipStream_t s) {
    if (t == DType::BF16) query<__bf16>(sh, io, s);
    else query<float>(sh, io, s);
}

void launch_latent_attn_decode(DType t, const LatentShape& sh, const LatentDecodeIo& io, hipStream_t s) {
    if (t == DType::BF16) decode<__bf16>(sh, io, s);
    else decode<float>(sh, io, s);
}

}  // namespace fh
