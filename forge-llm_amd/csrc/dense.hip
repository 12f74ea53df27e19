// Products with dense matrices (bfloat16 or 32-bit), y = a W^T, and the small kernels around them.
//
// M > 1: tiles on the matrix unit.  Workgroup = 4 waves (2 x 2), each TN x TM tiles of 32 x 32; the weights are the MFMA A operand,
// so a lane ends up with four consecutive columns n of one row m and the epilogue writes them at once (and has pairs of columns,
// rotary pairs and gate / up, in one lane).  A stage of 128 bytes of depth (64 bfloat16, 32 floats) goes from global memory
// straight into one of two LDS buffers while the other one is worked; LDS rows are 128 bytes, the 16-byte piece c of row r at
// position c ^ ((r >> 1) & 7), which keeps the fragment reads free of bank conflicts.  Rows past the end of a matrix read as
// zero through the buffer descriptors' range check.
// M = 1: dense_gemv.h.
#include <hip/hip_runtime.h>

#include <type_traits>

#include "common.h"
#include "dense.h"
#include "dense_gemv.h"
#include "device_utils.h"

namespace fh {

constexpr uint32_t ROW_BYTES = 128;
constexpr uint32_t DENSE_RSRC_FLAGS = 0x00020000;   // raw buffer, 32-bit data format
constexpr uint32_t DENSE_K_MAX = 32768;             // a GEMV keeps its vector as floats in LDS

#define FH_LDS3(p) ((__attribute__((address_space(3))) void*)(p))

template <typename T, int TN, int TM, DenseEpi MODE>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2)))
void dense_gemm_kernel(const T* __restrict__ w, const T* __restrict__ a, uint32_t lda, uint32_t M, uint32_t N, uint32_t K, uint32_t tiles_n,
                       DenseEpiArgs e) {
    extern __shared__ __attribute__((aligned(16))) uint8_t dense_lds[];
    constexpr uint32_t BN = 64 * TN, BM = 64 * TM, BK = ROW_BYTES / sizeof(T), ES = sizeof(T);
    constexpr uint32_t BUF = (BN + BM) * ROW_BYTES;
    const uint32_t tid = threadIdx.x, lane = tid & 63;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    const uint32_t wn = wave & 1, wm = wave >> 1, lrow = lane & 31, lh = lane >> 5;
    // Workgroups go round robin over the 8 XCDs: give each XCD a run of neighbouring tiles (they share operand rows in its L2).
    uint32_t tile = blockIdx.x;
    {
        const uint32_t total = gridDim.x, per = total / 8, x = tile % 8, i = tile / 8;
        if (i < per) tile = x * per + i;          // the last total % 8 tiles stay where they are
    }
    const uint32_t n0 = (tile % tiles_n) * BN, m0 = (tile / tiles_n) * BM;
    const uint32_t stages = K / BK;

    const __amdgpu_buffer_rsrc_t rw = __builtin_amdgcn_make_buffer_rsrc((void*)(w + (size_t)n0 * K), 0, min(N - n0, BN) * K * ES, DENSE_RSRC_FLAGS);
    const __amdgpu_buffer_rsrc_t ra =
        __builtin_amdgcn_make_buffer_rsrc((void*)(a + (size_t)m0 * lda), 0, ((min(M - m0, BM) - 1) * lda + K) * ES, DENSE_RSRC_FLAGS);
    // load i of wave v fills LDS rows (4 i + v) * 8 .. + 8, lane -> (row, position)
    const uint32_t ld_row = wave * 8 + (lane >> 3);
    const uint32_t ld_piece = (lane & 7) ^ ((ld_row >> 1) & 7);       // rows 32 i further on have the same swizzle
    const uint32_t w_off = ld_row * K * ES + ld_piece * 16, a_off = ld_row * lda * ES + ld_piece * 16;
    auto issue = [&](uint32_t stage, uint32_t buf) {
        uint8_t* base = dense_lds + buf * BUF + wave * 1024;
        const uint32_t k = stage * ROW_BYTES;
#pragma unroll
        for (uint32_t i = 0; i < BN / 32; i++)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(rw, FH_LDS3(base + i * 4096), 16, w_off + i * 32 * K * ES, k, 0, 0);
#pragma unroll
        for (uint32_t i = 0; i < BM / 32; i++)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(ra, FH_LDS3(base + BN * ROW_BYTES + i * 4096), 16, a_off + i * 32 * lda * ES, k, 0, 0);
    };
    v16f acc[TN][TM];
#pragma unroll
    for (int i = 0; i < TN; i++)
#pragma unroll
        for (int j = 0; j < TM; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) acc[i][j][r] = 0.f;

    const uint32_t sw = (lrow >> 1) & 7;
    auto frag = [&](const uint8_t* row, uint32_t kk) {
        if constexpr (sizeof(T) == 2) return *reinterpret_cast<const v8bf*>(row + (((2 * kk + lh) ^ sw) * 16));
        else {
            const v4f lo = *reinterpret_cast<const v4f*>(row + (((4 * kk + 2 * lh) ^ sw) * 16));
            const v4f hi = *reinterpret_cast<const v4f*>(row + (((4 * kk + 2 * lh + 1) ^ sw) * 16));
            return (v8f){lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
        }
    };
    issue(0, 0);
    __builtin_amdgcn_s_waitcnt(0);
    __syncthreads();
    for (uint32_t st = 0; st < stages; st++) {
        const uint32_t buf = st & 1;
        if (st + 1 < stages) issue(st + 1, buf ^ 1);
        const uint8_t* wb = dense_lds + buf * BUF + (wn * 32 * TN + lrow) * ROW_BYTES;
        const uint8_t* ab = dense_lds + buf * BUF + (BN + wm * 32 * TM + lrow) * ROW_BYTES;
#pragma unroll
        for (uint32_t kk = 0; kk < BK / 16; kk++) {
            typename Vec<T>::x8 fw[TN], fa[TM];
#pragma unroll
            for (int i = 0; i < TN; i++) fw[i] = frag(wb + i * 32 * ROW_BYTES, kk);
#pragma unroll
            for (int j = 0; j < TM; j++) fa[j] = frag(ab + j * 32 * ROW_BYTES, kk);
#pragma unroll
            for (int i = 0; i < TN; i++)
#pragma unroll
                for (int j = 0; j < TM; j++) acc[i][j] = mma32(fw[i], fa[j], acc[i][j]);
        }
        __builtin_amdgcn_s_waitcnt(0);          // the next stage's tiles are in LDS
        __syncthreads();
    }
#pragma unroll
    for (int j = 0; j < TM; j++) {
        const uint32_t m = m0 + (wm * TM + j) * 32 + lrow;
        if (m >= M) continue;
#pragma unroll
        for (int i = 0; i < TN; i++)
#pragma unroll
            for (int g = 0; g < 4; g++) {
                const uint32_t n = n0 + (wn * TN + i) * 32 + 8 * g + 4 * lh;
                if (n >= N) continue;
                const float v[4] = {acc[i][j][4 * g], acc[i][j][4 * g + 1], acc[i][j][4 * g + 2], acc[i][j][4 * g + 3]};
                dense_epilogue<T, MODE>(e, m, n, N, v);
            }
    }
}

// The vector of a one-row product goes into LDS as floats, made from what DenseIn names.
template <typename T, int KS, DenseEpi MODE, DenseIn::Kind IN>
__global__ __launch_bounds__(GEMV_THREADS) void dense_gemv_kernel(const T* __restrict__ w, DenseIn in, uint32_t N, uint32_t K, DenseEpiArgs e) {
    extern __shared__ __attribute__((aligned(16))) float gemv_lds[];
    const uint32_t tid = threadIdx.x;
    float* xs = gemv_lds;
    float* red = gemv_lds + K;
    gemv_body<T, KS, MODE>(w, N, K, blockIdx.x * gemv_rows<KS>(), xs, red, e, [&]() {
        if constexpr (IN == DenseIn::Rows) {
            const T* a = (const T*)in.rows;
            for (uint32_t k = tid * 8; k < K; k += GEMV_THREADS * 8) {
                const typename Vec<T>::x8 v = load8(a + k);
#pragma unroll
                for (int j = 0; j < 8; j++) xs[k + j] = (float)v[j];
            }
        } else if constexpr (IN == DenseIn::Normed) {
            // a thread keeps to its own elements until the product's barrier
            float s = 0.f;
            for (uint32_t k = tid * 4; k < K; k += GEMV_THREADS * 4) {
                const v4f v = *reinterpret_cast<const v4f*>(in.f32 + k);
                *reinterpret_cast<v4f*>(xs + k) = v;
                s += (v[0] + v[1]) + (v[2] + v[3]);                       // zero past ln.n
            }
            const float mean = block_sum(s, red, tid, GEMV_THREADS) / (float)in.ln.n;
            float ss = 0.f;
            for (uint32_t k = tid * 4; k < K; k += GEMV_THREADS * 4)
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    const float d = xs[k + j] - mean;
                    if (k + j < in.ln.n) ss = fmaf(d, d, ss);
                }
            const float inv = 1.0f / sqrtf(block_sum(ss, red, tid, GEMV_THREADS) / (float)in.ln.n + in.ln.eps);
            for (uint32_t k = tid * 4; k < K; k += GEMV_THREADS * 4) {
                const v4f lw = *reinterpret_cast<const v4f*>(in.ln.w + k), lb = *reinterpret_cast<const v4f*>(in.ln.b + k);
#pragma unroll
                for (int j = 0; j < 4; j++) xs[k + j] = (xs[k + j] - mean) * inv * lw[j] + lb[j];
            }
        } else {
            // head = a multiple of 32 columns: lane group of 16, 4 columns per lane and step
            const uint32_t n = in.heads * in.head;
            for (uint32_t k = n + tid; k < K; k += GEMV_THREADS) xs[k] = 0.f;
            for (uint32_t h = tid / 16; h < in.heads; h += GEMV_THREADS / 16) {
                const float* o = in.f32 + h * in.head;
                float ss = 0.f;
                for (uint32_t c = tid % 16 * 4; c < in.head; c += 64) {
                    const v4f v = *reinterpret_cast<const v4f*>(o + c);
#pragma unroll
                    for (int j = 0; j < 4; j++) ss = fmaf(v[j], v[j], ss);      // zero past head_n
                }
                ss = lane_xor_add<8>(ss); ss = lane_xor_add<4>(ss); ss = lane_xor_add<2>(ss); ss = lane_xor_add<1>(ss);
                const float inv = 1.0f / sqrtf(ss / (float)in.head_n + in.eps);
                for (uint32_t c = tid % 16 * 4; c < in.head; c += 64) {
                    const v4f v = *reinterpret_cast<const v4f*>(o + c), hw = *reinterpret_cast<const v4f*>(in.w + c);
                    const typename Vec<T>::x4 g = *reinterpret_cast<const typename Vec<T>::x4*>((const T*)in.gate + h * in.head + c);
#pragma unroll
                    for (int j = 0; j < 4; j++) xs[h * in.head + c + j] = v[j] * inv * hw[j] * (float)g[j];
                }
            }
        }
    });
}

// One workgroup per row; a thread holds NV groups of four elements.
template <typename T, int NV>
__global__ __launch_bounds__(256) void layer_norm_kernel(const float* __restrict__ x, uint32_t ldx, LayerNorm ln, uint32_t width, T* __restrict__ out, uint32_t ld_out) {
    __shared__ float red[4];
    const uint32_t m = blockIdx.x, tid = threadIdx.x;
    v4f v[NV];
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const uint32_t c = (tid + 256 * i) * 4;
        v[i] = c < width ? *reinterpret_cast<const v4f*>(x + (size_t)m * ldx + c) : (v4f){0.f, 0.f, 0.f, 0.f};
        s += (v[i][0] + v[i][1]) + (v[i][2] + v[i][3]);                  // zero past ln.n
    }
    const float mean = block_sum(s, red, tid, 256) / (float)ln.n;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const float d = v[i][j] - mean;
            if ((tid + 256 * i) * 4 + j < ln.n) ss = fmaf(d, d, ss);
        }
    const float inv = 1.0f / sqrtf(block_sum(ss, red, tid, 256) / (float)ln.n + ln.eps);
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const uint32_t c = (tid + 256 * i) * 4;
        if (c >= width) continue;
        const v4f w = *reinterpret_cast<const v4f*>(ln.w + c), b = *reinterpret_cast<const v4f*>(ln.b + c);
        float y[4];
#pragma unroll
        for (int j = 0; j < 4; j++) y[j] = (v[i][j] - mean) * inv * w[j] + b[j];
        store4<T>(out + (size_t)m * ld_out + c, y[0], y[1], y[2], y[3]);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void dense_embedding_kernel(const T* __restrict__ table, uint32_t ld_table, uint32_t width, float scale, const uint32_t* __restrict__ tokens,
                                                              float* __restrict__ x, uint32_t ldx, DynTanh next, T* __restrict__ out, uint32_t ld_out,
                                                              T* __restrict__ out2, uint32_t ld_out2, uint32_t* __restrict__ counts) {
    const uint32_t m = blockIdx.y, tok = tokens[m], i = blockIdx.x * 256 + threadIdx.x;
    if (i < ldx) {
        const float v = i < width ? (float)table[(size_t)tok * ld_table + i] * scale : 0.f;
        x[(size_t)m * ldx + i] = v;
        if (out) out[(size_t)m * ld_out + i] = (T)dyn_tanh(next, i, v);
        if (out2) out2[(size_t)m * ld_out2 + i] = (T)v;
    }
    if (i == 0 && counts) atomicAdd(counts + tok, 1u);
}

template <typename T>
__global__ __launch_bounds__(256) void gather_rows_kernel(const T* __restrict__ a, uint32_t lda, const uint32_t* __restrict__ rows, uint32_t width,
                                                          T* __restrict__ out, uint32_t ld_out) {
    const T* src = a + (size_t)rows[blockIdx.x] * lda;
    for (uint32_t i = threadIdx.x; i < width; i += blockDim.x) out[(size_t)blockIdx.x * ld_out + i] = src[i];
}

namespace {

template <typename T, int TN, int TM, DenseEpi MODE>
void go_gemm(const DenseWeight& w, const void* a, uint32_t lda, uint32_t M, const DenseEpiArgs& e, hipStream_t s) {
    constexpr uint32_t lds = (64 * TN + 64 * TM) * ROW_BYTES * 2;
    static const hipError_t lds_ok = hipFuncSetAttribute((const void*)dense_gemm_kernel<T, TN, TM, MODE>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)lds_ok;
    const uint32_t tn = (w.N + 64 * TN - 1) / (64 * TN), tm = (M + 64 * TM - 1) / (64 * TM);
    fh::launch(dense_gemm_kernel<T, TN, TM, MODE>, dim3(tn * tm), 256, lds, s, (const T*)w.p, (const T*)a, lda, M, w.N, w.K, tn, e);
}

template <typename T, int KS, DenseEpi MODE, DenseIn::Kind IN>
void go_gemv(const DenseWeight& w, const DenseIn& in, const DenseEpiArgs& e, hipStream_t s) {
    static const hipError_t lds_ok = hipFuncSetAttribute((const void*)dense_gemv_kernel<T, KS, MODE, IN>, hipFuncAttributeMaxDynamicSharedMemorySize, (DENSE_K_MAX + 16) * 4);
    (void)lds_ok;
    fh::launch(dense_gemv_kernel<T, KS, MODE, IN>, dim3((w.N + gemv_rows<KS>() - 1) / gemv_rows<KS>()), GEMV_THREADS, (w.K + 16) * 4, s, (const T*)w.p,
               in, w.N, w.K, e);
}

template <typename T, DenseEpi MODE, DenseIn::Kind IN>
void go_row(const DenseWeight& w, const DenseIn& in, const DenseEpiArgs& e, hipStream_t s) {
    switch (gemv_depth_split(w.N, w.K)) {
        case 1: go_gemv<T, 1, MODE, IN>(w, in, e, s); return;
        case 2: go_gemv<T, 2, MODE, IN>(w, in, e, s); return;
        default: go_gemv<T, 4, MODE, IN>(w, in, e, s); return;
    }
}

template <typename T, DenseEpi MODE>
void go(const DenseWeight& w, const DenseIn& in, uint32_t M, const DenseEpiArgs& e, hipStream_t s) {
    if (M == 1) {
        if constexpr (MODE == DenseEpi::RawGate || MODE == DenseEpi::ActPair)
            if (in.kind == DenseIn::Normed) { go_row<T, MODE, DenseIn::Normed>(w, in, e, s); return; }
        if constexpr (MODE == DenseEpi::Residual)
            if (in.kind == DenseIn::HeadGate) { go_row<T, MODE, DenseIn::HeadGate>(w, in, e, s); return; }
        if constexpr (MODE != DenseEpi::Rope && MODE != DenseEpi::Split && MODE != DenseEpi::GateMul) { go_row<T, MODE, DenseIn::Rows>(w, in, e, s); return; }
    }
    const void* a = in.rows;
    const uint32_t lda = in.lda;
    // the large tile when its tiles give most compute units work, else the small one
    const uint64_t big = (uint64_t)((w.N + 127) / 128) * ((M + 127) / 128);
    if (big >= 192) go_gemm<T, 2, 2, MODE>(w, a, lda, M, e, s);
    else go_gemm<T, 1, 1, MODE>(w, a, lda, M, e, s);
}

template <typename T>
void by_mode(const DenseWeight& w, const DenseIn& in, uint32_t M, DenseEpi mode, const DenseEpiArgs& e, hipStream_t s) {
    switch (mode) {
        case DenseEpi::F32: go<T, DenseEpi::F32>(w, in, M, e, s); break;
        case DenseEpi::RawGate: go<T, DenseEpi::RawGate>(w, in, M, e, s); break;
        case DenseEpi::Rope: go<T, DenseEpi::Rope>(w, in, M, e, s); break;
        case DenseEpi::Split: go<T, DenseEpi::Split>(w, in, M, e, s); break;
        case DenseEpi::GateMul: go<T, DenseEpi::GateMul>(w, in, M, e, s); break;
        case DenseEpi::ActPair: go<T, DenseEpi::ActPair>(w, in, M, e, s); break;
        case DenseEpi::Residual: go<T, DenseEpi::Residual>(w, in, M, e, s); break;
    }
}

}  // namespace

uint32_t dense_k_max() { return DENSE_K_MAX; }

void launch_dense(DType t, const DenseWeight& w, const DenseIn& in, uint32_t M, DenseEpi mode, const DenseEpiArgs& e, hipStream_t s) {
    if (M == 0 || w.N == 0) return;
    if (t == DType::BF16) by_mode<__bf16>(w, in, M, mode, e, s);
    else by_mode<float>(w, in, M, mode, e, s);
}

namespace {

template <typename T>
void layer_norm(const float* x, uint32_t ldx, const LayerNorm& ln, uint32_t width, uint32_t M, void* out, uint32_t ld_out, hipStream_t s) {
    auto go = [&](auto kernel) { fh::launch(kernel, dim3(M), 256, 0, s, x, ldx, ln, width, (T*)out, ld_out); };
    if (width <= 1024) go(layer_norm_kernel<T, 1>);
    else if (width <= 2048) go(layer_norm_kernel<T, 2>);
    else if (width <= 4096) go(layer_norm_kernel<T, 4>);
    else go(layer_norm_kernel<T, 16>);
}

}  // namespace

void launch_layer_norm(DType t, const float* x, uint32_t ldx, const LayerNorm& ln, uint32_t width, uint32_t M, void* out, uint32_t ld_out, hipStream_t s) {
    if (t == DType::BF16) layer_norm<__bf16>(x, ldx, ln, width, M, out, ld_out, s);
    else layer_norm<float>(x, ldx, ln, width, M, out, ld_out, s);
}

void launch_dense_embedding(DType t, const void* table, uint32_t ld_table, uint32_t width, float scale, const uint32_t* tokens_dev, uint32_t M, float* x,
                            uint32_t ldx, const DynTanh& next, void* out, uint32_t ld_out, void* out2, uint32_t ld_out2, uint32_t* counts, hipStream_t s) {
    if (t == DType::BF16)
        fh::launch(dense_embedding_kernel<__bf16>, dim3((ldx + 255) / 256, M), 256, 0, s, (const __bf16*)table, ld_table, width, scale, tokens_dev, x, ldx, next, (__bf16*)out, ld_out,
                   (__bf16*)out2, ld_out2, counts);
    else
        fh::launch(dense_embedding_kernel<float>, dim3((ldx + 255) / 256, M), 256, 0, s, (const float*)table, ld_table, width, scale, tokens_dev, x, ldx, next, (float*)out, ld_out,
                   (float*)out2, ld_out2, counts);
}

void launch_gather_rows(DType t, const void* a, uint32_t lda, const uint32_t* rows_dev, uint32_t n, uint32_t width, void* out, uint32_t ld_out, hipStream_t s) {
    if (t == DType::BF16) fh::launch(gather_rows_kernel<__bf16>, dim3(n), 256, 0, s, (const __bf16*)a, lda, rows_dev, width, (__bf16*)out, ld_out);
    else fh::launch(gather_rows_kernel<float>, dim3(n), 256, 0, s, (const float*)a, lda, rows_dev, width, (float*)out, ld_out);
}

}  // namespace fh
