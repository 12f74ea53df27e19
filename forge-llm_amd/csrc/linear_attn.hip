// Gated linear attention (a recurrence with a decay per key channel), all in 32-bit for both storage types:
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   a_t = sigmoid(W2 low_t + b)^(1 / tau).
//
// One row: linear_step_kernel.  A prompt's rows go in chunks of 64 tokens, each cut into four pieces of 16, in three launches:
//   chunk:  the decays; per chunk the state it adds, sum_j (decay from j to the chunk's end * k_j) v_j^T, and its whole decay;
//   scan:   the state ahead of every chunk, one after the other (elementwise);
//   output: o = decayed q against the state ahead of the chunk + the chunk's own pairs (t, j), then the heads' RMS norm and the gate.
//
// Every decay between two tokens is a product of numbers <= 1 of exactly the steps between them (running products inside a
// piece, from the start or to the end; products of whole pieces between pieces), never a quotient: nothing overflows or cancels
// however strong the decay.  Pairs inside a piece are worked on the vector unit (no factorization over (t, j) is safe there), all
// other products on the matrix unit in single precision.
#include <hip/hip_runtime.h>

#include "common.h"
#include "dense.h"
#include "device_utils.h"

namespace fh {

constexpr uint32_t LA_CHUNK = 64, LA_PIECE = 16, LA_PIECES = LA_CHUNK / LA_PIECE;
constexpr uint32_t LA_LS = LA_CHUNK + 4;     // LDS row stride in floats
constexpr uint32_t LA_MAX = 256;             // dim and vdim
constexpr uint32_t LA_RANK_MAX = 128, LA_RANK_STEP = 16;

__device__ __forceinline__ float decay_of(float z, float inv_tau) {
    // log sigmoid(z) = min(z, 0) - log(1 + e^-|z|)
    return expf((fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau);
}

// ---- one row -----------------------------------------------------------------------------------------------------------------
// Workgroup = (head, 32 value columns): 8 lanes of 4 columns, 32 row groups; a thread updates rows rg, rg + 32, ... (R of them).
template <int R>
__global__ __launch_bounds__(256) void linear_step_kernel(LinearShape sh, const float* __restrict__ raw, const float* __restrict__ w2, const float* __restrict__ b2,
                                                          float* __restrict__ state, float* __restrict__ o, uint32_t base_pos, const uint32_t* __restrict__ pos_dev) {
    __shared__ float as[LA_MAX], qs[LA_MAX], ks[LA_MAX];
    __shared__ v4f part[4][8];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, head = blockIdx.x, c0 = blockIdx.y * 32 + (tid & 7) * 4, rg = tid >> 3;
    const uint32_t pos = pos_dev ? *pos_dev : base_pos;
    float* S = state + (size_t)head * sh.dim * sh.vdim + c0;
    v4f s[R];
#pragma unroll
    for (int i = 0; i < R; i++) {
        const uint32_t d = rg + 32 * i;
        s[i] = pos && d < sh.dim ? *reinterpret_cast<const v4f*>(S + (size_t)d * sh.vdim) : (v4f){0.f, 0.f, 0.f, 0.f};
    }
    const v4f v = *reinterpret_cast<const v4f*>(raw + 2 * sh.qk() + head * sh.vdim + c0);
    if (tid < sh.dim) {
        const uint32_t ch = head * sh.dim + tid;
        const float* low = raw + 2 * sh.qk() + sh.heads * sh.vdim;
        float z = b2[ch];
#pragma unroll 8
        for (uint32_t r = 0; r < sh.rank; r++) z = fmaf(w2[(size_t)r * sh.qk() + ch], low[r], z);
        as[tid] = decay_of(z, sh.inv_tau);
        qs[tid] = raw[ch] * sh.q_scale;
        ks[tid] = raw[sh.qk() + ch];
    }
    __syncthreads();
    v4f acc = (v4f){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < R; i++) {
        const uint32_t d = rg + 32 * i;
        if (d >= sh.dim) continue;
        const float a = as[d], k = ks[d], q = qs[d];
#pragma unroll
        for (int j = 0; j < 4; j++) {
            s[i][j] = fmaf(a, s[i][j], k * v[j]);
            acc[j] = fmaf(q, s[i][j], acc[j]);
        }
        *reinterpret_cast<v4f*>(S + (size_t)d * sh.vdim) = s[i];
    }
#pragma unroll
    for (int j = 0; j < 4; j++) acc[j] = lane_xor_add<32>(lane_xor_add<16>(lane_xor_add<8>(acc[j])));
    if (lane < 8) part[wave][lane] = acc;
    __syncthreads();
    if (tid < 8) *reinterpret_cast<v4f*>(o + head * sh.vdim + c0) = (part[0][tid] + part[1][tid]) + (part[2][tid] + part[3][tid]);
}

// ---- prompt -------------------------------------------------------------------------------------------------------------------
// `rows` rows of `width` floats, ld apart, as a buffer: what lies past the last row reads as zero.  Offsets are in bytes.
__device__ __forceinline__ __amdgpu_buffer_rsrc_t rows_buffer(const float* p, uint32_t rows, uint32_t ld, uint32_t width) {
    return __builtin_amdgcn_make_buffer_rsrc((void*)p, 0, ((rows - 1) * ld + width) * 4, 0x00020000);
}
__device__ __forceinline__ float buffer_float(__amdgpu_buffer_rsrc_t b, uint32_t offset) {
    return __builtin_bit_cast(float, __builtin_amdgcn_raw_buffer_load_b32(b, offset, 0, 0));
}
// Eight values of one column, `step` bytes apart.
__device__ __forceinline__ v8f column8(__amdgpu_buffer_rsrc_t b, uint32_t offset, uint32_t step) {
    v8f f;
#pragma unroll
    for (uint32_t e = 0; e < 8; e++) f[e] = buffer_float(b, offset + e * step);
    return f;
}

// Workgroup = (chunk, head).  decay [M][heads * dim]; add [chunk][head][dim][vdim]; total [chunk][heads * dim].
__global__ __launch_bounds__(256) void linear_chunk_kernel(LinearShape sh, const float* __restrict__ raw, const float* __restrict__ w2, const float* __restrict__ b2,
                                                           uint32_t M, float* __restrict__ decay, float* __restrict__ add, float* __restrict__ total) {
    extern __shared__ __attribute__((aligned(16))) float lc_lds[];
    float* kt = lc_lds;                                       // [dim][LA_LS]: keys, decayed to their piece's end
    float* low = kt + sh.dim * LA_LS;                         // [64][rank + 4]
    float* dp = low + LA_CHUNK * (sh.rank + 4);               // [4][dim]: decay of a piece, then of all pieces behind it
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6)), lq = lane & 31, lh = lane >> 5;
    const uint32_t chunk = blockIdx.x, head = blockIdx.y, m0 = chunk * LA_CHUNK, rows = min(M - m0, LA_CHUNK), LR = sh.rank + 4, ld = sh.raw_row();
    const float* r0 = raw + (size_t)m0 * ld;
    const float* lowp = r0 + 2 * sh.qk() + sh.heads * sh.vdim;
    const uint32_t nv = sh.vdim / 32, n = nv * (sh.dim / 32);
    // the values of a tile; the wave's first are requested ahead of everything
    v8f vf[LA_PIECES];
    const __amdgpu_buffer_rsrc_t vbuf = rows_buffer(r0 + 2 * sh.qk() + head * sh.vdim, rows, ld, sh.vdim);
    auto fetch_values = [&](uint32_t i) {
#pragma unroll
        for (uint32_t s = 0; s < LA_PIECES; s++) vf[s] = column8(vbuf, ((16 * s + 8 * lh) * ld + i % nv * 32 + lq) * 4, ld * 4);
    };
    fetch_values(wave);
    // the keys of a channel over one piece, and the first of its row of the map
    const __amdgpu_buffer_rsrc_t kbuf = rows_buffer(r0 + sh.qk() + head * sh.dim, rows, ld, sh.dim);
    float k[LA_PIECE], w[LA_RANK_STEP], b;
    auto fetch_map = [&](uint32_t ch, uint32_t r) {
#pragma unroll
        for (uint32_t j = 0; j < LA_RANK_STEP; j++) w[j] = w2[(size_t)(r + j) * sh.qk() + ch];
    };
    auto fetch_channel = [&](uint32_t i) {
        const uint32_t c = i % sh.dim, t0 = i / sh.dim * LA_PIECE;
#pragma unroll
        for (uint32_t t = 0; t < LA_PIECE; t++) k[t] = buffer_float(kbuf, ((t0 + t) * ld + c) * 4);
        fetch_map(head * sh.dim + c, 0);
        b = b2[head * sh.dim + c];
    };
    if (tid < LA_PIECES * sh.dim) fetch_channel(tid);
    for (uint32_t i = tid; i < LA_CHUNK * (sh.rank / 4); i += 256) {
        const uint32_t t = i / (sh.rank / 4), c = i % (sh.rank / 4) * 4;
        *reinterpret_cast<v4f*>(low + t * LR + c) = t < rows ? *reinterpret_cast<const v4f*>(lowp + t * ld + c) : (v4f){0.f, 0.f, 0.f, 0.f};
    }
    __syncthreads();
    for (uint32_t i = tid; i < LA_PIECES * sh.dim; i += 256) {
        const uint32_t c = i % sh.dim, piece = i / sh.dim, ch = head * sh.dim + c, t0 = piece * LA_PIECE;
        float z[LA_PIECE];
        if (i != tid) fetch_channel(i);
#pragma unroll
        for (uint32_t t = 0; t < LA_PIECE; t++) z[t] = b;
        for (uint32_t r = 0; r < sh.rank; r += LA_RANK_STEP) {
            if (r) fetch_map(ch, r);
#pragma unroll
            for (uint32_t t = 0; t < LA_PIECE; t++)
#pragma unroll
                for (uint32_t g = 0; g < LA_RANK_STEP; g += 4) {
                    const v4f l = *reinterpret_cast<const v4f*>(low + (t0 + t) * LR + r + g);
#pragma unroll
                    for (uint32_t j = 0; j < 4; j++) z[t] = fmaf(w[g + j], l[j], z[t]);
                }
        }
#pragma unroll
        for (uint32_t t = 0; t < LA_PIECE; t++) {
            z[t] = t0 + t < rows ? decay_of(z[t], sh.inv_tau) : 1.f;
            if (t0 + t < rows) decay[(size_t)(m0 + t0 + t) * sh.qk() + ch] = z[t];
        }
        float p = 1.f;
#pragma unroll
        for (int t = LA_PIECE - 1; t >= 0; t--) { k[t] *= p; p *= z[t]; }
#pragma unroll
        for (uint32_t t = 0; t < LA_PIECE; t += 4) *reinterpret_cast<v4f*>(kt + c * LA_LS + t0 + t) = (v4f){k[t], k[t + 1], k[t + 2], k[t + 3]};
        dp[piece * sh.dim + c] = p;
    }
    __syncthreads();
    for (uint32_t c = tid; c < sh.dim; c += 256) {
        float p = 1.f;
#pragma unroll
        for (int s = LA_PIECES - 1; s >= 0; s--) {
            const float d = dp[s * sh.dim + c];
            dp[s * sh.dim + c] = p;
            p *= d;
        }
        total[(size_t)chunk * sh.qk() + head * sh.dim + c] = p;
    }
    __syncthreads();
    for (uint32_t i = wave; i < n; i += 4) {
        const uint32_t ct = i / nv * 32, vt = i % nv * 32;
        v16f acc;
#pragma unroll
        for (int r = 0; r < 16; r++) acc[r] = 0.f;
#pragma unroll
        for (uint32_t s = 0; s < LA_PIECES; s++) {
            const v8f a = load8(kt + (ct + lq) * LA_LS + 16 * s + 8 * lh) * dp[s * sh.dim + ct + lq];
            acc = mma32(a, vf[s], acc);
        }
        if (i + 4 < n) fetch_values(i + 4);
        float* y = add + (((size_t)chunk * sh.heads + head) * sh.dim + ct) * sh.vdim + vt + lq;
#pragma unroll
        for (int r = 0; r < 16; r++) y[(size_t)(8 * (r >> 2) + 4 * lh + (r & 3)) * sh.vdim] = acc[r];
    }
}

// add[chunk] <- the state ahead of the chunk; state <- the one behind the last.  A thread owns one element.
__global__ __launch_bounds__(256) void linear_scan_kernel(LinearShape sh, uint32_t chunks, const float* __restrict__ total, float* add, float* state, uint32_t base_pos) {
    const size_t n = sh.state(), i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const float* d = total + i / sh.vdim;
    float s = base_pos ? state[i] : 0.f;
    constexpr uint32_t B = 16;
    for (uint32_t c0 = 0; c0 < chunks; c0 += B) {
        float x[B], f[B];
#pragma unroll
        for (uint32_t b = 0; b < B; b++) {
            const uint32_t c = min(c0 + b, chunks - 1);
            x[b] = add[c * n + i];
            f[b] = d[(size_t)c * sh.qk()];
        }
#pragma unroll
        for (uint32_t b = 0; b < B; b++) {
            if (c0 + b >= chunks) break;
            add[(c0 + b) * n + i] = s;
            s = fmaf(f[b], s, x[b]);
        }
    }
    state[i] = s;
}

// Workgroup = (chunk, head), key channels 64 at a time.  A wave owns one piece of 16 tokens (loading, its own pairs, the running
// products), then its share of the pieces' pairs and of the output tiles.  Outputs are computed transposed: a lane owns one token.
// TILES: output tiles of a wave, at least.
template <typename T, int TILES>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(TILES <= 2 ? 3 : 2))) void linear_output_kernel(LinearShape sh, const float* __restrict__ raw, const float* __restrict__ decay, const float* __restrict__ before,
                                                            uint32_t M, const float* __restrict__ norm, const T* __restrict__ gate, T* __restrict__ out, uint32_t ld_out) {
    __shared__ __attribute__((aligned(16))) float qs[LA_CHUNK * LA_LS], ks[LA_CHUNK * LA_LS], ps[LA_CHUNK * LA_LS];    // ps: decays, then the pairs' weights
    __shared__ __attribute__((aligned(16))) float ahead[LA_PIECES][64], between[3][64];      // decay of the pieces ahead in the chunk; of piece 1, of 2, of both
    typedef typename Vec<T>::x4 x4;
    constexpr uint32_t LS = LA_LS;
    constexpr int EARLY = 1;                                 // output tiles whose operands are requested early
    const uint32_t tid = threadIdx.x, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(tid >> 6));
    uint32_t lane = tid & 63;
    const uint32_t chunk = blockIdx.x, head = blockIdx.y, m0 = chunk * LA_CHUNK, rows = min(M - m0, LA_CHUNK), ld = sh.raw_row();
    const float* r0 = raw + (size_t)m0 * ld;
    const uint32_t nv = sh.vdim / 32, ntile = 2 * nv;        // tile i: value columns i % nv, tokens 32 (i / nv) ..
    const float* S = before + ((size_t)chunk * sh.heads + head) * sh.dim * sh.vdim;
    const __amdgpu_buffer_rsrc_t vbuf = rows_buffer(r0 + 2 * sh.qk() + head * sh.vdim, rows, ld, sh.vdim);

    v16f acc[TILES];
#pragma unroll
    for (int i = 0; i < TILES; i++)
#pragma unroll
        for (int r = 0; r < 16; r++) acc[i][r] = 0.f;
    float own[LA_PIECE / 4] = {};                            // pairs (t, j = lane / 4) of the wave's piece, t = lane % 4 + 4 i
    v4f cross[2] = {(v4f){0.f, 0.f, 0.f, 0.f}, (v4f){0.f, 0.f, 0.f, 0.f}};
    // Pairs of pieces (later, earlier) = (1,0) (2,1) (3,2) (2,0) (3,1) (3,0), one hex digit each from the right, and the row of `between`
    // that lies between them (3: nothing does).  A wave takes pairs `wave` and `wave + 4`.
    constexpr uint32_t LATER = 0x332321, EARLIER = 0x010210, BETWEEN = 0x210333;

    for (uint32_t s0 = 0; s0 < sh.dim; s0 += 64) {
        asm volatile("" : "+v"(lane));                       // else the offsets of all loads stay in registers from pass to pass
        const uint32_t sw = min(64u, sh.dim - s0), lq = lane & 31, lh = lane >> 5, l16 = lane & 15, lg = lane >> 4;
        {
            // past the last token, and past the head's channels, all three are zero
            const __amdgpu_buffer_rsrc_t qb = rows_buffer(r0 + head * sh.dim + s0, rows, ld, sw), kb = rows_buffer(r0 + sh.qk() + head * sh.dim + s0, rows, ld, sw),
                                         ab = rows_buffer(decay + (size_t)m0 * sh.qk() + head * sh.dim + s0, rows, sh.qk(), sw);
            const uint32_t out_of_range = lane < sw ? 0 : 0x40000000;
            const uint32_t q0 = (wave * LA_PIECE * ld + lane) * 4 + out_of_range, a0 = (wave * LA_PIECE * sh.qk() + lane) * 4 + out_of_range;
            float q[LA_PIECE], k[LA_PIECE], a[LA_PIECE];
#pragma unroll
            for (uint32_t i = 0; i < LA_PIECE; i++) {
                q[i] = buffer_float(qb, q0 + i * ld * 4) * sh.q_scale;
                k[i] = buffer_float(kb, q0 + i * ld * 4);
                a[i] = buffer_float(ab, a0 + i * sh.qk() * 4);
            }
#pragma unroll
            for (uint32_t i = 0; i < LA_PIECE; i++) {
                const uint32_t at = (wave * LA_PIECE + i) * LS + lane;
                qs[at] = q[i];
                ks[at] = k[i];
                ps[at] = a[i];
            }
        }
        // the state ahead of the chunk, for the output tiles: requested ahead of the pairs
        const __amdgpu_buffer_rsrc_t sbuf = rows_buffer(S + (size_t)s0 * sh.vdim, sw, sh.vdim, sh.vdim);
        auto state8 = [&](uint32_t n, uint32_t s) { return column8(sbuf, ((s + 8 * lh) * sh.vdim + n % nv * 32 + lq) * 4, sh.vdim * 4); };
        v8f sf[EARLY][4];
#pragma unroll
        for (int i = 0; i < EARLY; i++)
#pragma unroll
            for (uint32_t s = 0; s < 4; s++) sf[i][s] = state8(wave + 4 * i, 16 * s);
        __syncthreads();
        {
            const uint32_t j = lane >> 2, at = wave * LA_PIECE * LS + (lane & 3) * 16;
            v4f k[4], kp[4];
#pragma unroll
            for (int g = 0; g < 4; g++) {
                k[g] = *reinterpret_cast<const v4f*>(ks + at + j * LS + 4 * g);
                kp[g] = (v4f){0.f, 0.f, 0.f, 0.f};
            }
#pragma unroll
            for (uint32_t t4 = 0; t4 < LA_PIECE; t4 += 4)
#pragma unroll 1
                for (uint32_t t = t4; t < t4 + 4; t++) {
                    float w = 0.f;
#pragma unroll
                    for (int g = 0; g < 4; g++) {
                        const v4f a = *reinterpret_cast<const v4f*>(ps + at + t * LS + 4 * g), q = *reinterpret_cast<const v4f*>(qs + at + t * LS + 4 * g);
#pragma unroll
                        for (int e = 0; e < 4; e++) {
                            kp[g][e] = t == j ? k[g][e] : kp[g][e] * a[e];        // 0 up to token j
                            w = fmaf(q[e], kp[g][e], w);
                        }
                    }
                    w = lane_xor_add<2>(lane_xor_add<1>(w));
                    own[t4 / 4] += (lane & 3) == t - t4 ? w : 0.f;
                }
        }
        __syncthreads();
        {
            float p = 1.f, b = 1.f;
#pragma unroll
            for (uint32_t t = 0; t < LA_PIECE; t++) {
                const uint32_t at = (wave * LA_PIECE + t) * LS + lane;
                p *= ps[at];
                qs[at] *= p;
            }
#pragma unroll
            for (int t = LA_PIECE - 1; t >= 0; t--) {
                const uint32_t at = (wave * LA_PIECE + t) * LS + lane;
                ks[at] *= b;
                b *= ps[at];
            }
            ahead[wave][lane] = p;
        }
        __syncthreads();
        if (wave == 0) {
            const float d0 = ahead[0][lane], d1 = ahead[1][lane], d2 = ahead[2][lane];
            ahead[0][lane] = 1.f;
            ahead[1][lane] = d0;
            ahead[2][lane] = d0 * d1;
            ahead[3][lane] = d0 * d1 * d2;
            between[0][lane] = d1;
            between[1][lane] = d2;
            between[2][lane] = d1 * d2;
        }
        __syncthreads();
#pragma unroll
        for (uint32_t i = 0; i < 2; i++) {
            const uint32_t n = wave + 4 * i;
            if (n >= 6) continue;
            const uint32_t a = LATER >> 4 * n & 15, b = EARLIER >> 4 * n & 15, bt = BETWEEN >> 4 * n & 15;
#pragma unroll 1
            for (uint32_t s = 0; s < sw; s += 32) {
                v8f q = load8(qs + (a * LA_PIECE + l16) * LS + s + 8 * lg);
                if (bt < 3) q *= load8(&between[bt][s + 8 * lg]);
                cross[i] = mma16(load8(ks + (b * LA_PIECE + l16) * LS + s + 8 * lg), q, cross[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < TILES; i++) {
            const uint32_t n = wave + 4 * i;
            if (n >= ntile) continue;
            const uint32_t t = n / nv * 32 + lq;
#pragma unroll
            for (uint32_t s = 0; s < 64; s += 16) {
                if (s >= sw) break;
                const v8f q = load8(qs + t * LS + s + 8 * lh) * load8(&ahead[t / LA_PIECE][s + 8 * lh]);
                acc[i] = mma32(i < EARLY ? sf[i < EARLY ? i : 0][s / 16] : state8(n, s), q, acc[i]);
                __builtin_amdgcn_sched_barrier(0);           // operands of a later step would take registers now
            }
        }
        __syncthreads();
    }

    const uint32_t lq = lane & 31, lh = lane >> 5, l16 = lane & 15, lg = lane >> 4;
    auto values8 = [&](uint32_t n, uint32_t s) { return column8(vbuf, ((s + 8 * lh) * ld + n % nv * 32 + lq) * 4, ld * 4); };
    v8f vf[EARLY][4];                                        // the chunk's values, for the first tiles
#pragma unroll
    for (int i = 0; i < EARLY; i++)
#pragma unroll
        for (uint32_t s = 0; s < 4; s++) vf[i][s] = values8(wave + 4 * i, 16 * s);
    // the weights of all pairs (t, j), j <= t
#pragma unroll
    for (uint32_t i = 0; i < LA_PIECE / 4; i++) ps[(wave * LA_PIECE + (lane & 3) + 4 * i) * LS + wave * LA_PIECE + (lane >> 2)] = own[i];
#pragma unroll
    for (uint32_t i = 0; i < 2; i++) {
        const uint32_t n = wave + 4 * i;
        if (n >= 6) continue;
        const uint32_t a = LATER >> 4 * n & 15, b = EARLIER >> 4 * n & 15;
        *reinterpret_cast<v4f*>(ps + (a * LA_PIECE + l16) * LS + b * LA_PIECE + 4 * lg) = cross[i];
    }
    // pieces 1 and 3 lie in the future of 0 and 2, inside the tiles read below
    for (uint32_t i = tid; i < 512; i += 256) ps[((i >> 8) * 32 + (i >> 4 & 15)) * LS + (i >> 8) * 32 + 16 + (i & 15)] = 0.f;
    __syncthreads();
    float* ssq = qs;                                         // [value tile][64]
#pragma unroll
    for (int i = 0; i < TILES; i++) {
        const uint32_t n = wave + 4 * i;
        if (n >= ntile) continue;
        const uint32_t tt = n / nv, t = tt * 32 + lq;
#pragma unroll
        for (uint32_t s = 0; s < 64; s += 16) {
            if (s >= 32 * (tt + 1)) break;
            acc[i] = mma32(i < EARLY ? vf[i < EARLY ? i : 0][s / 16] : values8(n, s), load8(ps + t * LS + s + 8 * lh), acc[i]);
            __builtin_amdgcn_sched_barrier(0);
        }
        float ss = 0.f;
#pragma unroll
        for (int r = 0; r < 16; r++) ss = fmaf(acc[i][r], acc[i][r], ss);
        ss = lane_xor_add<32>(ss);
        if (lh == 0) ssq[n % nv * 64 + t] = ss;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < TILES; i++) {
        const uint32_t n = wave + 4 * i;
        if (n >= ntile) continue;
        const uint32_t t = n / nv * 32 + lq;
        if (t >= rows) continue;
        float ss = 0.f;
        for (uint32_t k = 0; k < nv; k++) ss += ssq[k * 64 + t];
        const float inv = 1.0f / sqrtf(ss / (float)sh.vdim_n + sh.eps);
#pragma unroll
        for (int g = 0; g < 4; g++) {
            const uint32_t c = n % nv * 32 + 8 * g + 4 * lh;
            const v4f w = *reinterpret_cast<const v4f*>(norm + c);
            const size_t at = (size_t)(m0 + t) * ld_out + head * sh.vdim + c;
            const x4 gt = *reinterpret_cast<const x4*>(gate + at);
            float y[4];
#pragma unroll
            for (int e = 0; e < 4; e++) y[e] = acc[i][4 * g + e] * inv * w[e] * (float)gt[e];
            store4<T>(out + at, y[0], y[1], y[2], y[3]);
        }
    }
}

namespace {

uint32_t chunks_of(uint32_t M) { return (M + LA_CHUNK - 1) / LA_CHUNK; }

uint32_t chunk_lds(const LinearShape& sh) { return (sh.dim * LA_LS + LA_CHUNK * (sh.rank + 4) + LA_PIECES * sh.dim) * 4; }

template <typename T>
void output(const LinearShape& sh, const LinearIo& io, uint32_t M, const float* decay, const float* before, const float* norm, const void* gate, void* out,
            uint32_t ld_out, hipStream_t s) {
    auto go = [&](auto kernel) { fh::launch(kernel, dim3(chunks_of(M), sh.heads), 256, 0, s, sh, io.raw, decay, before, M, norm, (const T*)gate, (T*)out, ld_out); };
    if (sh.vdim <= 64) go(linear_output_kernel<T, 1>);
    else if (sh.vdim <= 128) go(linear_output_kernel<T, 2>);
    else go(linear_output_kernel<T, 4>);
}

}  // namespace

bool linear_shape_supported(const LinearShape& sh) { return sh.dim <= LA_MAX && sh.vdim <= LA_MAX && sh.rank <= LA_RANK_MAX; }

size_t linear_work_bytes(const LinearShape& sh, uint32_t M) {
    return ((size_t)M * sh.qk() + chunks_of(M) * (sh.state() + sh.qk())) * 4;
}

void launch_linear_prompt(DType t, const LinearShape& sh, const LinearIo& io, uint32_t M, float* work, const float* norm, const void* gate, void* out,
                          uint32_t ld_out, hipStream_t s) {
    const uint32_t chunks = chunks_of(M);
    float* add = work;
    float* total = add + chunks * sh.state();
    float* decay = total + (size_t)chunks * sh.qk();
    static const hipError_t ok = hipFuncSetAttribute((const void*)linear_chunk_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    (void)ok;
    fh::launch(linear_chunk_kernel, dim3(chunks, sh.heads), 256, chunk_lds(sh), s, sh, io.raw, io.w2, io.b2, M, decay, add, total);
    fh::launch(linear_scan_kernel, dim3((uint32_t)((sh.state() + 255) / 256)), 256, 0, s, sh, chunks, total, add, io.state, io.base_pos);
    if (t == DType::BF16) output<__bf16>(sh, io, M, decay, add, norm, gate, out, ld_out, s);
    else output<float>(sh, io, M, decay, add, norm, gate, out, ld_out, s);
}

void launch_linear_step(const LinearShape& sh, const LinearIo& io, float* o, hipStream_t s) {
    auto go = [&](auto kernel) { fh::launch(kernel, dim3(sh.heads, sh.vdim / 32), 256, 0, s, sh, io.raw, io.w2, io.b2, io.state, o, io.base_pos, io.pos_dev); };
    if (sh.dim <= 32) go(linear_step_kernel<1>);
    else if (sh.dim <= 64) go(linear_step_kernel<2>);
    else if (sh.dim <= 128) go(linear_step_kernel<4>);
    else go(linear_step_kernel<8>);
}

}  // namespace fh
