// Attention of a prompt's rows in bfloat16 or 32-bit: keys and values per head (or per group of heads), an optional key part that all
// heads share, an optional window, a gate on the output.  T: __bf16 or float (dense.h); scores, softmax and sums are 32-bit in both.
#include <hip/hip_runtime.h>

#include "common.h"
#include "dense.h"
#include "device_utils.h"

namespace fh {

constexpr float LOG2E = 1.4426950408889634f;

// Workgroup = 8 waves = 128 consecutive queries of one head: four groups of 32, each shared by two waves that take one half
// (32 keys) of every key tile and merge their (maximum, sum, output) at the end, which halves the longest chain of dependent
// tile steps.  Keys and values stream through LDS in tiles of 64 (K row-major: the head's own part, the shared part; V transposed), the
// next tile's loads in registers while this one is worked.  Both products are computed transposed (S^T = K Q^T, O^T = V^T P^T):
// a lane owns one query, so the softmax statistics are per-lane scalars, and the exponentiated scores are already the second
// product's operand.  Scores stay in the base-2 domain.
// DQ >= dim + rot and DV >= vdim: the register tiles' sizes; columns past the real ones are zero.
constexpr uint32_t LP_KT = 64, LP_QB = 128, LP_THREADS = 512;
template <typename T, int DQ, int DV> constexpr uint32_t prompt_lds() {
    const uint32_t tiles = (LP_KT * (DQ + 16 / sizeof(T)) + DV * (LP_KT + 8 / sizeof(T))) * sizeof(T), merge = 4 * 64 * 18 * 4;
    return tiles > merge ? tiles : merge;
}

template <typename T, int DQ, int DV>
__global__ __launch_bounds__(LP_THREADS) __attribute__((amdgpu_waves_per_eu(2)))
void attn_prompt_kernel(PromptAttn sh, const T* __restrict__ q, const T* __restrict__ kbuf, const T* __restrict__ vbuf, const T* __restrict__ shared,
                        const T* __restrict__ gate, T* __restrict__ out, uint32_t M, uint32_t base_pos) {
    typedef typename Vec<T>::x4 x4;
    typedef typename Vec<T>::x8 x8;
    constexpr uint32_t KT = LP_KT, QB = LP_QB, NT = LP_THREADS, PAD = 16 / sizeof(T);
    constexpr uint32_t KS = DQ + PAD, VS = KT + 8 / sizeof(T);         // LDS row strides
    constexpr uint32_t NS = DQ / 16, ND = DV / 32;
    constexpr uint32_t KTOTAL = KT * DQ / 8, VTOTAL = (KT / 2) * (DV / 4);       // pieces of a tile
    constexpr uint32_t KP = (KTOTAL + NT - 1) / NT, VP = (VTOTAL + NT - 1) / NT;
    extern __shared__ __attribute__((aligned(16))) uint8_t ap_lds[];
    T* Ks = reinterpret_cast<T*>(ap_lds);
    T* Vt = Ks + KT * KS;

    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 31, lh = lane >> 5;
    const uint32_t qg = wave >> 1, kh = wave & 1;        // query group, half of every key tile
    // latest (longest) query tiles first
    const uint32_t head = blockIdx.x % sh.heads, ntq = gridDim.x / sh.heads;
    const uint32_t q0 = (ntq - 1 - blockIdx.x / sh.heads) * QB;
    const uint32_t kvh = head / sh.group, kv_lo = sh.kv_lo, ld_out = sh.ld_out;
    const uint32_t dq = sh.dim + sh.rot, window = sh.window ? sh.window : 0xFFFFFFFFu;
    const float c2 = sh.scale * LOG2E;
    const uint32_t qrow = q0 + qg * 32 + lq, qpos = base_pos + qrow;

    x8 qf[NS];
#pragma unroll
    for (uint32_t s = 0; s < NS; s++) {
        const uint32_t d = 16 * s + 8 * lh;
        qf[s] = (qrow < M && d < dq) ? load8(q + ((size_t)qrow * sh.heads + head) * dq + d) : zero8<T>();
    }
    v16f oacc[ND];
#pragma unroll
    for (uint32_t d = 0; d < ND; d++)
#pragma unroll
        for (int r = 0; r < 16; r++) oacc[d][r] = 0.f;
    float m_run = -INFINITY, l_run = 0.f;

    const uint32_t total = base_pos + M;
    const uint32_t wg_max = base_pos + min(q0 + QB, M) - 1, wg_min = base_pos + q0;
    const bool wave_active = q0 + qg * 32 < M;
    const uint32_t wave_min = wg_min + qg * 32, wave_max = base_pos + min(q0 + qg * 32 + 32, M) - 1;
    auto first_visible = [&](uint32_t p) { return p >= window ? p - window + 1 : 0u; };
    const uint32_t wave_lo = first_visible(wave_min), last_lo = first_visible(wave_max);
    const uint32_t tile0 = first_visible(wg_min) / KT, ntiles = wg_max / KT + 1;

    const uint32_t kst = sh.k_row, vst = sh.v_row, cst = sh.shared_row;
    x8 kreg[KP];
    x4 va[VP], vb[VP];
    auto load_tile = [&](uint32_t kt) {
#pragma unroll
        for (uint32_t i = 0; i < KP; i++) {
            const uint32_t idx = tid + NT * i, key = idx / (DQ / 8), d = idx % (DQ / 8) * 8, t = kt * KT + key;
            if (idx >= KTOTAL || t >= total || d >= dq) kreg[i] = zero8<T>();
            else kreg[i] = d < sh.dim ? load8(kbuf + (size_t)(t - kv_lo) * kst + kvh * sh.dim + d)
                                      : load8(shared + (size_t)t * cst + (d - sh.dim));
        }
#pragma unroll
        for (uint32_t i = 0; i < VP; i++) {
            const uint32_t idx = tid + NT * i, kp = idx / (DV / 4), d = idx % (DV / 4) * 4, t = kt * KT + 2 * kp;
            const T* src = vbuf + (size_t)(t - kv_lo) * vst + kvh * sh.vdim + d;
            const bool in = idx < VTOTAL && d < sh.vdim;
            x4 z;
#pragma unroll
            for (int e = 0; e < 4; e++) z[e] = (T)0.f;
            va[i] = in && t < total ? *reinterpret_cast<const x4*>(src) : z;
            vb[i] = in && t + 1 < total ? *reinterpret_cast<const x4*>(src + vst) : z;
        }
    };
    auto store_tile = [&]() {
#pragma unroll
        for (uint32_t i = 0; i < KP; i++) {
            const uint32_t idx = tid + NT * i, key = idx / (DQ / 8), d = idx % (DQ / 8) * 8;
            if (idx < KTOTAL) store8(Ks + key * KS + d, kreg[i]);
        }
        // the two keys' values of one column side by side
#pragma unroll
        for (uint32_t i = 0; i < VP; i++) {
            const uint32_t idx = tid + NT * i, kp = idx / (DV / 4), d = idx % (DV / 4) * 4;
            if (idx >= VTOTAL) continue;
#pragma unroll
            for (int e = 0; e < 4; e++) {
                struct __attribute__((aligned(2 * sizeof(T)))) Pair { T a, b; } p = {va[i][e], vb[i][e]};
                *reinterpret_cast<Pair*>(Vt + (d + e) * VS + 2 * kp) = p;
            }
        }
    };

    load_tile(tile0);
    for (uint32_t kt = tile0; kt < ntiles; kt++) {
        __syncthreads();                      // the previous tile has been read
        store_tile();
        __syncthreads();
        if (kt + 1 < ntiles) load_tile(kt + 1);
        const uint32_t k0 = kt * KT + kh * 32;                                     // the wave's 32 keys
        if (!(wave_active && k0 <= wave_max && k0 + 32 > wave_lo)) continue;       // all in the wave's future, or before its windows
        // two accumulators: a product waits for the one before the last
        v16f sacc, sodd;
#pragma unroll
        for (int r = 0; r < 16; r++) sacc[r] = sodd[r] = 0.f;
#pragma unroll
        for (uint32_t s = 0; s < NS; s += 2) {
            sacc = mma32(load8(Ks + (kh * 32 + lq) * KS + 16 * s + 8 * lh), qf[s], sacc);
            sodd = mma32(load8(Ks + (kh * 32 + lq) * KS + 16 * (s + 1) + 8 * lh), qf[s + 1], sodd);
        }
        if (k0 + 31 > wave_min || k0 < last_lo) {
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const uint32_t t = k0 + 8 * (r >> 2) + 4 * lh + (r & 3);
                sacc[r] = (t <= qpos && qpos - t < window) ? (sacc[r] + sodd[r]) * c2 : -INFINITY;
            }
        } else {
#pragma unroll
            for (int r = 0; r < 16; r++) sacc[r] = (sacc[r] + sodd[r]) * c2;
        }
        float m_tile = sacc[0];
#pragma unroll
        for (int r = 1; r < 16; r++) m_tile = fmaxf(m_tile, sacc[r]);
        const float m_new = fmaxf(m_run, lane_xor_max<32>(m_tile));
        const float m_exp = m_new == -INFINITY ? 0.f : m_new;            // no key seen yet: every weight is 2^-inf = 0
        if (__builtin_amdgcn_ballot_w64(m_new > m_run) != 0) {
            const float alpha = m_run == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m_run - m_new);
            l_run *= alpha;
#pragma unroll
            for (uint32_t d = 0; d < ND; d++)
#pragma unroll
                for (int r = 0; r < 16; r++) oacc[d][r] *= alpha;
        }
        m_run = m_new;
        x8 pb[2];
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const float p = __builtin_amdgcn_exp2f(sacc[8 * j + e] - m_exp);
                l_run += p;
                pb[j][e] = (T)p;
            }
        // element e of lane half lh is key 16 j + 8 (e / 4) + 4 lh + e % 4 of the wave's half
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (uint32_t d = 0; d < ND; d++) {
                const T* vr = Vt + (d * 32 + lq) * VS + kh * 32 + 16 * j + 4 * lh;
                const x4 v0 = *reinterpret_cast<const x4*>(vr), v1 = *reinterpret_cast<const x4*>(vr + 8);
                oacc[d] = mma32((x8){v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]}, pb[j], oacc[d]);
            }
    }

    // ---- merge: the odd wave of a group hands its state over through LDS, 32 output columns at a time
    float* mg = reinterpret_cast<float*>(ap_lds) + (qg * 64 + lane) * 18;
    __syncthreads();
    if (kh) { mg[16] = m_run; mg[17] = l_run; }
    __syncthreads();
    const float m1 = mg[16], l1 = mg[17], m_all = fmaxf(m_run, m1);       // finite for rows < M: a query sees itself
    const float m_ref = m_all == -INFINITY ? 0.f : m_all;
    const float a0 = __builtin_amdgcn_exp2f(m_run - m_ref), a1 = __builtin_amdgcn_exp2f(m1 - m_ref);
    const float inv = 1.0f / lane_xor_add<32>(l_run * a0 + l1 * a1);
#pragma unroll
    for (uint32_t d = 0; d < ND; d++) {
        if (kh) {
#pragma unroll
            for (int r = 0; r < 16; r++) mg[r] = oacc[d][r];
        }
        __syncthreads();
        if (!kh && qrow < M) {
#pragma unroll
            for (int g = 0; g < 4; g++) {
                const uint32_t c = 32 * d + 8 * g + 4 * lh;
                if (c >= sh.vdim) continue;
                const size_t at = (size_t)qrow * ld_out + head * sh.vdim + c;
                const x4 gt = *reinterpret_cast<const x4*>(gate + at);
                float o[4];
#pragma unroll
                for (int i = 0; i < 4; i++) o[i] = (oacc[d][4 * g + i] * a0 + mg[4 * g + i] * a1) * inv * (float)gt[i];
                store4<T>(out + at, o[0], o[1], o[2], o[3]);
            }
        }
        __syncthreads();
    }
}

namespace {

template <typename T, int DQ, int DV>
void go(const PromptAttn& a, uint32_t M, uint32_t base_pos, hipStream_t s) {
    constexpr uint32_t lds = prompt_lds<T, DQ, DV>();
    static_assert(lds <= 160 * 1024, "LDS of a compute unit");
    static const hipError_t ok = hipFuncSetAttribute((const void*)attn_prompt_kernel<T, DQ, DV>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)ok;
    fh::launch(attn_prompt_kernel<T, DQ, DV>, dim3((M + LP_QB - 1) / LP_QB * a.heads), LP_THREADS, lds, s, a, (const T*)a.q, (const T*)a.k, (const T*)a.v,
               (const T*)a.shared, (const T*)a.gate, (T*)a.out, M, base_pos);
}

template <typename T>
void by_size(const PromptAttn& a, uint32_t M, uint32_t base_pos, hipStream_t s) {
    const uint32_t dq = a.dim + a.rot, dv = a.vdim;
#define FH_AP(DQ_, DV_) if (dq <= DQ_ && dv <= DV_) { go<T, DQ_, DV_>(a, M, base_pos, s); return; }
    FH_AP(64, 32)
    FH_AP(64, 64)
    FH_AP(96, 64)
    FH_AP(128, 128)
    FH_AP(192, 128)
    FH_AP(256, 256)
#undef FH_AP
}

}  // namespace

void launch_attn_prompt(DType t, const PromptAttn& a, uint32_t M, uint32_t base_pos, hipStream_t s) {
    if (t == DType::BF16) by_size<__bf16>(a, M, base_pos, s);
    else by_size<float>(a, M, base_pos, s);
}

}  // namespace fh
