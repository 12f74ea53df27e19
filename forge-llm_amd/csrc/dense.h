// Dense (bfloat16 or 32-bit) matrices: element types, matrix-unit fragments and the epilogues that the matrix-matrix and the
// matrix-vector kernels share.  T is the storage type of weights and activations: __bf16 or float.  Sums are 32-bit in both.
#pragma once

#include <hip/hip_runtime.h>
#include <math.h>
#include <stdint.h>

#include "common.h"
#include "device_utils.h"

namespace fh {

typedef float v4f __attribute__((ext_vector_type(4)));
typedef float v8f __attribute__((ext_vector_type(8)));
typedef float v16f __attribute__((ext_vector_type(16)));
typedef __bf16 v4bf __attribute__((ext_vector_type(4)));
typedef __bf16 v8bf __attribute__((ext_vector_type(8)));

// Four and eight elements of a row in registers.
template <typename T> struct Vec;
template <> struct Vec<__bf16> { typedef v4bf x4; typedef v8bf x8; };
template <> struct Vec<float> { typedef v4f x4; typedef v8f x8; };

template <typename T> __device__ __forceinline__ typename Vec<T>::x8 load8(const T* p) {
    if constexpr (sizeof(T) == 2) return *reinterpret_cast<const v8bf*>(p);
    else {
        const v4f a = reinterpret_cast<const v4f*>(p)[0], b = reinterpret_cast<const v4f*>(p)[1];
        return (v8f){a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
    }
}
template <typename T> __device__ __forceinline__ void store8(T* p, typename Vec<T>::x8 v) {
    if constexpr (sizeof(T) == 2) *reinterpret_cast<v8bf*>(p) = v;
    else {
        reinterpret_cast<v4f*>(p)[0] = (v4f){v[0], v[1], v[2], v[3]};
        reinterpret_cast<v4f*>(p)[1] = (v4f){v[4], v[5], v[6], v[7]};
    }
}
template <typename T> __device__ __forceinline__ typename Vec<T>::x8 zero8() {
    typename Vec<T>::x8 z;
#pragma unroll
    for (int e = 0; e < 8; e++) z[e] = (T)0.0f;
    return z;
}
template <typename T> __device__ __forceinline__ void store4(T* p, float a, float b, float c, float d) {
    typename Vec<T>::x4 v;
    v[0] = (T)a; v[1] = (T)b; v[2] = (T)c; v[3] = (T)d;
    *reinterpret_cast<typename Vec<T>::x4*>(p) = v;
}

// D += A B on the matrix unit with both operands as "8 elements per lane" fragments.  32x32 tile, depth 16: lane l holds row
// (column) l % 32 and the depths 8 (l / 32) + 0..7; the result lane l holds column l % 32 and, in register r, row
// 8 (r / 4) + 4 (l / 32) + r % 4.  The 32-bit form is eight depth-2 instructions over the same fragments (element e of the two
// lane halves forms one of them): full single precision.
__device__ __forceinline__ v16f mma32(v8bf a, v8bf b, v16f c) { return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ v16f mma32(v8f a, v8f b, v16f c) {
#pragma unroll
    for (int e = 0; e < 8; e++) c = __builtin_amdgcn_mfma_f32_32x32x2f32(a[e], b[e], c, 0, 0, 0);
    return c;
}
// 16x16 tile, depth 32: lane l holds row (column) l % 16 and the depths 8 (l / 16) + 0..7; the result lane l holds column l % 16
// and, in register r, row 4 (l / 16) + r.
__device__ __forceinline__ v4f mma16(v8bf a, v8bf b, v4f c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ v4f mma16(v8f a, v8f b, v4f c) {
#pragma unroll
    for (int e = 0; e < 8; e++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], c, 0, 0, 0);
    return c;
}

// Dynamic Tanh, an elementwise norm: tanh(alpha * x) * w + b.  w == nullptr: x itself.
__device__ __forceinline__ float dyn_tanh(const DynTanh& t, uint32_t n, float x) { return t.w ? tanhf(t.alpha * x) * t.w[n] + t.b[n] : x; }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
// 0.5 z (1 + tanh(u)) with u = sqrt(2 / pi) (z + 0.044715 z^3): the logistic function of 2 u, times z
__device__ __forceinline__ float gelu_tanh_f(float z) { return z / (1.0f + expf(-1.5957691216057308f * (z + 0.044715f * z * z * z))); }
__device__ __forceinline__ float act_f(Act a, float z) { return a == Act::Sigmoid ? sigmoid_f(z) : a == Act::Silu ? silu_f(z) : gelu_tanh_f(z); }

// Sum over the workgroup of `nt` threads; red: LDS, nt / 64 floats, free again after the next barrier.
__device__ __forceinline__ float block_sum(float v, float* red, uint32_t tid, uint32_t nt) {
    v = wave_sum(v);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = v;
    __syncthreads();
    float s = 0.f;
    for (uint32_t i = 0; i < nt / 64; i++) s += red[i];
    return s;
}

// What happens to the results (m, n .. n + 3) of a product; n is a multiple of 4.
template <typename T, DenseEpi MODE>
__device__ __forceinline__ void dense_epilogue(const DenseEpiArgs& e, uint32_t m, uint32_t n, uint32_t N, const float* v) {
    if constexpr (MODE == DenseEpi::F32) {
        float* y = e.f32 + (size_t)m * e.ld_f32 + n;
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (n + i < N) y[i] = e.cap > 0.f ? e.cap * tanhf(v[i] / e.cap) : v[i];
    } else if constexpr (MODE == DenseEpi::RawGate) {
        if (n < e.split) *reinterpret_cast<float4*>(e.f32 + (size_t)m * e.ld_f32 + n) = make_float4(v[0], v[1], v[2], v[3]);
        else store4<T>((T*)e.out + (size_t)m * e.ld_out + (n - e.split), act_f(e.act, v[0]), act_f(e.act, v[1]), act_f(e.act, v[2]), act_f(e.act, v[3]));
    } else if constexpr (MODE == DenseEpi::Rope) {
        const uint32_t j = n % e.head_stride;
        float a[4] = {v[0], v[1], v[2], v[3]};
        if (j >= e.rot_off && (j - e.rot_off) / 2 < e.rot_pairs) {
            const uint32_t p = (e.pos_dev ? *e.pos_dev : e.base_pos) + m, i = (j - e.rot_off) / 2;
            const float* ct = e.cos_t + (size_t)p * e.rot_pairs;
            const float* st = e.sin_t + (size_t)p * e.rot_pairs;
            const float c0 = ct[i], s0 = st[i];
            a[0] = v[0] * c0 - v[1] * s0;
            a[1] = v[1] * c0 + v[0] * s0;
            if (i + 1 < e.rot_pairs) {
                const float c1 = ct[i + 1], s1 = st[i + 1];
                a[2] = v[2] * c1 - v[3] * s1;
                a[3] = v[3] * c1 + v[2] * s1;
            }
        }
        store4<T>((T*)e.out + (size_t)m * e.ld_out + n, a[0], a[1], a[2], a[3]);
    } else if constexpr (MODE == DenseEpi::Split) {
        T* y = n < e.split ? (T*)e.out + (size_t)m * e.ld_out + n : (T*)e.out2 + (size_t)m * e.ld_out2 + (n - e.split);
        store4<T>(y, v[0], v[1], v[2], v[3]);
    } else if constexpr (MODE == DenseEpi::GateMul) {
        const T* g = (const T*)e.gate + (size_t)m * e.ld_out + n;
        store4<T>((T*)e.out + (size_t)m * e.ld_out + n, v[0] * (float)g[0], v[1] * (float)g[1], v[2] * (float)g[2], v[3] * (float)g[3]);
    } else if constexpr (MODE == DenseEpi::ActPair) {
        T* y = (T*)e.out + (size_t)m * e.ld_out + n / 2;
        y[0] = (T)(act_f(e.act, v[0]) * v[1]);
        y[1] = (T)(act_f(e.act, v[2]) * v[3]);
    } else if constexpr (MODE == DenseEpi::Residual) {
        // everything the four results need is requested at once
        float4* xp = reinterpret_cast<float4*>(e.f32 + (size_t)m * e.ld_f32 + n);
        const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
        const float4 x = e.add ? *xp : zero;
        const float4 pw = e.post.w ? *reinterpret_cast<const float4*>(e.post.w + n) : zero, pb = e.post.w ? *reinterpret_cast<const float4*>(e.post.b + n) : zero;
        const float4 nw = e.next.w ? *reinterpret_cast<const float4*>(e.next.w + n) : zero, nb = e.next.w ? *reinterpret_cast<const float4*>(e.next.b + n) : zero;
        float a[4] = {v[0], v[1], v[2], v[3]};
        auto norm4 = [&](const DynTanh& t, const float4& w, const float4& b) {
            if (!t.w) return;
            a[0] = tanhf(t.alpha * a[0]) * w.x + b.x;
            a[1] = tanhf(t.alpha * a[1]) * w.y + b.y;
            a[2] = tanhf(t.alpha * a[2]) * w.z + b.z;
            a[3] = tanhf(t.alpha * a[3]) * w.w + b.w;
        };
        norm4(e.post, pw, pb);
        a[0] += x.x; a[1] += x.y; a[2] += x.z; a[3] += x.w;
        *xp = make_float4(a[0], a[1], a[2], a[3]);
        if (!e.out) return;
        norm4(e.next, nw, nb);
        store4<T>((T*)e.out + (size_t)m * e.ld_out + n, a[0], a[1], a[2], a[3]);
    }
}

}  // namespace fh
