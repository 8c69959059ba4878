// Shared helpers of the mixer kernels (csrc/{stream,window_attn,lightning,latent,heads,rglru}.hip): element access for the two storage types
// (bf16 words, fp32), block reductions, and the hi / lo split of an fp32 operand for the matrix cores.
#pragma once
#include "common.h"

typedef unsigned int mx_u32x4 __attribute__((ext_vector_type(4)));   // (arrays of the uint4 struct end up in scratch memory)
typedef __bf16 mx_frag __attribute__((ext_vector_type(8)));     // MFMA 16x16x32 operand: 8 bf16 of one row / column

template <typename T> __device__ __forceinline__ float ld1(const T* p);
template <> __device__ __forceinline__ float ld1<uint16_t>(const uint16_t* p) { return bf_to_f(*p); }
template <> __device__ __forceinline__ float ld1<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void st1(T* p, float v);
template <> __device__ __forceinline__ void st1<uint16_t>(uint16_t* p, float v) { *p = f_to_bf(v); }
template <> __device__ __forceinline__ void st1<float>(float* p, float v) { *p = v; }

// V consecutive elements (V = 8: 16-byte aligned bf16 / 32-byte fp32 runs; V = 1: any alignment)
template <typename T, int V> struct vec_io;
template <> struct vec_io<uint16_t, 8> {
    static __device__ __forceinline__ void load(const uint16_t* p, float* f) {
        const uint4 v = *(const uint4*)p;
        f[0] = bf_lo(v.x); f[1] = bf_hi(v.x); f[2] = bf_lo(v.y); f[3] = bf_hi(v.y);
        f[4] = bf_lo(v.z); f[5] = bf_hi(v.z); f[6] = bf_lo(v.w); f[7] = bf_hi(v.w);
    }
    static __device__ __forceinline__ void store(uint16_t* p, const float* f) {
        *(uint4*)p = make_uint4(pack_bf2(f[0], f[1]), pack_bf2(f[2], f[3]), pack_bf2(f[4], f[5]), pack_bf2(f[6], f[7]));
    }
};
template <> struct vec_io<float, 8> {
    static __device__ __forceinline__ void load(const float* p, float* f) {
        const float4 a = ((const float4*)p)[0], b = ((const float4*)p)[1];
        f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
    }
    static __device__ __forceinline__ void store(float* p, const float* f) {
        ((float4*)p)[0] = make_float4(f[0], f[1], f[2], f[3]);
        ((float4*)p)[1] = make_float4(f[4], f[5], f[6], f[7]);
    }
};
template <typename T> struct vec_io<T, 1> {
    static __device__ __forceinline__ void load(const T* p, float* f) { f[0] = ld1(p); }
    static __device__ __forceinline__ void store(T* p, const float* f) { st1(p, f[0]); }
};

// logistic and SiLU: library exponential and division where the storage is fp32, the fast forms where the result is rounded to bf16
template <typename T> __device__ __forceinline__ float sigmoid_t(float z);
template <> __device__ __forceinline__ float sigmoid_t<float>(float z) { return 1.0f / (1.0f + expf(-z)); }
template <> __device__ __forceinline__ float sigmoid_t<uint16_t>(float z) {
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.4426950408889634f));
}
template <typename T> __device__ __forceinline__ float silu_t(float z) { return z * sigmoid_t<T>(z); }

// tanh-form GELU: z times the logistic of 2 sqrt(2 / pi) (z + 0.044715 z^3)
template <typename T> __device__ __forceinline__ float gelu_tanh_t(float z) { return z * sigmoid_t<T>(1.5957691216057308f * fmaf(0.044715f * z * z, z, z)); }

// activations by code: 1 SiLU, 2 tanh-form GELU, 3 square of relu
template <typename T> __device__ __forceinline__ float act_t(float z, int act) {
    if (act == 1) return silu_t<T>(z);
    if (act == 2) return gelu_tanh_t<T>(z);
    z = fmaxf(z, 0.f);
    return z * z;
}

// base^m for m >= 0 from log2(base) (-inf for base 0)
__device__ __forceinline__ float pow_log2(float l2, int m) { return m == 0 ? 1.0f : exp2f(l2 * (float)m); }

// sum over a workgroup of 256 threads; `red` is 4 floats of LDS, free again after the next barrier of the caller
__device__ __forceinline__ float block_sum_256(float v, float* red) {
    v = wave_sum(v);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return red[0] + red[1] + red[2] + red[3];
}

// an fp32 pair as bf16 pairs hi + lo: the sum is the fp32 value to 2^-17 relative
__device__ __forceinline__ void split_hi_lo(float a, float b, uint32_t& hi, uint32_t& lo) {
    hi = pack_bf2(a, b);
    lo = pack_bf2(a - bf_lo(hi), b - bf_hi(hi));
}

__device__ __forceinline__ mx_frag frag_of(uint32_t a, uint32_t b, uint32_t c, uint32_t d) {
    return __builtin_bit_cast(mx_frag, make_uint4(a, b, c, d));
}
// A fragment whose eight elements are two runs of four, 16 elements apart: p[0..3], p[16..19].  (The k index of an MFMA may be
// permuted as long as both operands agree: with this order an accumulator tile of one product is an operand of the next.)
__device__ __forceinline__ mx_frag frag_split(const uint16_t* p) {
    const uint2 a = *(const uint2*)p, b = *(const uint2*)(p + 16);
    return frag_of(a.x, a.y, b.x, b.y);
}
__device__ __forceinline__ f32x4_t mfma16(mx_frag a, mx_frag b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
