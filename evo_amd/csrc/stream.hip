// Token-local kernels of models whose residual stream is kept in fp32: scaled embedding, the norm of a sublayer's output added to the
// stream, the norm of their sum, the final norm, the gated norm behind a linear-attention mixer, the gate of a gated MLP.  One workgroup per row, fp32 math,
// one rounding on the way out; storage type T is bf16 or fp32.  Entry points: include/evo_mi355x.h.
#include "mixers_common.h"
#include "../../include/evo_mi355x.h"

#define STREAM_DISPATCH(KERNEL, VECOK, GRID, ...)                                                                          \
    do {                                                                                                                   \
        const dim3 g_(GRID), b_(256);                                                                                      \
        hipStream_t s_ = (hipStream_t)stream;                                                                              \
        if (f32) {                                                                                                         \
            if (VECOK) hipLaunchKernelGGL((KERNEL<float, 8>), g_, b_, 0, s_, __VA_ARGS__);                                 \
            else hipLaunchKernelGGL((KERNEL<float, 1>), g_, b_, 0, s_, __VA_ARGS__);                                       \
        } else {                                                                                                           \
            if (VECOK) hipLaunchKernelGGL((KERNEL<uint16_t, 8>), g_, b_, 0, s_, __VA_ARGS__);                              \
            else hipLaunchKernelGGL((KERNEL<uint16_t, 1>), g_, b_, 0, s_, __VA_ARGS__);                                    \
        }                                                                                                                  \
        return evo_launch_status();                                                                                        \
    } while (0)

// ---------------------------------------------------------------------------------------------- embedding
// x = scale * w[id]; an id outside the table gives a zero row and raises *bad_flag
template <typename T, int V>
__global__ __launch_bounds__(256) void embed_stream_kernel(const int64_t* __restrict__ ids, const void* __restrict__ w_, float* __restrict__ x,
                                                           uint16_t* __restrict__ xb, int D, int64_t vocab, float scale, int* __restrict__ bad_flag) {
    const T* w = (const T*)w_;
    const int64_t row = blockIdx.x;
    const int64_t id = ids[row];
    const bool ok = id >= 0 && id < vocab;
    if (!ok && bad_flag && threadIdx.x == 0) *bad_flag = 1;
    for (int c = threadIdx.x * V; c < D; c += 256 * V) {
        float f[V];
        if (ok) vec_io<T, V>::load(w + id * D + c, f);
#pragma unroll
        for (int e = 0; e < V; ++e) f[e] = ok ? f[e] * scale : 0.f;
        vec_io<float, V>::store(x + row * D + c, f);
        if (xb) vec_io<uint16_t, V>::store(xb + row * D + c, f);
    }
}

extern "C" int evo_embed_stream(const int64_t* ids, const void* w, float* x, void* xb, int64_t n_tok, int64_t D, int64_t vocab, float scale,
                                int* bad_flag, int64_t f32, void* stream) {
    if (n_tok < 0 || n_tok > 0x7fffffff || D <= 0 || D > 0x7fffffff || vocab <= 0) return -1;
    if (n_tok == 0) return 0;
    STREAM_DISPATCH(embed_stream_kernel, D % 8 == 0, (unsigned)n_tok, ids, w, x, (uint16_t*)xb, (int)D, vocab, scale, bad_flag);
}

// ---------------------------------------------------------------------------------------------- x += norm(y) * (off + w)
// SUM: x = norm(alpha x + y) * (off + w); `y` below is then the sum.
// y stays in registers between the two passes (rows up to 4,096 elements); x is written in fp32 and, for the next sublayer's matrix
// product, once more in bf16.
template <typename T, int V, bool SUM>
__device__ __forceinline__ void closing_norm(const void* __restrict__ y_, const void* __restrict__ w_, float* __restrict__ x,
                                             uint16_t* __restrict__ xb, int D, float alpha, float eps, float off) {
    constexpr int KEEP = V == 8 ? 2 : 4;                         // runs of V elements a thread keeps in registers (D <= 256 V KEEP)
    __shared__ float red[4];
    const T* w = (const T*)w_;
    const int64_t row = blockIdx.x;
    const T* y = (const T*)y_ + row * D;
    float keep[KEEP][V];
    float ss = 0.f;
    auto load = [&](int c, float* f) {
        vec_io<T, V>::load(y + c, f);
        if constexpr (SUM) {
            float r[V];
            vec_io<float, V>::load(x + row * D + c, r);
#pragma unroll
            for (int e = 0; e < V; ++e) f[e] = fmaf(alpha, r[e], f[e]);
        }
    };
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const int c = (threadIdx.x + 256 * i) * V;
        if (c < D) {
            load(c, keep[i]);
#pragma unroll
            for (int e = 0; e < V; ++e) ss = fmaf(keep[i][e], keep[i][e], ss);
        }
    }
    for (int c = (threadIdx.x + 256 * KEEP) * V; c < D; c += 256 * V) {
        float f[V];
        load(c, f);
#pragma unroll
        for (int e = 0; e < V; ++e) ss = fmaf(f[e], f[e], ss);
    }
    const float inv = 1.0f / sqrtf(block_sum_256(ss, red) / (float)D + eps);
    auto finish = [&](int c, const float* f) {
        float g[V], r[V];
        vec_io<T, V>::load(w + c, g);
        if constexpr (!SUM) vec_io<float, V>::load(x + row * D + c, r);
#pragma unroll
        for (int e = 0; e < V; ++e) r[e] = SUM ? f[e] * inv * (off + g[e]) : fmaf(f[e] * inv, off + g[e], r[e]);
        vec_io<float, V>::store(x + row * D + c, r);
        if (xb) vec_io<uint16_t, V>::store(xb + row * D + c, r);
    };
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const int c = (threadIdx.x + 256 * i) * V;
        if (c < D) finish(c, keep[i]);
    }
    for (int c = (threadIdx.x + 256 * KEEP) * V; c < D; c += 256 * V) {
        float f[V];
        load(c, f);
        finish(c, f);
    }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void postnorm_residual_kernel(const void* __restrict__ y, const void* __restrict__ w, float* __restrict__ x,
                                                                uint16_t* __restrict__ xb, int D, float eps, float off) {
    closing_norm<T, V, false>(y, w, x, xb, D, 1.f, eps, off);
}
template <typename T, int V>
__global__ __launch_bounds__(256) void sum_norm_kernel(const void* __restrict__ y, const void* __restrict__ w, float* __restrict__ x,
                                                       uint16_t* __restrict__ xb, int D, float alpha, float eps, float off) {
    closing_norm<T, V, true>(y, w, x, xb, D, alpha, eps, off);
}

extern "C" int evo_postnorm_residual(const void* y, const void* w, float* x, void* xb, int64_t M, int64_t D, float eps, float w_offset,
                                     int64_t f32, void* stream) {
    if (M < 0 || M > 0x7fffffff || D <= 0 || D > 0x3fffffff) return -1;
    if (M == 0) return 0;
    STREAM_DISPATCH(postnorm_residual_kernel, D % 8 == 0, (unsigned)M, y, w, x, (uint16_t*)xb, (int)D, eps, w_offset);
}

extern "C" int evo_sum_norm(const void* y, const void* w, float* x, void* xb, int64_t M, int64_t D, float alpha, float eps, float w_offset,
                            int64_t f32, void* stream) {
    if (!y || !w || !x || M < 0 || M > 0x7fffffff || D <= 0 || D > 0x3fffffff) return -1;
    if (M == 0) return 0;
    STREAM_DISPATCH(sum_norm_kernel, D % 8 == 0, (unsigned)M, y, w, x, (uint16_t*)xb, (int)D, alpha, eps, w_offset);
}

// ---------------------------------------------------------------------------------------------- out = norm(x) * (off + w), x the stream
template <typename T, int V>
__global__ __launch_bounds__(256) void rmsnorm_stream_kernel(const float* __restrict__ x_, const void* __restrict__ w_, void* __restrict__ out_, int D,
                                                             float eps, float off) {
    __shared__ float red[4];
    const T* w = (const T*)w_;
    const int64_t row = blockIdx.x;
    const float* x = x_ + row * D;
    T* out = (T*)out_ + row * D;
    float ss = 0.f;
    for (int c = threadIdx.x * V; c < D; c += 256 * V) {
        float f[V];
        vec_io<float, V>::load(x + c, f);
#pragma unroll
        for (int e = 0; e < V; ++e) ss = fmaf(f[e], f[e], ss);
    }
    const float inv = 1.0f / sqrtf(block_sum_256(ss, red) / (float)D + eps);
    for (int c = threadIdx.x * V; c < D; c += 256 * V) {
        float f[V], g[V];
        vec_io<float, V>::load(x + c, f);
        vec_io<T, V>::load(w + c, g);
#pragma unroll
        for (int e = 0; e < V; ++e) f[e] = f[e] * inv * (off + g[e]);
        vec_io<T, V>::store(out + c, f);
    }
}

extern "C" int evo_rmsnorm_stream(const float* x, const void* w, void* out, int64_t M, int64_t D, float eps, float w_offset, int64_t f32,
                                  void* stream) {
    if (M < 0 || M > 0x7fffffff || D <= 0 || D > 0x3fffffff) return -1;
    if (M == 0) return 0;
    STREAM_DISPATCH(rmsnorm_stream_kernel, D % 8 == 0, (unsigned)M, x, w, out, (int)D, eps, w_offset);
}

// ---------------------------------------------------------------------------------------------- out = norm(o) * w * sigmoid(g)
template <typename T, int V>
__global__ __launch_bounds__(256) void gated_norm_kernel(const void* __restrict__ o_, const void* __restrict__ g_, int64_t ldg,
                                                         const void* __restrict__ w_, void* __restrict__ out_, int D, float eps) {
    constexpr int KEEP = V == 8 ? 2 : 4;
    __shared__ float red[4];
    const T* w = (const T*)w_;
    const int64_t row = blockIdx.x;
    const T* o = (const T*)o_ + row * D;
    const T* g = (const T*)g_ + row * ldg;
    T* out = (T*)out_ + row * D;
    float keep[KEEP][V];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const int c = (threadIdx.x + 256 * i) * V;
        if (c < D) {
            vec_io<T, V>::load(o + c, keep[i]);
#pragma unroll
            for (int e = 0; e < V; ++e) ss = fmaf(keep[i][e], keep[i][e], ss);
        }
    }
    for (int c = (threadIdx.x + 256 * KEEP) * V; c < D; c += 256 * V) {
        float f[V];
        vec_io<T, V>::load(o + c, f);
#pragma unroll
        for (int e = 0; e < V; ++e) ss = fmaf(f[e], f[e], ss);
    }
    const float inv = 1.0f / sqrtf(block_sum_256(ss, red) / (float)D + eps);
    auto finish = [&](int c, const float* f) {
        float gg[V], ww[V], r[V];
        vec_io<T, V>::load(g + c, gg);
        vec_io<T, V>::load(w + c, ww);
#pragma unroll
        for (int e = 0; e < V; ++e) r[e] = f[e] * inv * ww[e] * sigmoid_t<T>(gg[e]);
        vec_io<T, V>::store(out + c, r);
    };
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const int c = (threadIdx.x + 256 * i) * V;
        if (c < D) finish(c, keep[i]);
    }
    for (int c = (threadIdx.x + 256 * KEEP) * V; c < D; c += 256 * V) {
        float f[V];
        vec_io<T, V>::load(o + c, f);
        finish(c, f);
    }
}

extern "C" int evo_gated_norm(const void* o, const void* g, int64_t ldg, const void* w, void* out, int64_t M, int64_t D, float eps, int64_t f32,
                              void* stream) {
    if (M < 0 || M > 0x7fffffff || D <= 0 || D > 0x3fffffff || ldg < D) return -1;
    if (M == 0) return 0;
    const bool vec = D % 8 == 0 && ldg % 8 == 0 && ((uintptr_t)g & 15) == 0;
    STREAM_DISPATCH(gated_norm_kernel, vec, (unsigned)M, o, g, ldg, w, out, (int)D, eps);
}

// ---------------------------------------------------------------------------------------------- a = silu(z[:, :I]) * z[:, I:]
template <typename T, int V>
__global__ __launch_bounds__(256) void silu_gate_kernel(const void* __restrict__ z_, void* __restrict__ a_, int64_t M, int64_t I) {
    const T* z = (const T*)z_;
    T* a = (T*)a_;
    const int64_t per = I / V, total = M * per;
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
        const int64_t row = i / per, c = (i - row * per) * V;
        float u[V], v[V];
        vec_io<T, V>::load(z + row * 2 * I + c, u);
        vec_io<T, V>::load(z + row * 2 * I + I + c, v);
#pragma unroll
        for (int e = 0; e < V; ++e) u[e] = silu_t<T>(u[e]) * v[e];
        vec_io<T, V>::store(a + row * I + c, u);
    }
}

extern "C" int evo_silu_gate(const void* z, void* a, int64_t M, int64_t I, int64_t f32, void* stream) {
    if (M < 0 || I <= 0) return -1;
    if (M == 0) return 0;
    const int64_t total = M * (I % 8 == 0 ? I / 8 : I);
    const unsigned grid = (unsigned)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
    STREAM_DISPATCH(silu_gate_kernel, I % 8 == 0, grid, z, a, M, I);
}

// ---------------------------------------------------------------------------------------------- z[:, :n] = act(z[:, :n]) in place
template <typename T, int V>
__global__ __launch_bounds__(256) void act_cols_kernel(void* __restrict__ z_, int64_t ld, int64_t M, int64_t n, int act) {
    T* z = (T*)z_;
    const int64_t per = n / V, total = M * per;
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
        const int64_t row = i / per;
        T* p = z + row * ld + (i - row * per) * V;
        float f[V];
        vec_io<T, V>::load(p, f);
#pragma unroll
        for (int e = 0; e < V; ++e) f[e] = act_t<T>(f[e], act);
        vec_io<T, V>::store(p, f);
    }
}

extern "C" int evo_act_cols(void* z, int64_t ld, int64_t M, int64_t n, int64_t act, int64_t f32, void* stream) {
    if (M < 0 || n <= 0 || ld < n || act < 1 || act > 3) return -1;
    if (M == 0) return 0;
    const bool vec = n % 8 == 0 && ld % 8 == 0 && ((uintptr_t)z & 15) == 0;
    const int64_t total = M * (vec ? n / 8 : n);
    const unsigned grid = (unsigned)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
    STREAM_DISPATCH(act_cols_kernel, vec, grid, z, ld, M, n, (int)act);
}
