// Attention with one cached key and value row per token and key head: preparation (per-head norms, rotation, cache append) and decode.
// Query heads share key / value heads in groups; a head may have two maps over the same values (differential attention).  Prompts attend in
// csrc/window_attn.hip.  Entry points: include/evo_mi355x.h.
#include "mixers_common.h"
#include "../../include/evo_mi355x.h"

#define LOG2E 1.4426950408889634f
#define FLOOR -1.0e30f                                           // running maximum before any key

// ------------------------------------------------------------------------------------------------ norms, rotation, cache append
struct HeadsArgs {
    void* z; int64_t ld; void* cache;                            // cache [rows, ring, rs] or null
    const void* qw; const void* kw; const float* inv_freq; const int64_t* pos; const int* seq; const int* cu;
    int nq, nk, dim, nv, n_rot, keep, ring, rs, unit;
    float amp, eps;
};

// this token's cache row, or null when no later token sees it
template <typename T> __device__ __forceinline__ T* cache_row(const HeadsArgs& a, int m, int64_t pos) {
    if (!a.cache) return nullptr;
    const int b = a.seq ? a.seq[m] : m, w = a.ring - a.keep;
    if (pos >= a.keep && a.cu && a.cu[b + 1] - m > w) return nullptr;
    const int64_t slot = pos < a.keep ? pos : a.keep + (pos - a.keep) % w;
    return (T*)a.cache + ((int64_t)b * a.ring + slot) * a.rs;
}

template <int N> __device__ __forceinline__ float lanes_sum(float v) {   // over groups of N consecutive lanes
    if (N >= 2) v += dpp_fetch<EVO_DPP_XOR1>(v);
    if (N >= 4) v += dpp_fetch<EVO_DPP_XOR2>(v);
    if (N >= 8) v += dpp_fetch<EVO_DPP_HALF_MIRROR>(v);
    if (N >= 16) v += dpp_fetch<EVO_DPP_MIRROR>(v);
    if (N >= 32) v += __shfl_xor(v, 16, 64);
    if (N >= 64) v += __shfl_xor(v, 32, 64);
    return v;
}

__device__ __forceinline__ void fill_turns(float2* turn, const HeadsArgs& a, int64_t pos) {
    for (int i = threadIdx.x; i < a.n_rot / 2; i += 256) {
        float c, s;
        sincosf((float)pos * a.inv_freq[i], &s, &c);
        turn[i] = make_float2(c * a.amp, s * a.amp);
    }
}

// LG lanes per vector, 16 elements each: a run of eight and its partners half a rotation further, or two runs that are not rotated.
// n_rot % 16 == 0, dim % 8 == 0, 16-byte aligned rows.
template <typename T, int LG>
__global__ __launch_bounds__(256) void heads_prep_kernel(HeadsArgs a) {
    extern __shared__ float2 turn[];                             // [n_rot / 2] cosine and sine of this token's angles, times the amplitude
    const int m = blockIdx.x, tid = threadIdx.x, u = tid % LG;
    const int64_t pos = a.pos[m];
    T* z = (T*)a.z + (int64_t)m * a.ld;
    T* slot = cache_row<T>(a, m, pos);
    const int half = a.n_rot / 2, rot = a.n_rot / 16;
    const int oa = u < rot ? 8 * u : a.n_rot + 16 * (u - rot), ob = u < rot ? half + 8 * u : oa + 8;
    const bool ha = oa < a.dim, hb = ob < a.dim;                 // (lanes past the vector idle)
    fill_turns(turn, a, pos);
    __syncthreads();
    for (int h = tid / LG; h < a.nq + a.nk; h += 256 / LG) {
        T* v = z + (int64_t)h * a.dim;
        float x[8], y[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = y[e] = 0.f;
        if (ha) vec_io<T, 8>::load(v + oa, x);
        if (hb) vec_io<T, 8>::load(v + ob, y);
        const T* w = (const T*)(h < a.nq ? a.qw : a.kw);
        auto inv_rms = [&]() {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss = fmaf(x[e], x[e], fmaf(y[e], y[e], ss));
            return 1.0f / sqrtf(lanes_sum<LG>(ss) / (float)a.dim + a.eps);
        };
        if (w) {
            const float inv = inv_rms();
            float g[8];
            if (ha) {
                vec_io<T, 8>::load(w + oa, g);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] *= inv * g[e];
            }
            if (hb) {
                vec_io<T, 8>::load(w + ob, g);
#pragma unroll
                for (int e = 0; e < 8; ++e) y[e] *= inv * g[e];
            }
        }
        if (u < rot) {
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float2 t = turn[8 * u + e];
                const float p = x[e], q = y[e];
                x[e] = p * t.x - q * t.y;
                y[e] = q * t.x + p * t.y;
            }
        }
        if (a.unit) {
            const float inv = inv_rms();
#pragma unroll
            for (int e = 0; e < 8; ++e) { x[e] *= inv; y[e] *= inv; }
        }
        if (ha) vec_io<T, 8>::store(v + oa, x);
        if (hb) vec_io<T, 8>::store(v + ob, y);
        if (slot && h >= a.nq) {
            T* k = slot + (int64_t)(h - a.nq) * a.dim;
            if (ha) vec_io<T, 8>::store(k + oa, x);
            if (hb) vec_io<T, 8>::store(k + ob, y);
        }
    }
    if (slot) {
        const T* v = z + (int64_t)(a.nq + a.nk) * a.dim;
        T* d = slot + (int64_t)a.nk * a.dim;
        for (int i = tid * 8; i + 7 < a.nv; i += 2048) {
            float x[8];
            vec_io<T, 8>::load(v + i, x);
            vec_io<T, 8>::store(d + i, x);
        }
        for (int i = a.nv / 8 * 8 + tid; i < a.nv; i += 256) d[i] = v[i];
    }
}

// Any sizes: a wave per vector
template <typename T>
__global__ __launch_bounds__(256) void heads_prep_any_kernel(HeadsArgs a) {
    extern __shared__ float2 turn[];                             // [n_rot / 2], then [4][dim] floats
    const int m = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int64_t pos = a.pos[m];
    T* z = (T*)a.z + (int64_t)m * a.ld;
    T* slot = cache_row<T>(a, m, pos);
    const int half = a.n_rot / 2;
    float* x = (float*)(turn + half) + wave * a.dim;
    fill_turns(turn, a, pos);
    __syncthreads();
    for (int h0 = 0; h0 < a.nq + a.nk; h0 += 4) {
        const int h = h0 + wave;
        const bool on = h < a.nq + a.nk;
        T* v = z + (int64_t)h * a.dim;
        const T* w = (const T*)(h < a.nq ? a.qw : a.kw);
        float ss = 0.f;
        for (int i = lane; on && i < a.dim; i += 64) { x[i] = ld1(v + i); ss = fmaf(x[i], x[i], ss); }
        if (w) {
            const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
            for (int i = lane; on && i < a.dim; i += 64) x[i] *= inv * ld1(w + i);
        }
        __syncthreads();                                         // (the pairs of a rotation belong to other lanes)
        for (int i = lane; on && i < half; i += 64) {
            const float p = x[i], q = x[i + half];
            x[i] = p * turn[i].x - q * turn[i].y;
            x[i + half] = q * turn[i].x + p * turn[i].y;
        }
        __syncthreads();
        float inv = 1.0f;
        if (a.unit) {
            ss = 0.f;
            for (int i = lane; on && i < a.dim; i += 64) ss = fmaf(x[i], x[i], ss);
            inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
        }
        for (int i = lane; on && i < a.dim; i += 64) {
            st1(v + i, x[i] * inv);
            if (slot && h >= a.nq) st1(slot + (int64_t)(h - a.nq) * a.dim + i, x[i] * inv);
        }
        __syncthreads();
    }
    if (slot)
        for (int i = tid; i < a.nv; i += 256) slot[(int64_t)a.nk * a.dim + i] = z[(int64_t)(a.nq + a.nk) * a.dim + i];
}

extern "C" int evo_heads_prep(void* z, int64_t ld, void* cache, const void* qw, const void* kw, const float* inv_freq, const int64_t* pos, const int* seq,
                              const int* cu, int64_t M, int64_t nq, int64_t nk, int64_t dim, int64_t nv, int64_t n_rot, int64_t keep, int64_t ring,
                              int64_t rs, float amp, float eps, int64_t unit, int64_t f32, void* stream) {
    if (!z || !pos || M <= 0 || M > 0x7fffffff || nq <= 0 || nk < 0 || dim <= 0 || dim > 2048 || nv < 0 || n_rot < 0 || n_rot > dim || n_rot % 2) return -1;
    if ((n_rot && !inv_freq) || (nq + nk) * dim + nv > ld || ld > 0x3fffffff || (cu && !seq) || !qw != !kw) return -1;
    if (cache && (keep < 0 || ring <= keep || ring > 0x3fffffff || rs < nk * dim + nv || rs > 0x3fffffff)) return -1;
    HeadsArgs a = {z, ld, cache, qw, kw, inv_freq, pos, seq, cu, (int)nq, (int)nk, (int)dim, (int)nv, (int)n_rot, (int)keep, (int)ring, (int)rs, (int)unit, amp, eps};
    const size_t lds = (size_t)n_rot * 4;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((unsigned)M), block(256);
    const int64_t lanes = n_rot / 16 + (dim - n_rot + 15) / 16;
    if (n_rot % 16 == 0 && dim % 8 == 0 && lanes <= 64 && ld % 8 == 0 && rs % 8 == 0 && (((uintptr_t)z | (uintptr_t)cache | (uintptr_t)qw | (uintptr_t)kw) & 15) == 0) {
#define HP(LG) do { if (f32) hipLaunchKernelGGL((heads_prep_kernel<float, LG>), grid, block, lds, s, a);                   \
                    else hipLaunchKernelGGL((heads_prep_kernel<uint16_t, LG>), grid, block, lds, s, a); } while (0)
        if (lanes <= 1) HP(1); else if (lanes <= 2) HP(2); else if (lanes <= 4) HP(4); else if (lanes <= 8) HP(8);
        else if (lanes <= 16) HP(16); else if (lanes <= 32) HP(32); else HP(64);
#undef HP
        return evo_launch_status();
    }
    if (f32) hipLaunchKernelGGL((heads_prep_any_kernel<float>), grid, block, lds + (size_t)dim * 16, s, a);
    else hipLaunchKernelGGL((heads_prep_any_kernel<uint16_t>), grid, block, lds + (size_t)dim * 16, s, a);
    return evo_launch_status();
}

// ------------------------------------------------------------------------------------------------ decode
// A slot of the cache holds some earlier token or nothing yet; min(pos + 1, ring) slots have been written and all of them are visible.
struct HDecArgs {
    const void* z; int64_t ld; const void* cache; const int64_t* pos; float* part_o; float* part_ml;
    int H, G, dim, dv, rs, ring, n_split, n_qb;                  // n_qb: blocks of 16 query heads per key head
    float sc2;                                                   // scale * log2(e)
};

// Matrix cores (bf16).  A workgroup: one (sequence, key head, up to 16 of its query heads) and its share of the slots, 32 at a time per wave
// and without a barrier among the waves:
//   scores   S^T = K q^T, query heads are the columns; fragments of K come straight from memory (a row is read once, by its own lane)
//   softmax  a lane holds four slots of each of two 16-slot blocks for one query head
//   sum      O^T = V^T P^T: the probabilities are an operand as they stand (split key order); V goes through a wave-private LDS tile and
//            is read as dwords, two adjacent dimensions of a slot: the even and the odd dimensions are two operands
// The waves' sums meet in LDS at the end.  The loads carry no branch: rows past the slots in use repeat a valid one and are masked.
// KS: 32-wide steps of a key, NG: 32-wide groups of a value, MAPS: maps per head ([map 1 | map 2] in keys and queries).
template <int KS, int NG, int MAPS>
__global__ __launch_bounds__(256) void heads_decode_kernel(HDecArgs a) {
    constexpr int VP = 32 * NG + 8, AP = 32 * NG + 4;            // pitches of the value tiles and of the meeting place
    extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
    __shared__ float ml[4][MAPS][16][2];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int split = blockIdx.x, hk = blockIdx.y / a.n_qb, qb = blockIdx.y % a.n_qb, b = blockIdx.z;
    const int Q = a.H / a.G, nq = Q - 16 * qb < 16 ? Q - 16 * qb : 16;    // query heads of this workgroup
    const int h0 = hk * Q + 16 * qb;
    const int dim = a.dim, dv = a.dv;
    uint16_t* vt = lds + wave * 32 * VP;                         // [32][VP]
    const uint16_t* base = (const uint16_t*)a.cache + (int64_t)b * a.ring * a.rs + (int64_t)hk * MAPS * dim;
    const uint16_t* vbase = (const uint16_t*)a.cache + (int64_t)b * a.ring * a.rs + (int64_t)a.G * MAPS * dim + (int64_t)hk * dv;
    mx_frag qf[MAPS][KS];
    {
        const uint16_t* q = (const uint16_t*)a.z + (int64_t)b * a.ld + (int64_t)(h0 + (c16 < nq ? c16 : nq - 1)) * MAPS * dim;
#pragma unroll
        for (int m = 0; m < MAPS; ++m)
#pragma unroll
            for (int ks = 0; ks < KS; ++ks) {
                const int d = 32 * ks + 8 * g;
                mx_u32x4 v = *(const mx_u32x4*)(q + m * dim + (d < dim ? d : dim - 8));
                const uint32_t on = d < dim ? 0xffffffffu : 0u;  // (dimensions past the head's: zero in q, anything in k)
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] &= on;
                qf[m][ks] = __builtin_bit_cast(mx_frag, v);
            }
    }
    mx_u32x4 kf[2][MAPS][KS], rv[2 * NG];
    auto load_k = [&](int s0) __attribute__((always_inline)) {
#pragma unroll
        for (int jb = 0; jb < 2; ++jb) {
            const int r = s0 + 16 * jb + c16;
            const uint16_t* p = base + (int64_t)(r < a.ring ? r : a.ring - 1) * a.rs;
#pragma unroll
            for (int m = 0; m < MAPS; ++m)
#pragma unroll
                for (int ks = 0; ks < KS; ++ks) {
                    const int d = 32 * ks + 8 * g;
                    kf[jb][m][ks] = *(const mx_u32x4*)(p + m * dim + (d < dim ? d : dim - 8));
                }
        }
    };
    auto load_v = [&](int s0) __attribute__((always_inline)) {   // item: eight values of a slot
#pragma unroll
        for (int i = 0; i < 2 * NG; ++i) {
            const int it = lane + 64 * i, r = s0 + it / (4 * NG), d = 8 * (it % (4 * NG));
            rv[i] = *(const mx_u32x4*)(vbase + (int64_t)(r < a.ring ? r : a.ring - 1) * a.rs + (d < dv ? d : dv - 8));
        }
    };
    const int step = a.n_split * 128;
    int s0 = (split * 4 + wave) * 32;
    load_k(s0);
    load_v(s0);
    const int64_t pos = a.pos[b];
    const int used = pos + 1 < a.ring ? (int)pos + 1 : a.ring;
    f32x4_t o[MAPS][NG][2];
    float mx[MAPS], den[MAPS];                                   // den: this lane's slots
#pragma unroll
    for (int m = 0; m < MAPS; ++m) {
        mx[m] = FLOOR;
        den[m] = 0.f;
#pragma unroll
        for (int n = 0; n < NG; ++n) o[m][n][0] = o[m][n][1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
    for (; s0 < used; s0 += step) {
        f32x4_t s[MAPS][2];
#pragma unroll
        for (int jb = 0; jb < 2; ++jb)
#pragma unroll
            for (int m = 0; m < MAPS; ++m) {
                s[m][jb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int ks = 0; ks < KS; ++ks) s[m][jb] = mfma16(__builtin_bit_cast(mx_frag, kf[jb][m][ks]), qf[m][ks], s[m][jb]);
            }
        __builtin_amdgcn_sched_barrier(0);
        load_k(s0 + step);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int i = 0; i < 2 * NG; ++i) {
            const int it = lane + 64 * i;
            *(mx_u32x4*)(vt + it / (4 * NG) * VP + 8 * (it % (4 * NG))) = rv[i];
        }
        __builtin_amdgcn_sched_barrier(0);
        load_v(s0 + step);
        __builtin_amdgcn_sched_barrier(0);
        mx_frag pf[MAPS];
#pragma unroll
        for (int m = 0; m < MAPS; ++m) {
            float top = mx[m];
#pragma unroll
            for (int jb = 0; jb < 2; ++jb)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    s[m][jb][r] = s0 + 16 * jb + 4 * g + r < used ? s[m][jb][r] * a.sc2 : -INFINITY;
                    top = fmaxf(top, s[m][jb][r]);
                }
            top = fmaxf(top, __shfl_xor(top, 16, 64));
            top = fmaxf(top, __shfl_xor(top, 32, 64));
            if (__builtin_amdgcn_ballot_w64(top > mx[m])) {
                const float f = __builtin_amdgcn_exp2f(mx[m] - top);
                mx[m] = top;
                den[m] *= f;
#pragma unroll
                for (int n = 0; n < NG; ++n)
#pragma unroll
                    for (int u = 0; u < 2; ++u)
#pragma unroll
                        for (int r = 0; r < 4; ++r) o[m][n][u][r] *= f;
            }
            uint32_t w[4];
#pragma unroll
            for (int jb = 0; jb < 2; ++jb) {
                float e[4];
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    e[r] = __builtin_amdgcn_exp2f(s[m][jb][r] - mx[m]);
                    den[m] += e[r];
                }
                w[2 * jb] = pack_bf2(e[0], e[1]);
                w[2 * jb + 1] = pack_bf2(e[2], e[3]);
            }
            pf[m] = frag_of(w[0], w[1], w[2], w[3]);
        }
        __builtin_amdgcn_wave_barrier();                         // (LDS accesses of a wave stay in order: the tile is complete)
#pragma unroll
        for (int n = 0; n < NG; ++n) {
            uint32_t x[8], ev[4], od[4];
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] = *(const uint32_t*)(vt + (16 * (e >> 2) + 4 * g + (e & 3)) * VP + 32 * n + 2 * c16);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                ev[e] = (x[2 * e] & 0xffffu) | x[2 * e + 1] << 16;
                od[e] = x[2 * e] >> 16 | (x[2 * e + 1] & 0xffff0000u);
            }
#pragma unroll
            for (int m = 0; m < MAPS; ++m) {
                o[m][n][0] = mfma16(frag_of(ev[0], ev[1], ev[2], ev[3]), pf[m], o[m][n][0]);
                o[m][n][1] = mfma16(frag_of(od[0], od[1], od[2], od[3]), pf[m], o[m][n][1]);
            }
        }
        __builtin_amdgcn_wave_barrier();
    }
    // the four waves' sums, on their common maximum
#pragma unroll
    for (int m = 0; m < MAPS; ++m) {
        den[m] += __shfl_xor(den[m], 16, 64);
        den[m] += __shfl_xor(den[m], 32, 64);
        if (g == 0) { ml[wave][m][c16][0] = mx[m]; ml[wave][m][c16][1] = den[m]; }
    }
    __syncthreads();                                             // (every wave is done with the value tiles, too)
    float* acc = (float*)lds;                                    // [MAPS][16][AP]
    float f[MAPS];
#pragma unroll
    for (int m = 0; m < MAPS; ++m) {
        const float top = fmaxf(fmaxf(ml[0][m][c16][0], ml[1][m][c16][0]), fmaxf(ml[2][m][c16][0], ml[3][m][c16][0]));
        f[m] = __builtin_amdgcn_exp2f(mx[m] - top);
        if (wave == 0 && g == 0 && c16 < nq) {
            float l = 0.f;
#pragma unroll
            for (int w = 0; w < 4; ++w) l = fmaf(ml[w][m][c16][1], __builtin_amdgcn_exp2f(ml[w][m][c16][0] - top), l);
            float* dst = a.part_ml + 2 * ((((int64_t)b * a.H + h0 + c16) * MAPS + m) * a.n_split + split);
            dst[0] = top;
            dst[1] = l;
        }
    }
    for (int w = 0; w < 4; ++w) {
        if (wave == w) {
#pragma unroll
            for (int m = 0; m < MAPS; ++m)
#pragma unroll
                for (int n = 0; n < NG; ++n)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        float2* p = (float2*)(acc + (m * 16 + c16) * AP + 32 * n + 8 * g + 2 * r);
                        float2 v = make_float2(o[m][n][0][r] * f[m], o[m][n][1][r] * f[m]);
                        if (w) { const float2 old = *p; v.x += old.x; v.y += old.y; }
                        *p = v;
                    }
        }
        __syncthreads();
    }
    for (int it = tid; it < MAPS * nq * (dv / 4); it += 256) {   // (dv % 8 == 0)
        const int m = it / (nq * (dv / 4)), c = it / (dv / 4) % nq, d = it % (dv / 4) * 4;
        *(float4*)(a.part_o + ((((int64_t)b * a.H + h0 + c) * MAPS + m) * a.n_split + split) * dv + d) = *(const float4*)(acc + (m * 16 + c) * AP + d);
    }
}

// Any sizes, both storage types: one wave per (split, head and map, sequence)
template <typename T>
__global__ __launch_bounds__(64) void heads_decode_any_kernel(HDecArgs a, int maps) {
    extern __shared__ float qs[];
    const int split = blockIdx.x, hm = blockIdx.y, b = blockIdx.z, lane = threadIdx.x;
    const int hk = hm / maps / (a.H / a.G), m_ = hm % maps;
    const T* q = (const T*)a.z + (int64_t)b * a.ld + (int64_t)hm * a.dim;
    for (int d = lane; d < a.dim; d += 64) qs[d] = ld1(q + d);
    __syncthreads();
    const int64_t pos = a.pos[b];
    const int used = pos + 1 < a.ring ? (int)pos + 1 : a.ring;
    const T* k = (const T*)a.cache + (int64_t)b * a.ring * a.rs + (int64_t)(hk * maps + m_) * a.dim;
    const T* v = (const T*)a.cache + (int64_t)b * a.ring * a.rs + (int64_t)a.G * maps * a.dim + (int64_t)hk * a.dv;
    float m = FLOOR, l = 0.f, o[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = 0.f;
    for (int s0 = split * 64; s0 < used; s0 += a.n_split * 64) {
        const int slot = s0 + lane;
        float s = -INFINITY;
        if (slot < used) {
            s = 0.f;
            for (int d = 0; d < a.dim; ++d) s = fmaf(qs[d], ld1(k + (int64_t)slot * a.rs + d), s);
            s *= a.sc2;
        }
        const float top = fmaxf(m, wave_max(s)), f = exp2f(m - top), p = exp2f(s - top);
        m = top;
        l = l * f + wave_sum(p);
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] *= f;
        const int n = used - s0 < 64 ? used - s0 : 64;
        for (int u = 0; u < n; ++u) {
            const float pu = __shfl(p, u, 64);
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (lane + 64 * e < a.dv) o[e] = fmaf(pu, ld1(v + (int64_t)(s0 + u) * a.rs + lane + 64 * e), o[e]);
        }
    }
    const int64_t p = ((int64_t)b * a.H * maps + hm) * a.n_split + split;
#pragma unroll
    for (int e = 0; e < 8; ++e)
        if (lane + 64 * e < a.dv) a.part_o[p * a.dv + lane + 64 * e] = o[e];
    if (lane == 0) { a.part_ml[2 * p] = m; a.part_ml[2 * p + 1] = l; }
}

extern "C" int evo_heads_decode(const void* z, int64_t ld, const void* cache, const int64_t* pos, float* part_o, float* part_ml, int64_t B, int64_t H,
                                int64_t kv_heads, int64_t maps, int64_t dim, int64_t dv, int64_t ring, int64_t rs, int64_t n_split, float scale,
                                int64_t f32, int64_t mfma, void* stream) {
    if (!z || !cache || !pos || !part_o || !part_ml || B <= 0 || B > 65535 || H <= 0 || H > 16384 || kv_heads <= 0 || H % kv_heads) return -1;
    if ((maps != 1 && maps != 2) || dim <= 0 || dim > 8192 || dv <= 0 || dv > 512 || ring <= 0 || ring > 0x3fffffff || n_split <= 0 || n_split > 1024) return -1;
    if (ld < H * maps * dim || rs < kv_heads * (maps * dim + dv) || rs > 0x3fffffff) return -1;
    const int64_t Q = H / kv_heads;
    HDecArgs a = {z, ld, cache, pos, part_o, part_ml, (int)H, (int)kv_heads, (int)dim, (int)dv, (int)rs, (int)ring, (int)n_split, (int)((Q + 15) / 16), scale * LOG2E};
    hipStream_t s = (hipStream_t)stream;
    if (!f32 && mfma && dim % 8 == 0 && dv % 8 == 0 && ld % 8 == 0 && rs % 8 == 0 && dim <= (maps == 2 ? 128 : 256) && dv <= 256 &&
        (((uintptr_t)z | (uintptr_t)cache | (uintptr_t)part_o) & 15) == 0) {
        const dim3 grid((unsigned)n_split, (unsigned)(kv_heads * a.n_qb), (unsigned)B);
#define HD(KS, NG, MAPS)                                                                                                   \
    do {                                                                                                                   \
        constexpr int tiles = 4 * 32 * (32 * NG + 8) * 2, meet = MAPS * 16 * (32 * NG + 4) * 4, bytes = tiles > meet ? tiles : meet;   \
        if (bytes > 60 * 1024) (void)hipFuncSetAttribute((const void*)heads_decode_kernel<KS, NG, MAPS>, hipFuncAttributeMaxDynamicSharedMemorySize, bytes); \
        hipLaunchKernelGGL((heads_decode_kernel<KS, NG, MAPS>), grid, dim3(256), (size_t)bytes, s, a);                     \
    } while (0)
#define HDV(KS, MAPS) do { if (dv <= 64) HD(KS, 2, MAPS); else if (dv <= 128) HD(KS, 4, MAPS); else HD(KS, 8, MAPS); } while (0)
        if (maps == 2) { if (dim <= 64) HDV(2, 2); else HDV(4, 2); }
        else if (dim <= 64) HDV(2, 1); else if (dim <= 128) HDV(4, 1); else HDV(8, 1);
#undef HDV
#undef HD
        return evo_launch_status();
    }
    const dim3 grid((unsigned)n_split, (unsigned)(H * maps), (unsigned)B);
    if (f32) hipLaunchKernelGGL((heads_decode_any_kernel<float>), grid, dim3(64), (size_t)dim * 4, s, a, (int)maps);
    else hipLaunchKernelGGL((heads_decode_any_kernel<uint16_t>), grid, dim3(64), (size_t)dim * 4, s, a, (int)maps);
    return evo_launch_status();
}

// o = the merged parts of a head; two maps: gain * unit_rms(o1 - lam o2) over its dv values
template <typename T, int MAPS>
__global__ __launch_bounds__(128) void heads_merge_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, void* __restrict__ o_, int H,
                                                          int dv, int n_split, float lam, float gain, float eps) {
    extern __shared__ float wt[];                                // [MAPS][n_split] weights of the parts
    __shared__ float red[2];
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int64_t p0 = ((int64_t)b * H + h) * MAPS * n_split;
    if (wave < MAPS) {
        const float* ml = part_ml + 2 * (p0 + (int64_t)wave * n_split);
        float top = FLOOR;
        for (int s = lane; s < n_split; s += 64) top = fmaxf(top, ml[2 * s]);
        top = wave_max(top);
        float l = 0.f;
        for (int s = lane; s < n_split; s += 64) l = fmaf(ml[2 * s + 1], exp2f(ml[2 * s] - top), l);
        l = wave_sum(l);
        for (int s = lane; s < n_split; s += 64) wt[wave * n_split + s] = exp2f(ml[2 * s] - top) / l;
    }
    __syncthreads();
    float x[4], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int d = tid + 128 * e;
        x[e] = 0.f;
        if (d < dv) {
            float a[MAPS];
#pragma unroll
            for (int m = 0; m < MAPS; ++m) {
                a[m] = 0.f;
                const float* po = part_o + (p0 + (int64_t)m * n_split) * dv + d;
#pragma unroll 8
                for (int s = 0; s < n_split; ++s) a[m] = fmaf(po[(int64_t)s * dv], wt[m * n_split + s], a[m]);
            }
            x[e] = MAPS == 2 ? a[0] - lam * a[MAPS - 1] : a[0];
        }
        ss = fmaf(x[e], x[e], ss);
    }
    float f = 1.0f;
    if constexpr (MAPS == 2) {
        ss = wave_sum(ss);
        if (lane == 0) red[wave] = ss;
        __syncthreads();
        f = gain / sqrtf((red[0] + red[1]) / (float)dv + eps);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (tid + 128 * e < dv) st1((T*)o_ + ((int64_t)b * H + h) * dv + tid + 128 * e, x[e] * f);
}

extern "C" int evo_heads_merge(const float* part_o, const float* part_ml, void* o, int64_t B, int64_t H, int64_t maps, int64_t dv, int64_t n_split, float lam,
                               float gain, float eps, int64_t f32, void* stream) {
    if (!part_o || !part_ml || !o || B <= 0 || B > 65535 || H <= 0 || (maps != 1 && maps != 2) || dv <= 0 || dv > 512 || n_split <= 0 || n_split > 1024) return -1;
    const dim3 grid((unsigned)H, (unsigned)B), block(128);
    const size_t lds = (size_t)maps * n_split * 4;
    hipStream_t s = (hipStream_t)stream;
#define HM(T, MAPS) hipLaunchKernelGGL((heads_merge_kernel<T, MAPS>), grid, block, lds, s, part_o, part_ml, o, (int)H, (int)dv, (int)n_split, lam, gain, eps)
    if (f32) { if (maps == 2) HM(float, 2); else HM(float, 1); }
    else { if (maps == 2) HM(uint16_t, 2); else HM(uint16_t, 1); }
#undef HM
    return evo_launch_status();
}
