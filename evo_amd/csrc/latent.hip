// Latent attention: keys and values of every head are linear maps of one normed latent c per token, plus one rotated key part shared by
// all heads; sliding window; one sink per head in the softmax denominator.  Entry points: include/evo_mi355x.h.
//   prompts:  q | down-projection row -> latent_prep (norm, rotation, cache append) -> k, v of every head by one dense layer -> window
//             attention (csrc/window_attn.hip)
//   decode:   the key map is moved to the query side (q_abs = W_uk^T q), scores and the weighted sum run on the cached latents themselves,
//             the value map is applied to the one combined latent:  latent_absorb -> latent_decode (split over the window) -> latent_up
#include "mixers_common.h"
#include "../../include/evo_mi355x.h"

#define LOG2E 1.4426950408889634f

// ------------------------------------------------------------------------------------------------ norm, rotation, cache append
struct PrepArgs {
    void* q; int64_t ldq;                                        // row m: H heads of [dn | dr] (rotated in place), then [R | dr] (read)
    void* c; void* kr; void* cache;                              // c [M, R] / kr [M, dr] or null; cache [rows, ring, rs] or null
    const void* w; const float* inv_freq; const int64_t* pos; const int* seq; const int* cu;
    int H, dn, dr, R, n_rot, ring, rs;
    float eps;
};

template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(PrepArgs a) {
    extern __shared__ float2 turn[];                             // [n_rot / 2] cosine and sine of this token's angles
    __shared__ float red[4];
    const int m = blockIdx.x, tid = threadIdx.x;
    const int b = a.seq ? a.seq[m] : m;
    T* q = (T*)a.q + (int64_t)m * a.ldq;
    const int64_t pos = a.pos[m];
    const int half = a.n_rot / 2, dh = a.dn + a.dr;
    const T* dkv = q + a.H * dh;
    T* slot = nullptr;
    if (a.cache && (!a.cu || a.cu[b + 1] - m <= a.ring)) slot = (T*)a.cache + ((int64_t)b * a.ring + pos % a.ring) * a.rs;
    for (int i = tid; i < half; i += 256) sincosf((float)pos * a.inv_freq[i], &turn[i].y, &turn[i].x);
    float ss = 0.f;
    for (int r = tid; r < a.R; r += 256) { const float v = ld1(dkv + r); ss = fmaf(v, v, ss); }
    const float inv = 1.0f / sqrtf(block_sum_256(ss, red) / (float)a.R + a.eps);
    for (int r = tid; r < a.R; r += 256) {
        const float v = ld1(dkv + r) * inv * ld1((const T*)a.w + r);
        if (a.c) st1((T*)a.c + (int64_t)m * a.R + r, v);
        if (slot) st1(slot + r, v);
    }
    // rotation: pair (i, i + half) of the first n_rot elements of every head's rotated part, and of the shared key part (index H)
    // (the reduction's barrier above is behind every thread's angles)
    for (int it = tid; it < (a.H + 1) * half; it += 256) {
        const int h = it / half, i = it - h * half;
        const float cs = turn[i].x, sn = turn[i].y;
        if (h < a.H) {
            T* x = q + h * dh + a.dn;
            const float u = ld1(x + i), v = ld1(x + i + half);
            st1(x + i, u * cs - v * sn);
            st1(x + i + half, v * cs + u * sn);
        } else {
            const float u = ld1(dkv + a.R + i), v = ld1(dkv + a.R + i + half);
            const float x = u * cs - v * sn, y = v * cs + u * sn;
            if (a.kr) { st1((T*)a.kr + (int64_t)m * a.dr + i, x); st1((T*)a.kr + (int64_t)m * a.dr + i + half, y); }
            if (slot) { st1(slot + a.R + i, x); st1(slot + a.R + i + half, y); }
        }
    }
    for (int i = a.n_rot + tid; i < a.dr; i += 256) {            // the part of the shared key that is not rotated
        const float v = ld1(dkv + a.R + i);
        if (a.kr) st1((T*)a.kr + (int64_t)m * a.dr + i, v);
        if (slot) st1(slot + a.R + i, v);
    }
}

extern "C" int evo_latent_prep(void* q, int64_t ldq, void* c, void* kr, void* cache, const void* w, const float* inv_freq, const int64_t* pos,
                               const int* seq, const int* cu, int64_t M, int64_t H, int64_t dn, int64_t dr, int64_t R, int64_t n_rot, int64_t ring,
                               int64_t rs, float eps, int64_t f32, void* stream) {
    if (!q || !w || !inv_freq || !pos || M <= 0 || M > 0x7fffffff || H <= 0 || dn < 0 || dr < 0 || R <= 0 || n_rot < 0 || n_rot > dr || n_rot % 2 || n_rot > 8192) return -1;
    if (ldq < H * (dn + dr) + R + dr || (cache && (ring <= 0 || rs < R + dr)) || (cu && !seq) || (H + 1) * (dn + dr) > 0x3fffffff) return -1;
    PrepArgs a = {q, ldq, c, kr, cache, w, inv_freq, pos, seq, cu, (int)H, (int)dn, (int)dr, (int)R, (int)n_rot, (int)ring, (int)rs, eps};
    if (f32) hipLaunchKernelGGL((latent_prep_kernel<float>), dim3((unsigned)M), dim3(256), (size_t)n_rot * 4, (hipStream_t)stream, a);
    else hipLaunchKernelGGL((latent_prep_kernel<uint16_t>), dim3((unsigned)M), dim3(256), (size_t)n_rot * 4, (hipStream_t)stream, a);
    return evo_launch_status();
}

// ------------------------------------------------------------------------------------------------ decode: query side of the key map
// out[b][h] = [W_uk,h^T q_n (R) | rotated q (dr) | zeros up to rs].  Workgroup: 64 V latent columns of one head, NB sequences; eight waves
// share the dn rows of the map, a lane owns V adjacent columns.
template <typename T, int NB, int V>
__global__ __launch_bounds__(512) void latent_absorb_kernel(const void* __restrict__ q_, int64_t ldq, const void* __restrict__ w_, void* __restrict__ out_,
                                                            int B, int H, int dn, int dr, int R, int rs) {
    extern __shared__ float sm[];                                // q parts [NB][dn], partial sums [8][NB][64 V]
    float* part = sm + NB * dn;
    const int h = blockIdx.y, b0 = blockIdx.z * NB, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int nb = B - b0 < NB ? B - b0 : NB, dh = dn + dr;
#pragma unroll
    for (int i = 0; i < NB; ++i)
        for (int n = tid; n < dn; n += 512) sm[i * dn + n] = i < nb ? ld1((const T*)q_ + (int64_t)(b0 + i) * ldq + (int64_t)h * dh + n) : 0.f;
    __syncthreads();
    const int r0 = blockIdx.x * 64 * V, r = r0 + lane * V;
    const T* w = (const T*)w_ + (int64_t)h * dn * R + r;
    float acc[NB][V];
#pragma unroll
    for (int i = 0; i < NB; ++i)
#pragma unroll
        for (int e = 0; e < V; ++e) acc[i][e] = 0.f;
    if (r < R) {
        int n = wave;
        for (; n + 24 < dn; n += 32) {
            float f[4][V];
#pragma unroll
            for (int u = 0; u < 4; ++u) vec_io<T, V>::load(w + (int64_t)(n + 8 * u) * R, f[u]);
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int i = 0; i < NB; ++i)
#pragma unroll
                    for (int e = 0; e < V; ++e) acc[i][e] = fmaf(f[u][e], sm[i * dn + n + 8 * u], acc[i][e]);
        }
        for (; n < dn; n += 8) {
            float f[V];
            vec_io<T, V>::load(w + (int64_t)n * R, f);
#pragma unroll
            for (int i = 0; i < NB; ++i)
#pragma unroll
                for (int e = 0; e < V; ++e) acc[i][e] = fmaf(f[e], sm[i * dn + n], acc[i][e]);
        }
    }
#pragma unroll
    for (int i = 0; i < NB; ++i) vec_io<float, V>::store(part + ((wave * NB + i) * 64 + lane) * V, acc[i]);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NB; ++i) {
        if (i >= nb) break;
        T* out = (T*)out_ + ((int64_t)(b0 + i) * H + h) * rs;
        for (int c = tid; c < 64 * V; c += 512) {
            float v = 0.f;
#pragma unroll
            for (int k = 0; k < 8; ++k) v += part[(k * NB + i) * 64 * V + c];
            if (r0 + c < R) st1(out + r0 + c, v);
        }
        if (blockIdx.x == 0)
            for (int c = R + tid; c < rs; c += 512)
                st1(out + c, c < R + dr ? ld1((const T*)q_ + (int64_t)(b0 + i) * ldq + (int64_t)h * dh + dn + c - R) : 0.f);
    }
}

extern "C" int evo_latent_absorb(const void* q, int64_t ldq, const void* wuk, void* out, int64_t B, int64_t H, int64_t dn, int64_t dr, int64_t R,
                                 int64_t rs, int64_t f32, void* stream) {
    if (!q || !wuk || !out || B <= 0 || H <= 0 || H > 65535 || dn <= 0 || dn > 4096 || dr < 0 || R <= 0 || rs < R + dr || ldq < H * (dn + dr)) return -1;
    const int nb = B > 2 ? 4 : (int)B, v = R % 8 == 0 && ((uintptr_t)wuk & 15) == 0 ? 8 : 1;
    const dim3 grid((unsigned)((R + 64 * v - 1) / (64 * v)), (unsigned)H, (unsigned)((B + nb - 1) / nb)), block(512);
    const size_t lds = (size_t)nb * (dn + 512 * v) * 4;          // (<= 128 KB)
    hipStream_t s = (hipStream_t)stream;
#define AB(T, NB, V)                                                                                                       \
    do {                                                                                                                   \
        if (lds > 64 * 1024) (void)hipFuncSetAttribute((const void*)latent_absorb_kernel<T, NB, V>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
        hipLaunchKernelGGL((latent_absorb_kernel<T, NB, V>), grid, block, lds, s, q, ldq, wuk, out, (int)B, (int)H, (int)dn, (int)dr, (int)R, (int)rs); \
    } while (0)
#define ABV(T, V) do { if (nb == 1) AB(T, 1, V); else if (nb == 2) AB(T, 2, V); else AB(T, 4, V); } while (0)
    if (f32) { if (v == 8) ABV(float, 8); else ABV(float, 1); }
    else { if (v == 8) ABV(uint16_t, 8); else ABV(uint16_t, 1); }
#undef ABV
#undef AB
    return evo_launch_status();
}

// ------------------------------------------------------------------------------------------------ decode: scores and sum on the latents
// The cache of a sequence is a ring: token j sits at slot j % ring.  A slot's age is (pos - slot) mod ring; it is seen when the age is below
// the window and not above pos.  Slots are walked in memory order: the order of keys does not matter to a softmax.
struct DecArgs {
    const void* q; const void* cache; const int64_t* pos; float* part_o; float* part_ml;   // part_ml: [.., 2] running max (log2 domain), denominator
    int H, R, rs, ring, window, n_split;
    float sc2;                                                   // scale * log2(e)
};
__device__ __forceinline__ bool slot_seen(int slot, int64_t pos, int cur, const DecArgs& a) {
    int age = cur - slot;
    age = age < 0 ? age + a.ring : age;
    return slot < a.ring && age < a.window && age <= pos;
}

// Matrix cores (bf16).  A workgroup of eight waves: 16 CB heads of one sequence against its share of 64-slot tiles.  A tile comes once from
// memory into LDS (the next one is on its way in registers meanwhile) and is read as rows for the scores and as pairs of columns for the sum:
//   scores   S^T = tile q^T; wave (row block, half of the row) -> two halves of [heads][64 slots] in LDS
//   softmax  a wave owns 2 CB heads, a lane one slot; running maximum and denominator stay with the head's wave; probabilities -> LDS (bf16)
//   sum      a wave owns every eighth 32-wide group of latents; a dword holds latents 2 i, 2 i + 1 of a slot: the even and the odd latents of
//            a group are two operands, no transposed copy exists
// NR: 32-wide groups of latents, KS: of the whole row (rs = 32 KS).  The loads carry no branch: with one among them the wait for a tile's rows
// cannot be told from the wait for the next tile's.
template <int NR, int KS, int CB>
__global__ __launch_bounds__(512, 2) void latent_decode_kernel(DecArgs a) {
    constexpr int KH = (KS + 1) / 2;                             // 32-wide steps of half a row
    constexpr int GPW = (NR + 7) / 8;                            // latent groups per wave
    constexpr int LI = (KS + 1) / 2;                             // 16-byte pieces of a tile per thread
    constexpr int SP = 68, PP = 72;                              // pitches of the score and probability rows
    extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int split = blockIdx.x, h0 = blockIdx.y * 16 * CB, b = blockIdx.z;
    constexpr int rs = 32 * KS, pr = rs + 8;
    uint16_t* tile = lds;                                        // [64][pr]
    float* sc = (float*)(tile + 64 * pr);                        // [2][16 CB][SP]
    float* fac = sc + 2 * 16 * CB * SP;                          // [16 CB]
    uint16_t* pb = (uint16_t*)(fac + 16 * CB);                   // [16 CB][PP]
    const int rb = wave & 3, kh = wave >> 2;
    const int ks0 = kh ? KH : 0, ks1 = kh ? KS : KH;
    mx_frag qf[CB][KH];
#pragma unroll
    for (int cb = 0; cb < CB; ++cb)
#pragma unroll
        for (int i = 0; i < KH; ++i) {
            const int h = h0 + 16 * cb + c16, ks = ks0 + i < KS ? ks0 + i : KS - 1;
            mx_u32x4 v = *(const mx_u32x4*)((const uint16_t*)a.q + ((int64_t)b * a.H + (h < a.H ? h : a.H - 1)) * rs + 32 * ks + 8 * g);
            const uint32_t keep = ks0 + i < ks1 ? 0xffffffffu : 0u;              // (an odd row's last step exists in one half only)
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] &= keep;
            qf[cb][i] = __builtin_bit_cast(mx_frag, v);
        }
    const uint16_t* base = (const uint16_t*)a.cache + (int64_t)b * a.ring * rs;
    mx_u32x4 nx[LI];
    const int row_t = tid >> 3, col_t = (tid & 7) * 8;           // eight threads share a row: 128 contiguous bytes per request
    const int col_l = (KS & 1) && col_t >= 32 ? col_t - 32 : col_t;   // last group of an odd row: its four pieces twice
    auto load = [&](int s0) __attribute__((always_inline)) {
        const uint16_t* p = base + (int64_t)(s0 + row_t < a.ring ? s0 + row_t : a.ring - 1) * rs;   // (no wait for the position: slots never written are masked)
#pragma unroll
        for (int i = 0; i < LI; ++i) nx[i] = *(const mx_u32x4*)(p + (i == LI - 1 ? col_l : col_t) + 64 * i);
    };
    if (split * 64 < a.ring) load(split * 64);
    const int64_t pos = a.pos[b];
    const int cur = (int)((uint64_t)pos < 0x80000000u ? (uint32_t)pos % (uint32_t)a.ring : pos % a.ring);
    const int used = pos + 1 < a.ring ? (int)pos + 1 : a.ring;   // slots that have ever been written by this sequence
    f32x4_t o[GPW][2][CB];
#pragma unroll
    for (int i = 0; i < GPW; ++i)
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int cb = 0; cb < CB; ++cb) o[i][u][cb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    float mx[2 * CB], den[2 * CB];                               // of heads wave 2 CB + i; den: this lane's slots
#pragma unroll
    for (int i = 0; i < 2 * CB; ++i) { mx[i] = -INFINITY; den[i] = 0.f; }
    const int step = a.n_split * 64;
    for (int s0 = split * 64; s0 < used; s0 += step) {
#pragma unroll
        for (int i = 0; i < LI; ++i) *(mx_u32x4*)(tile + row_t * pr + (i == LI - 1 ? col_l : col_t) + 64 * i) = nx[i];
        __syncthreads();
        if (s0 + step < used) load(s0 + step);
        f32x4_t s[CB];
#pragma unroll
        for (int cb = 0; cb < CB; ++cb) s[cb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < KH; ++i) {
            const int ks = ks0 + i < KS ? ks0 + i : KS - 1;
            const mx_frag kf = __builtin_bit_cast(mx_frag, *(const uint4*)(tile + (16 * rb + c16) * pr + 32 * ks + 8 * g));
#pragma unroll
            for (int cb = 0; cb < CB; ++cb) s[cb] = mfma16(kf, qf[cb][i], s[cb]);
        }
#pragma unroll
        for (int cb = 0; cb < CB; ++cb) *(f32x4_t*)(sc + (kh * 16 * CB + 16 * cb + c16) * SP + 16 * rb + 4 * g) = s[cb];
        __syncthreads();
        const bool seen = slot_seen(s0 + lane, pos, cur, a);
#pragma unroll
        for (int i = 0; i < 2 * CB; ++i) {
            const int h = wave * 2 * CB + i;
            const float x = seen ? (sc[h * SP + lane] + sc[(16 * CB + h) * SP + lane]) * a.sc2 : -INFINITY;
            const float top = fmaxf(mx[i], wave_max(x));
            const bool any = top > -INFINITY;                    // (a tile may hold no seen slot at all)
            const float f = any ? __builtin_amdgcn_exp2f(mx[i] - top) : 1.f, p = seen && any ? __builtin_amdgcn_exp2f(x - top) : 0.f;
            mx[i] = top;
            den[i] = den[i] * f + p;
            pb[h * PP + lane] = f_to_bf(p);
            if (lane == 0) fac[h] = f;
        }
        __syncthreads();
        float f[CB];
#pragma unroll
        for (int cb = 0; cb < CB; ++cb) f[cb] = fac[16 * cb + c16];
        mx_frag pf[CB][2];
#pragma unroll
        for (int cb = 0; cb < CB; ++cb)
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) pf[cb][kk] = frag_split(pb + (16 * cb + c16) * PP + 32 * kk + 4 * g);
#pragma unroll
        for (int i = 0; i < GPW; ++i) {
            const int grp = wave + 8 * i;
            if (grp < NR) {
#pragma unroll
                for (int u = 0; u < 2; ++u)
#pragma unroll
                    for (int cb = 0; cb < CB; ++cb)
#pragma unroll
                        for (int r = 0; r < 4; ++r) o[i][u][cb][r] *= f[cb];
#pragma unroll
                for (int kk = 0; kk < 2; ++kk) {
                    uint32_t x[8], ev[4], od[4];
#pragma unroll
                    for (int e = 0; e < 8; ++e) x[e] = *(const uint32_t*)(tile + (32 * kk + 16 * (e >> 2) + 4 * g + (e & 3)) * pr + 32 * grp + 2 * c16);
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        ev[e] = (x[2 * e] & 0xffffu) | x[2 * e + 1] << 16;
                        od[e] = x[2 * e] >> 16 | (x[2 * e + 1] & 0xffff0000u);
                    }
#pragma unroll
                    for (int cb = 0; cb < CB; ++cb) {
                        o[i][0][cb] = mfma16(frag_of(ev[0], ev[1], ev[2], ev[3]), pf[cb][kk], o[i][0][cb]);
                        o[i][1][cb] = mfma16(frag_of(od[0], od[1], od[2], od[3]), pf[cb][kk], o[i][1][cb]);
                    }
                }
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 2 * CB; ++i) {
        const int h = h0 + wave * 2 * CB + i;
        const float l = wave_sum(den[i]);
        if (lane == 0 && h < a.H) {
            const int64_t p = ((int64_t)b * a.H + h) * a.n_split + split;
            a.part_ml[2 * p] = mx[i];
            a.part_ml[2 * p + 1] = l;
        }
    }
#pragma unroll
    for (int i = 0; i < GPW; ++i)
#pragma unroll
        for (int cb = 0; cb < CB; ++cb) {
            const int grp = wave + 8 * i, h = h0 + 16 * cb + c16;
            if (grp < NR && h < a.H) {
                float* po = a.part_o + (((int64_t)b * a.H + h) * a.n_split + split) * a.R;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int col = 32 * grp + 8 * g + 2 * r;
                    if (col + 1 < a.R && (a.R & 1) == 0) *(float2*)(po + col) = make_float2(o[i][0][cb][r], o[i][1][cb][r]);
                    else {
                        if (col < a.R) po[col] = o[i][0][cb][r];
                        if (col + 1 < a.R) po[col + 1] = o[i][1][cb][r];
                    }
                }
            }
        }
}

// Any sizes, both storage types: one wave per (split, head, sequence)
template <typename T>
__global__ __launch_bounds__(64) void latent_decode_any_kernel(DecArgs a, int dq) {
    extern __shared__ float qf[];
    const int split = blockIdx.x, h = blockIdx.y, b = blockIdx.z, lane = threadIdx.x;
    const T* q = (const T*)a.q + ((int64_t)b * a.H + h) * a.rs;
    for (int d = lane; d < dq; d += 64) qf[d] = ld1(q + d);
    __syncthreads();
    const int64_t pos = a.pos[b];
    const int cur = (int)(pos % a.ring);
    const T* base = (const T*)a.cache + (int64_t)b * a.ring * a.rs;
    const int64_t p = ((int64_t)b * a.H + h) * a.n_split + split;
    float m = -INFINITY, l = 0.f;
    float* po = a.part_o + p * a.R;
    const int used = pos + 1 < a.ring ? (int)pos + 1 : a.ring;
    for (int pass = 0; pass < (a.R + 511) / 512; ++pass) {       // 512 latent columns per pass (the scores are recomputed per pass)
        float o[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = 0.f;
        m = -INFINITY; l = 0.f;
        for (int s0 = split * 64; s0 < used; s0 += a.n_split * 64) {
            const int slot = s0 + lane;
            float s = -INFINITY;
            if (slot < used && slot_seen(slot, pos, cur, a)) {
                s = 0.f;
                for (int d = 0; d < dq; ++d) s = fmaf(qf[d], ld1(base + (int64_t)slot * a.rs + d), s);
                s *= a.sc2;
            }
            const float top = fmaxf(m, wave_max(s));
            if (top == -INFINITY) continue;
            const float f = exp2f(m - top), pr = exp2f(s - top);
            m = top;
            l = l * f + wave_sum(pr);
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] *= f;
            const int n = used - s0 < 64 ? used - s0 : 64;
            for (int u = 0; u < n; ++u) {
                const float pu = __shfl(pr, u, 64);
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const int r = pass * 512 + lane + 64 * e;
                    if (r < a.R) o[e] = fmaf(pu, ld1(base + (int64_t)(s0 + u) * a.rs + r), o[e]);
                }
            }
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int r = pass * 512 + lane + 64 * e;
            if (r < a.R) po[r] = o[e];
        }
    }
    if (lane == 0) { a.part_ml[2 * p] = m; a.part_ml[2 * p + 1] = l; }
}

extern "C" int evo_latent_decode(const void* q, const void* cache, const int64_t* pos, float* part_o, float* part_ml, int64_t B, int64_t H, int64_t R,
                                 int64_t dr, int64_t rs, int64_t ring, int64_t window, int64_t n_split, float scale, int64_t f32, int64_t mfma,
                                 void* stream) {
    if (!q || !cache || !pos || !part_o || !part_ml || B <= 0 || B > 65535 || H <= 0 || H > 65535 || R <= 0 || dr < 0 || rs < R + dr || R + dr > 8192) return -1;
    if (ring <= 0 || ring > 0x3fffffff || window <= 0 || window > ring || n_split <= 0 || n_split > 64) return -1;
    DecArgs a = {q, cache, pos, part_o, part_ml, (int)H, (int)R, (int)rs, (int)ring, (int)window, (int)n_split, scale * LOG2E};
    hipStream_t s = (hipStream_t)stream;
    static const int steps[8] = {1, 2, 3, 4, 6, 8, 12, 16};      // latent groups the matrix-core kernel exists for, in rows one or two groups longer
    int nr = 0;
    for (int i = 7; i >= 0; --i)
        if (steps[i] * 32 >= R && (rs == 32 * (steps[i] + 1) || rs == 32 * (steps[i] + 2))) nr = steps[i];
    const int cb = mfma == 16 || H <= 16 ? 1 : 2;
    const size_t lds = (size_t)64 * (rs + 8) * 2 + (size_t)cb * 16 * (2 * 68 * 4 + 4 + 72 * 2);
    if (!f32 && mfma && nr && (((uintptr_t)q | (uintptr_t)cache) & 15) == 0) {
        const dim3 grid((unsigned)n_split, (unsigned)((H + 16 * cb - 1) / (16 * cb)), (unsigned)B), block(512);
#define LD1(NR, KS, CB)                                                                                                    \
    do {                                                                                                                   \
        if (lds > 64 * 1024) (void)hipFuncSetAttribute((const void*)latent_decode_kernel<NR, KS, CB>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
        hipLaunchKernelGGL((latent_decode_kernel<NR, KS, CB>), grid, block, lds, s, a);                                    \
    } while (0)
#define LD2(NR, KS) do { if (cb == 1) LD1(NR, KS, 1); else LD1(NR, KS, 2); } while (0)
#define LD(NR) do { if (rs == 32 * (NR + 1)) LD2(NR, NR + 1); else LD2(NR, NR + 2); } while (0)
        switch (nr) {
            case 1: LD(1); break;
            case 2: LD(2); break;
            case 3: LD(3); break;
            case 4: LD(4); break;
            case 6: LD(6); break;
            case 8: LD(8); break;
            case 12: LD(12); break;
            default: LD(16); break;
        }
#undef LD
#undef LD2
#undef LD1
        return evo_launch_status();
    }
    const dim3 grid((unsigned)n_split, (unsigned)H, (unsigned)B);
    if (f32) hipLaunchKernelGGL((latent_decode_any_kernel<float>), grid, dim3(64), (size_t)(R + dr) * 4, s, a, (int)(R + dr));
    else hipLaunchKernelGGL((latent_decode_any_kernel<uint16_t>), grid, dim3(64), (size_t)(R + dr) * 4, s, a, (int)(R + dr));
    return evo_launch_status();
}

// ------------------------------------------------------------------------------------------------ decode: merge, sink, value map
// o[b][h dv + v] = W_uv,h[v] . (sum_s w_s part_o[s]) / (sum_s w_s l_s + 2^(sink - top)).  Workgroup: one head, NB sequences (they share the
// weights), `rows` value rows; the merged latents sit in LDS, a wave takes a value row at a time.
template <typename T, int NB, int V>
__global__ __launch_bounds__(512) void latent_up_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, const float* __restrict__ sink,
                                                        const void* __restrict__ w_, void* __restrict__ o_, int B, int H, int R, int dv, int n_split,
                                                        int rows) {
    extern __shared__ float sm[];                                // [NB][R] latents, [NB][n_split] weights of the parts
    float* lat = sm;
    float* wt = sm + NB * R;
    const int h = blockIdx.y, b0 = blockIdx.z * NB, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    if (wave < NB) {                                             // a wave per sequence: the parts' weights
        const int b = b0 + wave;
        const float* ml = part_ml + ((int64_t)(b < B ? b : B - 1) * H + h) * n_split * 2;
        const float sk = sink[h] * LOG2E;
        float top = sk;
        for (int s = lane; s < n_split; s += 64) top = fmaxf(top, ml[2 * s]);
        top = wave_max(top);
        float l = 0.f;
        for (int s = lane; s < n_split; s += 64) l = fmaf(ml[2 * s + 1], exp2f(ml[2 * s] - top), l);
        l = wave_sum(l) + exp2f(sk - top);
        for (int s = lane; s < n_split; s += 64) wt[wave * n_split + s] = exp2f(ml[2 * s] - top) / l;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NB; ++i) {
        const int b = b0 + i < B ? b0 + i : B - 1;
        const float* po = part_o + ((int64_t)b * H + h) * n_split * R;
        for (int r = tid; r < R; r += 512) {
            float acc = 0.f;
#pragma unroll 8
            for (int s = 0; s < n_split; ++s) acc = fmaf(po[(int64_t)s * R + r], wt[i * n_split + s], acc);
            lat[i * R + r] = acc;
        }
    }
    __syncthreads();
    const int v_end = dv < (int)(blockIdx.x + 1) * rows ? dv : (blockIdx.x + 1) * rows;
    if (V == 8 && R <= 512) {                                    // a row is one request per lane; the lane's latents stay in registers
        float own[NB][V];
        const bool in = lane * V < R;
#pragma unroll
        for (int i = 0; i < NB; ++i)
#pragma unroll
            for (int e = 0; e < V; ++e) own[i][e] = in ? lat[i * R + lane * V + e] : 0.f;
#pragma unroll 4
        for (int v = blockIdx.x * rows + wave; v < v_end; v += 8) {
            float f[V];
            vec_io<T, V>::load((const T*)w_ + ((int64_t)h * dv + v) * R + (in ? lane * V : 0), f);
#pragma unroll
            for (int i = 0; i < NB; ++i) {
                float x = 0.f;
#pragma unroll
                for (int e = 0; e < V; ++e) x = fmaf(f[e], own[i][e], x);
                x = wave_sum(x);
                if (lane == 0 && b0 + i < B) st1((T*)o_ + (int64_t)(b0 + i) * H * dv + (int64_t)h * dv + v, x);
            }
        }
        return;
    }
#pragma unroll 4
    for (int v = blockIdx.x * rows + wave; v < v_end; v += 8) {
        const T* w = (const T*)w_ + ((int64_t)h * dv + v) * R;
        float acc[NB];
#pragma unroll
        for (int i = 0; i < NB; ++i) acc[i] = 0.f;
        for (int r = lane * V; r < R; r += 64 * V) {
            float f[V];
            vec_io<T, V>::load(w + r, f);
#pragma unroll
            for (int i = 0; i < NB; ++i)
#pragma unroll
                for (int e = 0; e < V; ++e) acc[i] = fmaf(f[e], lat[i * R + r + e], acc[i]);
        }
#pragma unroll
        for (int i = 0; i < NB; ++i) {
            const float x = wave_sum(acc[i]);
            if (lane == 0 && b0 + i < B) st1((T*)o_ + (int64_t)(b0 + i) * H * dv + (int64_t)h * dv + v, x);
        }
    }
}

// The same for 16 sequences at a time on the matrix cores (bf16, R % 32 == 0): 128 value rows of one head, a wave owns 16 of them
template <int NS>
__global__ __launch_bounds__(512) void latent_up_mfma_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, const float* __restrict__ sink,
                                                             const uint16_t* __restrict__ w, uint16_t* __restrict__ o, int B, int H, int R, int dv, int n_split) {
    extern __shared__ __attribute__((aligned(16))) uint16_t lat[];   // [NS][R + 8] merged latents, then [NS][n_split] weights of the parts
    const int h = blockIdx.y, b0 = blockIdx.z * NS, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int pr = R + 8, c16 = lane & 15, g = lane >> 4;
    float* wt = (float*)(lat + NS * pr);
    const int v0 = blockIdx.x * 128 + 16 * wave;
    for (int i = wave; i < NS; i += 8) {
        const int b = b0 + i < B ? b0 + i : B - 1;
        const float* ml = part_ml + ((int64_t)b * H + h) * n_split * 2;
        const float m = lane < n_split ? ml[2 * lane] : -INFINITY, d = lane < n_split ? ml[2 * lane + 1] : 0.f;     // (n_split <= 64)
        const float sk = sink[h] * LOG2E, top = fmaxf(sk, wave_max(m)), f = exp2f(m - top);
        const float l = wave_sum(d * f) + exp2f(sk - top);
        if (lane < n_split) wt[i * n_split + lane] = f / l;
    }
    __syncthreads();
    for (int it = tid; it < NS * (R / 4); it += 512) {
        const int i = it / (R / 4), r = it % (R / 4) * 4, b = b0 + i < B ? b0 + i : B - 1;
        const float* po = part_o + ((int64_t)b * H + h) * n_split * R + r;
        float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
        for (int s = 0; s < n_split; ++s) {
            const float4 x = *(const float4*)(po + (int64_t)s * R);
            const float f = wt[i * n_split + s];
            acc.x = fmaf(x.x, f, acc.x); acc.y = fmaf(x.y, f, acc.y); acc.z = fmaf(x.z, f, acc.z); acc.w = fmaf(x.w, f, acc.w);
        }
        *(uint2*)(lat + i * pr + r) = make_uint2(pack_bf2(acc.x, acc.y), pack_bf2(acc.z, acc.w));
    }
    __syncthreads();
    if (v0 >= dv) return;
    const uint16_t* wr = w + ((int64_t)h * dv + (v0 + c16 < dv ? v0 + c16 : dv - 1)) * R + 8 * g;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    const int cl = c16 < NS ? c16 : 0;                           // (columns beyond NS repeat the first and are not stored)
#pragma unroll 8
    for (int k = 0; k < R; k += 32)
        acc = mfma16(__builtin_bit_cast(mx_frag, *(const uint4*)(wr + k)), __builtin_bit_cast(mx_frag, *(const uint4*)(lat + cl * pr + k + 8 * g)), acc);
    if (c16 < NS && b0 + c16 < B) {
        uint16_t* op = o + (int64_t)(b0 + c16) * H * dv + (int64_t)h * dv + v0 + 4 * g;
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (v0 + 4 * g + r < dv) op[r] = f_to_bf(acc[r]);
    }
}

extern "C" int evo_latent_up(const float* part_o, const float* part_ml, const float* sink, const void* wuv, void* o, int64_t B, int64_t H, int64_t R,
                             int64_t dv, int64_t n_split, int64_t f32, int64_t mfma, void* stream) {
    if (!part_o || !part_ml || !sink || !wuv || !o || B <= 0 || H <= 0 || H > 65535 || R <= 0 || R > 8192 || dv <= 0 || n_split <= 0 || n_split > 64) return -1;
    if (!f32 && mfma && B > 2 && R % 32 == 0 && R <= 1024 && (((uintptr_t)wuv | (uintptr_t)part_o) & 15) == 0) {
        const int ns = B <= 8 ? 8 : 16;
        const dim3 grid((unsigned)((dv + 127) / 128), (unsigned)H, (unsigned)((B + ns - 1) / ns));
        const size_t lds = (size_t)ns * ((R + 8) * 2 + n_split * 4);
        if (ns == 8) hipLaunchKernelGGL((latent_up_mfma_kernel<8>), grid, dim3(512), lds, (hipStream_t)stream, part_o, part_ml, sink, (const uint16_t*)wuv,
                                        (uint16_t*)o, (int)B, (int)H, (int)R, (int)dv, (int)n_split);
        else hipLaunchKernelGGL((latent_up_mfma_kernel<16>), grid, dim3(512), lds, (hipStream_t)stream, part_o, part_ml, sink, (const uint16_t*)wuv,
                                (uint16_t*)o, (int)B, (int)H, (int)R, (int)dv, (int)n_split);
        return evo_launch_status();
    }
    const int nb = B > 2 ? 4 : (int)B;
    const int rows = H * ((B + nb - 1) / nb) >= 128 ? (int)dv : (int)((dv + 3) / 4);     // few heads and sequences: four workgroups share a head's rows
    const dim3 grid((unsigned)((dv + rows - 1) / rows), (unsigned)H, (unsigned)((B + nb - 1) / nb)), block(512);
    const size_t lds = (size_t)nb * (R + n_split) * 4;
    hipStream_t s = (hipStream_t)stream;
    const bool vec = R % 8 == 0 && ((uintptr_t)wuv & 15) == 0;
#define UP(T, NB, V)                                                                                                       \
    do {                                                                                                                   \
        if (lds > 64 * 1024) (void)hipFuncSetAttribute((const void*)latent_up_kernel<T, NB, V>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
        hipLaunchKernelGGL((latent_up_kernel<T, NB, V>), grid, block, lds, s, part_o, part_ml, sink, wuv, o, (int)B, (int)H, (int)R, (int)dv, (int)n_split, rows); \
    } while (0)
#define UPV(T, V) do { if (nb == 1) UP(T, 1, V); else if (nb == 2) UP(T, 2, V); else UP(T, 4, V); } while (0)
    if (f32) { if (vec) UPV(float, 8); else UPV(float, 1); }
    else { if (vec) UPV(uint16_t, 8); else UPV(uint16_t, 1); }
#undef UPV
#undef UP
    return evo_launch_status();
}
