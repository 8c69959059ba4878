// Softmax attention of packed prompts: causal, optionally over a sliding window whose first tokens stay visible, optionally with one sink per
// head in the denominator; query heads share key / value heads in groups; two attention maps over the same values may be combined on the way
// out (differential attention).  Entry point: include/evo_mi355x.h.
#include "mixers_common.h"
#include "../../include/evo_mi355x.h"

#define LOG2E 1.4426950408889634f

struct WinArgs {
    const void* q; const void* kn; const void* v; const void* kr; void* o;
    const int* cu_q; const int* cu_k; const float* sink;         // sink, kr: may be null
    int64_t ldq, ldkv;                                           // q row pitch; pitch of the kn / v rows
    int H, grp, dn, dr, dv, window, keep, n_qb;                  // grp query heads share a key / value head; kr rows are dr elements, o rows H dv
    float scale, lam, gain, eps;                                 // two maps: o = gain * unit_rms(o1 - lam o2)
};
#define FLOOR -1.0e30f                                           // running maximum before any key: finite, so that no difference of infinities arises

// Visible keys of query i (indexes into the sequence's keys, whose last ones are the queries'): j <= i and (i - j < window or j < keep).  A
// caller that leaves out keys between the kept ones and the window may do so: only order matters to both conditions.
//
// Matrix-core form (bf16).  A workgroup: 64 QC query rows of one (sequence, head); wave w owns 16 QC of them as MFMA COLUMNS: scores come
// as S^T = K Q^T (a lane holds one query's scores of four keys per 16-key block), so the softmax needs two cross-lane steps, the
// probabilities are the next product's operand as they stand (split key order), and O^T = V^T P^T is rescaled by one factor per lane.
// VEC: every row piece of eight elements is 16-byte aligned.
// MAPS == 2: the two column blocks of a wave are the two maps of the same 16 queries -- rows of q and k hold [map 1 | map 2] per head --, the
// values are shared, and the maps meet in the epilogue.  KEEP: a.keep is not zero.  NW: waves
// (8: wide heads, whose sums leave a SIMD room for two waves of one workgroup only).  NH: a tile's keys are gone through in NH parts (2: half
// the registers for scores).
template <int KS, int DVB, int QC, bool VEC, bool KEEP, int MAPS, int MINW, int NW = 4, int NH = 1>
__global__ __launch_bounds__(64 * NW, MINW) void window_attn_kernel(WinArgs a, int B) {
    static_assert(MAPS == 1 || QC == 2, "two maps are two column blocks");
    constexpr int DQ = 32 * KS, PR = MAPS * DQ + 8, PT = 64 + 4, DVP = 16 * DVB, QW = 16 * QC / MAPS, QB = NW * QW;   // QW: queries of a wave
    constexpr int KG = DQ / 64, VG = DVP / 64;                   // groups of 64 key / value dimensions
    constexpr int KU = 8 / NW, VI = VG * 4 / NW;                 // keys per thread; groups of value dimensions per thread
    static_assert(NW == 4 || VG % 2 == 0, "eight waves share the value groups by halves");
    __shared__ __attribute__((aligned(16))) uint16_t k_rows[64 * PR], v_cols[DVP * PT];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    // the query blocks of a (sequence, head) share most of their keys: consecutive work items stay on one XCD (block b runs on XCD b % 8)
    const int per_xcd = gridDim.x >> 3;
    const int item = (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3);
    const int qb = item % a.n_qb, h = item / a.n_qb % a.H, b = item / a.n_qb / a.H;
    if (b >= B) return;                                          // (the grid is rounded up to a multiple of 8)
    const int q0 = a.cu_q[b], nq = a.cu_q[b + 1] - q0, k0 = a.cu_k[b], nk = a.cu_k[b + 1] - k0;
    if (qb * QB >= nq) return;
    const int off = nk - nq;                                     // key index of query 0
    const int dh = a.dn + a.dr, dn = a.dn, dv = a.dv, hk = h / a.grp;
    const uint16_t* kr = (const uint16_t*)a.kr + (int64_t)k0 * a.dr;
    const uint16_t* kn = (const uint16_t*)a.kn + (int64_t)k0 * a.ldkv + (int64_t)hk * dn * MAPS;
    const uint16_t* vg = (const uint16_t*)a.v + (int64_t)k0 * a.ldkv + (int64_t)hk * dv;
    mx_frag qf[QC][KS];
    int qi[QC];                                                  // this lane's query of each column block, as a key index
#pragma unroll
    for (int c = 0; c < QC; ++c) {
        const int i = qb * QB + wave * QW + (MAPS == 2 ? 0 : 16 * c) + c16;
        qi[c] = i + off;
        const uint16_t* p = (const uint16_t*)a.q + (int64_t)(q0 + (i < nq ? i : nq - 1)) * a.ldq + (int64_t)(h * MAPS + (MAPS == 2 ? c : 0)) * dh;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const int d = 32 * ks + 8 * g;
            uint4 v = make_uint4(0u, 0u, 0u, 0u);
            if constexpr (VEC) { if (d < dh) v = *(const uint4*)(p + d); }
            else {
                uint32_t w[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) w[e] = d + e < dh ? p[d + e] : 0u;
                v = make_uint4(w[0] | w[1] << 16, w[2] | w[3] << 16, w[4] | w[5] << 16, w[6] | w[7] << 16);
            }
            qf[c][ks] = __builtin_bit_cast(mx_frag, v);
        }
    }
    const float sc2 = a.scale * LOG2E;
    f32x4_t o[QC][DVB];
    float mx[QC], den[QC];                                       // den: this lane's share (its keys); the sink sits in lane group 0's
#pragma unroll
    for (int c = 0; c < QC; ++c) {
        mx[c] = a.sink ? a.sink[h] * LOG2E : FLOOR;
        den[c] = a.sink && g == 0 ? 1.0f : 0.0f;
#pragma unroll
        for (int db = 0; db < DVB; ++db) o[c][db] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }

    // eight threads share a row: thread (row rt = tid / 8, dims ct + 64 i) of keys rt and (four waves) rt + 32, values of keys 2 vt and 2 vt + 1
    // (eight waves: half of the value dims each).  A tile's base is uniform, offsets within it are 32 bits; eight waves make them anew for every
    // tile: held across tiles they spill.
    mx_u32x4 rk[MAPS * KG][KU], rv[VI][2];
    auto any8 = [](const uint16_t* x, int nx, const uint16_t* y, int ny, int d) {       // eight dims of [x (nx) | y (ny) | zeros], any alignment
        uint32_t w[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = d + e < nx ? x[d + e] : (d + e < nx + ny ? y[d + e - nx] : 0u);
        return mx_u32x4{w[0] | w[1] << 16, w[2] | w[3] << 16, w[4] | w[5] << 16, w[6] | w[7] << 16};
    };
    // (keys past the end and dimensions past the head's repeat valid ones -- their scores are masked, the queries are zero there, their
    //  outputs are not stored --, so that the aligned form has no branch among its requests)
    const uint32_t row_bytes = (uint32_t)a.ldkv * 2;
    auto here = [](int v) __attribute__((always_inline)) {
        if constexpr (NW == 8) asm volatile("" : "+v"(v));
        return v;
    };
    auto load_k = [&](int j0) __attribute__((always_inline)) {
        const char* tile = (const char*)(kn + j0 * a.ldkv);
        const int t = here(tid), rt = t >> 3, ct = (t & 7) * 8;
#pragma unroll
        for (int u = 0; u < KU; ++u) {
            const int r = rt + 32 * u < nk - j0 ? rt + 32 * u : nk - 1 - j0;
            const uint16_t *pn = kn + (j0 + r) * a.ldkv, *pr_ = kr + (int64_t)(j0 + r) * a.dr;
#pragma unroll
            for (int i = 0; i < MAPS * KG; ++i) {
                const int d = ct + 64 * (i % KG), dc = d < dh ? d : dh - 8;
                if constexpr (!VEC) rk[i][u] = any8(pn + (i / KG) * dn, dn, pr_, a.dr, d);
                else if constexpr (MAPS == 2)                    // (a shared key part goes with one map only)
                    rk[i][u] = *(const mx_u32x4*)(tile + ((uint32_t)r * row_bytes + 2u * (uint32_t)((i / KG) * dn + dc)));
                else rk[i][u] = *(const mx_u32x4*)(dc < dn ? pn + dc : pr_ + (dc - dn));
            }
        }
    };
    auto load_v = [&](int j0) __attribute__((always_inline)) {
        const char* tile = (const char*)(vg + j0 * a.ldkv);
        const int t = here(tid), vt = (t >> 3) & 31, vi0 = (t >> 8) * VI, ct = (t & 7) * 8;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int r = 2 * vt + u < nk - j0 ? 2 * vt + u : nk - 1 - j0;
#pragma unroll
            for (int i = 0; i < VI; ++i) {
                const int d = ct + 64 * (vi0 + i);
                if constexpr (!VEC) rv[i][u] = any8(vg + (j0 + r) * a.ldkv, dv, vg, 0, d);
                else rv[i][u] = *(const mx_u32x4*)(tile + ((uint32_t)r * row_bytes + 2u * (uint32_t)(d < dv ? d : dv - 8)));
            }
        }
    };
    auto stage = [&]() __attribute__((always_inline)) {
        const int t = here(tid), rt = t >> 3, vt = rt & 31, vi0 = (t >> 8) * VI, ct = (t & 7) * 8;
#pragma unroll
        for (int i = 0; i < MAPS * KG; ++i)
#pragma unroll
            for (int u = 0; u < KU; ++u) *(mx_u32x4*)(k_rows + (rt + 32 * u) * PR + ct + 64 * i) = rk[i][u];
#pragma unroll
        for (int i = 0; i < VI; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const uint32_t x = rv[i][0][e], y = rv[i][1][e];
                uint16_t* c = v_cols + (ct + 64 * (vi0 + i) + 2 * e) * PT + 2 * vt;
                *(uint32_t*)c = (x & 0xffffu) | y << 16;
                *(uint32_t*)(c + PT) = x >> 16 | (y & 0xffff0000u);
            }
    };

    const int last_q = (qb + 1) * QB < nq ? (qb + 1) * QB - 1 : nq - 1;
    int j_lo = qb * QB + off - a.window + 1;
    j_lo = j_lo < 0 ? 0 : j_lo & ~63;
    const int j_hi = last_q + off;                               // last key any row of this block sees
    const int w_first = qb * QB + wave * QW + off, w_last = w_first + QW - 1;   // this wave's queries as key indexes
    const int keep = !KEEP ? 0 : (a.keep < j_lo ? a.keep : j_lo);   // kept keys ahead of the window's tiles: tiles [0, keep) come first
    auto after = [&](int j) { return KEEP && j < j_lo && j + 64 >= keep ? j_lo : j + 64; };
    int j0 = keep > 0 ? 0 : j_lo;
    load_k(j0);
    load_v(j0);
    for (int next = j0; j0 <= j_hi; j0 = next) {
        stage();
        __syncthreads();
        next = after(j0);
        const bool more = next <= j_hi;
        const bool mine = j0 <= w_last && (j0 + 63 > w_first - a.window || (KEEP && j0 < a.keep));   // some query of this wave sees some key of the tile
        constexpr int NJ = 4 / NH;                               // 16-key blocks of a part
#pragma unroll
        for (int hh = 0; hh < NH; ++hh) {
        f32x4_t s[QC][NJ];
        if (mine) {
#pragma unroll
            for (int jb = 0; jb < NJ; ++jb) {
#pragma unroll
                for (int c = 0; c < QC; ++c) s[c][jb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int ks = 0; ks < KS; ++ks) {
                    const uint16_t* kp = k_rows + (16 * (hh * NJ + jb) + c16) * PR + 32 * ks + 8 * g;
                    const mx_frag kf = __builtin_bit_cast(mx_frag, *(const uint4*)kp);
#pragma unroll
                    for (int c = 0; c < QC; ++c)
                        s[c][jb] = mfma16(MAPS == 2 && c == 1 ? __builtin_bit_cast(mx_frag, *(const uint4*)(kp + DQ)) : kf, qf[c][ks], s[c][jb]);
                }
                if (jb & 1) __builtin_amdgcn_sched_barrier(0);   // (bounds the fragments read ahead)
            }
        }
        // the next tile's requests go out in two parts, between the phases: with all of them ahead of the scores the register file spills
        __builtin_amdgcn_sched_barrier(0);
        if (hh == NH - 1 && more) load_k(next);
        __builtin_amdgcn_sched_barrier(0);
        mx_frag pf[QC][NJ / 2];
        if (mine) {
            if (j0 + 63 > w_first || (j0 <= w_last - a.window && (!KEEP || j0 + 63 >= a.keep))) {   // the tile holds an edge of some query's window
#pragma unroll
                for (int c = 0; c < QC; ++c)
#pragma unroll
                    for (int jb = 0; jb < NJ; ++jb)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int j = j0 + 16 * (hh * NJ + jb) + 4 * g + r, age = qi[c] - j;
                            s[c][jb][r] = age >= 0 && (age < a.window || (KEEP && j < a.keep)) ? s[c][jb][r] * sc2 : -INFINITY;
                        }
            } else {
#pragma unroll
                for (int c = 0; c < QC; ++c)
#pragma unroll
                    for (int jb = 0; jb < NJ; ++jb)
#pragma unroll
                        for (int r = 0; r < 4; ++r) s[c][jb][r] *= sc2;
            }
#pragma unroll
            for (int c = 0; c < QC; ++c) {
                float top = mx[c];
#pragma unroll
                for (int jb = 0; jb < NJ; ++jb) top = fmaxf(top, fmaxf(fmaxf(s[c][jb][0], s[c][jb][1]), fmaxf(s[c][jb][2], s[c][jb][3])));
                top = fmaxf(top, __shfl_xor(top, 16, 64));
                top = fmaxf(top, __shfl_xor(top, 32, 64));
                if (__builtin_amdgcn_ballot_w64(top > mx[c])) {          // the running maximum moved in some column: rescale
                    const float f = __builtin_amdgcn_exp2f(mx[c] - top);
                    mx[c] = top;
                    den[c] *= f;
#pragma unroll
                    for (int db = 0; db < DVB; ++db)
#pragma unroll
                        for (int r = 0; r < 4; ++r) o[c][db][r] *= f;
                }
                uint32_t w[2 * NJ];
#pragma unroll
                for (int jb = 0; jb < NJ; ++jb) {
                    float e[4];
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        e[r] = __builtin_amdgcn_exp2f(s[c][jb][r] - mx[c]);
                        den[c] += e[r];
                    }
                    w[2 * jb] = pack_bf2(e[0], e[1]);
                    w[2 * jb + 1] = pack_bf2(e[2], e[3]);
                }
#pragma unroll
                for (int jj = 0; jj < NJ / 2; ++jj) pf[c][jj] = frag_of(w[4 * jj], w[4 * jj + 1], w[4 * jj + 2], w[4 * jj + 3]);
            }
        }
        __builtin_amdgcn_sched_barrier(0);
        if (hh == NH - 1 && more) load_v(next);
        __builtin_amdgcn_sched_barrier(0);
        if (mine) {
#pragma unroll
            for (int jj = 0; jj < NJ / 2; ++jj)
#pragma unroll
                for (int db = 0; db < DVB; ++db) {
                    const mx_frag vf = frag_split(v_cols + (16 * db + c16) * PT + 32 * (hh * (NJ / 2) + jj) + 4 * g);
#pragma unroll
                    for (int c = 0; c < QC; ++c) o[c][db] = mfma16(vf, pf[c][jj], o[c][db]);
                    if ((db & 3) == 3) __builtin_amdgcn_sched_barrier(0);
                }
        }
        }
        __syncthreads();
    }
    float inv[QC];
#pragma unroll
    for (int c = 0; c < QC; ++c) {
        float l = den[c];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        inv[c] = 1.0f / l;
    }
    if constexpr (MAPS == 2) {                                   // the difference of the maps, its unit norm over the head's values
        const float i1 = inv[0], i2 = inv[1] * a.lam;
        float ss = 0.f;
#pragma unroll
        for (int db = 0; db < DVB; ++db)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float x = o[0][db][r] * i1 - o[1][db][r] * i2;
                o[0][db][r] = x;
                if (16 * db + 4 * g + r < dv) ss = fmaf(x, x, ss);
            }
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        inv[0] = a.gain / sqrtf(ss / (float)dv + a.eps);
    }
#pragma unroll
    for (int c = 0; c < QC / MAPS; ++c) {
        const int i = qi[c] - off;
        if (i < nq) {
            uint16_t* op = (uint16_t*)a.o + (int64_t)(q0 + i) * a.H * dv + (int64_t)h * dv;
#pragma unroll
            for (int db = 0; db < DVB; ++db) {
                const int d = 16 * db + 4 * g;
                if (d + 3 < dv && (dv & 3) == 0)
                    *(uint2*)(op + d) = make_uint2(pack_bf2(o[c][db][0] * inv[c], o[c][db][1] * inv[c]), pack_bf2(o[c][db][2] * inv[c], o[c][db][3] * inv[c]));
                else {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (d + r < dv) op[d + r] = f_to_bf(o[c][db][r] * inv[c]);
                }
            }
        }
    }
}

// Any sizes, both storage types: one wave per (query, head); lanes are keys for the scores, value columns for the sum
template <typename T, int MAPS>
__global__ __launch_bounds__(64) void window_attn_any_kernel(WinArgs a) {
    extern __shared__ float qs[];                                // dn + dr floats
    const int qr = blockIdx.x, h = blockIdx.y, b = blockIdx.z, lane = threadIdx.x;
    const int q0 = a.cu_q[b], nq = a.cu_q[b + 1] - q0, k0 = a.cu_k[b], nk = a.cu_k[b + 1] - k0;
    if (qr >= nq) return;
    const int dh = a.dn + a.dr, ki = qr + nk - nq, hk = h / a.grp;
    const T* vg = (const T*)a.v + (int64_t)k0 * a.ldkv + (int64_t)hk * a.dv;
    const T* kr = (const T*)a.kr + (int64_t)k0 * a.dr;
    const int j_lo = ki - a.window + 1 < 0 ? 0 : ki - a.window + 1, keep = a.keep < j_lo ? a.keep : j_lo;
    float o[MAPS][8];
#pragma unroll
    for (int map = 0; map < MAPS; ++map) {
        const T* q = (const T*)a.q + (int64_t)(q0 + qr) * a.ldq + (int64_t)(h * MAPS + map) * dh;
        __syncthreads();
        for (int d = lane; d < dh; d += 64) qs[d] = ld1(q + d);
        __syncthreads();
        const T* kn = (const T*)a.kn + (int64_t)k0 * a.ldkv + (int64_t)(hk * MAPS + map) * a.dn;
        float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.0f : 0.0f;
#pragma unroll
        for (int e = 0; e < 8; ++e) o[map][e] = 0.f;
        for (int part = keep > 0 ? 0 : 1; part < 2; ++part)      // the kept keys ahead of the window, then the window
            for (int j0 = part ? j_lo : 0, end = part ? ki + 1 : keep; j0 < end; j0 += 64) {
                const int j = j0 + lane;
                float s = -INFINITY;
                if (j < end) {
                    s = 0.f;
                    for (int d = 0; d < a.dn; ++d) s = fmaf(qs[d], ld1(kn + j * a.ldkv + d), s);
                    for (int d = 0; d < a.dr; ++d) s = fmaf(qs[a.dn + d], ld1(kr + (int64_t)j * a.dr + d), s);
                    s *= a.scale;
                }
                const float top = fmaxf(m, wave_max(s)), f = expf(m - top), p = expf(s - top);
                m = top;
                l = l * f + wave_sum(p);
#pragma unroll
                for (int e = 0; e < 8; ++e) o[map][e] *= f;
                const int n = end - j0 < 64 ? end - j0 : 64;
                for (int u = 0; u < n; ++u) {
                    const float pu = __shfl(p, u, 64);
                    const T* vr = vg + (j0 + u) * a.ldkv;
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (lane + 64 * e < a.dv) o[map][e] = fmaf(pu, ld1(vr + lane + 64 * e), o[map][e]);
                }
            }
#pragma unroll
        for (int e = 0; e < 8; ++e) o[map][e] /= l;
    }
    float gain = 1.0f;
    if constexpr (MAPS == 2) {
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            o[0][e] -= a.lam * o[1][e];
            if (lane + 64 * e < a.dv) ss = fmaf(o[0][e], o[0][e], ss);
        }
        gain = a.gain / sqrtf(wave_sum(ss) / (float)a.dv + a.eps);
    }
    T* op = (T*)a.o + (int64_t)(q0 + qr) * a.H * a.dv + (int64_t)h * a.dv;
#pragma unroll
    for (int e = 0; e < 8; ++e)
        if (lane + 64 * e < a.dv) st1(op + lane + 64 * e, o[0][e] * gain);
}

extern "C" int evo_window_attn(const void* q, int64_t ldq, const void* kn, const void* v, int64_t ldkv, const void* kr, void* o, const int* cu_q,
                               const int* cu_k, const float* sink, int64_t B, int64_t H, int64_t kv_heads, int64_t maps, int64_t dn, int64_t dr,
                               int64_t dv, int64_t window, int64_t keep, int64_t max_q, float scale, float lam, float gain, float eps, int64_t f32,
                               int64_t mfma, void* stream) {
    if (!q || !kn || !v || !o || !cu_q || !cu_k || B <= 0 || B > 65535 || H <= 0 || H > 65535 || kv_heads <= 0 || H % kv_heads != 0) return -1;
    if (dn < 0 || dr < 0 || (dr > 0 && !kr) || dn + dr <= 0 || dn + dr > 8192 || dv <= 0 || dv > 512 || window <= 0 || keep < 0 || max_q <= 0 || max_q > 0x3fffffff) return -1;
    if ((maps != 1 && maps != 2) || (maps == 2 && (dr > 0 || sink)) || ldq < H * maps * (dn + dr) || ldkv < kv_heads * dv || ldkv < kv_heads * maps * dn) return -1;
    const int w = window > 0x3fffffff ? 0x3fffffff : (int)window, kp = keep > 0x3fffffff ? 0x3fffffff : (int)keep;
    WinArgs a = {q, kn, v, kr, o, cu_q, cu_k, sink, ldq, ldkv, (int)H, (int)(H / kv_heads), (int)dn, (int)dr, (int)dv, w, kp, 0, scale, lam, gain, eps};
    hipStream_t s = (hipStream_t)stream;
    const int64_t dq = dn + dr;
    if (!f32 && mfma && dq <= (maps == 2 ? 128 : 256) && dv <= 256) {
        const bool vec = dn % 8 == 0 && dr % 8 == 0 && dv % 8 == 0 && ldq % 8 == 0 && ldkv % 8 == 0 && ldkv <= 0xffffff &&
                         (((uintptr_t)q | (uintptr_t)kn | (uintptr_t)v | (uintptr_t)kr) & 15) == 0;
#define WA1(KS, DVB, QC, VEC, KEEP, MAPS, MINW, NW)                                                                        \
    do {                                                                                                                   \
        a.n_qb = (int)((max_q + 16 * NW * QC / MAPS - 1) / (16 * NW * QC / MAPS));                                         \
        const int64_t items = (int64_t)a.n_qb * H * B;                                                                     \
        if (items > 0x7ffffff0) return -1;                                                                                 \
        hipLaunchKernelGGL((window_attn_kernel<KS, DVB, QC, VEC, KEEP, MAPS, MINW, NW, (MAPS == 2 && NW == 8 ? 2 : 1)>), dim3((unsigned)((items + 7) / 8 * 8)), dim3(64 * NW), 0, s, a, (int)B); \
    } while (0)
#define WAN(KS, DVB, QC, VEC, MAPS, MINW, NW) do { if (kp) WA1(KS, DVB, QC, VEC, true, MAPS, MINW, NW); else WA1(KS, DVB, QC, VEC, false, MAPS, MINW, NW); } while (0)
#define WA(KS, DVB, QC, VEC, MAPS, MINW) WAN(KS, DVB, QC, VEC, MAPS, MINW, 4)
#define WAV(KS, QC) do { if (dv <= 64) WA(KS, 4, QC, true, 1, 2); else if (dv <= 128) WA(KS, 8, QC, true, 1, 2); else WA(KS, 16, 1, true, 1, 2); } while (0)
#define WA2(KS) do { if (dv <= 64) WA(KS, 4, 2, true, 2, 2); else if (dv <= 128) WA(KS, 8, 2, true, 2, 2); \
                     else if (!kp) WA1(KS, 16, 2, true, false, 2, 2, 8); \
                     else WA1(KS, 16, 2, true, true, 2, (KS > 2 ? 1 : 2), (KS > 2 ? 4 : 8)); } while (0)   /* (kept tokens cost registers) */
        if (maps == 2) { if (!vec) WA(4, 16, 2, false, 2, 1); else if (dq <= 64) WA2(2); else WA2(4); }
        else if (!vec) { if (dq <= 64 && dv <= 64) WA(2, 4, 2, false, 1, 2); else WA(8, 16, 1, false, 1, 2); }
        else if (dq <= 64) WAV(2, 2);
        else if (dq <= 128) WAV(4, 2);
        else if (dq <= 192) {                                    // (kept tokens cost registers: one column block)
            if (dv <= 64) WA(6, 4, 2, true, 1, 2);
            else if (dv > 128) WA(6, 16, 1, true, 1, 2);
            else if (kp) WA1(6, 8, 1, true, true, 1, 2, 4);
            else WA1(6, 8, 2, true, false, 1, 2, 4);
        }
        else if (dv <= 64) WA(8, 4, 1, true, 1, 2);
        else if (dv <= 128) WA(8, 8, 1, true, 1, 2);
        else WA(8, 16, 1, true, 1, 1);
#undef WA2
#undef WAV
#undef WA
#undef WAN
#undef WA1
        return evo_launch_status();
    }
    const dim3 grid((unsigned)max_q, (unsigned)H, (unsigned)B);
#define WY(T, MAPS) hipLaunchKernelGGL((window_attn_any_kernel<T, MAPS>), grid, dim3(64), (size_t)dq * 4, s, a)
    if (f32) { if (maps == 2) WY(float, 2); else WY(float, 1); }
    else { if (maps == 2) WY(uint16_t, 2); else WY(uint16_t, 1); }
#undef WY
    return evo_launch_status();
}
