// Gated linear recurrence behind a short causal convolution (a recurrent block of Griffin's kind):
//   u = conv(x) + c;   r, i = sigmoid(block-diagonal maps of u);   a = exp(decay r);   S <- a S + sqrt(1 - a^2) i u;   o = S gelu(y)
// one fp32 state per channel.  A row of z is [y (W) | x (W)].  Per-sequence cache [1 + taps, W] fp32: S, then a ring of the last inputs of the
// convolution (position p in row 1 + p % taps: the rows a step reads are not the one it writes).  Entry points: include/evo_mi355x.h.
//
// Prompt form (bf16): a workgroup owns up to 128 channels of one block of one sequence's segment and walks it in tiles of 64 tokens.  The
// convolution's result -- every channel of the block -- is staged in LDS as the operand of both gate maps, whose weights stay in registers for
// the whole walk; a wave owns 16 channels, a lane four consecutive tokens of one of them per 16-token block, so the recurrence is four steps
// in registers, a scan over the four lane groups and one carried value per channel.  Long sequences that leave CUs idle are cut into segments:
// (1) every segment's decay product and end state from zero, (2) a scan over segments, (3) outputs.
#include "mixers_common.h"
#include "../../include/evo_mi355x.h"
#include <type_traits>

#define LOG2E 1.4426950408889634f
#define RT 64                                                    // tokens per tile
#define TAPS 4                                                   // convolution taps the matrix-core kernels hold (fewer: zeros in front)

struct RgArgs {
    const void* z; const void* in_b; void* o; float* state; float* seg;   // seg [B][n_seg][2][W]
    const void *conv, *conv_b, *ra, *ra_b, *ri, *ri_b;
    const float* decay; const int64_t* pos; const int* seq; const int* cu; const int* resume;
    int64_t ld;
    int W, nb, bs, taps, n_seg, seg_len, n_cg, act, rows;
};

typedef __bf16 rg_bf16x2 __attribute__((ext_vector_type(2)));
__device__ __forceinline__ float dot2(uint32_t a, uint32_t b, float c) {
    return __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(rg_bf16x2, a), __builtin_bit_cast(rg_bf16x2, b), c, false);
}
// the values of a lane's neighbours in the four 16-lane rows of a wave: swap16 -> (even row of its pair, odd row), swap32 -> (lower half, upper half)
__device__ __forceinline__ void swap16(float v, float& even, float& odd) {
    const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    even = __uint_as_float(r[0]); odd = __uint_as_float(r[1]);
}
__device__ __forceinline__ void swap32(float v, float& low, float& high) {
    const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    low = __uint_as_float(r[0]); high = __uint_as_float(r[1]);
}
// gates of one channel: decay a and input sqrt(1 - a^2) i u from the maps' results.  sqrt(x) / E = x rsqrt(x E^2); x is 0 (a = 1) or at least 2^-24.
__device__ __forceinline__ void gate(float zr, float zi, float c2, float u, float& al, float& add) {
    al = __builtin_amdgcn_exp2f(c2 * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-LOG2E * zr)));
    const float x = fmaxf(fmaf(-al, al, 1.0f), 1e-30f), e = 1.0f + __builtin_amdgcn_exp2f(-LOG2E * zi);
    add = x * __builtin_amdgcn_rsqf(x * e * e) * u;
}

// ------------------------------------------------------------------------------------------------ prompts
// KS: 32-wide steps of a block, NW: waves.  OUT: outputs and the sequence's end state; otherwise a segment's (product of a, end state from zero).
template <int KS, int NW, bool OUT>
__global__ __launch_bounds__(64 * NW) void rglru_chunk_kernel(RgArgs a) {
    constexpr int KP = 32 * KS, PR = KP + 8, NT = 64 * NW, NC = 16 * NW, YP = NC + 8;
    constexpr int IT = (16 * 4 * KS + NT - 1) / NT;              // staged runs (four tokens x eight channels) per thread
    constexpr bool AHEAD = KS < 12;                              // the next tile's rows are requested a tile ahead (wide blocks: no registers left)
    extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
    uint16_t* const tile = lds;                                  // [2][RT][PR]
    uint32_t* const cw = (uint32_t*)(lds + 2 * RT * PR);         // [2][KP] taps as bf16 pairs, oldest first; [KP] the bias
    float* const cb = (float*)(cw + 2 * KP);
    uint16_t* const yo = (uint16_t*)(cb + KP);                   // [2][RT][YP] y, replaced by the outputs where they are made
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int cg = blockIdx.x % a.n_cg, seg = blockIdx.x / a.n_cg, n = blockIdx.y, b = blockIdx.z;
    const int bs = a.bs, W = a.W, row0 = a.cu[b];
    const int len_all = a.cu[b + 1] - row0, s_lo = seg * a.seg_len;
    int s_hi = s_lo + a.seg_len;
    s_hi = s_hi < len_all ? s_hi : len_all;
    if (s_lo >= s_hi) return;
    const bool go_on = a.resume && a.resume[b];
    const int ch = cg * 16 * NW + 16 * wave + c16, cc = ch < bs ? ch : bs - 1;   // this lane's channel of the block (clamped for loads)
    const int wch = n * bs + cc;                                 // ... of the whole width
    const uint16_t* zx = (const uint16_t*)a.z + (int64_t)row0 * a.ld + W + n * bs;
    const uint16_t* zy = (const uint16_t*)a.z + (int64_t)row0 * a.ld + n * bs;
    float* st = a.state ? a.state + (int64_t)b * (1 + a.taps) * W + n * bs : nullptr;

    for (int i = tid; i < KP; i += NT) {                         // taps and bias of this block's channels
        uint32_t w[TAPS];
#pragma unroll
        for (int t = 0; t < TAPS; ++t) {
            const int k = t - (TAPS - a.taps);
            w[t] = i < bs && k >= 0 ? ((const uint16_t*)a.conv)[(int64_t)(n * bs + i) * a.taps + k] : 0u;
        }
        cw[i] = w[0] | w[1] << 16;
        cw[KP + i] = w[2] | w[3] << 16;
        cb[i] = i < bs ? ld1((const uint16_t*)a.conv_b + n * bs + i) : 0.f;
    }
    for (int i = tid; i < 2 * RT * (PR - bs); i += NT) tile[i / (PR - bs) * PR + bs + i % (PR - bs)] = 0;   // columns behind the block
    mx_frag wr[KS], wi[KS];                                      // rows of the gate maps: this lane's channel
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
        const int k = 32 * ks + 8 * g;
        const int64_t off = ((int64_t)n * bs + cc) * bs + (k < bs ? k : bs - 8);   // (beyond the block the tile is zero)
        wr[ks] = __builtin_bit_cast(mx_frag, *(const mx_u32x4*)((const uint16_t*)a.ra + off));
        wi[ks] = __builtin_bit_cast(mx_frag, *(const mx_u32x4*)((const uint16_t*)a.ri + off));
    }
    const float br = ld1((const uint16_t*)a.ra_b + wch), bi = ld1((const uint16_t*)a.ri_b + wch), c2 = a.decay[wch] * LOG2E;

    // staged run: tokens 4 q .. 4 q + 3, channels 8 d .. 8 d + 7 of the block
    const int nd = bs / 8;
    mx_u32x4 xr[AHEAD ? IT : 1][TAPS + 3];
    const uint32_t row_bytes = (uint32_t)a.ld * 2;
    auto load_run = [&](int t0, int i, mx_u32x4* x) __attribute__((always_inline)) {   // (uniform base, 32-bit offsets: rows t0 - 3 + 4 q + u, clamped)
        int it = tid + NT * i;
        it = it < 16 * nd ? it : 16 * nd - 1;
        const int q = it / nd, d = it - q * nd, tb = t0 < len_all ? t0 : len_all - 1;
        const int lo = tb < TAPS - 1 ? TAPS - 1 - tb : 0, hi = len_all - 1 - tb + TAPS - 1;
        const char* base = (const char*)(zx + (int64_t)(tb - (TAPS - 1)) * a.ld);
#pragma unroll
        for (int u = 0; u < TAPS + 3; ++u) {
            int r = 4 * q + u;
            r = r < lo ? lo : (r < hi ? r : hi);
            x[u] = *(const mx_u32x4*)(base + (uint32_t)((uint32_t)r * row_bytes + 16u * (uint32_t)d));
        }
    };
    auto load_x = [&](int t0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < (AHEAD ? IT : 0); ++i) load_run(t0, i, xr[i]);
    };
    auto convolve = [&](int t0, uint16_t* dst) __attribute__((always_inline)) {
#pragma unroll AHEAD ? IT : 1
        for (int i = 0; i < IT; ++i) {
            const int it = tid + NT * i, xi = AHEAD ? i : 0;
            if (!AHEAD) load_run(t0, i, xr[0]);
            if (it >= 16 * nd) break;
            const int q = it / nd, d = it - q * nd;
            if (t0 == 0 && q == 0) {                             // before this portion: the cached inputs, zeros before the sequence
#pragma unroll
                for (int u = 0; u < TAPS - 1; ++u) {
                    const int back = TAPS - 1 - u;               // tokens before the portion's first
                    const int64_t p = a.pos[row0] - back;
                    const bool have = go_on && p >= 0 && back < a.taps;
                    float h[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
                    if (have) vec_io<float, 8>::load(st + (1 + (int)(p % a.taps)) * (int64_t)W + 8 * d, h);
                    xr[xi][u] = mx_u32x4{pack_bf2(h[0], h[1]), pack_bf2(h[2], h[3]), pack_bf2(h[4], h[5]), pack_bf2(h[6], h[7])};
                }
            }
            // two taps per instruction: operands are pairs of adjacent tokens of one channel
            float acc[4][8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const uint32_t w0 = cw[8 * d + e], w1 = cw[KP + 8 * d + e], pick = e & 1 ? 0x07060302u : 0x05040100u;
                const float c = cb[8 * d + e];
                uint32_t pr[TAPS + 3];
#pragma unroll
                for (int u = 1; u < TAPS + 3; ++u) pr[u] = __builtin_amdgcn_perm(xr[xi][u][e >> 1], xr[xi][u - 1][e >> 1], pick);
#pragma unroll
                for (int v = 0; v < 4; ++v) acc[v][e] = dot2(pr[v + 3], w1, dot2(pr[v + 1], w0, c));
            }
#pragma unroll
            for (int v = 0; v < 4; ++v)
                *(uint4*)(dst + (4 * q + v) * PR + 8 * d) = make_uint4(pack_bf2(acc[v][0], acc[v][1]), pack_bf2(acc[v][2], acc[v][3]),
                                                                       pack_bf2(acc[v][4], acc[v][5]), pack_bf2(acc[v][6], acc[v][7]));
        }
    };

    float S = 0.f, A = 1.f;                                      // the carried state (the same in the four lane groups); OUT = false: the product of a
    if (OUT) {
        if (a.seg && (seg > 0 || go_on)) S = a.seg[(((int64_t)b * a.n_seg + seg) * 2 + 1) * W + wch];
        else if (go_on) S = st[cc];
    }
    // y and the outputs move 16 bytes at a time: thread (row, run of eight channels) of two runs, the same ones in both directions
    mx_u32x4 yv[2];
    auto load_y = [&](int t0) __attribute__((always_inline)) {
        if (!OUT) return;
        const int tb = t0 < s_hi ? t0 : s_hi - 1;
        const char* base = (const char*)(zy + (int64_t)tb * a.ld);
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const int it = tid + NT * k, r = it / (NC / 8), c = cg * NC + 8 * (it % (NC / 8));
            yv[k] = *(const mx_u32x4*)(base + (uint32_t)((uint32_t)(r < s_hi - tb ? r : s_hi - 1 - tb) * row_bytes + 2u * (uint32_t)(c < bs ? c : bs - 8)));
        }
    };
    auto store_o = [&](int t0, const uint16_t* src) __attribute__((always_inline)) {
        char* base = (char*)((uint16_t*)a.o + ((int64_t)row0 + t0) * W + n * bs);
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const int it = tid + NT * k, r = it / (NC / 8), j = it % (NC / 8), c = cg * NC + 8 * j;
            const uint4 v = *(const uint4*)(src + r * YP + 8 * j);
            if (t0 + r < s_hi && c < bs) *(uint4*)(base + (uint32_t)((uint32_t)r * (uint32_t)W * 2u + 2u * (uint32_t)c)) = v;
        }
    };
    load_x(s_lo);
    load_y(s_lo);
    __syncthreads();                                             // (taps)
    int buf = 0;
    for (int t0 = s_lo; t0 < s_hi; t0 += RT, buf ^= 1) {
        uint16_t* const ut = tile + buf * RT * PR;
        uint16_t* const yt = yo + buf * RT * YP;
        convolve(t0, ut);
        if (OUT) {
#pragma unroll
            for (int k = 0; k < 2; ++k) {
                const int it = tid + NT * k;
                *(mx_u32x4*)(yt + it / (NC / 8) * YP + 8 * (it % (NC / 8))) = yv[k];
            }
        }
        __syncthreads();                                         // (the other buffers' readers are past this tile's barrier as well)
        load_x(t0 + RT);                                         // (past the end: valid rows again, not used)
        load_y(t0 + RT);
        if (OUT && t0 > s_lo) store_o(t0 - RT, yo + (buf ^ 1) * RT * YP);
        __builtin_amdgcn_sched_barrier(0);
        // the gate maps of a 16-token block run ahead of the arithmetic on the one before
        f32x4_t zr[2], zi[2];
        auto maps = [&](int tb) __attribute__((always_inline)) {
            f32x4_t r = {br, br, br, br}, i = {bi, bi, bi, bi};
#pragma unroll
            for (int ks = 0; ks < KS; ++ks) {
                const mx_frag uf = __builtin_bit_cast(mx_frag, *(const uint4*)(ut + (16 * tb + c16) * PR + 32 * ks + 8 * g));
                r = mfma16(uf, wr[ks], r);
                i = mfma16(uf, wi[ks], i);
            }
            zr[tb & 1] = r;
            zi[tb & 1] = i;
        };
        auto walk = [&](auto full) __attribute__((always_inline)) {
#pragma unroll
        for (int tb = 0; tb < 4; ++tb) {
            if (tb < 3) maps(tb + 1);
            float pa[4], ps[4];                                  // running (product of a, state from zero) over this lane's four tokens
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float u = bf_to_f(ut[(16 * tb + 4 * g + r) * PR + cc]);
                float al, add;
                gate(zr[tb & 1][r], zi[tb & 1][r], c2, u, al, add);
                if (!decltype(full)::value && t0 + 16 * tb + 4 * g + r >= s_hi) { al = 1.f; add = 0.f; }   // past the end: the state stays
                pa[r] = r ? pa[r - 1] * al : al;
                ps[r] = r ? fmaf(ps[r - 1], al, add) : add;
            }
            // composition over the four lane groups: every lane gets the even and odd member of its pair of groups, then both pairs
            float ea, oa, es, os, la, ha, ls, hs;
            swap16(pa[3], ea, oa);
            swap16(ps[3], es, os);
            swap32(ea * oa, la, ha);
            swap32(fmaf(es, oa, os), ls, hs);
            const float mid = fmaf(la, S, ls);                   // state behind the lower two groups
            float in = g >= 2 ? mid : S;
            if (g & 1) in = fmaf(ea, in, es);
            if (!OUT) A *= la * ha;
            S = fmaf(ha, mid, hs);
            if (OUT) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    uint16_t* e = yt + (16 * tb + 4 * g + r) * YP + 16 * wave + c16;
                    *e = f_to_bf(fmaf(pa[r], in, ps[r]) * bf_to_f(*e));
                }
            }
        }
        };
        maps(0);
        if (t0 + RT <= s_hi) walk(std::true_type());
        else walk(std::false_type());
    }
    if (OUT) {
        __syncthreads();
        store_o((s_hi - 1 - s_lo) / RT * RT + s_lo, yo + (buf ^ 1) * RT * YP);
    }
    if (g == 0 && ch < bs) {
        if (!OUT) {
            float* p = a.seg + ((int64_t)b * a.n_seg + seg) * 2 * W + wch;
            p[0] = A;
            p[W] = S;
        } else if (st && s_hi == len_all) st[cc] = S;
    }
}

// segments' (product, end state from zero) -> incoming states, in place of the latter
__global__ __launch_bounds__(256) void rglru_carry_kernel(RgArgs a) {
    const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
    if (c >= a.W) return;
    const int len = a.cu[b + 1] - a.cu[b], n = (len + a.seg_len - 1) / a.seg_len;
    float S = a.resume && a.resume[b] ? a.state[(int64_t)b * (1 + a.taps) * a.W + c] : 0.f;
    for (int s = 0; s < n; ++s) {
        float* p = a.seg + ((int64_t)b * a.n_seg + s) * 2 * a.W + c;
        const float in = S;
        S = fmaf(p[0], S, p[a.W]);
        p[a.W] = in;
    }
}

// the last inputs of the convolution -> the ring
template <typename T>
__global__ __launch_bounds__(256) void rglru_tail_kernel(RgArgs a) {
    const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
    if (c >= a.W) return;
    const int row0 = a.cu ? a.cu[b] : b, len = a.cu ? a.cu[b + 1] - row0 : 1, n = len < a.taps ? len : a.taps;
    const float bias = a.in_b ? ld1((const T*)a.in_b + a.W + c) : 0.f;
    for (int t = len - n; t < len; ++t)
        a.state[((int64_t)b * (1 + a.taps) + 1 + a.pos[row0 + t] % a.taps) * a.W + c] = ld1((const T*)a.z + (row0 + t) * a.ld + a.W + c) + bias;
}

static bool rg_sizes(const void* z, const void* o, const void* conv, const void* conv_b, const void* ra, const void* ra_b, const void* ri, const void* ri_b,
                     const float* decay, const int64_t* pos, int64_t ld, int64_t B, int64_t W, int64_t nb, int64_t taps) {
    return z && o && conv && conv_b && ra && ra_b && ri && ri_b && decay && pos && B > 0 && B <= 65535 && W > 0 && W <= 0x7ffffff && nb > 0 && nb <= 65535 &&
           W % nb == 0 && taps > 0 && taps <= 0xffff && ld >= 2 * W && ld <= 0x3fffffff;
}

extern "C" int evo_rglru_chunk_bf16(const void* z, int64_t ld, void* o, float* state, float* seg, const void* conv, const void* conv_b, const void* ra,
                                    const void* ra_b, const void* ri, const void* ri_b, const float* decay, const int64_t* pos, const int* cu,
                                    const int* resume, int64_t B, int64_t W, int64_t nb, int64_t taps, int64_t max_len, int64_t seg_len, void* stream) {
    if (!rg_sizes(z, o, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, ld, B, W, nb, taps) || !cu || (resume && !state)) return -1;
    const int64_t bs = W / nb;
    if (bs % 8 || bs > 384 || taps > TAPS || max_len <= 0 || max_len > 0x3fffffff || seg_len <= 0 || seg_len % RT || ld % 8) return -1;
    if ((((uintptr_t)z | (uintptr_t)ra | (uintptr_t)ri | (uintptr_t)o | (uintptr_t)state) & 15) || ld > 0xffffff || W > 0xffffff) return -1;
    const int64_t n_seg = (max_len + seg_len - 1) / seg_len;
    if (n_seg > 1 && !seg) return -1;
    const int nw = bs <= 64 ? 4 : 8;
    const int64_t n_cg = (bs + 16 * nw - 1) / (16 * nw);
    if (n_seg * n_cg > 0x7fffffff) return -1;
    RgArgs a = {z, nullptr, o, state, n_seg > 1 ? seg : nullptr, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, nullptr, cu, resume,
                ld, (int)W, (int)nb, (int)bs, (int)taps, (int)n_seg, (int)seg_len, (int)n_cg, 0, (int)B};
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((unsigned)(n_seg * n_cg), (unsigned)nb, (unsigned)B);
#define RC(KS, NW)                                                                                                         \
    do {                                                                                                                   \
        constexpr int bytes = 2 * RT * (32 * KS + 8) * 2 + 3 * 32 * KS * 4 + 2 * RT * (16 * NW + 8) * 2;                                       \
        if (bytes > 64 * 1024) {                                                                                           \
            (void)hipFuncSetAttribute((const void*)rglru_chunk_kernel<KS, NW, false>, hipFuncAttributeMaxDynamicSharedMemorySize, bytes); \
            (void)hipFuncSetAttribute((const void*)rglru_chunk_kernel<KS, NW, true>, hipFuncAttributeMaxDynamicSharedMemorySize, bytes);  \
        }                                                                                                                  \
        if (n_seg > 1) {                                                                                                   \
            hipLaunchKernelGGL((rglru_chunk_kernel<KS, NW, false>), grid, dim3(64 * NW), bytes, s, a);                     \
            hipLaunchKernelGGL(rglru_carry_kernel, dim3((unsigned)((W + 255) / 256), (unsigned)B), dim3(256), 0, s, a);    \
        }                                                                                                                  \
        hipLaunchKernelGGL((rglru_chunk_kernel<KS, NW, true>), grid, dim3(64 * NW), bytes, s, a);                          \
    } while (0)
    if (bs <= 64) RC(2, 4); else if (bs <= 96) RC(3, 8); else if (bs <= 128) RC(4, 8); else if (bs <= 192) RC(6, 8); else if (bs <= 256) RC(8, 8); else RC(12, 8);
#undef RC
    if (state) hipLaunchKernelGGL((rglru_tail_kernel<uint16_t>), dim3((unsigned)((W + 255) / 256), (unsigned)B), dim3(256), 0, s, a);
    return evo_launch_status();
}

// ------------------------------------------------------------------------------------------------ decode
// One token per sequence.  A workgroup: 16 CG channels of one block for up to 16 sequences; the block's convolution outputs are rebuilt in LDS (a
// few KB from L2), a wave is one of the two gate maps, one half of its sum and 16 of the channels, a thread ends with one channel of one
// sequence.  The rows of a ring are requested before the position is known: which tap a row meets is settled afterwards.
template <int KS, int CG>
__global__ __launch_bounds__(256 * CG) void rglru_step_kernel(RgArgs a) {
    constexpr int KP = 32 * KS, PR = KP + 8, KH = (KS + 1) / 2, NT = 256 * CG, NC = 16 * CG;
    __shared__ __attribute__((aligned(16))) uint16_t ut[16 * PR];
    __shared__ __attribute__((aligned(16))) float cw[(TAPS + 1) * KP];   // taps, oldest first, then a row of zeros
    __shared__ float part[2][2][16][NC + 1];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int n = blockIdx.y, b0 = blockIdx.z * 16, bs = a.bs, W = a.W, taps = a.taps, rows = a.rows - b0 < 16 ? a.rows - b0 : 16;
    const int c0 = blockIdx.x * NC, map = wave & 1, half = (wave >> 1) & 1, cg = wave >> 2;
    mx_frag wf[KH];
    {
        const int c = c0 + 16 * cg + c16;
        const uint16_t* w = (const uint16_t*)(map ? a.ri : a.ra) + ((int64_t)n * bs + (c < bs ? c : bs - 1)) * bs;
#pragma unroll
        for (int i = 0; i < KH; ++i) {
            const int k = 32 * (half * KH + i) + 8 * g;
            wf[i] = __builtin_bit_cast(mx_frag, *(const mx_u32x4*)(w + (k < bs ? k : bs - 8)));
        }
    }
    const uint16_t* z = (const uint16_t*)a.z;
    // what this thread's channel of this thread's sequence needs at the end
    const int mi = tid / NC, mc = c0 + tid % NC, wc = n * bs + (mc < bs ? mc : bs - 1), mb = b0 + (mi < rows ? mi : rows - 1);
    float* st = a.state + (int64_t)mb * (1 + taps) * W + wc;
    const float S0 = st[0], dec = a.decay[wc] * LOG2E, br = ld1((const uint16_t*)a.ra_b + wc), bi = ld1((const uint16_t*)a.ri_b + wc);
    float mx = ld1(z + mb * a.ld + W + wc), my = ld1(z + mb * a.ld + wc);
    if (a.in_b) { mx += ld1((const uint16_t*)a.in_b + W + wc); my += ld1((const uint16_t*)a.in_b + wc); }
    const uint32_t mpos = (uint32_t)a.pos[mb];

    constexpr int CI = ((TAPS + 1) * KP + NT - 1) / NT;          // (all requests first: one memory latency)
    float tap[CI];
#pragma unroll
    for (int k = 0; k < CI; ++k) {
        const int i = tid + NT * k, t = i / KP, c = i % KP;
        tap[k] = ld1((const uint16_t*)a.conv + (int64_t)(n * bs + (c < bs ? c : bs - 1)) * taps + (t < taps ? t : 0));
        if (t >= taps || c >= bs) tap[k] = 0.f;
    }
    constexpr int ND = KP / 8, IT = (16 * ND + NT - 1) / NT;     // runs of eight channels of one sequence, per thread
    float acc[IT][8], h[IT][TAPS][8], x[IT][8];
    uint32_t p[IT];                                              // (positions are far below 2^31)
#pragma unroll
    for (int k = 0; k < IT; ++k) {
        const int it = tid + NT * k, i = it / ND, d = 8 * (it % ND), b = b0 + (i < rows ? i : rows - 1), dc = d < bs ? d : 0;
        p[k] = (uint32_t)a.pos[b];
        vec_io<uint16_t, 8>::load(z + b * a.ld + W + n * bs + dc, x[k]);
        vec_io<uint16_t, 8>::load((const uint16_t*)a.conv_b + n * bs + dc, acc[k]);
#pragma unroll
        for (int t = 0; t < TAPS; ++t)                           // (fewer taps: the last row again, with weight zero)
            vec_io<float, 8>::load(a.state + ((int64_t)b * (1 + taps) + 1 + (t < taps ? t : taps - 1)) * W + n * bs + dc, h[k][t]);
        if (a.in_b) {
            float ib[8];
            vec_io<uint16_t, 8>::load((const uint16_t*)a.in_b + W + n * bs + dc, ib);
#pragma unroll
            for (int e = 0; e < 8; ++e) x[k][e] += ib[e];
        }
    }
#pragma unroll
    for (int k = 0; k < CI; ++k)
        if (tid + NT * k < (TAPS + 1) * KP) cw[tid + NT * k] = tap[k];
    __syncthreads();
#pragma unroll
    for (int k = 0; k < IT; ++k) {
        const int it = tid + NT * k, i = it / ND, d = 8 * (it % ND);
        if (it >= 16 * ND) break;
        const int cur = (int)(p[k] % (uint32_t)taps);
        auto add = [&](int row, const float* v) {
            float w[8];
            vec_io<float, 8>::load(cw + row * KP + d, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[k][e] = fmaf(w[e], v[e], acc[k][e]);
        };
        add(taps - 1, x[k]);
#pragma unroll
        for (int t = 0; t < TAPS; ++t) {
            const int back = cur - t + (cur < t ? taps : 0);     // tokens between this one and the row's
            const bool have = t < taps && back > 0 && (uint32_t)back <= p[k];
            float v[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = have ? h[k][t][e] : 0.f;
            add(have ? taps - 1 - back : taps, v);
        }
        const bool on = i < rows && d < bs;
        *(uint4*)(ut + i * PR + d) = make_uint4(on ? pack_bf2(acc[k][0], acc[k][1]) : 0u, on ? pack_bf2(acc[k][2], acc[k][3]) : 0u,
                                                on ? pack_bf2(acc[k][4], acc[k][5]) : 0u, on ? pack_bf2(acc[k][6], acc[k][7]) : 0u);
    }
    __syncthreads();
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < KH; ++i)
        if (half * KH + i < KS) s = mfma16(__builtin_bit_cast(mx_frag, *(const uint4*)(ut + c16 * PR + 32 * (half * KH + i) + 8 * g)), wf[i], s);
#pragma unroll
    for (int r = 0; r < 4; ++r) part[half][map][4 * g + r][16 * cg + c16] = s[r];
    __syncthreads();
    if (mi >= rows || mc >= bs) return;
    const int ci = tid % NC;
    float al, add;
    gate(part[0][0][mi][ci] + part[1][0][mi][ci] + br, part[0][1][mi][ci] + part[1][1][mi][ci] + bi, dec, bf_to_f(ut[mi * PR + mc]), al, add);
    const float S = fmaf(al, S0, add);
    if (a.act) my = gelu_tanh_t<uint16_t>(my);
    st[0] = S;
    st[(int64_t)(1 + mpos % (uint32_t)taps) * W] = mx;
    ((uint16_t*)a.o)[(int64_t)mb * W + wc] = f_to_bf(S * my);
}

extern "C" int evo_rglru_step_bf16(const void* z, int64_t ld, const void* in_b, void* o, float* state, const void* conv, const void* conv_b, const void* ra,
                                   const void* ra_b, const void* ri, const void* ri_b, const float* decay, const int64_t* pos, int64_t B, int64_t W,
                                   int64_t nb, int64_t taps, int64_t act, void* stream) {
    if (!rg_sizes(z, o, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, ld, B, W, nb, taps) || !state) return -1;
    const int64_t bs = W / nb;
    if (bs % 8 || bs > 384 || taps > TAPS || ld % 8 || (((uintptr_t)z | (uintptr_t)ra | (uintptr_t)ri | (uintptr_t)in_b | (uintptr_t)conv_b | (uintptr_t)state) & 15)) return -1;
    RgArgs a = {z, in_b, o, state, nullptr, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, nullptr, nullptr, nullptr,
                ld, (int)W, (int)nb, (int)bs, (int)taps, 1, 0, 1, (int)act, (int)B};
    // more channels per workgroup rebuild the convolution less often, fewer spread the weights over more workgroups
    const int cg = B <= 4 ? 1 : (B <= 32 || bs > 256 ? 2 : 4);
    const dim3 grid((unsigned)((bs + 16 * cg - 1) / (16 * cg)), (unsigned)nb, (unsigned)((B + 15) / 16));
#define RS1(KS, CG) hipLaunchKernelGGL((rglru_step_kernel<KS, CG>), grid, dim3(256 * CG), 0, (hipStream_t)stream, a)
#define RS(KS) do { if (cg == 1) RS1(KS, 1); else if (cg == 2) RS1(KS, 2); else RS1(KS, 4); } while (0)
    if (bs <= 64) RS(2); else if (bs <= 96) RS(3); else if (bs <= 128) RS(4); else if (bs <= 192) RS(6); else if (bs <= 256) RS(8);
    else if (cg == 1) RS1(12, 1); else RS1(12, 2);
#undef RS1
#undef RS
    return evo_launch_status();
}

// ------------------------------------------------------------------------------------------------ any sizes, both storage types
// gates: four tokens of one block per workgroup; -> ab [M][2][W] = (a, sqrt(1 - a^2) i u)
template <typename T>
__global__ __launch_bounds__(256) void rglru_gates_any_kernel(RgArgs a, float* __restrict__ ab, int M) {
    extern __shared__ float us[];                                // [4][bs]
    const int n = blockIdx.y, m0 = blockIdx.x * 4, bs = a.bs, W = a.W, nt = M - m0 < 4 ? M - m0 : 4;
    for (int it = threadIdx.x; it < 4 * bs; it += 256) {
        const int i = it / bs, c = n * bs + it % bs, m = m0 + (i < nt ? i : nt - 1);
        const int b = a.seq ? a.seq[m] : m, t = a.cu ? m - a.cu[b] : 0;      // t: tokens of this portion before this one
        const bool go_on = !a.cu || (a.resume && a.resume[b]);
        const int64_t p = a.pos[m];
        const T* cw = (const T*)a.conv + (int64_t)c * a.taps;
        const float bias = a.in_b ? ld1((const T*)a.in_b + W + c) : 0.f;
        float u = ld1((const T*)a.conv_b + c);
        for (int back = 0; back < a.taps; ++back) {
            float x = 0.f;
            if (back <= t) x = ld1((const T*)a.z + (int64_t)(m - back) * a.ld + W + c) + bias;
            else if (go_on && p - back >= 0) x = a.state[((int64_t)b * (1 + a.taps) + 1 + (p - back) % a.taps) * W + c];
            u = fmaf(ld1(cw + a.taps - 1 - back), x, u);
        }
        us[it] = u;
    }
    __syncthreads();
    for (int c = threadIdx.x; c < bs; c += 256) {
        const int wc = n * bs + c;
        const T *wr = (const T*)a.ra + (int64_t)wc * bs, *wi = (const T*)a.ri + (int64_t)wc * bs;
        float zr[4], zi[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) { zr[i] = ld1((const T*)a.ra_b + wc); zi[i] = ld1((const T*)a.ri_b + wc); }
        for (int k = 0; k < bs; ++k) {
            const float p = ld1(wr + k), q = ld1(wi + k);
#pragma unroll
            for (int i = 0; i < 4; ++i) { zr[i] = fmaf(p, us[i * bs + k], zr[i]); zi[i] = fmaf(q, us[i * bs + k], zi[i]); }
        }
        for (int i = 0; i < nt; ++i) {
            const float l = a.decay[wc] / (1.0f + expf(-zr[i]));
            float* d = ab + (int64_t)(m0 + i) * 2 * W + wc;
            d[0] = expf(l);
            d[W] = sqrtf(-expm1f(2.0f * l)) / (1.0f + expf(-zi[i])) * us[i * bs + c];
        }
    }
}

template <typename T>
__global__ __launch_bounds__(64) void rglru_scan_any_kernel(RgArgs a, const float* __restrict__ ab) {
    const int c = blockIdx.x * 64 + threadIdx.x, b = blockIdx.y, W = a.W;
    if (c >= W) return;
    const int row0 = a.cu ? a.cu[b] : b, len = a.cu ? a.cu[b + 1] - row0 : 1;
    float* st = a.state ? a.state + (int64_t)b * (1 + a.taps) * W + c : nullptr;
    float S = (!a.cu || (a.resume && a.resume[b])) && st ? st[0] : 0.f;
    const float bias = a.in_b ? ld1((const T*)a.in_b + c) : 0.f;
    for (int t = 0; t < len; ++t) {
        const int64_t m = row0 + t;
        S = fmaf(ab[m * 2 * W + c], S, ab[m * 2 * W + W + c]);
        float y = ld1((const T*)a.z + m * a.ld + c) + bias;
        if (a.act) y = gelu_tanh_t<T>(y);
        st1((T*)a.o + m * W + c, S * y);
    }
    if (st && len > 0) st[0] = S;
}

extern "C" int evo_rglru_any(const void* z, int64_t ld, const void* in_b, void* o, float* state, float* ab, const void* conv, const void* conv_b,
                             const void* ra, const void* ra_b, const void* ri, const void* ri_b, const float* decay, const int64_t* pos, const int* seq,
                             const int* cu, const int* resume, int64_t M, int64_t B, int64_t W, int64_t nb, int64_t taps, int64_t act, int64_t f32,
                             void* stream) {
    if (!rg_sizes(z, o, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, ld, B, W, nb, taps) || !ab || M <= 0 || M > 0x7ffffff0 || !cu != !seq) return -1;
    if ((!cu && (!state || M != B)) || (resume && !state) || W / nb > 4096) return -1;
    RgArgs a = {z, in_b, o, state, nullptr, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, seq, cu, resume,
                ld, (int)W, (int)nb, (int)(W / nb), (int)taps, 1, 0, 1, (int)act, (int)B};
    hipStream_t s = (hipStream_t)stream;
    const dim3 g1((unsigned)((M + 3) / 4), (unsigned)nb), g2((unsigned)((W + 63) / 64), (unsigned)B), g3((unsigned)((W + 255) / 256), (unsigned)B);
    const size_t lds = (size_t)(W / nb) * 16;                    // (<= 64 KB)
#define RA(T)                                                                                                              \
    do {                                                                                                                   \
        hipLaunchKernelGGL((rglru_gates_any_kernel<T>), g1, dim3(256), lds, s, a, ab, (int)M);                             \
        hipLaunchKernelGGL((rglru_scan_any_kernel<T>), g2, dim3(64), 0, s, a, (const float*)ab);                           \
        if (state) hipLaunchKernelGGL((rglru_tail_kernel<T>), g3, dim3(256), 0, s, a);                                     \
    } while (0)
    if (f32) RA(float); else RA(uint16_t);
#undef RA
    return evo_launch_status();
}
