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

__device__ __forceinline__ float rcp1p_exp2(float e) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(e)); }   // 1 / (1 + 2^e)

// ------------------------------------------------------------------------------------------------ prompts
// KS: 32-wide steps of a block, NW: waves.  OUT: outputs and the sequence's end state; otherwise a segment's (product of a, end state from zero).
template <int KS, int NW, bool OUT>
__global__ __launch_bounds__(64 * NW) void rglru_chunk_kernel(RgArgs a) {
    constexpr int KP = 32 * KS, PR = KP + 8, NT = 64 * NW;
    constexpr int IT = (16 * 4 * KS + NT - 1) / NT;              // staged runs (four tokens x eight channels) per thread
    constexpr bool AHEAD = KS < 12;                              // the next tile's rows are requested a tile ahead (wide blocks: no registers left)
    extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
    uint16_t* const tile = lds;                                  // [2][RT][PR]
    float* const cw = (float*)(lds + 2 * RT * PR);               // [TAPS + 1][KP]: taps, oldest first, then the bias
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
    const uint16_t* zy = (const uint16_t*)a.z + (int64_t)row0 * a.ld + wch;
    float* st = a.state ? a.state + (int64_t)b * (1 + a.taps) * W + n * bs : nullptr;

    for (int i = tid; i < KP; i += NT) {                         // taps and bias of this block's channels
        for (int t = 0; t < TAPS; ++t) {
            const int k = t - (TAPS - a.taps);
            cw[t * KP + i] = i < bs && k >= 0 ? ld1((const uint16_t*)a.conv + (int64_t)(n * bs + i) * a.taps + k) : 0.f;
        }
        cw[TAPS * KP + i] = i < bs ? ld1((const uint16_t*)a.conv_b + n * bs + i) : 0.f;
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
    auto load_run = [&](int t0, int i, mx_u32x4* x) __attribute__((always_inline)) {
        int it = tid + NT * i;
        it = it < 16 * nd ? it : 16 * nd - 1;
        const int q = it / nd, d = it - q * nd;
#pragma unroll
        for (int u = 0; u < TAPS + 3; ++u) {
            int t = t0 + 4 * q + u - (TAPS - 1);
            t = t < 0 ? 0 : (t < len_all ? t : len_all - 1);
            x[u] = *(const mx_u32x4*)(zx + t * a.ld + 8 * d);
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
            float acc[4][8];
            {
                const float4 p = *(const float4*)(cw + TAPS * KP + 8 * d), r = *(const float4*)(cw + TAPS * KP + 8 * d + 4);
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    acc[v][0] = p.x; acc[v][1] = p.y; acc[v][2] = p.z; acc[v][3] = p.w;
                    acc[v][4] = r.x; acc[v][5] = r.y; acc[v][6] = r.z; acc[v][7] = r.w;
                }
            }
            float w[TAPS][8];
#pragma unroll
            for (int t = 0; t < TAPS; ++t) {
                const float4 p = *(const float4*)(cw + t * KP + 8 * d), r = *(const float4*)(cw + t * KP + 8 * d + 4);
                w[t][0] = p.x; w[t][1] = p.y; w[t][2] = p.z; w[t][3] = p.w; w[t][4] = r.x; w[t][5] = r.y; w[t][6] = r.z; w[t][7] = r.w;
            }
#pragma unroll
            for (int u = 0; u < TAPS + 3; ++u) {
                float x[8];
#pragma unroll
                for (int e = 0; e < 4; ++e) { x[2 * e] = bf_lo(xr[xi][u][e]); x[2 * e + 1] = bf_hi(xr[xi][u][e]); }
                if (t0 == 0 && 4 * q + u < TAPS - 1) {           // before this portion: the cached inputs, zeros before the sequence
                    const int back = TAPS - 1 - 4 * q - u;       // tokens before the portion's first, 1 .. TAPS - 1
                    const int64_t p = a.pos[row0] - back;
                    const bool have = go_on && p >= 0 && back < a.taps;
                    const float* h = st + (1 + (have ? (int)(p % a.taps) : 0)) * (int64_t)W + 8 * d;
#pragma unroll
                    for (int e = 0; e < 8; ++e) x[e] = have ? h[e] : 0.f;
                }
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    const int t = u - v;                         // tap of input u for token v
                    if (t < 0 || t >= TAPS) continue;
#pragma unroll
                    for (int e = 0; e < 8; ++e) acc[v][e] = fmaf(w[t][e], x[e], acc[v][e]);
                }
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
    load_x(s_lo);
    __syncthreads();                                             // (taps)
    int buf = 0;
    for (int t0 = s_lo; t0 < s_hi; t0 += RT, buf ^= 1) {
        uint16_t* const ut = tile + buf * RT * PR;
        convolve(t0, ut);
        __syncthreads();                                         // (the other buffer's readers are past this tile's barrier as well)
        load_x(t0 + RT);                                         // (past the end: valid rows again, not used)
        uint16_t yv[16];
        if (OUT) {
#pragma unroll
            for (int k = 0; k < 16; ++k) {
                const int t = t0 + 16 * (k >> 2) + 4 * g + (k & 3);
                yv[k] = zy[(int64_t)(t < s_hi ? t : s_hi - 1) * a.ld];
            }
        }
        __builtin_amdgcn_sched_barrier(0);
        const bool full = t0 + RT <= s_hi;
#pragma unroll
        for (int tb = 0; tb < 4; ++tb) {
            f32x4_t zr = {br, br, br, br}, zi = {bi, bi, bi, bi};
#pragma unroll
            for (int ks = 0; ks < KS; ++ks) {
                const mx_frag uf = __builtin_bit_cast(mx_frag, *(const uint4*)(ut + (16 * tb + c16) * PR + 32 * ks + 8 * g));
                zr = mfma16(uf, wr[ks], zr);
                zi = mfma16(uf, wi[ks], zi);
            }
            float pa[4], ps[4];                                  // running (product of a, state from zero) over this lane's four tokens
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float u = bf_to_f(ut[(16 * tb + 4 * g + r) * PR + cc]);
                float al = __builtin_amdgcn_exp2f(c2 * rcp1p_exp2(-LOG2E * zr[r]));
                float add = __builtin_amdgcn_sqrtf(fmaxf(fmaf(-al, al, 1.0f), 0.f)) * rcp1p_exp2(-LOG2E * zi[r]) * u;
                if (!full && t0 + 16 * tb + 4 * g + r >= s_hi) { al = 1.f; add = 0.f; }   // past the end: the state stays
                pa[r] = r ? pa[r - 1] * al : al;
                ps[r] = r ? fmaf(ps[r - 1], al, add) : add;
            }
            // inclusive scan over the four lane groups, then this group's incoming state
            float ga = pa[3], gs = ps[3];
            float ua = __shfl_up(ga, 16, 64), us = __shfl_up(gs, 16, 64);
            if (g >= 1) { gs = fmaf(us, ga, gs); ga *= ua; }
            ua = __shfl_up(ga, 32, 64); us = __shfl_up(gs, 32, 64);
            if (g >= 2) { gs = fmaf(us, ga, gs); ga *= ua; }
            const float end = fmaf(ga, S, gs);                   // state behind this group's tokens
            float in = __shfl_up(end, 16, 64);
            if (g == 0) in = S;
            if (!OUT) A *= __shfl(ga, 48 + c16, 64);
            S = __shfl(end, 48 + c16, 64);
            if (OUT) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = t0 + 16 * tb + 4 * g + r;
                    const float v = fmaf(pa[r], in, ps[r]) * bf_to_f(yv[4 * tb + r]);
                    if (t < s_hi && ch < bs) ((uint16_t*)a.o)[((int64_t)row0 + t) * W + wch] = f_to_bf(v);
                }
            }
        }
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
    if (((uintptr_t)z | (uintptr_t)ra | (uintptr_t)ri) & 15) return -1;
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
        constexpr int bytes = 2 * RT * (32 * KS + 8) * 2 + (TAPS + 1) * 32 * KS * 4;                                       \
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
// One token per sequence.  A workgroup: 16 channels of one block for up to 16 sequences; the block's convolution outputs are rebuilt in LDS (a
// few KB from L2), the four waves are the two gate maps x the halves of the sum, a thread ends with one channel of one sequence.
template <int KS>
__global__ __launch_bounds__(256) void rglru_step_kernel(RgArgs a) {
    constexpr int KP = 32 * KS, PR = KP + 8, KH = (KS + 1) / 2;
    __shared__ __attribute__((aligned(16))) uint16_t ut[16 * PR];
    __shared__ float part[4][16][17];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int n = blockIdx.y, b0 = blockIdx.z * 16, bs = a.bs, W = a.W, rows = a.rows - b0 < 16 ? a.rows - b0 : 16;
    const int c0 = blockIdx.x * 16, gate = wave & 1, ks0 = (wave >> 1) * KH;
    mx_frag wf[KH];
    {
        const uint16_t* w = (const uint16_t*)(gate ? a.ri : a.ra) + ((int64_t)n * bs + (c0 + c16 < bs ? c0 + c16 : bs - 1)) * bs;
#pragma unroll
        for (int i = 0; i < KH; ++i) {
            const int k = 32 * (ks0 + i) + 8 * g;
            wf[i] = __builtin_bit_cast(mx_frag, *(const mx_u32x4*)(w + (k < bs ? k : bs - 8)));
        }
    }
    const uint16_t* z = (const uint16_t*)a.z;
    const int nd = KP / 8;
    for (int it = tid; it < 16 * nd; it += 256) {                // eight channels of one sequence
        const int i = it / nd, d = 8 * (it - i * nd);
        uint4 u = make_uint4(0u, 0u, 0u, 0u);
        if (i < rows && d < bs) {
            const int b = b0 + i;
            const int64_t p = a.pos[b];
            float x[8], acc[8];
            vec_io<uint16_t, 8>::load(z + b * a.ld + W + n * bs + d, x);
            if (a.in_b) {
                float ib[8];
                vec_io<uint16_t, 8>::load((const uint16_t*)a.in_b + W + n * bs + d, ib);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] += ib[e];
            }
            const uint16_t* cw = (const uint16_t*)a.conv + (int64_t)(n * bs + d) * a.taps;
            vec_io<uint16_t, 8>::load((const uint16_t*)a.conv_b + n * bs + d, acc);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[e] = fmaf(ld1(cw + e * a.taps + a.taps - 1), x[e], acc[e]);
            for (int back = 1; back < a.taps; ++back) {
                if (p - back < 0) break;
                float h[8];
                vec_io<float, 8>::load(a.state + ((int64_t)b * (1 + a.taps) + 1 + (p - back) % a.taps) * W + n * bs + d, h);
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[e] = fmaf(ld1(cw + e * a.taps + a.taps - 1 - back), h[e], acc[e]);
            }
            u = make_uint4(pack_bf2(acc[0], acc[1]), pack_bf2(acc[2], acc[3]), pack_bf2(acc[4], acc[5]), pack_bf2(acc[6], acc[7]));
        }
        *(uint4*)(ut + i * PR + d) = u;
    }
    __syncthreads();
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < KH; ++i)
        if (ks0 + i < KS) s = mfma16(__builtin_bit_cast(mx_frag, *(const uint4*)(ut + c16 * PR + 32 * (ks0 + i) + 8 * g)), wf[i], s);
#pragma unroll
    for (int r = 0; r < 4; ++r) part[wave][4 * g + r][c16] = s[r];
    __syncthreads();
    const int i = tid >> 4, c = c0 + (tid & 15);                 // one channel of one sequence
    if (i >= rows || c >= bs) return;
    const int b = b0 + i, wc = n * bs + c;
    const float zr = part[0][i][tid & 15] + part[2][i][tid & 15] + ld1((const uint16_t*)a.ra_b + wc);
    const float zi = part[1][i][tid & 15] + part[3][i][tid & 15] + ld1((const uint16_t*)a.ri_b + wc);
    float x = ld1(z + b * a.ld + W + wc), y = ld1(z + b * a.ld + wc);
    if (a.in_b) { x += ld1((const uint16_t*)a.in_b + W + wc); y += ld1((const uint16_t*)a.in_b + wc); }
    if (a.act) y = gelu_tanh_t<uint16_t>(y);
    float* st = a.state + (int64_t)b * (1 + a.taps) * W + wc;
    const float al = __builtin_amdgcn_exp2f(a.decay[wc] * LOG2E * rcp1p_exp2(-LOG2E * zr));
    const float S = fmaf(al, st[0], __builtin_amdgcn_sqrtf(fmaxf(fmaf(-al, al, 1.0f), 0.f)) * rcp1p_exp2(-LOG2E * zi) * bf_to_f(ut[i * PR + c]));
    st[0] = S;
    st[(int64_t)(1 + a.pos[b] % a.taps) * W] = x;
    ((uint16_t*)a.o)[(int64_t)b * W + wc] = f_to_bf(S * y);
}

extern "C" int evo_rglru_step_bf16(const void* z, int64_t ld, const void* in_b, void* o, float* state, const void* conv, const void* conv_b, const void* ra,
                                   const void* ra_b, const void* ri, const void* ri_b, const float* decay, const int64_t* pos, int64_t B, int64_t W,
                                   int64_t nb, int64_t taps, int64_t act, void* stream) {
    if (!rg_sizes(z, o, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, ld, B, W, nb, taps) || !state) return -1;
    const int64_t bs = W / nb;
    if (bs % 8 || bs > 384 || ld % 8 || (((uintptr_t)z | (uintptr_t)ra | (uintptr_t)ri | (uintptr_t)in_b | (uintptr_t)conv_b | (uintptr_t)state) & 15)) return -1;
    RgArgs a = {z, in_b, o, state, nullptr, conv, conv_b, ra, ra_b, ri, ri_b, decay, pos, nullptr, nullptr, nullptr,
                ld, (int)W, (int)nb, (int)bs, (int)taps, 1, 0, 1, (int)act, (int)B};
    const dim3 grid((unsigned)((bs + 15) / 16), (unsigned)nb, (unsigned)((B + 15) / 16));
#define RS(KS) hipLaunchKernelGGL((rglru_step_kernel<KS>), grid, dim3(256), 0, (hipStream_t)stream, a)
    if (bs <= 64) RS(2); else if (bs <= 96) RS(3); else if (bs <= 128) RS(4); else if (bs <= 192) RS(6); else if (bs <= 256) RS(8); else RS(12);
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
