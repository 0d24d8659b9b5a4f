// dense_small.hip — y[t][n] = act(W[n] . x[t] + bias) for up to 64 tokens per pass over dense weights: every weight is read once per 64 tokens, straight from HBM into
// the A operand of 16 x 16 matrix-core tiles (rows of W = rows of the tile, tokens = its columns). HBM-bound: a workgroup owns 16 or 32 rows, its eight waves take
// interleaved 64-k blocks of them and add up through LDS. Both number formats: bf16 (v_mfma_f32_16x16x32_bf16) and f32 (v_mfma_f32_16x16x4_f32); the order of k inside a
// block is the one in which a lane's 16-byte loads lie (both operands agree on it).
// With a few tokens the prologue x + norm(y) runs in every workgroup (one launch less; the residual row is written by the first).
// The same body serves one matrix per attention head (groups of rows with activations of their own) and experts: with a few tokens one workgroup row per (token, expert)
// pair, which routes its token in the prologue, and a down product over the concatenation of a token's experts; with more one row per expert that has tokens.
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "pm355_route.h"
#include "../../include/prima_mi355.h"

namespace {

enum { DENSE = 0, PAIR = 1, CONCAT = 2, SORTED = 3 };
struct SmallP {
    const void * W; const void * act; void * y; const float * bias; pm_add_norm pro;
    int K, T, lda, ldy, y_type, n_store, act_fn;
    int group, g_act, g_out, g_store; pm_split_merge merge;
    // experts: values between two of them; SORTED: rows in / out are sorted pairs (in_sorted / out_sorted) or tokens / pairs
    pm_route r; int64_t e_stride; int in_sorted, out_sorted, weigh;
};
// The norm prologue pays where a launch is short: up to this width x tokens (rounded up to a power of two). Wider rows cost every workgroup more than one norm launch does
// (width 2048: 8.3 us against 6.7 + 3.0; 4096: 20.8 against 15.5 + 4.2; 8192: 87 against 57 + 7)
constexpr int PRO_MAX = 2048;

template <typename T> struct Frag;                         // one 16-byte load per lane
template <> struct Frag<uint16_t> {
    static constexpr int PER_BLOCK = 2;                    // loads per lane and 64-k block
    static __device__ __forceinline__ f32x4 mma(u32x4 a, u32x4 b, f32x4 c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
    }
};
template <> struct Frag<float> {
    static constexpr int PER_BLOCK = 4;
    static __device__ __forceinline__ f32x4 mma(u32x4 a, u32x4 b, f32x4 c) {
        const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
        for (int e = 0; e < 4; ++e) c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[e], y[e], c, 0, 0, 0);
        return c;
    }
};

// x + norm(y) of token wave / (8 / TP) in VP values per lane: everything the rows need is requested before the first weights (loads return in order), the sums run
// while those are on their way. Result -> LDS (T, stride ldl) and, from workgroup 0, the residual stream.
template <typename T, int TP> struct AddNorm {
    static constexpr int NW = 8 / TP, VP = PRO_MAX / 512;
    float y[VP], x[VP], w[VP], b[VP], w2[VP];
    int t, l;
    __device__ __forceinline__ void request(const SmallP & p, int wave, int lane) {
        const pm_add_norm & q = p.pro;
        t = wave / NW; l = (wave % NW) * 64 + lane;
        const int tt = t < p.T ? t : 0;
#pragma unroll
        for (int i = 0; i < VP; ++i) {
            const int c = i * NW * 64 + l, cc = c < q.width ? c : q.width - 1;
            y[i] = ld_g(q.y + (size_t) tt * q.ldy + cc);
            x[i] = q.x ? ld_g(q.x + (size_t) tt * q.ldx + cc) : 0.0f;
            w[i] = ld_g(q.w + cc);
            b[i] = q.b ? ld_g(q.b + cc) : 0.0f;
            w2[i] = q.w2 ? ld_g(q.w2 + cc) : 1.0f;
        }
    }
    __device__ __forceinline__ float token_sum(float s, float * red, int wave, int lane) const {
        s = wave_sum(s);
        if (lane == 0) red[wave] = s;
        __syncthreads();
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < NW; ++i) o += red[t * NW + i];
        return o;
    }
    __device__ __forceinline__ void finish(const SmallP & p, T * rows, int ldl, float * red, int wave, int lane) {
        const pm_add_norm & q = p.pro;
        float s = 0.0f, mean = 0.0f;
        if (!q.rms) {
#pragma unroll
            for (int i = 0; i < VP; ++i) s += i * NW * 64 + l < q.width ? y[i] : 0.0f;
            mean = token_sum(s, red, wave, lane) / (float) q.width;
        }
        float s2 = 0.0f;
#pragma unroll
        for (int i = 0; i < VP; ++i) { const float d = i * NW * 64 + l < q.width ? y[i] - mean : 0.0f; s2 = fmaf(d, d, s2); }
        const float rs = 1.0f / sqrtf(token_sum(s2, red + 8, wave, lane) / (float) q.width + q.eps);
        float s3 = 0.0f;
#pragma unroll
        for (int i = 0; i < VP; ++i) { x[i] += (y[i] - mean) * rs * w[i] + b[i]; s3 += i * NW * 64 + l < q.width ? x[i] * x[i] : 0.0f; }
        const float r2 = q.w2 ? 1.0f / sqrtf(token_sum(s3, red + 16, wave, lane) / (float) q.width + q.eps) : 1.0f;
        if (t < p.T) {
#pragma unroll
            for (int i = 0; i < VP; ++i) {
                const int c = i * NW * 64 + l;
                const T v = from_f<T>(x[i] * (r2 * w2[i]));
                if (c < q.width) {
                    rows[t * ldl + c] = v;
                    if (blockIdx.x == 0 && q.x_out) q.x_out[(size_t) t * q.ldo + c] = x[i];
                    if (blockIdx.x == 0 && q.act_out) ((T *) q.act_out)[(size_t) t * q.ld_act + c] = v;
                } else if (c < p.K) rows[t * ldl + c] = from_f<T>(0.0f);
            }
        }
        for (int c = NW * VP * 64 + l; c < p.K && t < p.T; c += NW * 64) rows[t * ldl + c] = from_f<T>(0.0f);
        __syncthreads();
    }
};

// SRC, where the activations come from: 0 global memory (they ride in the load groups: the vector-memory counter is in order, a later load must not be waited for in front
// of an earlier one), -1 LDS (copied once), 1 / 2 / 4 the norm prologue for that many tokens (LDS).
// LINE (bf16, activations in LDS, up to 8 tokens): the 16 tile rows are 8 rows of W x 2 halves of a 64-k block and the 16 columns 8 tokens x the same 2 halves, so that one
// load instruction covers whole 128-byte lines (a line that two instructions touch is requested twice); of the result the blocks with equal halves count.
template <typename T, int NT, int RM, int SRC, int EXP> __global__ __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(4))) void dense_small_kernel(SmallP p) {
    constexpr bool LINE = sizeof(T) == 2 && SRC != 0;
    constexpr int ROWS = LINE ? 8 : 16, TOK = LINE ? 8 : 16, EPL = 16 / sizeof(T);
    // PB loads per lane and 64-k block, U blocks per load group: about eight 16-byte weight loads per lane, two groups in flight
    constexpr int PB = LINE ? 1 : Frag<T>::PER_BLOCK, NB = SRC == 0 ? NT : 0, UG = 8 / (PB * (RM + NB)), U = UG < 1 ? 1 : UG;
    constexpr bool TWO = NB < 4;                           // (NT = 4: one group, its registers are taken by the products)
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float * red = (float *) smem;                                                                  // [8 waves][NT][RM][16 columns][16 rows]
    const int wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 15, g = lane >> 4;
    const int r0 = blockIdx.x * ROWS * RM;
    // this workgroup's matrix, activations and tokens
    const T * W = (const T *) p.W, * act = (const T *) p.act;
    int t0 = blockIdx.y * TOK * NT, n_tok = p.T, base = 0;
    float weight = 1.0f;
    const int32_t * cat = nullptr;                         // CONCAT: the token's experts
    (void) cat;
    if constexpr (EXP == PAIR) {                           // base: the pair, which is also its row of y
        __shared__ int ids[64]; __shared__ float w[64];
        const int top = p.r.top, t = blockIdx.y / top, k = blockIdx.y % top;
        if (wave == 0) {
            route_token(p.r.logits + (size_t) t * p.r.ldl, p.r.E, top, p.r.groups, p.r.keep, (float *) smem, (float *) smem + 1024, ids, w);
            if (blockIdx.x == 0 && k == 0 && lane < top) { p.r.id[t * top + lane] = ids[lane]; p.r.w[t * top + lane] = w[lane]; }
        }
        __syncthreads();
        W += (size_t) __builtin_amdgcn_readfirstlane(ids[k]) * p.e_stride;
        weight = w[k]; base = blockIdx.y; act += (size_t) t * p.lda; t0 = 0; n_tok = 1;
    }
    if constexpr (EXP == CONCAT) { const int t = blockIdx.y; cat = uniform_const_ptr(p.r.id + t * p.r.top); base = t; act += (size_t) t * p.lda; t0 = 0; n_tok = 1; }
    if constexpr (EXP == SORTED) {
        if ((int) blockIdx.y >= ld_g(p.r.active)) return;
        const int e = __builtin_amdgcn_readfirstlane(ld_g(p.r.active + 1 + blockIdx.y));
        base = __builtin_amdgcn_readfirstlane(ld_g(p.r.off + e)); n_tok = __builtin_amdgcn_readfirstlane(ld_g(p.r.off + e + 1)) - base;
        W += (size_t) e * p.e_stride; t0 = 0;
    }
    if (EXP == DENSE && p.group) act += (size_t) (r0 / p.group) * p.g_act;
    // activation row of the tile's token t (< n_tok)
    auto row_in = [&](int t) __attribute__((always_inline)) -> const T * {
        if constexpr (EXP == PAIR || EXP == CONCAT) return act;
        if constexpr (EXP == SORTED) return act + (size_t) (p.in_sorted ? base + t : ld_g(p.r.order + base + t) / p.r.top) * p.lda;
        return act + (size_t) t * p.lda;
    };
    const int nb1 = p.K >> 6, nblk = EXP == CONCAT ? nb1 * p.r.top : nb1, mine = (nblk - wave + 7) >> 3;      // 64-k blocks wave, wave + 8, ..
    const int koff = (LINE ? (lr >> 3) * 32 : 0) + g * EPL;
    const T * wrow[RM];
#pragma unroll
    for (int m = 0; m < RM; ++m) wrow[m] = W + (size_t) (r0 + m * ROWS + lr % ROWS) * p.K + koff;
    auto w_at = [&](int blk) __attribute__((always_inline)) -> int64_t {      // of a 64-k block in a row of W
        if constexpr (EXP == CONCAT) { const int s = blk / nb1; return (int64_t) cat[s] * p.e_stride + ((blk - s * nb1) << 6); }
        return blk << 6;
    };
    do {
    const T * arow[NT];
    if (SRC == 0) {
#pragma unroll
        for (int n = 0; n < NT; ++n) { const int t = t0 + n * 16 + lr; arow[n] = row_in(t < n_tok ? t : n_tok - 1) + koff; }
    }
    struct Group { u32x4 w[U][RM][PB], x[U][NB ? NB : 1][PB]; };
    auto load = [&](Group & a, int grp) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = grp * U + u, blk = wave + (i < mine ? i : mine - 1) * 8, k = blk << 6;   // (past the end: the last block again, not multiplied)
            const int64_t wk = w_at(blk);
#pragma unroll
            for (int s = 0; s < PB; ++s) {
#pragma unroll
                for (int n = 0; n < NB; ++n) a.x[u][n][s] = *(const PM_G u32x4 *) (arow[n] + k + s * (64 / PB));
#pragma unroll
                for (int m = 0; m < RM; ++m) a.w[u][m][s] = ld_nt16(wrow[m] + wk + s * (64 / PB));
            }
        }
    };
    AddNorm<T, SRC < 1 ? 1 : SRC> norm;
    if (SRC > 0) norm.request(p, wave, lane);
    Group ga, gb;
    (void) gb;
    if (mine > 0) load(ga, 0);                             // the first weights are on their way while the activations are made
    if (SRC != 0) {
        const int kk = nblk << 6, ldl = kk + EPL;
        T * rows = (T *) (smem + 8 * NT * RM * 1024);
        const int here = n_tok - t0 < TOK ? n_tok - t0 : TOK;
        if (SRC > 0) norm.finish(p, rows, ldl, red, wave, lane);
        else if (EXP == DENSE && sizeof(T) == 2 && p.merge.part) {
            // the activations are sums over key splits (wave t: the shares of token t's splits)
            __shared__ float share[8 * 64];
            const int h = r0 / p.group < p.merge.H ? r0 / p.group : p.merge.H - 1;
            const size_t ht = (p.merge.H + 15) / 16;
            const pm_split_merge & q = p.merge;
            if (wave < here) {
                const size_t slot = (size_t) (t0 + wave) * ht + h / 16;
                const float * ml = q.ml + ((slot * q.splits + (lane < q.splits ? lane : 0)) * 16 + h % 16) * 2;
                const float m = lane < q.splits ? ld_g(ml) : -1e30f, l = lane < q.splits ? ld_g(ml + 1) : 0.0f, f = __builtin_amdgcn_exp2f(m - wave_max(m));
                share[wave * 64 + lane] = f / wave_sum(l * f);
            }
            __syncthreads();
            const int n2 = kk / 2;
            for (int i = threadIdx.x; i < here * n2; i += 512) {
                const int t = i / n2, c = (i - t * n2) * 2;
                const float * src = q.part + ((((size_t) (t0 + t) * ht + h / 16) * q.splits) * 16 + h % 16) * kk + c;
                float a0 = 0.0f, a1 = 0.0f;
                for (int s0 = 0; s0 < q.splits; s0 += 16) {
                    float2 v[16];
#pragma unroll
                    for (int s = 0; s < 16; ++s) v[s] = __builtin_bit_cast(float2, *(const PM_G u32x2 *) (src + (size_t) (s0 + s < q.splits ? s0 + s : 0) * 16 * kk));
#pragma unroll
                    for (int s = 0; s < 16; ++s) { const float w = s0 + s < q.splits ? share[t * 64 + s0 + s] : 0.0f; a0 = fmaf(v[s].x, w, a0); a1 = fmaf(v[s].y, w, a1); }
                }
                rows[t * ldl + c] = from_f<T>(a0); rows[t * ldl + c + 1] = from_f<T>(a1);
            }
            __syncthreads();
        } else {
            const int n16 = kk / EPL;
            for (int t = 0; t < here; ++t) {
                const T * src = row_in(t0 + t);
                for (int i = threadIdx.x; i < n16; i += 512) *(u32x4 *) (rows + t * ldl + i * EPL) = *(const PM_G u32x4 *) (src + i * EPL);
            }
            __syncthreads();
        }
        const int t = lr % TOK;
        arow[0] = rows + (t < here ? t : here - 1) * ldl + koff;
    }
    f32x4 acc[NT][RM];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < RM; ++m) acc[n][m] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    auto mma = [&](const Group & a, int grp, bool full) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = grp * U + u, k = (wave + i * 8) << 6;
            if (!full && i >= mine) break;
#pragma unroll
            for (int s = 0; s < PB; ++s)
#pragma unroll
                for (int n = 0; n < NT; ++n) {
                    u32x4 x;
                    if (NB) x = a.x[u][n][s]; else x = *(const u32x4 *) (arow[n] + k + s * (64 / PB));
#pragma unroll
                    for (int m = 0; m < RM; ++m) acc[n][m] = Frag<T>::mma(a.w[u][m][s], x, acc[n][m]);
                }
        }
    };
    // two register sets, the next group's loads in front of this group's products
    const int ng = (mine + U - 1) / U;
    int i = 0;
    if (!TWO) for (; i < ng; ++i) { if (i) load(ga, i); mma(ga, i, false); }
    else for (; i + 2 < ng; i += 2) { load(gb, i + 1); mma(ga, i, true); load(ga, i + 2); mma(gb, i + 1, true); }
    if (TWO && ng - i == 2) { load(gb, i + 1); mma(ga, i, true); mma(gb, i + 1, false); }
    else if (TWO && ng - i == 1) mma(ga, i, false);
    // A wave with nothing left to multiply comes here by a jump, and behind one of those jumps ROCm 7.2's compiler left out the wait states between a product and the store
    // that reads it (seen in the assembly of the sorted-experts kernels, and in their results): they are spelled out. 20 states: the longest such wait there is
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < RM; ++m) asm volatile("" : "+v"(acc[n][m]));
    asm volatile("s_nop 15\n\ts_nop 3");
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < RM; ++m) asm volatile("" : "+v"(acc[n][m]));
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < RM; ++m) *(f32x4 *) (red + (((wave * NT + n) * RM + m) * 16 + lr) * 16 + g * 4) = acc[n][m];
    __syncthreads();
    for (int o = threadIdx.x; o < NT * RM * ROWS * TOK; o += 512) {
        const int r = o % ROWS, m = o / ROWS % RM, t = o / ROWS / RM, n = t / TOK, tt = t % TOK;      // rows fastest: a token's rows are stored as one segment
        const int row = r0 + m * ROWS + r;
        int tok = t0 + t, col = row;
        if (tok >= n_tok) continue;
        if (EXP == DENSE && p.group) {
            const int h = row / p.group, hr = row - h * p.group;
            if (hr >= p.g_store) continue;
            col = h * p.g_out + hr;
        }
        if (col >= p.n_store) continue;
        float v = 0.0f;
#pragma unroll
        for (int w = 0; w < 8; ++w) {
            const float * q = red + (((w * NT + n) * RM + m) * 16 + tt) * 16 + r;
            v += q[0];
            if (LINE) v += q[8 * 16 + 8];
        }
        if (p.bias) v += p.bias[row];
        v = act_apply(p.act_fn, v);
        if constexpr (EXP == PAIR) { v *= weight; tok = base; }
        if constexpr (EXP == CONCAT) tok = base;
        if constexpr (EXP == SORTED) {
            const int pair = ld_g(p.r.order + base + tok);
            if (p.weigh) v *= ld_g(p.r.w + pair);
            tok = p.out_sorted ? base + tok : pair;
        }
        st_type(p.y, (size_t) tok * p.ldy + col, p.y_type, v);
    }
    if (EXP == SORTED) { t0 += TOK * NT; __syncthreads(); }
    } while (EXP == SORTED && t0 < n_tok);
}

template <typename T, int NT, int RM, int SRC, int EXP = DENSE> int launch(const SmallP & p, int N, int y, hipStream_t st) {
    constexpr bool LINE = sizeof(T) == 2 && SRC != 0;
    constexpr int rows = (LINE ? 8 : 16) * RM, toks = (LINE ? 8 : 16) * NT;
    const int here = EXP == PAIR || EXP == CONCAT ? 1 : EXP == SORTED || p.T > toks ? toks : p.T;
    size_t lds = (size_t) 8 * NT * RM * 1024 + (SRC ? (size_t) here * ((size_t) p.K * (EXP == CONCAT ? p.r.top : 1) * sizeof(T) + 16) : 0);
    if (EXP == PAIR && lds < 8192) lds = 8192;
    pm_allow_big_lds((const void *) dense_small_kernel<T, NT, RM, SRC, EXP>, lds);
    hipLaunchKernelGGL((dense_small_kernel<T, NT, RM, SRC, EXP>), dim3(N / rows, EXP == DENSE ? (p.T + toks - 1) / toks : y), dim3(512), lds, st, p);
    return 0;
}
// a wave's load group should not outgrow its share of K
int rows_per_lane(int K) { return (K / 64 + 7) / 8 >= 8 ? 1 : 2; }
constexpr size_t LDS_ACT = 72 * 1024;

template <typename T> int launch_type(const pm_dense_args & a, const SmallP & p, hipStream_t st) {
    const int N = a.group ? a.N : (a.n_store + 63) / 64 * 64;
    const int rm = rows_per_lane(a.K);
    if (a.pro) {
        if (!pm_dense_pro_ok(a.T, a.pro->width)) return PM355_E_UNSUPPORTED;
        if constexpr (sizeof(T) == 2) if (rm == 2) return a.T == 1 ? launch<T, 1, 2, 1>(p, N, 0, st) : a.T == 2 ? launch<T, 1, 2, 2>(p, N, 0, st) : launch<T, 1, 2, 4>(p, N, 0, st);
        return a.T == 1 ? launch<T, 1, 1, 1>(p, N, 0, st) : a.T == 2 ? launch<T, 1, 1, 2>(p, N, 0, st) : launch<T, 1, 1, 4>(p, N, 0, st);
    }
    if constexpr (sizeof(T) == 2)
        if (a.T <= 8 && (size_t) a.T * (a.K * 2 + 16) <= LDS_ACT) return rm == 1 ? launch<T, 1, 1, -1>(p, N, 0, st) : launch<T, 1, 2, -1>(p, N, 0, st);
    const bool wide = N / 32 >= 512;
    if (a.merge) return PM355_E_SHAPE;                     // (pm_dense_merge_ok)
    if (a.T <= 16) return wide ? launch<T, 1, 2, 0>(p, N, 0, st) : launch<T, 1, 1, 0>(p, N, 0, st);
    if (a.T <= 32) return wide ? launch<T, 2, 2, 0>(p, N, 0, st) : launch<T, 2, 1, 0>(p, N, 0, st);
    if constexpr (sizeof(T) == 2) if (wide) return launch<T, 4, 2, 0>(p, N, 0, st);
    return launch<T, 4, 1, 0>(p, N, 0, st);
}
// one product of the experts: N rows of K values per expert
template <typename T, int EXP> int launch_experts(const SmallP & p, int N, int y, hipStream_t st) {
    if constexpr (sizeof(T) == 2) {
        const size_t one = (size_t) p.K * (EXP == CONCAT ? p.r.top : 1) * 2 + 16;
        if (one * (EXP == SORTED ? 8 : 1) <= LDS_ACT) return rows_per_lane(EXP == CONCAT ? p.K * p.r.top : p.K) == 1 ? launch<T, 1, 1, -1, EXP>(p, N, y, st) : launch<T, 1, 2, -1, EXP>(p, N, y, st);
    }
    return launch<T, 1, 1, 0, EXP>(p, N, y, st);
}
template <typename T> int experts_type(const pm_expert_args & a, hipStream_t st) {
    SmallP p = {};
    p.r = a.r;
    const int pairs = a.T * a.r.top, few = a.r.E < pairs ? a.r.E : pairs;
    // up: hid = weight * act(W_up x)
    p.W = a.up; p.e_stride = a.up_stride; p.act = a.x; p.lda = a.ldx; p.K = a.width_p; p.y = a.hid; p.ldy = a.ffp; p.y_type = a.type; p.n_store = a.ffp; p.act_fn = a.act_fn; p.T = a.T;
    p.in_sorted = 0; p.out_sorted = 1; p.weigh = 1;
    int rc = a.T <= PM_ROUTE_PAIR_MAX ? launch_experts<T, PAIR>(p, a.ffp, pairs, st) : launch_experts<T, SORTED>(p, a.ffp, few, st);
    if (rc) return rc;
    p.W = a.down; p.e_stride = a.down_stride; p.act = a.hid; p.K = a.ffp; p.y = a.y; p.ldy = a.ldy; p.y_type = a.y_type; p.n_store = a.width; p.act_fn = PM355_ACT_NONE;
    p.in_sorted = 1; p.out_sorted = 0; p.weigh = 0;
    if (a.T <= PM_ROUTE_PAIR_MAX) { p.lda = a.ffp * a.r.top; return launch_experts<T, CONCAT>(p, a.width_p, a.T, st); }
    p.lda = a.ffp;
    return launch_experts<T, SORTED>(p, a.width_p, few, st);
}

} // namespace

// (every workgroup of a head merges that head's sums again: with more tokens a launch of its own costs less)
bool pm_dense_merge_ok(int T, int K) { return T <= 2 && (size_t) T * (K * 2 + 16) <= LDS_ACT; }
bool pm_dense_pro_ok(int T, int width) { return T >= 1 && T <= 4 && width * (T == 1 ? 1 : T == 2 ? 2 : 4) <= PRO_MAX; }

int pm_launch_dense_small(const pm_dense_args & a, hipStream_t st) {
    SmallP p = {};
    p.W = a.W; p.act = a.act; p.y = a.y; p.bias = a.bias; p.K = a.K; p.T = a.T; p.lda = a.lda; p.ldy = a.ldy; p.y_type = a.y_type; p.n_store = a.n_store; p.act_fn = a.act_fn;
    p.group = a.group; p.g_act = a.g_act; p.g_out = a.g_out; p.g_store = a.g_store;
    if (a.pro) p.pro = *a.pro;
    if (a.merge) p.merge = *a.merge;
    if (a.merge && (!a.group || a.type != PM_BF16 || a.merge->splits < 1 || a.merge->splits > 64 || !pm_dense_merge_ok(a.T, a.K))) return PM355_E_SHAPE;
    if (a.K % 64 || a.N % 64 || (!a.group && a.n_store > a.N) || a.T < 1 || (a.type != PM_BF16 && a.type != PM_F32)) return PM355_E_SHAPE;
    if (a.group && (a.group % 32 || a.pro || a.bias || (size_t) a.g_act * pm_dense_bytes(a.type) % 16)) return PM355_E_SHAPE;
    return a.type == PM_BF16 ? launch_type<uint16_t>(a, p, st) : launch_type<float>(a, p, st);
}

int pm_launch_experts_small(const pm_expert_args & a, hipStream_t st) {
    if (a.T < 1 || a.width_p % 64 || a.ffp % 64 || a.r.E < 1 || a.r.E > 1024 || a.r.top < 1 || a.r.top > 64 || a.r.groups > 1024 || (a.type != PM_BF16 && a.type != PM_F32)) return PM355_E_SHAPE;
    return a.type == PM_BF16 ? experts_type<uint16_t>(a, st) : experts_type<float>(a, st);
}
