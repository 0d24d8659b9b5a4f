// dense_small.hip — y[t][n] = act(W[n] . x[t] + bias) for up to 64 tokens per pass over dense weights: every weight is read once per 64 tokens, straight from HBM into
// the A operand of 16 x 16 matrix-core tiles (rows of W = rows of the tile, tokens = its columns). HBM-bound: a workgroup owns 16 or 32 rows, its eight waves take
// interleaved 64-k blocks of them and add up through LDS. Both number formats: bf16 (v_mfma_f32_16x16x32_bf16) and f32 (v_mfma_f32_16x16x4_f32); the order of k inside a
// block is the one in which a lane's 16-byte loads lie (both operands agree on it).
// With a few tokens the prologue x + layer_norm(y) runs in every workgroup (one launch less; the residual row is written by the first).
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"

namespace {

struct SmallP {
    const void * W; const void * act; void * y; const float * bias; pm_add_norm pro;
    int K, T, lda, ldy, y_type, n_store, act_fn;
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

// x + layer_norm(y) of token wave / (8 / TP) in VP values per lane: everything the rows need is requested before the first weights (loads return in order), the sums run
// while those are on their way. Result -> LDS (T, stride ldl) and, from workgroup 0, the residual stream.
template <typename T, int TP> struct AddNorm {
    static constexpr int NW = 8 / TP, VP = PRO_MAX / 512;
    float y[VP], x[VP], w[VP], b[VP];
    int t, l;
    __device__ __forceinline__ void request(const SmallP & p, int wave, int lane) {
        const pm_add_norm & q = p.pro;
        t = wave / NW; l = (wave % NW) * 64 + lane;
        const int tt = t < p.T ? t : 0;
#pragma unroll
        for (int i = 0; i < VP; ++i) {
            const int c = i * NW * 64 + l, cc = c < q.width ? c : q.width - 1;
            y[i] = ld_g(q.y + (size_t) tt * q.ldy + cc);
            x[i] = ld_g(q.x + (size_t) tt * q.ldx + cc);
            w[i] = ld_g(q.w + cc);
            b[i] = ld_g(q.b + cc);
        }
    }
    __device__ __forceinline__ void finish(const SmallP & p, T * rows, int ldl, float * red, int wave, int lane) {
        const pm_add_norm & q = p.pro;
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < VP; ++i) s += i * NW * 64 + l < q.width ? y[i] : 0.0f;
        s = wave_sum(s);
        if (lane == 0) red[wave] = s;
        __syncthreads();
        float mean = 0.0f;
#pragma unroll
        for (int i = 0; i < NW; ++i) mean += red[t * NW + i];
        mean /= (float) q.width;
        float s2 = 0.0f;
#pragma unroll
        for (int i = 0; i < VP; ++i) { const float d = i * NW * 64 + l < q.width ? y[i] - mean : 0.0f; s2 = fmaf(d, d, s2); }
        s2 = wave_sum(s2);
        if (lane == 0) red[8 + wave] = s2;
        __syncthreads();
        float var = 0.0f;
#pragma unroll
        for (int i = 0; i < NW; ++i) var += red[8 + t * NW + i];
        const float rs = 1.0f / sqrtf(var / (float) q.width + q.eps);
        if (t < p.T) {
#pragma unroll
            for (int i = 0; i < VP; ++i) {
                const int c = i * NW * 64 + l;
                if (c < q.width) {
                    const float v = x[i] + ((y[i] - mean) * rs * w[i] + b[i]);
                    rows[t * ldl + c] = from_f<T>(v);
                    if (blockIdx.x == 0) q.x_out[(size_t) t * q.ldo + c] = v;
                } else if (c < p.K) rows[t * ldl + c] = from_f<T>(0.0f);
            }
        }
        __syncthreads();
    }
};

// SRC, where the activations come from: 0 global memory (they ride in the load groups: the vector-memory counter is in order, a later load must not be waited for in front
// of an earlier one), -1 LDS (copied once), 1 / 2 / 4 the norm prologue for that many tokens (LDS).
// LINE (bf16, activations in LDS, up to 8 tokens): the 16 tile rows are 8 rows of W x 2 halves of a 64-k block and the 16 columns 8 tokens x the same 2 halves, so that one
// load instruction covers whole 128-byte lines (a line that two instructions touch is requested twice); of the result the blocks with equal halves count.
template <typename T, int NT, int RM, int SRC> __global__ __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(4))) void dense_small_kernel(SmallP p) {
    constexpr bool LINE = sizeof(T) == 2 && SRC != 0;
    constexpr int ROWS = LINE ? 8 : 16, TOK = LINE ? 8 : 16, EPL = 16 / sizeof(T);
    // PB loads per lane and 64-k block, U blocks per load group: about eight 16-byte weight loads per lane, two groups in flight
    constexpr int PB = LINE ? 1 : Frag<T>::PER_BLOCK, NB = SRC == 0 ? NT : 0, UG = 8 / (PB * (RM + NB)), U = UG < 1 ? 1 : UG;
    constexpr bool TWO = NB < 4;                           // (NT = 4: one group, its registers are taken by the products)
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float * red = (float *) smem;                                                                  // [8 waves][NT][RM][16 columns][16 rows]
    const int wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 15, g = lane >> 4;
    const int r0 = blockIdx.x * ROWS * RM, t0 = blockIdx.y * TOK * NT;
    const int nblk = p.K >> 6, mine = (nblk - wave + 7) >> 3;                                      // 64-k blocks wave, wave + 8, ..
    const int koff = (LINE ? (lr >> 3) * 32 : 0) + g * EPL;
    const T * wrow[RM];
#pragma unroll
    for (int m = 0; m < RM; ++m) wrow[m] = (const T *) p.W + (size_t) (r0 + m * ROWS + lr % ROWS) * p.K + koff;
    const T * arow[NT];
    if (SRC == 0) {
#pragma unroll
        for (int n = 0; n < NT; ++n) { const int t = t0 + n * 16 + lr; arow[n] = (const T *) p.act + (size_t) (t < p.T ? t : p.T - 1) * p.lda + koff; }
    }
    struct Group { u32x4 w[U][RM][PB], x[U][NB ? NB : 1][PB]; };
    auto load = [&](Group & a, int grp) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = grp * U + u, k = (wave + (i < mine ? i : mine - 1) * 8) << 6;            // (past the end: the last block again, not multiplied)
#pragma unroll
            for (int s = 0; s < PB; ++s) {
#pragma unroll
                for (int n = 0; n < NB; ++n) a.x[u][n][s] = *(const PM_G u32x4 *) (arow[n] + k + s * (64 / PB));
#pragma unroll
                for (int m = 0; m < RM; ++m) a.w[u][m][s] = ld_nt16(wrow[m] + k + s * (64 / PB));
            }
        }
    };
    AddNorm<T, SRC < 1 ? 1 : SRC> norm;
    if (SRC > 0) norm.request(p, wave, lane);
    Group ga, gb;
    (void) gb;
    if (mine > 0) load(ga, 0);                             // the first weights are on their way while the activations are made
    if (SRC != 0) {
        const int ldl = p.K + EPL;
        T * rows = (T *) (smem + 8 * NT * RM * 1024);
        if (SRC > 0) norm.finish(p, rows, ldl, red, wave, lane);
        else {
            const int n16 = p.K / EPL;
            for (int t = 0; t < p.T; ++t)
                for (int i = threadIdx.x; i < n16; i += 512) *(u32x4 *) (rows + t * ldl + i * EPL) = *(const PM_G u32x4 *) ((const T *) p.act + (size_t) t * p.lda + i * EPL);
            __syncthreads();
        }
        const int t = lr % TOK;
        arow[0] = rows + (t < p.T ? t : p.T - 1) * ldl + koff;
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
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < RM; ++m) *(f32x4 *) (red + (((wave * NT + n) * RM + m) * 16 + lr) * 16 + g * 4) = acc[n][m];
    __syncthreads();
    for (int o = threadIdx.x; o < NT * RM * ROWS * TOK; o += 512) {
        const int r = o % ROWS, m = o / ROWS % RM, t = o / ROWS / RM, n = t / TOK, tt = t % TOK;      // rows fastest: a token's rows are stored as one segment
        const int row = r0 + m * ROWS + r, tok = t0 + t;
        if (row >= p.n_store || tok >= p.T) continue;
        float v = 0.0f;
#pragma unroll
        for (int w = 0; w < 8; ++w) {
            const float * q = red + (((w * NT + n) * RM + m) * 16 + tt) * 16 + r;
            v += q[0];
            if (LINE) v += q[8 * 16 + 8];
        }
        if (p.bias) v += p.bias[row];
        if (p.act_fn == PM355_ACT_RELU2) { v = fmaxf(v, 0.0f); v *= v; }
        st_type(p.y, (size_t) tok * p.ldy + row, p.y_type, v);
    }
}

template <typename T, int NT, int RM, int SRC> int launch(const SmallP & p, int N, hipStream_t st) {
    constexpr bool LINE = sizeof(T) == 2 && SRC != 0;
    constexpr int rows = (LINE ? 8 : 16) * RM, toks = (LINE ? 8 : 16) * NT;
    const size_t lds = (size_t) 8 * NT * RM * 1024 + (SRC ? (size_t) p.T * (p.K * sizeof(T) + 16) : 0);
    pm_allow_big_lds((const void *) dense_small_kernel<T, NT, RM, SRC>, lds);
    hipLaunchKernelGGL((dense_small_kernel<T, NT, RM, SRC>), dim3(N / rows, (p.T + toks - 1) / toks), dim3(512), lds, st, p);
    return 0;
}
template <typename T> int launch_type(const pm_dense_args & a, const SmallP & p, hipStream_t st) {
    const int N = (a.n_store + 63) / 64 * 64, per_wave = (a.K / 64 + 7) / 8;
    const int rm = per_wave >= 8 ? 1 : 2;                  // (a wave's load group should not outgrow its share of K)
    if (a.pro) {
        if (!pm_dense_pro_ok(a.T, a.pro->width)) return PM355_E_UNSUPPORTED;
        if constexpr (sizeof(T) == 2) if (rm == 2) return a.T == 1 ? launch<T, 1, 2, 1>(p, N, st) : a.T == 2 ? launch<T, 1, 2, 2>(p, N, st) : launch<T, 1, 2, 4>(p, N, st);
        return a.T == 1 ? launch<T, 1, 1, 1>(p, N, st) : a.T == 2 ? launch<T, 1, 1, 2>(p, N, st) : launch<T, 1, 1, 4>(p, N, st);
    }
    if constexpr (sizeof(T) == 2)
        if (a.T <= 8 && (size_t) a.T * (a.K * 2 + 16) <= 72 * 1024) return rm == 1 ? launch<T, 1, 1, -1>(p, N, st) : launch<T, 1, 2, -1>(p, N, st);
    const bool wide = N / 32 >= 512;
    if (a.T <= 16) return wide ? launch<T, 1, 2, 0>(p, N, st) : launch<T, 1, 1, 0>(p, N, st);
    if (a.T <= 32) return wide ? launch<T, 2, 2, 0>(p, N, st) : launch<T, 2, 1, 0>(p, N, st);
    if constexpr (sizeof(T) == 2) if (wide) return launch<T, 4, 2, 0>(p, N, st);
    return launch<T, 4, 1, 0>(p, N, st);
}

} // namespace

bool pm_dense_pro_ok(int T, int width) { return T >= 1 && T <= 4 && width * (T == 1 ? 1 : T == 2 ? 2 : 4) <= PRO_MAX; }

int pm_launch_dense_small(const pm_dense_args & a, hipStream_t st) {
    SmallP p = {};
    p.W = a.W; p.act = a.act; p.y = a.y; p.bias = a.bias; p.K = a.K; p.T = a.T; p.lda = a.lda; p.ldy = a.ldy; p.y_type = a.y_type; p.n_store = a.n_store; p.act_fn = a.act_fn;
    if (a.pro) p.pro = *a.pro;
    if (a.K % 64 || a.N % 64 || a.n_store > a.N || a.T < 1 || (a.type != PM_BF16 && a.type != PM_F32)) return PM355_E_SHAPE;
    return a.type == PM_BF16 ? launch_type<uint16_t>(a, p, st) : launch_type<float>(a, p, st);
}
