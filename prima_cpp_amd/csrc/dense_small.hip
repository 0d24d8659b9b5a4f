// dense_small.hip — y[t][n] = act(W[n] . x[t] + bias) for up to 64 tokens per pass over dense weights: every weight is read once per 64 tokens, straight from HBM into
// the A operand of 16 x 16 matrix-core tiles (rows of W = rows of the tile, tokens = its columns). HBM-bound: a workgroup owns 16 or 32 rows, its eight waves take
// interleaved 64-k blocks of them and add up through LDS. Both number formats: bf16 (v_mfma_f32_16x16x32_bf16) and f32 (v_mfma_f32_16x16x4_f32); the order of k inside a
// block is the one in which a lane's 16-byte loads lie (both operands agree on it).
// With a few tokens the prologue x + layer_norm(y) runs in every workgroup (one launch less; the residual row is written by the first).
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"
#include <type_traits>

namespace {

struct SmallP {
    const void * W; const void * act; void * y; const float * bias; pm_add_norm pro;
    int K, T, lda, ldy, y_type, n_store, act_fn;
};
constexpr int PRO_MAX = 8192;                              // width x tokens (rounded up to a power of two) that the prologue holds in registers

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

// rows r of [0, T): x + layer_norm(y) -> LDS (T, stride ldl) and, from workgroup 0, the residual stream. 8 / TP waves per token.
template <typename T, int TP> __device__ __forceinline__ void add_norm_prologue(const SmallP & p, T * rows, int ldl, float * red) {
    constexpr int NW = 8 / TP, VPL = PRO_MAX / TP / (NW * 64);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, t = wave / NW, l = (wave % NW) * 64 + lane;
    const pm_add_norm & q = p.pro;
    const bool on = t < p.T;
    const int tt = on ? t : 0;
    float v[VPL];
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < VPL; ++i) { const int c = i * NW * 64 + l; v[i] = c < q.width ? q.y[(size_t) tt * q.ldy + c] : 0.0f; s += v[i]; }
    s = wave_sum(s);
    if (lane == 0) red[wave] = s;
    __syncthreads();
    float mean = 0.0f;
#pragma unroll
    for (int i = 0; i < NW; ++i) mean += red[t * NW + i];
    mean /= (float) q.width;
    float s2 = 0.0f;
#pragma unroll
    for (int i = 0; i < VPL; ++i) { const int c = i * NW * 64 + l; const float d = c < q.width ? v[i] - mean : 0.0f; s2 = fmaf(d, d, s2); }
    s2 = wave_sum(s2);
    if (lane == 0) red[8 + wave] = s2;
    __syncthreads();
    float var = 0.0f;
#pragma unroll
    for (int i = 0; i < NW; ++i) var += red[8 + t * NW + i];
    const float rs = 1.0f / sqrtf(var / (float) q.width + q.eps);
    if (on) {
#pragma unroll
        for (int i = 0; i < VPL; ++i) {
            const int c = i * NW * 64 + l;
            if (c < q.width) {
                const float x = q.x[(size_t) t * q.ldx + c] + ((v[i] - mean) * rs * q.w[c] + q.b[c]);
                rows[t * ldl + c] = from_f<T>(x);
                if (blockIdx.x == 0) q.x_out[(size_t) t * q.ldo + c] = x;
            } else if (c < p.K) rows[t * ldl + c] = from_f<T>(0.0f);
        }
    }
    __syncthreads();
}

template <typename T, int NT, int RM, int TP> __global__ __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(4))) void dense_small_kernel(SmallP p) {
    // U blocks per load group (eight 16-byte loads per lane; two groups are in flight), EPL elements per 16 bytes
    constexpr int PB = Frag<T>::PER_BLOCK, EPL = 16 / sizeof(T), UG = 8 / (PB * RM) / (NT == 4 ? 2 : 1), U = UG < 1 ? 1 : UG;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float * red = (float *) smem;                                                                  // [8 waves][NT][RM][16 tokens][16 rows]
    const int wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 15, g = lane >> 4;
    const int r0 = blockIdx.x * 16 * RM, t0 = blockIdx.y * 16 * NT;
    const int nblk = p.K >> 6, mine = (nblk - wave + 7) >> 3;                                      // 64-k blocks wave, wave + 8, ..
    const T * wrow[RM];
#pragma unroll
    for (int m = 0; m < RM; ++m) wrow[m] = (const T *) p.W + (size_t) (r0 + m * 16 + lr) * p.K + g * EPL;
    auto load = [&](u32x4 (&a)[U][RM][PB], int grp) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = grp * U + u, k = (wave + (i < mine ? i : mine - 1) * 8) << 6;            // (past the end: the last block again, not multiplied)
#pragma unroll
            for (int m = 0; m < RM; ++m)
#pragma unroll
                for (int s = 0; s < PB; ++s) a[u][m][s] = ld_nt16(wrow[m] + k + s * (64 / PB));
        }
    };
    u32x4 wa[U][RM][PB], wb[U][RM][PB];
    if (mine > 0) load(wa, 0);                             // the first weights are on their way while the prologue runs
    const T * arow[NT];
    if (TP) {
        const int ldl = p.K + EPL;
        T * rows = (T *) (smem + 8 * NT * RM * 1024);
        add_norm_prologue<T, TP ? TP : 1>(p, rows, ldl, red);
        arow[0] = rows + (lr < p.T ? lr : p.T - 1) * ldl + g * EPL;
    } else {
#pragma unroll
        for (int n = 0; n < NT; ++n) { const int t = t0 + n * 16 + lr; arow[n] = (const T *) p.act + (size_t) (t < p.T ? t : p.T - 1) * p.lda + g * EPL; }
    }
    f32x4 acc[NT][RM];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < RM; ++m) acc[n][m] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    auto mma = [&](const u32x4 (&w)[U][RM][PB], int grp, bool full) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = grp * U + u, k = (wave + i * 8) << 6;
            if (!full && i >= mine) break;
#pragma unroll
            for (int s = 0; s < PB; ++s)
#pragma unroll
                for (int n = 0; n < NT; ++n) {
                    const u32x4 b = TP ? *(const u32x4 *) (arow[n] + k + s * (64 / PB)) : *(const PM_G u32x4 *) (arow[n] + k + s * (64 / PB));
#pragma unroll
                    for (int m = 0; m < RM; ++m) acc[n][m] = Frag<T>::mma(w[u][m][s], b, acc[n][m]);
                }
        }
    };
    // two register sets, the next group's loads in front of this group's products
    const int ng = (mine + U - 1) / U;
    int g2 = 0;
    for (; g2 + 2 < ng; g2 += 2) { load(wb, g2 + 1); mma(wa, g2, true); load(wa, g2 + 2); mma(wb, g2 + 1, true); }
    if (ng - g2 == 2) { load(wb, g2 + 1); mma(wa, g2, true); mma(wb, g2 + 1, false); }
    else if (ng - g2 == 1) mma(wa, g2, false);
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < RM; ++m) *(f32x4 *) (red + (((wave * NT + n) * RM + m) * 16 + lr) * 16 + g * 4) = acc[n][m];
    __syncthreads();
    for (int o = threadIdx.x; o < NT * RM * 256; o += 512) {
        const int r = o & 15, m = (o >> 4) % RM, t = (o >> 4) / RM;                     // rows fastest: a token's rows are stored as one segment
        const int n = t >> 4, tt = t & 15;
        float v = 0.0f;
#pragma unroll
        for (int w = 0; w < 8; ++w) v += red[(((w * NT + n) * RM + m) * 16 + tt) * 16 + r];
        const int row = r0 + m * 16 + r, tok = t0 + t;
        if (row < p.n_store && tok < p.T) {
            if (p.bias) v += p.bias[row];
            if (p.act_fn == PM355_ACT_RELU2) { v = fmaxf(v, 0.0f); v *= v; }
            st_type(p.y, (size_t) tok * p.ldy + row, p.y_type, v);
        }
    }
}

template <typename T, int NT, int RM, int TP> int launch(const SmallP & p, int N, hipStream_t st) {
    const size_t lds = (size_t) 8 * NT * RM * 1024 + (TP ? (size_t) p.T * (p.K * sizeof(T) + 16) : 0);
    pm_allow_big_lds((const void *) dense_small_kernel<T, NT, RM, TP>, lds);
    hipLaunchKernelGGL((dense_small_kernel<T, NT, RM, TP>), dim3(N / (16 * RM), (p.T + 16 * NT - 1) / (16 * NT)), dim3(512), lds, st, p);
    return 0;
}
template <typename T> int launch_type(const pm_dense_args & a, const SmallP & p, hipStream_t st) {
    const int N = (a.n_store + 63) / 64 * 64;
    if (a.pro) {
        // every workgroup runs the prologue: few enough of them that all are resident (two per CU)
        if (!pm_dense_pro_ok(a.T, a.pro->width)) return PM355_E_UNSUPPORTED;
        auto go = [&](auto rm) {
            constexpr int RM = decltype(rm)::value;
            return a.T == 1 ? launch<T, 1, RM, 1>(p, N, st) : a.T == 2 ? launch<T, 1, RM, 2>(p, N, st) : launch<T, 1, RM, 4>(p, N, st);
        };
        return N / 16 <= 512 ? go(std::integral_constant<int, 1>()) : N / 32 <= 512 ? go(std::integral_constant<int, 2>()) : go(std::integral_constant<int, 4>());
    }
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
