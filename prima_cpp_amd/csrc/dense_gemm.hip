// dense_gemm.hip — y[t][n] = act(W[n] . x[t] + bias) for prompt-sized batches, bf16 x bf16 with f32 accumulation on v_mfma_f32_32x32x16_bf16.
// Both operands travel by LDS-DMA as whole 128-byte lines (64 k per stage) into two stages; 16-byte chunks are XOR-swizzled on the source side (chunk c of row r at
// c ^ ((r >> 1) & 7): the sixteen lanes a ds_read_b128 serves hit sixteen bank groups). One barrier per stage: behind it the stage of the previous step is free and takes
// the next k-step's DMA, which has this step's MFMAs to land. Tiles 256 x 256 (eight waves, 128 tokens x 64 rows each) or 128 x 128 (four waves, 64 x 64), chosen by how
// many rounds the grid takes; tiles of one XCD form compact blocks of the output so that its L2 serves both operands.
// The same loop multiplies experts (token tiles from the routing tables, rows gathered and scattered by pair) and expands latent cache pages into keys and transposed values.
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"
#include <type_traits>

namespace {

enum { DENSE = 0, EXPERTS = 1, KEYS = 2, VALUES = 3 };
struct GemmP {
    const uint16_t * W; const uint16_t * X; void * y; const float * bias;
    int K, N, T, lda, ldy, y_type, n_store, act_fn, nt, nn;      // nt, nn: token / row tiles
    // EXPERTS: tiles = [count, {expert, first sorted pair, pairs} ..]; input rows are tokens (gather) or sorted pairs, output rows sorted pairs or pairs (scatter)
    const int32_t * tiles, * order; const float * weight; int64_t e_stride; int top, gather, scatter;
    // KEYS: X rows are those of cache pages; VALUES: the rows of W are (tokens become the columns of the output)
    const int32_t * pages; int H, per, rows_h, pad;              // heads, values per head, rows of W per head, padded head size of the output
    int splits, split_steps;                                     // DENSE: k ranges of so many 64-k steps; with more than one, y = f32 sums [splits][T][ldy] (reduce_kernel)
};

template <int N> __device__ __forceinline__ void vm_wait() { asm volatile("s_waitcnt vmcnt(%0)" :: "n"(N) : "memory"); }

template <int BM, int BN, int WM, int WN, int STAGES, int KIND> __global__ __launch_bounds__(BM / WM * (BN / WN) * 64) void dense_gemm_kernel(GemmP p) {
    constexpr int WAVES = BM / WM * (BN / WN), MI = WM / 32, NI = WN / 32, PIECES = (BM + BN) / 8 / WAVES, STAGE = (BM + BN) * 128;
    extern __shared__ __attribute__((aligned(1024))) char smem[];
    const int wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 31, h_ = lane >> 5;
    const int wm = wave / (BN / WN), wn = wave % (BN / WN);
    // tile order: XCD x = blockIdx % 8 takes a contiguous run of tiles; runs walk blocks of 8 token tiles column by column
    const int nt = KIND == EXPERTS ? __builtin_amdgcn_readfirstlane(ld_g(p.tiles)) : p.nt;      // (the grid has room for the most tiles there can be)
    const int tiles = nt * p.nn, total = KIND == DENSE ? tiles * p.splits : tiles, per = (total + 7) / 8;
    int slot = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if (slot >= total || (int) (blockIdx.x >> 3) >= per) return;
    const int split = KIND == DENSE ? slot / tiles : 0;
    slot -= split * tiles;
    const int band = slot / (8 * p.nn), left = nt - band * 8, bh = left < 8 ? left : 8, in = slot - band * 8 * p.nn;
    int t0 = (band * 8 + in % bh) * BM, n_tok = p.T;
    const int n0 = (in / bh) * BN;
    const uint16_t * W = p.W;
    if constexpr (KIND == EXPERTS) {                       // t0, n_tok: sorted pairs of this tile
        const int32_t * tt = p.tiles + 1 + 3 * (band * 8 + in % bh);
        W += (int64_t) __builtin_amdgcn_readfirstlane(ld_g(tt)) * p.e_stride;
        t0 = __builtin_amdgcn_readfirstlane(ld_g(tt + 1)); n_tok = t0 + __builtin_amdgcn_readfirstlane(ld_g(tt + 2));
    }

    // DMA pieces of this wave (8 rows of 128 bytes each): the first half of the waves brings the tokens, the second half the rows of W
    static_assert(STAGES == 2 || STAGES == 4, "stages are found by a mask, waits are spelled for these");
    static_assert(BM == BN, "a wave's pieces belong to one operand");
    const bool tok = wave < WAVES / 2;
    const char * base = tok ? (const char *) (KIND == VALUES ? W + (size_t) t0 * p.K : p.X + (KIND == EXPERTS ? 0 : (size_t) t0 * p.lda)) : (const char *) (W + (size_t) n0 * p.K);
    const int last = tok ? n_tok - 1 - t0 : p.N - 1 - n0;
    const bool paged = KIND == KEYS ? tok : KIND == VALUES ? !tok : false;
    const char * pbase[PIECES];                            // (paged: a piece's eight rows lie in one page)
    (void) pbase;
    const uint32_t pitch = (uint32_t) (tok && KIND != VALUES ? p.lda : p.K) * 2u;
    const uint32_t lds0 = (uint32_t) (uintptr_t) (__attribute__((address_space(3))) char *) smem + (uint32_t) wave * PIECES * 1024u;
    uint32_t off[PIECES];
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
        const int r = (wave * PIECES + i) * 8 + (lane >> 3), rr = tok ? r : r - BM;
        int row = rr < last ? rr : last;
        if constexpr (KIND == EXPERTS) if (tok) { row += t0; if (p.gather) row = ld_g(p.order + row) / p.top; }
        const uint32_t swz = (uint32_t) ((lane & 7) ^ ((r >> 1) & 7)) * 16u;
        if (KIND >= KEYS && paged) {
            const int at = (tok ? t0 : n0) + (wave * PIECES + i) * 8 - (tok ? 0 : BM), lim = (tok ? n_tok : p.N) - 8, a8 = at < lim ? at : lim;      // (whole pages: a multiple of 8)
            pbase[i] = (const char *) p.X + ((size_t) __builtin_amdgcn_readfirstlane(ld_g(p.pages + a8 / PM_PAGE)) * PM_PAGE + a8 % PM_PAGE) * (size_t) p.lda * 2;
            off[i] = (uint32_t) (lane >> 3) * (uint32_t) p.lda * 2u + swz;
        } else off[i] = (uint32_t) row * pitch + swz;
    }
    const int k0 = KIND == DENSE ? split * p.split_steps : 0;
    auto request = [&](int k, int stage) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < PIECES; ++i) pm_dma16((KIND >= KEYS && paged ? pbase[i] : base) + (size_t) (k0 + k) * 128, off[i], lds0 + (uint32_t) stage * STAGE + (uint32_t) i * 1024u);
    };
    f32x16 acc[MI][NI];
#pragma unroll
    for (int m = 0; m < MI; ++m)
#pragma unroll
        for (int n = 0; n < NI; ++n)
#pragma unroll
            for (int e = 0; e < 16; ++e) acc[m][n][e] = 0.0f;
    uint32_t arow[MI], brow[NI]; int asw[MI], bsw[NI];
#pragma unroll
    for (int m = 0; m < MI; ++m) { const int r = wm * WM + m * 32 + lr; arow[m] = (uint32_t) r * 128u; asw[m] = (r >> 1) & 7; }
#pragma unroll
    for (int n = 0; n < NI; ++n) { const int r = BM + wn * WN + n * 32 + lr; brow[n] = (uint32_t) r * 128u; bsw[n] = (r >> 1) & 7; }

    float bias[NI];
#pragma unroll
    for (int n = 0; n < NI; ++n) { const int col = n0 + wn * WN + n * 32 + lr; bias[n] = KIND == DENSE && p.bias && col < p.n_store ? ld_g(p.bias + col) : 0.0f; }
    const int steps = KIND == DENSE && p.split_steps < (p.K >> 6) - k0 ? p.split_steps : (p.K >> 6) - k0;
#pragma unroll
    for (int i = 0; i < STAGES - 1; ++i) if (i < steps) request(i, i);
    for (int k = 0; k < steps; ++k) {
        const int ahead = steps - 1 - k;                   // this step's lines have landed (requests complete in order) ..
        if (STAGES > 2 && ahead >= STAGES - 2) vm_wait<PIECES * (STAGES - 2)>();
        else if (STAGES > 3 && ahead == 1) vm_wait<PIECES>();
        else vm_wait<0>();
        __syncthreads();                                   // .. for every wave, and every wave is done with the stage in front of this one
        if (k + STAGES - 1 < steps) request(k + STAGES - 1, (k + STAGES - 1) & (STAGES - 1));
        const char * s = smem + (k & (STAGES - 1)) * STAGE;
        // fragments of the next 16 k are on their way while this 16 k's products run
        bf16x8 a[2][MI], b[2][NI];
        auto read = [&](int j) __attribute__((always_inline)) {
#pragma unroll
            for (int n = 0; n < NI; ++n) b[j & 1][n] = *(const bf16x8 *) (s + brow[n] + (uint32_t) (((j * 2 + h_) ^ bsw[n]) * 16));
#pragma unroll
            for (int m = 0; m < MI; ++m) a[j & 1][m] = *(const bf16x8 *) (s + arow[m] + (uint32_t) (((j * 2 + h_) ^ asw[m]) * 16));
        };
        read(0);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j < 3) read(j + 1);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int m = 0; m < MI; ++m)
#pragma unroll
                for (int n = 0; n < NI; ++n) acc[m][n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[j & 1][m], b[j & 1][n], acc[m][n], 0, 0, 0);
            __builtin_amdgcn_sched_barrier(0);
        }
    }
    int * s_pair = (int *) smem;
    float * s_weight = (float *) (smem + BM * 4);
    if constexpr (KIND == EXPERTS) {                       // what the stores need about their rows
        __syncthreads();
        for (int i = threadIdx.x; i < BM; i += WAVES * 64) {
            const int pair = ld_g(p.order + (t0 + i < n_tok ? t0 + i : n_tok - 1));
            s_pair[i] = p.scatter ? pair : t0 + i;
            s_weight[i] = p.weight ? ld_g(p.weight + pair) : 1.0f;
        }
        __syncthreads();
    }
    // tokens are the tile's rows, W rows its columns: a register's 32 lanes store 32 consecutive outputs of one token
#pragma unroll
    for (int n = 0; n < NI; ++n) {
        const int col = n0 + wn * WN + n * 32 + lr;
        const bool ok = col < p.n_store;
        // (32 rows of the tile lie in one page, or belong to one head)
        if constexpr (KIND == KEYS) {                      // K[page][head][slot][pad]
            const int h = col / p.per, d = col - h * p.per;
#pragma unroll
            for (int m = 0; m < MI; ++m) {
                const int tok0 = t0 + wm * WM + m * 32;
                uint16_t * o = (uint16_t *) p.y + (((size_t) (tok0 / PM_PAGE) * p.H + h) * PM_PAGE + tok0 % PM_PAGE) * p.pad + d;
                if (!ok || tok0 >= p.T) continue;          // (whole pages)
#pragma unroll
                for (int e = 0; e < 16; ++e) st_g(o + (size_t) ((e & 3) + 8 * (e >> 2) + 4 * h_) * p.pad, f2bf(acc[m][n][e]));
            }
            continue;
        }
        if constexpr (KIND == VALUES) {                    // V[page][head][pad][slot]: rows of the tile are W's, columns the keys
#pragma unroll
            for (int m = 0; m < MI; ++m) {
                const int row0 = t0 + wm * WM + m * 32, h = row0 / p.rows_h, d0 = row0 - h * p.rows_h;
                uint16_t * o = (uint16_t *) p.y + (((size_t) (col / PM_PAGE) * p.H + h) * p.pad + d0) * PM_PAGE + col % PM_PAGE;
                if (!ok || h >= p.H) continue;
#pragma unroll
                for (int e = 0; e < 16; ++e) {
                    const int in = (e & 3) + 8 * (e >> 2) + 4 * h_;
                    if (d0 + in < p.per) st_g(o + (size_t) in * PM_PAGE, f2bf(acc[m][n][e]));
                }
            }
            continue;
        }
        (void) ok;
    }
    if constexpr (KIND <= EXPERTS) {
        // (everything the stores need is in registers or LDS: a load among them would wait for the stores in front of it)
#pragma unroll
        for (int n = 0; n < NI; ++n) asm volatile("" : "+v"(bias[n]));
#pragma unroll
        for (int m = 0; m < MI; ++m)
#pragma unroll
            for (int n = 0; n < NI; ++n)
#pragma unroll
                for (int e = 0; e < 16; ++e) acc[m][n][e] += bias[n];
        if (p.act_fn) {
#pragma unroll
            for (int m = 0; m < MI; ++m)
#pragma unroll
                for (int n = 0; n < NI; ++n)
#pragma unroll
                    for (int e = 0; e < 16; ++e) acc[m][n][e] = act_apply(p.act_fn, acc[m][n][e]);
        }
        auto put = [&](auto * y, bool whole) __attribute__((always_inline)) {
#pragma unroll
            for (int m = 0; m < MI; ++m)
#pragma unroll
                for (int e = 0; e < 16; ++e) {
                    const int in = wm * WM + m * 32 + (e & 3) + 8 * (e >> 2) + 4 * h_;
                    if (!whole && t0 + in >= n_tok) continue;
                    float w = 1.0f;
                    int tok = t0 + in;
                    if constexpr (KIND == EXPERTS) { w = s_weight[in]; tok = s_pair[in]; }
                    auto * row = y + (size_t) (KIND == DENSE ? split * p.T + tok : tok) * p.ldy + n0 + wn * WN + lr;
#pragma unroll
                    for (int n = 0; n < NI; ++n)
                        if (whole || n0 + wn * WN + n * 32 + lr < p.n_store) st_g(row + n * 32, from_f<std::remove_reference_t<decltype(*y)>>(KIND == EXPERTS ? acc[m][n][e] * w : acc[m][n][e]));
                }
        };
        const bool whole = t0 + BM <= n_tok && n0 + BN <= p.n_store;
        if (p.y_type == PM_BF16) { if (whole) put((uint16_t *) p.y, true); else put((uint16_t *) p.y, false); }
        else { if (whole) put((float *) p.y, true); else put((float *) p.y, false); }
    }
}

// sums of k ranges -> act(sum + bias)
__global__ __launch_bounds__(256) void reduce_kernel(const float * part, int splits, int T, int ldp, const float * bias, int act_fn, void * y, int ldy, int y_type, int n_store) {
    const int quads = ldp / 4;
    const long i = (long) blockIdx.x * 256 + threadIdx.x;
    if (i >= (long) T * quads) return;
    const int t = (int) (i / quads), c = (int) (i - (long) t * quads) * 4;
    const float * src = part + (size_t) t * ldp + c;
    f32x4 v = *(const PM_G f32x4 *) src;
    for (int s = 1; s < splits; s += 4) {                  // four loads at a time
        f32x4 r[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) r[j] = *(const PM_G f32x4 *) (src + (size_t) (s + j < splits ? s + j : 0) * T * ldp);
#pragma unroll
        for (int j = 0; j < 4; ++j) if (s + j < splits) v += r[j];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) if (c + e < n_store) st_type(y, (size_t) t * ldy + c + e, y_type, act_apply(act_fn, v[e] + (bias ? ld_g(bias + c + e) : 0.0f)));
}

template <int BM, int BN, int WM, int WN, int STAGES, int KIND> int launch_stages(GemmP p, hipStream_t st) {
    constexpr int threads = BM / WM * (BN / WN) * 64;
    if (p.splits < 1) { p.splits = 1; p.split_steps = p.K >> 6; }
    if (KIND != EXPERTS) p.nt = (p.T + BM - 1) / BM;
    p.nn = (p.n_store + BN - 1) / BN;
    const size_t lds = (size_t) STAGES * (BM + BN) * 128;
    pm_allow_big_lds((const void *) dense_gemm_kernel<BM, BN, WM, WN, STAGES, KIND>, lds);
    const int per = (p.nt * p.nn * p.splits + 7) / 8;
    hipLaunchKernelGGL((dense_gemm_kernel<BM, BN, WM, WN, STAGES, KIND>), dim3(per * 8), dim3(threads), lds, st, p);
    return 0;
}
// up to one tile per CU: twice the stages hide the memory's latency; more: two tiles share a CU
template <int KIND> int launch_128(const GemmP & p, hipStream_t st) {
    if constexpr (KIND != EXPERTS) if ((long) ((p.T + 127) / 128) * ((p.n_store + 127) / 128) * (p.splits > 1 ? p.splits : 1) <= 256) return launch_stages<128, 128, 64, 64, 4, KIND>(p, st);
    return launch_stages<128, 128, 64, 64, 2, KIND>(p, st);
}

} // namespace

int pm_launch_dense_small(const pm_dense_args & a, hipStream_t st);

int pm_launch_dense_gemm(const pm_dense_args & a, hipStream_t st) {
    if (a.type != PM_BF16 || a.K % 64 || a.N % 64 || a.n_store > a.N || a.T < 1 || a.pro) return PM355_E_SHAPE;
    GemmP p = {};
    p.W = (const uint16_t *) a.W; p.X = (const uint16_t *) a.act; p.y = a.y; p.bias = a.bias; p.K = a.K; p.N = a.N; p.T = a.T; p.lda = a.lda; p.ldy = a.ldy; p.y_type = a.y_type;
    p.n_store = a.n_store; p.act_fn = a.act_fn;
    // rounds of the grid x time of a tile: a 256-tile does four times a 128-tile's work on a whole CU in ~3.4x its time (two 128-tiles share a CU)
    const long big = (long) ((a.T + 255) / 256) * ((a.n_store + 255) / 256), small = (long) ((a.T + 127) / 128) * ((a.n_store + 127) / 128);
    // too few tiles for the chip: ranges of k to different workgroups, their sums to scratch
    const int steps = a.K >> 6, ldp = (a.n_store + 3) / 4 * 4;
    const int most = steps / 4 < (int) (256 / small) ? steps / 4 : (int) (256 / small);
    if (a.split && small <= 128 && most > 1 && (size_t) most * a.T * ldp <= a.split_floats) {
        p.split_steps = (steps + most - 1) / most; p.splits = (steps + p.split_steps - 1) / p.split_steps;
        p.y = a.split; p.ldy = ldp; p.y_type = PM_F32; p.bias = nullptr; p.act_fn = PM355_ACT_NONE;
        launch_128<DENSE>(p, st);
        hipLaunchKernelGGL(reduce_kernel, dim3((unsigned) (((long) a.T * (ldp / 4) + 255) / 256)), dim3(256), 0, st, a.split, p.splits, a.T, ldp, a.bias, a.act_fn, a.y, a.ldy, a.y_type, a.n_store);
        return 0;
    }
    const double cb = (double) ((big + 255) / 256) * 1.7, cs = (double) ((small + 511) / 512);
    return cb <= cs ? launch_stages<256, 256, 128, 64, 2, DENSE>(p, st) : launch_128<DENSE>(p, st);
}

int pm_launch_dense(const pm_dense_args & a, hipStream_t st) {
    return a.pro || a.group || a.type != PM_BF16 || a.T <= 64 ? pm_launch_dense_small(a, st) : pm_launch_dense_gemm(a, st);
}

int pm_launch_experts_gemm(const pm_expert_args & a, hipStream_t st) {
    const int64_t pairs = (int64_t) a.T * a.r.top;
    if (a.type != PM_BF16 || a.T < 1 || a.width_p % 64 || a.ffp % 64 || (int64_t) a.T * a.ldx * 2 >= 1ll << 32 || pairs * a.ffp * 2 >= 1ll << 32) return PM355_E_SHAPE;
    GemmP p = {};
    p.tiles = a.r.tiles; p.order = a.r.order; p.top = a.r.top;
    if (a.r.tile != 128 && a.r.tile != 256) return PM355_E_SHAPE;
    auto go = [&]() { return a.r.tile == 256 ? launch_stages<256, 256, 128, 64, 2, EXPERTS>(p, st) : launch_128<EXPERTS>(p, st); };
    p.nt = (int) (pairs / a.r.tile + (a.r.E < pairs ? a.r.E : pairs));                  // (most tiles there can be: every expert's last one may be short)
    p.W = (const uint16_t *) a.up; p.e_stride = a.up_stride; p.X = (const uint16_t *) a.x; p.lda = a.ldx; p.K = a.width_p; p.N = p.n_store = a.ffp; p.y = a.hid; p.ldy = a.ffp;
    p.y_type = PM_BF16; p.act_fn = a.act_fn; p.gather = 1; p.weight = a.r.w;
    go();
    p.W = (const uint16_t *) a.down; p.e_stride = a.down_stride; p.X = (const uint16_t *) a.hid; p.lda = a.ffp; p.K = a.ffp; p.N = a.width_p; p.n_store = a.width; p.y = a.y; p.ldy = a.ldy;
    p.y_type = a.y_type; p.act_fn = PM355_ACT_NONE; p.gather = 0; p.scatter = 1; p.weight = nullptr;
    return go();
}

int pm_launch_latent_expand(const pm_latent_expand & x, hipStream_t st) {
    if (x.n_pages < 1 || x.kvp % 64 || x.ld % 64) return PM355_E_SHAPE;
    GemmP p = {};
    p.pages = x.pages; p.X = (const uint16_t *) x.cache; p.lda = x.ld; p.K = x.kvp; p.H = x.H;
    GemmP k = p;
    k.W = (const uint16_t *) x.Wk; k.T = x.n_pages * PM_PAGE; k.n_store = x.H * x.dim; k.N = pm_dense_pad(k.n_store); k.y = x.K; k.per = x.dim; k.pad = x.dkp;
    launch_128<KEYS>(k, st);
    p.W = (const uint16_t *) x.Wv; p.T = pm_dense_pad(x.H * x.vrows); p.N = p.n_store = x.n_pages * PM_PAGE; p.y = x.V; p.per = x.vdim; p.rows_h = x.vrows; p.pad = x.dvp;
    return launch_128<VALUES>(p, st);
}
