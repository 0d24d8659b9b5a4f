// dense_gemm.hip — y[t][n] = act(W[n] . x[t] + bias) for prompt-sized batches, bf16 x bf16 with f32 accumulation on v_mfma_f32_32x32x16_bf16.
// Both operands travel by LDS-DMA as whole 128-byte lines (64 k per stage) into two stages; 16-byte chunks are XOR-swizzled on the source side (chunk c of row r at
// c ^ ((r >> 1) & 7): the sixteen lanes a ds_read_b128 serves hit sixteen bank groups). One barrier per stage: behind it the stage of the previous step is free and takes
// the next k-step's DMA, which has this step's MFMAs to land. Tiles 256 x 256 (eight waves, 128 tokens x 64 rows each) or 128 x 128 (four waves, 64 x 64), chosen by how
// many rounds the grid takes; tiles of one XCD form compact blocks of the output so that its L2 serves both operands.
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"
#include <stdlib.h>

namespace {

struct GemmP {
    const uint16_t * W; const uint16_t * X; void * y; const float * bias;
    int K, N, T, lda, ldy, y_type, n_store, act_fn, nt, nn;      // nt, nn: token / row tiles
};

template <int BM, int BN, int WM, int WN> __global__ __launch_bounds__(BM / WM * (BN / WN) * 64) void dense_gemm_kernel(GemmP p) {
    constexpr int WAVES = BM / WM * (BN / WN), MI = WM / 32, NI = WN / 32, PIECES = (BM + BN) / 8 / WAVES, STAGE = (BM + BN) * 128;
    extern __shared__ __attribute__((aligned(1024))) char smem[];
    const int wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 31, h = lane >> 5;
    const int wm = wave / (BN / WN), wn = wave % (BN / WN);
    // tile order: XCD x = blockIdx % 8 takes a contiguous run of tiles; runs walk blocks of 8 token tiles column by column
    const int total = p.nt * p.nn, per = (total + 7) / 8;
    const int slot = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if (slot >= total || (int) (blockIdx.x >> 3) >= per) return;
    const int band = slot / (8 * p.nn), left = p.nt - band * 8, bh = left < 8 ? left : 8, in = slot - band * 8 * p.nn;
    const int t0 = (band * 8 + in % bh) * BM, n0 = (in / bh) * BN;

    // DMA pieces of this wave (8 rows of 128 bytes each): the first half of the waves brings the tokens, the second half the rows of W
    static_assert(BM == BN, "a wave's pieces belong to one operand");
    const bool tok = wave < WAVES / 2;
    const char * base = tok ? (const char *) (p.X + (size_t) t0 * p.lda) : (const char *) (p.W + (size_t) n0 * p.K);
    const int last = tok ? p.T - 1 - t0 : p.N - 1 - n0;
    const uint32_t pitch = (uint32_t) (tok ? p.lda : p.K) * 2u;
    const uint32_t lds0 = (uint32_t) (uintptr_t) (__attribute__((address_space(3))) char *) smem + (uint32_t) wave * PIECES * 1024u;
    uint32_t off[PIECES];
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
        const int r = (wave * PIECES + i) * 8 + (lane >> 3), rr = tok ? r : r - BM;
        off[i] = (uint32_t) (rr < last ? rr : last) * pitch + (uint32_t) ((lane & 7) ^ ((r >> 1) & 7)) * 16u;
    }
    auto request = [&](int k, int stage) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < PIECES; ++i) pm_dma16(base + (size_t) k * 128, off[i], lds0 + (uint32_t) stage * STAGE + (uint32_t) i * 1024u);
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

    const int steps = p.K >> 6;
    request(0, 0);
    for (int k = 0; k < steps; ++k) {
        pm_vm_drain();                                     // this step's lines have landed ..
        __syncthreads();                                   // .. for every wave, and every wave is done with the other stage
        if (k + 1 < steps) request(k + 1, (k + 1) & 1);
        const char * s = smem + (k & 1) * STAGE;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            bf16x8 a[MI], b[NI];
#pragma unroll
            for (int n = 0; n < NI; ++n) b[n] = *(const bf16x8 *) (s + brow[n] + (uint32_t) (((j * 2 + h) ^ bsw[n]) * 16));
#pragma unroll
            for (int m = 0; m < MI; ++m) a[m] = *(const bf16x8 *) (s + arow[m] + (uint32_t) (((j * 2 + h) ^ asw[m]) * 16));
#pragma unroll
            for (int m = 0; m < MI; ++m)
#pragma unroll
                for (int n = 0; n < NI; ++n) acc[m][n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[m], b[n], acc[m][n], 0, 0, 0);
        }
    }
    // tokens are the tile's rows, W rows its columns: a register's 32 lanes store 32 consecutive outputs of one token
#pragma unroll
    for (int n = 0; n < NI; ++n) {
        const int col = n0 + wn * WN + n * 32 + lr;
        const bool ok = col < p.n_store;
        const float bias = (ok && p.bias) ? p.bias[col] : 0.0f;
#pragma unroll
        for (int m = 0; m < MI; ++m)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const int tok = t0 + wm * WM + m * 32 + (e & 3) + 8 * (e >> 2) + 4 * h;
                float v = acc[m][n][e] + bias;
                if (p.act_fn == PM355_ACT_RELU2) { v = fmaxf(v, 0.0f); v *= v; }
                if (ok && tok < p.T) st_type(p.y, (size_t) tok * p.ldy + col, p.y_type, v);
            }
    }
}

template <int BM, int BN, int WM, int WN> int launch(GemmP p, hipStream_t st) {
    constexpr int threads = BM / WM * (BN / WN) * 64;
    p.nt = (p.T + BM - 1) / BM; p.nn = (p.n_store + BN - 1) / BN;
    const size_t lds = (size_t) 2 * (BM + BN) * 128;
    pm_allow_big_lds((const void *) dense_gemm_kernel<BM, BN, WM, WN>, lds);
    const int per = (p.nt * p.nn + 7) / 8;
    hipLaunchKernelGGL((dense_gemm_kernel<BM, BN, WM, WN>), dim3(per * 8), dim3(threads), lds, st, p);
    return 0;
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
    const double cb = (double) ((big + 255) / 256) * 1.7, cs = (double) ((small + 511) / 512);
    return cb <= cs ? launch<256, 256, 128, 64>(p, st) : launch<128, 128, 64, 64>(p, st);
}

int pm_launch_dense(const pm_dense_args & a, hipStream_t st) {
    return a.pro || a.type != PM_BF16 || a.T <= 64 ? pm_launch_dense_small(a, st) : pm_launch_dense_gemm(a, st);
}
