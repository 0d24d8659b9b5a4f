// attn_paged.hip — attention over paged KV caches: unit-norm q / k, capped scores, chunk and window masks, softmax with a sink, mixed values, output gate - each one a parameter
// (pm_attn_layer). Pages hold 64 tokens of one sequence per KV head: K rows [64][dkp], V transposed [dvp][64], so that both products read their matrix-core operands as
// 16-byte pieces. Four kernels:
//   prepare   q / k unit norm, value mixing, K / V into the pages (prompts; decode fuses it)
//   plain     one workgroup per (token, head) on the vector pipe: the 32-bit model and any head size
//   decode    one token x KV head (its query heads are the columns of 16 x 16 matrix-core tiles), keys split over waves and workgroups, the last workgroup merges
//   tiles     128 prompt tokens x head, 32 queries per wave as the columns of 32 x 32 tiles, pages by LDS-DMA into two stages
// In both matrix-core kernels S^T = K Q^T is computed with the key rows permuted so that a lane's score registers ARE its P operand of O^T = V^T P^T.
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"
#include <math.h>

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr float NONE = -1e30f;                             // running maximum before the first visible key

__device__ __forceinline__ int q_off(const pm_attn_layer & a, int h) { return h * a.dk; }
__device__ __forceinline__ int k_off(const pm_attn_layer & a, int g) { return a.H * a.dk + g * a.dk; }
__device__ __forceinline__ int v_off(const pm_attn_layer & a, int g) { return (a.H + a.G) * a.dk + g * a.dv; }
__device__ __forceinline__ int g_off(const pm_attn_layer & a, int h) { return (a.H + a.G) * a.dk + a.G * a.dv + h * a.dv; }

// 1 / root mean square of n projections (one wave), 1 without the norm
__device__ __forceinline__ float unit_scale(const pm_attn_layer & a, size_t at, int n) {
    if (!(a.flags & PM355_MIX_QK_NORM)) return 1.0f;
    float s = 0.0f;
    for (int d = threadIdx.x & 63; d < n; d += 64) { const float v = ld_any(a.raw, at + d, a.raw_type); s = fmaf(v, v, s); }
    return 1.0f / sqrtf(wave_sum(s) / (float) n + a.eps);
}
__device__ __forceinline__ float mixed_value(const pm_attn_layer & a, int t, int col, float v) {
    if (a.mixes == 1) v = (1.0f - a.lambda) * v + a.lambda * a.vfirst[(size_t) t * a.ld_vfirst + col];
    if (a.mixes == 2) a.vfirst[(size_t) t * a.ld_vfirst + col] = v;
    return v;
}

// blocks [0, T): q and k of a token; then one block per (64 tokens, KV head): values, transposed through LDS so that a page row is stored as one piece
template <typename T> __global__ __launch_bounds__(256) void attn_prepare_kernel(pm_attn_layer a, pm_batch_dev b, int n_tok) {
    __shared__ float tile[64 * 65];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    if ((int) blockIdx.x < n_tok) {
        const int t = blockIdx.x, pos = b.pos[t], page = b.table[(size_t) b.seq[t] * b.table_ld + pos / PM_PAGE], slot = pos % PM_PAGE;
        const int n = a.H + a.G;
        int i = wave;
        if (a.dkp <= 128) for (; i + 12 < n; i += 16) {    // four heads' loads at a time
            float v[4][2], rs[4];
            size_t at[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int hd = i + j * 4;
                at[j] = (size_t) t * a.ldraw + (hd < a.H ? q_off(a, hd) : k_off(a, hd - a.H));
                v[j][0] = lane < a.dk ? ld_any(a.raw, at[j] + lane, a.raw_type) : 0.0f;
                v[j][1] = lane + 64 < a.dk ? ld_any(a.raw, at[j] + lane + 64, a.raw_type) : 0.0f;
            }
#pragma unroll
            for (int j = 0; j < 4; ++j)
                rs[j] = a.flags & PM355_MIX_QK_NORM ? 1.0f / sqrtf(wave_sum(fmaf(v[j][1], v[j][1], v[j][0] * v[j][0])) / (float) a.dk + a.eps) : 1.0f;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int hd = i + j * 4;
                T * dst = hd < a.H ? (T *) a.q + ((size_t) t * a.H + hd) * a.dkp : (T *) a.kc + (((size_t) page * a.G + (hd - a.H)) * PM_PAGE + slot) * a.dkp;
                dst[lane] = from_f<T>(v[j][0] * rs[j]);
                if (a.dkp == 128) dst[lane + 64] = from_f<T>(v[j][1] * rs[j]);
            }
        }
        for (; i < n; i += 4) {
            const bool isq = i < a.H;
            const size_t at = (size_t) t * a.ldraw + (isq ? q_off(a, i) : k_off(a, i - a.H));
            const float rs = unit_scale(a, at, a.dk);
            T * dst = isq ? (T *) a.q + ((size_t) t * a.H + i) * a.dkp : (T *) a.kc + (((size_t) page * a.G + (i - a.H)) * PM_PAGE + slot) * a.dkp;
            for (int d = lane; d < a.dkp; d += 64) dst[d] = from_f<T>(d < a.dk ? ld_any(a.raw, at + d, a.raw_type) * rs : 0.0f);
        }
        return;
    }
    const int blk = blockIdx.x - n_tok, g = blk % a.G, t0 = blk / a.G * 64, nt = n_tok - t0 < 64 ? n_tok - t0 : 64;
    const int tl = t0 + (lane < nt ? lane : 0), pos = b.pos[tl];
    T * vrow = (T *) a.vc + ((size_t) b.table[(size_t) b.seq[tl] * b.table_ld + pos / PM_PAGE] * a.G + g) * a.dvp * PM_PAGE + pos % PM_PAGE;
    for (int d0 = 0; d0 < a.dv; d0 += 64) {
        __syncthreads();
        const int d = d0 + lane;
        for (int i = wave; i < nt; i += 4)
            if (d < a.dv) tile[i * 65 + lane] = mixed_value(a, t0 + i, g * a.dv + d, ld_any(a.raw, (size_t) (t0 + i) * a.ldraw + v_off(a, g) + d, a.raw_type));
        __syncthreads();
        for (int i = wave; i < 64; i += 4)
            if (d0 + i < a.dv && lane < nt) vrow[(size_t) (d0 + i) * PM_PAGE] = from_f<T>(tile[lane * 65 + i]);
    }
}

template <typename T> __global__ __launch_bounds__(256) void attn_plain_kernel(pm_attn_layer a, pm_batch_dev b) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ float wm[4], wl[4];
    const int t = blockIdx.x, h = blockIdx.y, g = h / (a.H / a.G), wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    float * q = sm, * p = sm + a.dkp + wave * (64 + a.dvp), * acc = p + 64;
    for (int d = threadIdx.x; d < a.dkp; d += 256) q[d] = to_f<T>(((const T *) a.q)[((size_t) t * a.H + h) * a.dkp + d]);
    for (int d = lane; d < a.dvp; d += 64) acc[d] = 0.0f;
    __syncthreads();
    const int pos = b.pos[t], first = first_key(pos, a.mask, a.mask_size);
    const int32_t * pages = b.table + (size_t) b.seq[t] * b.table_ld;
    float m = NONE, l = 0.0f;
    for (int pg = first / PM_PAGE + wave; pg <= pos / PM_PAGE; pg += 4) {
        const size_t at = (size_t) pages[pg] * a.G + g;
        const T * k = (const T *) a.kc + (at * PM_PAGE + lane) * a.dkp;
        const int key = pg * PM_PAGE + lane;
        const bool ok = key >= first && key <= pos;
        float s = 0.0f;
        for (int d = 0; d < a.dk; ++d) s = fmaf(q[d], to_f<T>(k[d]), s);
        s *= a.scale;
        if (a.cap > 0.0f) s = a.cap * tanhf(s / a.cap);
        const float mn = fmaxf(m, wave_max(ok ? s : NONE)), e = ok ? expf(s - mn) : 0.0f, corr = expf(m - mn);
        l = l * corr + wave_sum(e); m = mn;
        p[lane] = e;
        __builtin_amdgcn_wave_barrier();
        for (int d = lane; d < a.dv; d += 64) {
            const T * v = (const T *) a.vc + (at * a.dvp + d) * PM_PAGE;
            float o = acc[d] * corr;
            for (int j = 0; j < PM_PAGE; ++j) o = fmaf(p[j], to_f<T>(v[j]), o);
            acc[d] = o;
        }
        __builtin_amdgcn_wave_barrier();
    }
    if (lane == 0) { wm[wave] = m; wl[wave] = l; }
    __syncthreads();
    float M = a.flags & PM355_MIX_SINK ? a.sink[h] : NONE;
    for (int w = 0; w < 4; ++w) M = fmaxf(M, wm[w]);
    float L = a.flags & PM355_MIX_SINK ? expf(a.sink[h] - M) : 0.0f, f[4];
    for (int w = 0; w < 4; ++w) { f[w] = expf(wm[w] - M); L += wl[w] * f[w]; }
    for (int d = threadIdx.x; d < a.dv; d += 256) {
        float o = 0.0f;
        for (int w = 0; w < 4; ++w) o += sm[a.dkp + w * (64 + a.dvp) + 64 + d] * f[w];
        o /= L;
        if (a.flags & PM355_MIX_OUT_GATE) o *= 1.0f / (1.0f + expf(-ld_any(a.raw, (size_t) t * a.ldraw + g_off(a, h) + d, a.raw_type)));
        ((T *) a.out)[(size_t) t * a.ldo + h * a.dv + d] = from_f<T>(o);
    }
}

__device__ __forceinline__ bf16x8 ld_b8(const uint16_t * p) { return __builtin_bit_cast(bf16x8, *(const PM_G u32x4 *) p); }

// values published inside a launch for a workgroup on any XCD: write-through stores, loads that no cache answers
__device__ __forceinline__ void st_shared(float * p, float v) { __hip_atomic_store((PM_G float *) p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
__device__ __forceinline__ float ld_shared(const float * p) { return __hip_atomic_load((const PM_G float *) p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }

constexpr int DW = 8;                                      // waves of a decode workgroup: 32 keys each = 256 keys per round
template <int DK, int DV> __global__ __launch_bounds__(DW * 64) void attn_decode_kernel(pm_attn_layer a, pm_batch_dev b, const int32_t * rows, int fused, int splits) {
    constexpr int KS = DK / 32, VT = DV / 16, QL = DK / 64;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    float * acc_l = (float *) smem;                        // [DW waves][16 heads][DV]; its front is the query tile before the key loop
    float * m_l = acc_l + DW * 16 * DV, * l_l = m_l + DW * 16;
    uint16_t * q_l = (uint16_t *) smem;                    // [16][DK + 8]
    __shared__ int is_last;
    const int R = a.H / a.G, HT = (R + 15) / 16, g = blockIdx.y / HT, h0 = g * R + blockIdx.y % HT * 16, nh = R - blockIdx.y % HT * 16 < 16 ? R - blockIdx.y % HT * 16 : 16;
    const int t = rows ? rows[blockIdx.x] : blockIdx.x, wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 15, lg = lane >> 4;
    const int pos = b.pos[t], first = first_key(pos, a.mask, a.mask_size);
    const int32_t * pages = b.table + (size_t) b.seq[t] * b.table_ld;
    // this workgroup's pages
    const int p0 = first / PM_PAGE, np = pos / PM_PAGE - p0 + 1, per = (np + splits - 1) / splits, s = blockIdx.z;
    const int lo = p0 + s * per, hi = p0 + ((s + 1) * per < np ? (s + 1) * per : np);
    const int krow = 8 * (lr >> 2) + (lr & 3);             // key of score row lr in tile 0 (tile 1: + 4)
    bf16x8 k0[KS], k1[KS], v[VT];
    auto load = [&](int c) __attribute__((always_inline)) {          // the keys and values of chunk c (32 keys), matrix-core operands as they lie
        const size_t at = (size_t) pages[c >> 1] * a.G + g;
        const uint16_t * kp = (const uint16_t *) a.kc + (at * PM_PAGE + (c & 1) * 32 + krow) * DK + lg * 8;
        const uint16_t * vp = (const uint16_t *) a.vc + (at * DV + lr) * PM_PAGE + (c & 1) * 32 + lg * 8;
#pragma unroll
        for (int i = 0; i < KS; ++i) { k0[i] = ld_b8(kp + i * 32); k1[i] = ld_b8(kp + 4 * DK + i * 32); }
#pragma unroll
        for (int i = 0; i < VT; ++i) v[i] = ld_b8(vp + i * 16 * PM_PAGE);
    };
    // a wave's first chunk is on its way while the queries are prepared - unless it lies in the page that takes the token's own key and value
    int c = lo * 2 + wave;
    const bool any = c < hi * 2, early = any && !(fused && (c >> 1) == pos / PM_PAGE);
    if (early) load(c);

#pragma unroll
    for (int i = 0; i < 16 / DW; ++i) {
        const int h = wave + i * DW;
        float x[QL], ss = 0.0f;
        const size_t at = fused ? (size_t) t * a.ldraw + q_off(a, h0 + h) : ((size_t) t * a.H + h0 + h) * DK;
#pragma unroll
        for (int j = 0; j < QL; ++j) {
            const int d = lane + j * 64;
            x[j] = h >= nh || d >= a.dk ? 0.0f : fused ? ld_any(a.raw, at + d, a.raw_type) : bf2f(((const uint16_t *) a.q)[at + d]);
            ss = fmaf(x[j], x[j], ss);
        }
        const float rs = fused && (a.flags & PM355_MIX_QK_NORM) ? 1.0f / sqrtf(wave_sum(ss) / (float) a.dk + a.eps) : 1.0f;
#pragma unroll
        for (int j = 0; j < QL; ++j) q_l[h * (DK + 8) + lane + j * 64] = f2bf(x[j] * rs);
    }
    if (fused && pos / PM_PAGE >= lo && pos / PM_PAGE < hi) {
        // the token's own key and value: the workgroup that attends them stores them first (pages are not shared between splits)
        const size_t at = (size_t) pages[pos / PM_PAGE] * a.G + g;
        if (wave == 0) {
            const size_t kat = (size_t) t * a.ldraw + k_off(a, g);
            const float rs = unit_scale(a, kat, a.dk);
            for (int d = lane; d < a.dk; d += 64) ((uint16_t *) a.kc)[(at * PM_PAGE + pos % PM_PAGE) * DK + d] = f2bf(ld_any(a.raw, kat + d, a.raw_type) * rs);
        } else for (int d = threadIdx.x - 64; d < a.dv; d += (DW - 1) * 64)
            ((uint16_t *) a.vc)[(at * DV + d) * PM_PAGE + pos % PM_PAGE] = f2bf(mixed_value(a, t, g * a.dv + d, ld_any(a.raw, (size_t) t * a.ldraw + v_off(a, g) + d, a.raw_type)));
        pm_vm_drain();                                     // (stored before any wave of this workgroup passes the barrier and loads them)
    }
    __syncthreads();
    if (any && !early) load(c);
    bf16x8 q[KS];
#pragma unroll
    for (int i = 0; i < KS; ++i) q[i] = *(const bf16x8 *) (q_l + lr * (DK + 8) + i * 32 + lg * 8);
    __syncthreads();                                       // (the tile's LDS is the accumulators')

    f32x4 acc[VT];
#pragma unroll
    for (int i = 0; i < VT; ++i) acc[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    float m = NONE, l = 0.0f;
    const float c_in = a.cap > 0.0f ? 2.0f * LOG2E / a.cap : 0.0f;
    for (bool loaded = true; c < hi * 2; c += DW) {
        const int key0 = c * 32;
        if (!loaded) load(c);
        loaded = false;
        if (key0 > pos || key0 + 31 < first) continue;
        f32x4 s0 = {0.0f, 0.0f, 0.0f, 0.0f}, s1 = s0;
#pragma unroll
        for (int i = 0; i < KS; ++i) {
            s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0[i], q[i], s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1[i], q[i], s1, 0, 0, 0);
        }
        float x[8], mx = NONE;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int key = key0 + lg * 8 + j;
            float f = (j < 4 ? s0[j & 3] : s1[j & 3]) * a.scale;
            if (a.cap > 0.0f) f = cap_score(f, a.cap, c_in);
            x[j] = (key >= first && key <= pos) ? f * LOG2E : -INFINITY;
            mx = fmaxf(mx, x[j]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16)); mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float mn = fmaxf(m, mx), corr = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        float sum = 0.0f;
        bf16x8 pv;
#pragma unroll
        for (int j = 0; j < 8; ++j) { const float e = __builtin_amdgcn_exp2f(x[j] - mn); sum += e; pv[j] = (__bf16) e; }
        l = l * corr + sum;
#pragma unroll
        for (int i = 0; i < VT; ++i) {
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[i][e] *= corr;
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[i], pv, acc[i], 0, 0, 0);
        }
    }
    l += __shfl_xor(l, 16); l += __shfl_xor(l, 32);
#pragma unroll
    for (int i = 0; i < VT; ++i) *(f32x4 *) (acc_l + (wave * 16 + lr) * DV + i * 16 + lg * 4) = acc[i];
    if (lg == 0) { m_l[wave * 16 + lr] = m; l_l[wave * 16 + lr] = l; }
    __syncthreads();
    const bool sink = a.flags & PM355_MIX_SINK;
    auto store = [&](int h, int d, float o) {
        if (a.flags & PM355_MIX_OUT_GATE) o *= sigmoid_f(ld_any(a.raw, (size_t) t * a.ldraw + g_off(a, h0 + h) + d, a.raw_type));
        ((uint16_t *) a.out)[(size_t) t * a.ldo + (h0 + h) * a.dv + d] = f2bf(o);
    };
    const size_t slot = (size_t) blockIdx.x * gridDim.y + blockIdx.y;
    float * part = a.part + slot * splits * 16 * (DV + 2);
    for (int o = threadIdx.x; o < nh * DV; o += DW * 64) {
        const int h = o / DV, d = o % DV;
        const float sk = splits == 1 && sink ? a.sink[h0 + h] * LOG2E : NONE;
        float M = sk;
#pragma unroll
        for (int w = 0; w < DW; ++w) M = fmaxf(M, m_l[w * 16 + h]);
        float x = 0.0f, L = splits == 1 && sink ? __builtin_amdgcn_exp2f(sk - M) : 0.0f;
#pragma unroll
        for (int w = 0; w < DW; ++w) { const float f = __builtin_amdgcn_exp2f(m_l[w * 16 + h] - M); x += acc_l[(w * 16 + h) * DV + d] * f; L += l_l[w * 16 + h] * f; }
        if (splits == 1) { if (d < a.dv) store(h, d, x / L); }
        else {
            float * r = part + (s * 16 + h) * (DV + 2);
            st_shared(r + d, x);
            if (d == 0) { st_shared(r + DV, M); st_shared(r + DV + 1, L); }
        }
    }
    if (splits == 1) return;
    // partials out, then a ticket; the last split of this (token, KV head) merges all of them and re-arms the ticket
    pm_vm_drain();
    __syncthreads();
    if (threadIdx.x == 0) {
        unsigned * tk = a.ticket + slot;
        is_last = __hip_atomic_fetch_add(tk, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (unsigned) splits - 1;
        if (is_last) __hip_atomic_store(tk, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    __syncthreads();
    if (!is_last) return;
    float * ml = acc_l;                                    // [splits][16][2]
    for (int o = threadIdx.x; o < splits * 32; o += DW * 64) if ((o >> 1 & 15) < nh) ml[o] = ld_shared(part + (o >> 1) * (DV + 2) + DV + (o & 1));
    __syncthreads();
    for (int o = threadIdx.x; o < nh * DV; o += DW * 64) {
        const int h = o / DV, d = o % DV;
        if (d >= a.dv) continue;
        const float sk = sink ? a.sink[h0 + h] * LOG2E : NONE;
        float M = sk;
        for (int i = 0; i < splits; ++i) M = fmaxf(M, ml[(i * 16 + h) * 2]);
        float x = 0.0f, L = sink ? __builtin_amdgcn_exp2f(sk - M) : 0.0f;
        for (int i0 = 0; i0 < splits; i0 += 8) {
            float r[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) r[i] = ld_shared(part + ((i0 + i < splits ? i0 + i : splits - 1) * 16 + h) * (DV + 2) + d);
#pragma unroll
            for (int i = 0; i < 8; ++i)
                if (i0 + i < splits) { const float f = __builtin_amdgcn_exp2f(ml[((i0 + i) * 16 + h) * 2] - M); x += r[i] * f; L += ml[((i0 + i) * 16 + h) * 2 + 1] * f; }
        }
        store(h, d, x / L);
    }
}

// FIXED: |score| is bounded (unit-norm q and k) well inside the range of exp in f32, so no running maximum is kept, and the cap is a polynomial in a small argument
template <int DK, int DV, bool FIXED> __global__ __launch_bounds__(256, 2) void attn_tiles_kernel(pm_attn_layer a, pm_batch_dev b, const pm_attn_tile * tiles, int n_tiles, float poly) {
    constexpr int KS = DK / 16, VT = DV / 32, KB = 128 * DK, STAGE = KB + 128 * DV;      // bytes of a page: K 64 x DK x 2, V DV x 64 x 2
    constexpr int OC = DV < 128 ? DV : 128;
    extern __shared__ __attribute__((aligned(1024))) char smem[];
    const int wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 31, hf = lane >> 5;
    // an XCD (blockIdx % 8) keeps to its share of the heads: the query heads of a KV head meet in one L2
    int h, tile;
    if (a.H % 8 == 0) { const int per = a.H / 8, j = blockIdx.x >> 3; h = (blockIdx.x & 7) * per + j % per; tile = j / per; }
    else { h = blockIdx.x % a.H; tile = blockIdx.x / a.H; }
    tile = n_tiles - 1 - tile;                             // (the longest ones first)
    const pm_attn_tile tl = tiles[tile];
    const int g = h / (a.H / a.G);
    const int32_t * pages = b.table + (a.flat ? 0 : (size_t) tl.seq * b.table_ld);
    const int qi = wave * 32 + lr, qc = qi < tl.n ? qi : tl.n - 1;
    const int pos = tl.pos + qc, first = first_key(pos, a.mask, a.mask_size);
    const int w_on = wave * 32 < tl.n, w_q1 = (wave * 32 + 31 < tl.n ? wave * 32 + 31 : tl.n - 1);
    const int w_pos0 = tl.pos + wave * 32, w_pos1 = tl.pos + w_q1;                       // positions of the wave's first and last query
    const int w_first0 = w_on ? first_key(w_pos0, a.mask, a.mask_size) : 0, w_first1 = w_on ? first_key(w_pos1, a.mask, a.mask_size) : 0;
    const int pg0 = first_key(tl.pos, a.mask, a.mask_size) / PM_PAGE, pg1 = (tl.pos + tl.n - 1) / PM_PAGE;

    bf16x8 q[KS];
    const uint16_t * qp = (const uint16_t *) a.q + ((size_t) (tl.row + qc) * a.H + h) * DK + hf * 8;
#pragma unroll
    for (int i = 0; i < KS; ++i) q[i] = ld_b8(qp + i * 16);

    // DMA: a page is K pieces then V pieces of 1 KiB; wave w brings pieces w, w + 4, ..
    const uint32_t lds0 = (uint32_t) (uintptr_t) (__attribute__((address_space(3))) char *) smem;
    auto request = [&](int pg, int stage) __attribute__((always_inline)) {
        const size_t at = (size_t) __builtin_amdgcn_readfirstlane(a.flat ? tl.seq + pg : pages[pg]) * a.G + g;
        const char * kb = (const char *) a.kc + at * KB, * vb = (const char *) a.vc + at * (128 * DV);
#pragma unroll
        for (int i = 0; i < DK / 32; ++i) {
            const uint32_t o = (uint32_t) (wave + i * 4) * 1024u + (uint32_t) lane * 16u, row = o / (DK * 2), ch = o % (DK * 2) / 16;
            pm_dma16(kb, row * (DK * 2) + (ch ^ (DK % 128 ? (row >> 1) & 7 : row & 15)) * 16, lds0 + stage * STAGE + (wave + i * 4) * 1024);
        }
#pragma unroll
        for (int i = 0; i < DV / 32; ++i) {
            const uint32_t o = (uint32_t) (wave + i * 4) * 1024u + (uint32_t) lane * 16u, row = o / 128, ch = o % 128 / 16;
            pm_dma16(vb, row * 128 + (ch ^ ((row >> 1) & 7)) * 16, lds0 + stage * STAGE + KB + (wave + i * 4) * 1024);
        }
    };
    f32x16 acc[VT];
#pragma unroll
    for (int i = 0; i < VT; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e) acc[i][e] = 0.0f;
    float m = FIXED ? 0.0f : NONE, l = 0.0f;
    const float cap = a.cap, c_in = cap > 0.0f ? 2.0f * LOG2E / cap : 0.0f, c_sc = a.scale * LOG2E;
    // FIXED: log2e * cap * tanh(z / cap), z = scale * (q . k), as  z' (1 + u (-1/3 + u (2/15 - u 17/315))), u = (z / cap)^2 = poly * (q . k)^2
    const int kr = (lr & ~12) | ((lr & 4) << 1) | ((lr & 8) >> 1);                       // key row of score row lr (bits 2 and 3 swapped)
    request(pg0, 0);
    for (int pg = pg0; pg <= pg1; ++pg) {
        const int stage = (pg - pg0) & 1;
        pm_vm_drain();
        __syncthreads();
        if (pg < pg1) request(pg + 1, stage ^ 1);
        const int key0 = pg * PM_PAGE;
        if (!w_on || key0 > w_pos1 || key0 + PM_PAGE <= w_first0) continue;
        const bool open = key0 >= w_first1 && key0 + PM_PAGE - 1 <= w_pos0;              // every key visible to every query of the wave
        const char * ks = smem + stage * STAGE, * vs = ks + KB;
        f32x16 s[2];
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int e = 0; e < 16; ++e) s[t][e] = 0.0f;
        const uint32_t sw = DK % 128 ? (kr >> 1) & 7 : kr & 15;
#pragma unroll
        for (int i = 0; i < KS; ++i)
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const bf16x8 k = *(const bf16x8 *) (ks + (t * 32 + kr) * (DK * 2) + (((uint32_t) (i * 2 + hf)) ^ sw) * 16);
                s[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(k, q[i], s[t], 0, 0, 0);
            }
        float mx = NONE;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                float x = s[t][e];
                if (FIXED) {
                    const float u = x * x * poly;
                    x = (x * c_sc) * fmaf(u, fmaf(u, fmaf(u, -17.0f / 315.0f, 2.0f / 15.0f), -1.0f / 3.0f), 1.0f);
                } else {
                    x *= a.scale;
                    if (cap > 0.0f) x = cap_score(x, cap, c_in);
                    x *= LOG2E;
                }
                if (!open) {
                    const int key = key0 + t * 32 + 16 * (e >> 3) + 8 * hf + (e & 7);
                    if (key < first || key > pos) x = -INFINITY;
                }
                s[t][e] = x;
                if (!FIXED) mx = fmaxf(mx, x);
            }
        if (!FIXED) {
            mx = fmaxf(mx, __shfl_xor(mx, 32));
            const float mn = fmaxf(m, mx);
            if (__any(mn > m)) {
                const float corr = __builtin_amdgcn_exp2f(m - mn);
                l *= corr; m = mn;
#pragma unroll
                for (int i = 0; i < VT; ++i)
#pragma unroll
                    for (int e = 0; e < 16; ++e) acc[i][e] *= corr;
            }
        }
        bf16x8 p[4];
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const float x = __builtin_amdgcn_exp2f(FIXED ? s[t][e] : s[t][e] - m);
                l += x;
                p[t * 2 + (e >> 3)][e & 7] = (__bf16) x;
            }
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int i = 0; i < VT; ++i) {
                const uint32_t row = (uint32_t) (i * 32 + lr);
                const bf16x8 v = *(const bf16x8 *) (vs + row * 128 + (((uint32_t) (j * 2 + hf)) ^ ((row >> 1) & 7)) * 16);
                acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v, p[j], acc[i], 0, 0, 0);
            }
    }
    l += __shfl_xor(l, 32);
    float f = 1.0f;
    if (a.flags & PM355_MIX_SINK) {
        const float sk = a.sink[h] * LOG2E;
        if (FIXED) l += __builtin_amdgcn_exp2f(sk);
        else { const float M = fmaxf(m, sk); f = __builtin_amdgcn_exp2f(m - M); l = l * f + __builtin_amdgcn_exp2f(sk - M); }
    }
    f /= l;
    // queries are the columns of the accumulators: through LDS, then a wave stores a query's outputs as one piece, gate applied
    float * o = (float *) smem + wave * 32 * (OC + 4);
#pragma unroll
    for (int c = 0; c < DV / OC; ++c) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < OC / 32; ++i)
#pragma unroll
            for (int e = 0; e < 16; e += 4) {
                const f32x16 & s = acc[c * (OC / 32) + i];
                *(f32x4 *) (o + lr * (OC + 4) + i * 32 + 8 * (e >> 2) + 4 * hf) = f32x4{s[e] * f, s[e + 1] * f, s[e + 2] * f, s[e + 3] * f};
            }
        __syncthreads();
        if (w_on)
            for (int r = 0; r <= w_q1 - wave * 32; ++r) {
                const size_t row = (size_t) tl.row + wave * 32 + r;
#pragma unroll
                for (int d0 = 0; d0 < OC; d0 += 64) {
                    const int d = c * OC + d0 + lane;
                    if (d >= a.dv) continue;
                    float v = o[r * (OC + 4) + d0 + lane];
                    if (a.flags & PM355_MIX_OUT_GATE) v *= sigmoid_f(ld_any(a.raw, row * a.ldraw + g_off(a, h) + d, a.raw_type));
                    ((uint16_t *) a.out)[row * a.ldo + h * a.dv + d] = f2bf(v);
                }
            }
    }
}

template <int DK, int DV> int launch_tiles(const pm_attn_layer & a, const pm_batch_dev & b, const pm_attn_tile * tiles, int n, hipStream_t st) {
    constexpr int OC = DV < 128 ? DV : 128;
    const size_t stage = (size_t) 2 * 128 * (DK + DV), out = (size_t) 4 * 32 * (OC + 4) * 4, lds = stage > out ? stage : out;
    const float bound = (float) a.dk * fabsf(a.scale) * 1.02f;
    const bool fixed = (a.flags & PM355_MIX_QK_NORM) && bound <= 40.0f && (a.cap <= 0.0f || bound <= 0.3f * a.cap);
    const float poly = a.cap > 0.0f ? (a.scale / a.cap) * (a.scale / a.cap) : 0.0f;
    auto go = [&](auto kern) { pm_allow_big_lds((const void *) kern, lds); hipLaunchKernelGGL(kern, dim3(n * a.H), dim3(256), lds, st, a, b, tiles, n, poly); };
    if (fixed) go(attn_tiles_kernel<DK, DV, true>); else go(attn_tiles_kernel<DK, DV, false>);
    return 0;
}
template <int DK, int DV> int launch_decode(const pm_attn_layer & a, const pm_batch_dev & b, const int32_t * rows, int n, int fused, int splits, hipStream_t st) {
    const int R = a.H / a.G, HT = (R + 15) / 16;
    constexpr size_t lds = (size_t) DW * 16 * (DV + 2) * 4;      // (covers the query tile: 16 x (DK + 8) halves, and the merge's 64 x 32 floats)
    static_assert(lds >= (size_t) 16 * (DK + 8) * 2 && lds >= 64 * 32 * 4, "LDS");
    pm_allow_big_lds((const void *) attn_decode_kernel<DK, DV>, lds);
    hipLaunchKernelGGL((attn_decode_kernel<DK, DV>), dim3(n, a.G * HT, splits), dim3(DW * 64), lds, st, a, b, rows, fused, splits);
    return 0;
}

} // namespace

#define PM_HEAD_SIZES(CALL) \
    if (a.dkp == 64 && a.dvp == 64) return CALL(64, 64); \
    if (a.dkp == 128 && a.dvp == 64) return CALL(128, 64); \
    if (a.dkp == 64 && a.dvp == 128) return CALL(64, 128); \
    if (a.dkp == 128 && a.dvp == 128) return CALL(128, 128); \
    if (a.dkp == 256 && a.dvp == 256) return CALL(256, 256)

void pm_launch_attn_prepare(const pm_attn_layer & a, const pm_batch_dev & b, int T, hipStream_t st) {
    const dim3 grid(T + (T + 63) / 64 * a.G);
    if (a.type == PM_BF16) hipLaunchKernelGGL(attn_prepare_kernel<uint16_t>, grid, dim3(256), 0, st, a, b, T);
    else hipLaunchKernelGGL(attn_prepare_kernel<float>, grid, dim3(256), 0, st, a, b, T);
}
void pm_launch_attn_plain(const pm_attn_layer & a, const pm_batch_dev & b, int T, hipStream_t st) {
    const size_t lds = (size_t) (a.dkp + 4 * (64 + a.dvp)) * 4;
    auto go = [&](auto kern) { pm_allow_big_lds((const void *) kern, lds); hipLaunchKernelGGL(kern, dim3(T, a.H), dim3(256), lds, st, a, b); };
    if (a.type == PM_BF16) go(attn_plain_kernel<uint16_t>); else go(attn_plain_kernel<float>);
}
int pm_launch_attn_tiles(const pm_attn_layer & a, const pm_batch_dev & b, const pm_attn_tile * d_tiles, int n_tiles, hipStream_t st) {
#define PM_CALL(K, V) launch_tiles<K, V>(a, b, d_tiles, n_tiles, st)
    if (a.type != PM_BF16) return PM355_E_UNSUPPORTED;
    if (a.dkp == 192 && a.dvp == 128) return PM_CALL(192, 128);
    PM_HEAD_SIZES(PM_CALL);
    return PM355_E_UNSUPPORTED;
#undef PM_CALL
}

// keys of a (token, KV head) are split over workgroups until the grid fills the chip, but not below four pages each
int pm_attn_decode_splits(int n_tokens, int G, int max_keys) {
    const int most = (max_keys + 255) / 256, want = (768 + n_tokens * G - 1) / (n_tokens * G);
    const int s = want < most ? want : most;
    return s < 1 ? 1 : s > 64 ? 64 : s;
}
size_t pm_attn_decode_part_floats(int n_tokens, int G, int H, int dvp) {
    // (splits(n, G, ..) * n * G < 768 + 2 n G workgroup rows of 16 heads, per group of 16 query heads)
    const size_t HT = (size_t) (H / G + 15) / 16;
    return ((size_t) 768 + 2 * (size_t) n_tokens * G) * HT * 16 * (dvp + 2);
}
int pm_launch_attn_decode_paged(const pm_attn_layer & a, const pm_batch_dev & b, const int32_t * d_rows, int n, int fused, int max_keys, hipStream_t st) {
    if (a.type != PM_BF16) return PM355_E_UNSUPPORTED;
    int splits = pm_attn_decode_splits(n, a.G, max_keys);
    if (!a.part || !a.ticket || pm_attn_decode_part_floats(n, a.G, a.H, a.dvp) > a.part_floats) splits = 1;
#define PM_CALL(K, V) launch_decode<K, V>(a, b, d_rows, n, fused, splits, st)
    PM_HEAD_SIZES(PM_CALL);
    return PM355_E_UNSUPPORTED;
#undef PM_CALL
}
