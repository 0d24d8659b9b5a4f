// attn_latent.hip — latent attention over paged caches of one row per token: [normed latent c: kvp values | rotated key part: ld - kvp], shared by all heads. A head's score
// is q_unrotated . (W_uk c) + q_rotated . k_rotated and its value W_uv c. Decoded tokens (and short portions) apply W_uk^T to the query and W_uv to the weighted sum instead, so
// that every head attends over the cached rows themselves; longer portions expand the rows they see into keys and values and take the prompt kernel of attn_paged.hip.
//   prepare   query latent normed, latent normed and key part rotated into the page
//   rotate    rotated part of the queries
//   decode    one token x 16 heads x key split: 32 cached rows per step by LDS-DMA into a ring of stages, eight waves share the scores' k range and then the values' columns;
//             the values are the same LDS rows, read transposed (ds_read_b64_tr_b16). With one token per entry the cache store and the rotation happen inside
//   plain     one workgroup per (token, head) on the vector pipe: the 32-bit model and any size
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"
#include <math.h>

namespace {

constexpr float LOG2E = 1.4426950408889634f, NONE = -1e30f;
constexpr int DW = 8, STEP = 32;                           // waves of a decode workgroup, keys per step
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) s16x4 * lds_s4;

// entry i of a rotated vector; at(k): entry k of the unrotated one; cs: cos, sin of the token
template <typename F> __device__ __forceinline__ float rotated(const F & at, int i, int rot_dims, const float * cs) {
    const int half = rot_dims / 2;
    if (i < half) return at(i) * cs[2 * i] - at(i + half) * cs[2 * i + 1];
    if (i < 2 * half) return at(i) * cs[2 * (i - half)] + at(i - half) * cs[2 * (i - half) + 1];
    return at(i);
}
// the token's cache row from its projections: scale of the latent's norm (one wave), then n threads store it
// (loops of predicated loads would wait for one load after the other: these ask for eight at a time, indexes clamped)
__device__ __forceinline__ float latent_scale(const pm_latent_layer & a, int t) {
    const size_t at = (size_t) t * a.ldraw + a.q_rank;
    float s = 0.0f;
    for (int d0 = threadIdx.x & 63; d0 < a.kv_rank; d0 += 512) {
        float v[8];
        if (a.raw_type == PM_F32) {
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = ld_g((const float *) a.raw + at + (d0 + 64 * j < a.kv_rank ? d0 + 64 * j : d0));
        } else {
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = bf2f(ld_g((const uint16_t *) a.raw + at + (d0 + 64 * j < a.kv_rank ? d0 + 64 * j : d0)));
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) s = d0 + 64 * j < a.kv_rank ? fmaf(v[j], v[j], s) : s;
    }
    return 1.0f / sqrtf(wave_sum(s) / (float) a.kv_rank + a.eps);
}
// entries r0 .. r0 + 7 of a rotated bf16 vector, zero from `rot` on
__device__ __forceinline__ bf16x8 rotated8(const uint16_t * q, int r0, int rot, int rot_dims, const float * cs) {
    const int half = rot_dims / 2;
    float u[8], w[8], c[8], s[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        const int r = r0 + e < rot ? r0 + e : rot - 1, i = r < half ? r : r < 2 * half ? r - half : 0, o = r < half ? r + half : r < 2 * half ? r - half : r;
        u[e] = bf2f(ld_g(q + r)); w[e] = bf2f(ld_g(q + o)); c[e] = ld_g(cs + 2 * i); s[e] = ld_g(cs + 2 * i + 1);
    }
    bf16x8 y;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        const int r = r0 + e;
        const float t = r < half ? u[e] * c[e] - w[e] * s[e] : u[e] * c[e] + w[e] * s[e];
        y[e] = (__bf16) (r >= rot ? 0.0f : r < 2 * half ? t : u[e]);
    }
    return y;
}
template <typename T> __device__ __forceinline__ void store_row(const pm_latent_layer & a, int t, T * row, float rs, int i0, int n) {
    const size_t at = (size_t) t * a.ldraw + a.q_rank;
    for (int d = i0; d < a.kv_rank; d += n) row[d] = from_f<T>(ld_any(a.raw, at + d, a.raw_type) * (rs * a.kv_norm[d]));
    for (int i = i0; i < a.rot; i += n)
        row[a.kvp + i] = from_f<T>(rotated([&](int k) { return ld_any(a.raw, at + a.kv_rank + k, a.raw_type); }, i, a.rot_dims, a.cs + (size_t) t * a.rot_dims));
}

template <typename T> __global__ __launch_bounds__(256) void prepare_kernel(pm_latent_layer a, pm_batch_dev b) {
    __shared__ float red[4];
    const int t = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    if (a.kv_norm) {
        const int pos = b.pos[t];
        T * row = (T *) a.cache + ((size_t) b.table[(size_t) b.seq[t] * b.table_ld + pos / PM_PAGE] * PM_PAGE + pos % PM_PAGE) * a.ld;
        store_row<T>(a, t, row, latent_scale(a, t), threadIdx.x, 256);
    }
    if (!a.cq) return;
    float s = 0.0f;
    for (int d = threadIdx.x; d < a.q_rank; d += 256) { const float v = ld_any(a.raw, (size_t) t * a.ldraw + d, a.raw_type); s = fmaf(v, v, s); }
    s = wave_sum(s);
    if (lane == 0) red[wave] = s;
    __syncthreads();
    const float rs = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float) a.q_rank + a.eps);
    for (int d = threadIdx.x; d < a.q_rank; d += 256) ((T *) a.cq)[(size_t) t * a.ld_cq + d] = from_f<T>(ld_any(a.raw, (size_t) t * a.ldraw + d, a.raw_type) * (rs * a.q_norm[d]));
}
template <typename T> __global__ __launch_bounds__(256) void rotate_kernel(pm_latent_layer a) {
    const int t = blockIdx.x, half = a.rot_dims / 2, n = a.rot - half, rp = a.ld - a.kvp;
    const float * cs = a.cs + (size_t) t * a.rot_dims;
    for (int i = threadIdx.x; i < a.H * n; i += 256) {     // a thread per pair (and per entry that stays)
        const int h = i / n, k = i % n;
        T * q = (T *) a.qh + ((size_t) t * a.H + h) * a.qs + a.dim, * o = (T *) a.qa + ((size_t) t * a.H + h) * a.ld + a.kvp;
        if (k < half) {
            const float u = to_f<T>(q[k]), v = to_f<T>(q[k + half]), c = cs[2 * k], s = cs[2 * k + 1];
            q[k] = o[k] = from_f<T>(u * c - v * s);
            q[k + half] = o[k + half] = from_f<T>(v * c + u * s);
        } else o[k + half] = q[k + half];
    }
    for (int i = threadIdx.x; i < a.H * (rp - a.rot); i += 256) ((T *) a.qa)[((size_t) t * a.H + i / (rp - a.rot)) * a.ld + a.kvp + a.rot + i % (rp - a.rot)] = from_f<T>(0.0f);
}
// the shared rotated key part of expanded pages
__global__ __launch_bounds__(256) void spread_kernel(pm_latent_expand x) {
    const int p = blockIdx.x, h = blockIdx.y;
    const uint16_t * src = (const uint16_t *) x.cache + (size_t) x.pages[p] * PM_PAGE * x.ld + x.kvp;
    uint16_t * dst = (uint16_t *) x.K + ((size_t) p * x.H + h) * PM_PAGE * x.dkp + x.dim;
    for (int i = threadIdx.x; i < PM_PAGE * x.rot; i += 256) dst[(size_t) (i / x.rot) * x.dkp + i % x.rot] = src[(size_t) (i / x.rot) * x.ld + i % x.rot];
}

template <typename T> __global__ __launch_bounds__(256) void plain_kernel(pm_latent_layer a, pm_batch_dev b) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ float wm[4], wl[4];
    const int t = blockIdx.x, h = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    float * q = sm, * p = sm + a.ld + wave * (64 + a.kvp), * acc = p + 64;
    for (int d = threadIdx.x; d < a.ld; d += 256) q[d] = to_f<T>(((const T *) a.qa)[((size_t) t * a.H + h) * a.ld + d]);
    for (int d = lane; d < a.kvp; d += 64) acc[d] = 0.0f;
    __syncthreads();
    const int pos = b.pos[t], first = first_key(pos, a.mask, a.mask_size);
    const int32_t * pages = b.table + (size_t) b.seq[t] * b.table_ld;
    float m = NONE, l = 0.0f;
    for (int pg = first / PM_PAGE + wave; pg <= pos / PM_PAGE; pg += 4) {
        const T * rows = (const T *) a.cache + (size_t) pages[pg] * PM_PAGE * a.ld, * k = rows + (size_t) lane * a.ld;
        const int key = pg * PM_PAGE + lane;
        const bool ok = key >= first && key <= pos;
        float s = 0.0f;
        for (int d = 0; d < a.ld; ++d) s = fmaf(q[d], to_f<T>(k[d]), s);
        s *= a.scale;
        const float mn = fmaxf(m, wave_max(ok ? s : NONE)), e = ok ? expf(s - mn) : 0.0f, corr = expf(m - mn);
        l = l * corr + wave_sum(e); m = mn;
        p[lane] = e;
        __builtin_amdgcn_wave_barrier();
        for (int d = lane; d < a.kvp; d += 64) {
            float o = acc[d] * corr;
            for (int j = 0; j < PM_PAGE; ++j) o = fmaf(p[j], to_f<T>(rows[(size_t) j * a.ld + d]), o);
            acc[d] = o;
        }
        __builtin_amdgcn_wave_barrier();
    }
    if (lane == 0) { wm[wave] = m; wl[wave] = l; }
    __syncthreads();
    float M = NONE, L = 0.0f, f[4];
    for (int w = 0; w < 4; ++w) M = fmaxf(M, wm[w]);
    for (int w = 0; w < 4; ++w) { f[w] = expf(wm[w] - M); L += wl[w] * f[w]; }
    for (int d = threadIdx.x; d < a.kvp; d += 256) {
        float o = 0.0f;
        for (int w = 0; w < 4; ++w) o += sm[a.ld + w * (64 + a.kvp) + 64 + d] * f[w];
        ((T *) a.out)[(size_t) t * a.ldo + h * a.kvp + d] = from_f<T>(o / L);
    }
}

// waits until at most n of the wave's vector-memory operations are outstanding (rounded down to a count the instruction is spelled for)
__device__ __forceinline__ void vm_wait(int n) {
    if (n >= 24) asm volatile("s_waitcnt vmcnt(24)" ::: "memory");
    else if (n >= 16) asm volatile("s_waitcnt vmcnt(16)" ::: "memory");
    else if (n >= 12) asm volatile("s_waitcnt vmcnt(12)" ::: "memory");
    else if (n >= 10) asm volatile("s_waitcnt vmcnt(10)" ::: "memory");
    else if (n >= 8) asm volatile("s_waitcnt vmcnt(8)" ::: "memory");
    else if (n >= 6) asm volatile("s_waitcnt vmcnt(6)" ::: "memory");
    else if (n == 5) asm volatile("s_waitcnt vmcnt(5)" ::: "memory");
    else if (n == 4) asm volatile("s_waitcnt vmcnt(4)" ::: "memory");
    else if (n == 3) asm volatile("s_waitcnt vmcnt(3)" ::: "memory");
    else if (n == 2) asm volatile("s_waitcnt vmcnt(2)" ::: "memory");
    else if (n == 1) asm volatile("s_waitcnt vmcnt(1)" ::: "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
}

// VT: 16-column value tiles per wave (kvp <= 128 VT). A wave's 16-byte pieces of the scores' k range and its DMA pieces per step are at most VT + 2
template <int VT> __global__ __launch_bounds__(DW * 64) void latent_decode_kernel(pm_latent_layer a, pm_batch_dev b, int fused, int splits, int stages,
                                                                                                      float * ml) {
    constexpr int QS = VT + 2;
    extern __shared__ __attribute__((aligned(1024))) char smem[];
    const uint32_t pitch = (uint32_t) a.ld * 2u, stage_bytes = pitch * STEP;
    float * sp = (float *) (smem + stages * stage_bytes);  // [4 k ranges][2 key tiles][64 lanes][4]
    const int h0 = blockIdx.y * 16, nh = a.H - h0 < 16 ? a.H - h0 : 16, t = blockIdx.x;
    const int wave = __builtin_amdgcn_readfirstlane((int) threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 15, lg = lane >> 4;
    const int pos = __builtin_amdgcn_readfirstlane(ld_g(b.pos + t)), first = first_key(pos, a.mask, a.mask_size);
    const int32_t * pages = uniform_const_ptr(b.table + (size_t) ld_g(b.seq + t) * b.table_ld);
    const int p0 = first / PM_PAGE, np = pos / PM_PAGE - p0 + 1, per = (np + splits - 1) / splits, s = blockIdx.z;
    const int lo = p0 + s * per, hi = p0 + ((s + 1) * per < np ? (s + 1) * per : np);
    const int c0 = lo * 2 > first / STEP ? lo * 2 : first / STEP, c1 = hi * 2 < pos / STEP + 1 ? hi * 2 : pos / STEP + 1;

    if (fused && a.kv_norm && pos / PM_PAGE >= lo && pos / PM_PAGE < hi) {
        // the token's own row: the workgroups that attend its page store it first (all heads' workgroups write the same values)
        store_row<uint16_t>(a, t, (uint16_t *) a.cache + ((size_t) pages[pos / PM_PAGE] * PM_PAGE + pos % PM_PAGE) * a.ld, latent_scale(a, t), threadIdx.x, DW * 64);
        pm_vm_drain();
    }
    __syncthreads();
    // LDS rows are swizzled in 16-byte pieces: sixteen lanes that read one piece of sixteen rows hit different banks
    const bool wide = (a.ld & 127) == 0;
    auto swz = [&](uint32_t row) __attribute__((always_inline)) -> uint32_t { return wide ? row & 15u : (row >> 1) & 7u; };
    const int n_piece = a.ld / 16, mine = (n_piece - wave + DW - 1) / DW;
    const uint32_t lds0 = (uint32_t) (uintptr_t) (__attribute__((address_space(3))) char *) smem;
    uint32_t voff[QS];
#pragma unroll
    for (int i = 0; i < QS; ++i) {
        const uint32_t o = (uint32_t) (wave + i * DW) * 1024u + (uint32_t) lane * 16u, row = o / pitch, ch = (o - row * pitch) / 16u;
        voff[i] = row * pitch + (ch ^ swz(row)) * 16u;
    }
    auto request = [&](int c, int stage) __attribute__((always_inline)) {
        const char * base = (const char *) a.cache + ((size_t) pages[c >> 1] * PM_PAGE + (c & 1) * STEP) * pitch;
#pragma unroll
        for (int i = 0; i < QS; ++i) if (i < mine) pm_dma16(base, voff[i], lds0 + (uint32_t) stage * stage_bytes + (uint32_t) (wave + i * DW) * 1024u);
    };
    for (int i = 0; i < stages - 1; ++i) if (c0 + i < c1) request(c0 + i, i);

    // this wave's pieces of the queries: key tile kt, k pieces kq, kq + 4, ..
    const int kt = wave & 1, kq = wave >> 1, ks = a.ld / 32;
    bf16x8 q[QS];
    const uint16_t * qa = (const uint16_t *) a.qa + ((size_t) t * a.H + h0 + (lr < nh ? lr : 0)) * a.ld;
    const uint16_t * qr = (const uint16_t *) a.qh + ((size_t) t * a.H + h0 + (lr < nh ? lr : 0)) * a.qs + a.dim;
#pragma unroll
    for (int i = 0; i < QS; ++i) {
        const int k = (kq + 4 * i) * 32 + lg * 8;
        q[i] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
        if (kq + 4 * i >= ks) continue;
        if (k < a.kvp || !fused) q[i] = __builtin_bit_cast(bf16x8, *(const PM_G u32x4 *) (qa + k));
        else q[i] = rotated8(qr, k - a.kvp, a.rot, a.rot_dims, a.cs + (size_t) t * a.rot_dims);
        if (lr >= nh) q[i] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
    const uint32_t krow = 8 * (lr >> 2) + 4 * kt + (lr & 3);            // key of score row lr
    const uint32_t kbase = krow * pitch, ksw = swz(krow);
    const uint32_t v0 = 8 * lg + (lr >> 2), v1 = v0 + 4;                // rows this lane addresses in the transposed reads
    const uint32_t vb0 = v0 * pitch + (lr & 1) * 8, vb1 = v1 * pitch + (lr & 1) * 8, vs0 = swz(v0), vs1 = swz(v1);
    f32x4 acc[VT];
#pragma unroll
    for (int i = 0; i < VT; ++i) acc[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    float m = NONE, l = 0.0f;
    const float c_sc = a.scale * LOG2E;
    const int vt = a.kvp / 16;
    int stage = 0;
    for (int c = c0; c < c1; ++c) {
        const int ahead = c1 - 1 - c < stages - 2 ? c1 - 1 - c : stages - 2;
        vm_wait(ahead * mine);
        __syncthreads();                                   // this step's rows are there for every wave, and the stage in front of it is free
        if (c + stages - 1 < c1) request(c + stages - 1, stage ? stage - 1 : stages - 1);
        const char * rows = smem + stage * stage_bytes;
        f32x4 x4 = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int i = 0; i < QS; ++i)
            if (kq + 4 * i < ks) {
                const bf16x8 k = *(const bf16x8 *) (rows + kbase + ((((uint32_t) (kq + 4 * i) * 4u + lg) ^ ksw) * 16u));
                x4 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, q[i], x4, 0, 0, 0);
            }
        *(f32x4 *) (sp + ((kq * 2 + kt) * 64 + lane) * 4) = x4;
        __syncthreads();
        float x[8], mx = NONE;
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            f32x4 v = *(const f32x4 *) (sp + (j * 64 + lane) * 4);
#pragma unroll
            for (int w = 1; w < 4; ++w) v += *(const f32x4 *) (sp + ((w * 2 + j) * 64 + lane) * 4);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = c * STEP + lg * 8 + j * 4 + e;
                x[j * 4 + e] = key >= first && key <= pos ? v[e] * c_sc : -INFINITY;
                mx = fmaxf(mx, x[j * 4 + e]);
            }
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
            const int dt = wave + i * DW;
            if (dt >= vt) continue;
            const uint32_t ch = (uint32_t) dt * 2u + ((lr & 3) >> 1);
            const s16x4 x0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4) (rows + vb0 + (ch ^ vs0) * 16u));
            const s16x4 x1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4) (rows + vb1 + (ch ^ vs1) * 16u));
            const s16x8 v = {x0[0], x0[1], x0[2], x0[3], x1[0], x1[1], x1[2], x1[3]};
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[i][e] *= corr;
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v), pv, acc[i], 0, 0, 0);
        }
        if (++stage == stages) stage = 0;
    }
    l += __shfl_xor(l, 16); l += __shfl_xor(l, 32);
    if (splits == 1) {
        const float f = 1.0f / l;
        uint16_t * o = (uint16_t *) a.out + (size_t) t * a.ldo + (size_t) (h0 + lr) * a.kvp + lg * 4;
        if (lr < nh)
#pragma unroll
            for (int i = 0; i < VT; ++i) {
                const int dt = wave + i * DW;
                if (dt < vt) *(PM_G u32x2 *) (o + dt * 16) = u32x2{(uint32_t) f2bf(acc[i][0] * f) | (uint32_t) f2bf(acc[i][1] * f) << 16, (uint32_t) f2bf(acc[i][2] * f) | (uint32_t) f2bf(acc[i][3] * f) << 16};
            }
        return;
    }
    const size_t slot = ((size_t) blockIdx.x * gridDim.y + blockIdx.y) * splits + s;
    if (lr < nh) {
        float * r = a.part + (slot * 16 + lr) * a.kvp + lg * 4;
#pragma unroll
        for (int i = 0; i < VT; ++i) {
            const int dt = wave + i * DW;
            if (dt < vt) *(PM_G f32x4 *) (r + dt * 16) = acc[i];
        }
        if (wave == 0 && lg == 0) *(PM_G u32x2 *) (ml + (slot * 16 + lr) * 2) = u32x2{__builtin_bit_cast(uint32_t, m), __builtin_bit_cast(uint32_t, l)};
    }
}
// split sums of one (token, head) -> its weighted latent
__global__ __launch_bounds__(256) void latent_merge_kernel(pm_latent_layer a, const float * ml, int splits) {
    __shared__ float share[64];
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const size_t slot = ((size_t) t * ((a.H + 15) / 16) + h / 16) * splits;
    if (threadIdx.x < 64) {
        const float * q = ml + ((slot + (lane < splits ? lane : 0)) * 16 + h % 16) * 2;
        const float m = lane < splits ? ld_g(q) : NONE, l = lane < splits ? ld_g(q + 1) : 0.0f, f = __builtin_amdgcn_exp2f(m - wave_max(m));
        share[lane] = f / wave_sum(l * f);
    }
    __syncthreads();
    for (int d = threadIdx.x; d < a.kvp; d += 256) {
        const float * r = a.part + (slot * 16 + h % 16) * a.kvp + d;
        float y = 0.0f;
        for (int i0 = 0; i0 < splits; i0 += 8) {
            float v[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) v[i] = ld_g(r + (size_t) (i0 + i < splits ? i0 + i : 0) * 16 * a.kvp);
#pragma unroll
            for (int i = 0; i < 8; ++i) y = fmaf(v[i], i0 + i < splits ? share[i0 + i] : 0.0f, y);
        }
        ((uint16_t *) a.out)[(size_t) t * a.ldo + (size_t) h * a.kvp + d] = f2bf(y);
    }
}

constexpr size_t LDS_MAX = 150 * 1024, SCORES = 8192;
int stages_for(int ld) {
    const size_t one = (size_t) ld * 2 * STEP;
    int n = (int) ((LDS_MAX - SCORES) / one);
    return n > 8 ? 8 : n;
}
int splits_for(int n, int H, int max_keys) {
    const int HT = (H + 15) / 16, most = (max_keys + 63) / 64, want = (256 + n * HT - 1) / (n * HT), s = want < most ? want : most;
    return s < 1 ? 1 : s > 64 ? 64 : s;
}

} // namespace

void pm_launch_latent_prepare(const pm_latent_layer & a, const pm_batch_dev & b, int T, hipStream_t st) {
    if (a.type == PM_BF16) hipLaunchKernelGGL(prepare_kernel<uint16_t>, dim3(T), dim3(256), 0, st, a, b); else hipLaunchKernelGGL(prepare_kernel<float>, dim3(T), dim3(256), 0, st, a, b);
}
void pm_launch_latent_rotate(const pm_latent_layer & a, int T, hipStream_t st) {
    if (a.type == PM_BF16) hipLaunchKernelGGL(rotate_kernel<uint16_t>, dim3(T), dim3(256), 0, st, a); else hipLaunchKernelGGL(rotate_kernel<float>, dim3(T), dim3(256), 0, st, a);
}
void pm_launch_latent_spread(const pm_latent_expand & x, hipStream_t st) { hipLaunchKernelGGL(spread_kernel, dim3(x.n_pages, x.H), dim3(256), 0, st, x); }
void pm_launch_latent_plain(const pm_latent_layer & a, const pm_batch_dev & b, int n, hipStream_t st) {
    const size_t lds = (size_t) (a.ld + 4 * (64 + a.kvp)) * 4;
    auto go = [&](auto kern) { pm_allow_big_lds((const void *) kern, lds); hipLaunchKernelGGL(kern, dim3(n, a.H), dim3(256), lds, st, a, b); };
    if (a.type == PM_BF16) go(plain_kernel<uint16_t>); else go(plain_kernel<float>);
}
bool pm_latent_decode_ok(int kvp, int ld) { return kvp % 64 == 0 && ld % 64 == 0 && ld >= kvp && kvp <= 1024 && ld <= 128 * ((kvp <= 128 ? 1 : kvp <= 256 ? 2 : kvp <= 512 ? 4 : 8) + 2) && stages_for(ld) >= 2; }
size_t pm_latent_part_floats(int n_tokens, int H, int kvp) { return ((size_t) 512 + 2 * (size_t) n_tokens * ((H + 15) / 16)) * 16 * (kvp + 2); }
int pm_launch_latent_decode(const pm_latent_layer & a, const pm_batch_dev & b, int n, int fused, int max_keys, pm_split_merge * merge, hipStream_t st) {
    if (a.type != PM_BF16 || !pm_latent_decode_ok(a.kvp, a.ld) || n < 1) return PM355_E_UNSUPPORTED;
    int splits = splits_for(n, a.H, max_keys);
    if (!a.part || pm_latent_part_floats(n, a.H, a.kvp) > a.part_floats) splits = 1;
    const int stages = stages_for(a.ld), HT = (a.H + 15) / 16;
    float * ml = a.part + (size_t) n * HT * splits * 16 * a.kvp;
    const size_t lds = (size_t) stages * a.ld * 2 * STEP + SCORES;
    auto go = [&](auto kern) { pm_allow_big_lds((const void *) kern, lds); hipLaunchKernelGGL(kern, dim3(n, HT, splits), dim3(DW * 64), lds, st, a, b, fused, splits, stages, ml); };
    if (a.kvp <= 128) go(latent_decode_kernel<1>); else if (a.kvp <= 256) go(latent_decode_kernel<2>); else if (a.kvp <= 512) go(latent_decode_kernel<4>); else go(latent_decode_kernel<8>);
    if (merge) *merge = pm_split_merge{a.part, ml, splits, a.H};
    else if (splits > 1) hipLaunchKernelGGL(latent_merge_kernel, dim3(n, a.H), dim3(256), 0, st, a, ml, splits);
    return 0;
}
