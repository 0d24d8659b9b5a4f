// dense_ops.hip — what surrounds the matrix products of a layer-described model: weight conversion, embeddings, norms (f32), rotation tables, greedy tokens.
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"

namespace {

__global__ void convert_kernel(int src_type, const void * src, int type, void * dst, int K, long n, int Kp, int group, int gstride, int transpose) {
    for (long i = (long) blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long) gridDim.x * blockDim.x) {
        const long r = i / K, k = i % K, g = group ? r / group : 0, in = group ? r - g * group : r;
        st_type(dst, transpose ? (size_t) (g * gstride + k) * Kp + in : (size_t) (g * gstride + in) * Kp + k, type, ld_any(src, i, src_type));
    }
}
__global__ void ssm_decay_kernel(float * a, long n) {
    for (long i = (long) blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long) gridDim.x * blockDim.x) a[i] = -expf(a[i]) * 1.4426950408889634f;
}

__device__ __forceinline__ uint32_t hash32(uint64_t x) {
    x ^= x >> 33; x *= 0xff51afd7ed558ccdULL; x ^= x >> 33; x *= 0xc4ceb9fe1a85ec53ULL; x ^= x >> 33;
    return (uint32_t) x;
}
__global__ void fill_kernel(int type, void * dst, int K, long n, int Kp, uint64_t seed, float mean, float amp) {
    for (long i = (long) blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long) gridDim.x * blockDim.x)
        st_type(dst, (size_t) (i / K) * Kp + i % K, type, mean + amp * ((float) (hash32(seed * 0x9E3779B97F4A7C15ULL + (uint64_t) i) & 0xFFFFFF) / 8388608.0f - 1.0f));
}

__device__ __forceinline__ float block_sum(float v, float * red) {
    v = wave_sum(v);
    const int wave = threadIdx.x >> 6, n = blockDim.x >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[wave] = v;
    __syncthreads();
    float s = 0.0f;
    for (int i = 0; i < n; ++i) s += red[i];
    return s;
}

// eight consecutive values from a 16-byte aligned row
__device__ __forceinline__ void ld8(const void * p, size_t i, int type, float * v) {
    if (type == PM_BF16) {
        const u32x4 r = *(const PM_G u32x4 *) ((const uint16_t *) p + i);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = bf2f((uint16_t) (r[e >> 1] >> (e & 1) * 16));
    } else {
        const f32x4 a = *(const PM_G f32x4 *) ((const float *) p + i), b = *(const PM_G f32x4 *) ((const float *) p + i + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) { v[e] = a[e]; v[4 + e] = b[e]; }
    }
}
__device__ __forceinline__ void st8(void * p, size_t i, int type, const float * v) {
    if (type == PM_BF16) {
        u32x4 r;
#pragma unroll
        for (int e = 0; e < 4; ++e) r[e] = (uint32_t) f2bf(v[2 * e]) | (uint32_t) f2bf(v[2 * e + 1]) << 16;
        *(PM_G u32x4 *) ((uint16_t *) p + i) = r;
    } else {
        *(PM_G f32x4 *) ((float *) p + i) = f32x4{v[0], v[1], v[2], v[3]};
        *(PM_G f32x4 *) ((float *) p + i + 4) = f32x4{v[4], v[5], v[6], v[7]};
    }
}
// one token per workgroup, the row in registers (8 x EMBED_ROUNDS values per thread); the first workgroups bring page tables, previous tokens and counters up to date (their
// readers are later launches; a portion's previous token is read and replaced by the workgroup of its first token)
constexpr int EMBED_ROUNDS = 4;
__global__ __launch_bounds__(1024) void embed_kernel(pm_embed_args a, pm_batch_dev b) {
    __shared__ float red[16];
    const int t = blockIdx.x;
    if (t == 0) {
        for (int i = threadIdx.x; i < b.n_upd[0]; i += blockDim.x) b.table[b.upd[2 * i]] = b.upd[2 * i + 1];
        for (int i = threadIdx.x; i < a.n_clear; i += blockDim.x) a.clear[i] = 0;
    }
    auto token = [&](int r) { const int k = b.tok[r]; return k < 0 ? b.last[b.seq[r]] : k; };
    const int tok = token(t);
    int64_t row = -1;
    if (a.bigram) {
        const int i = b.idx[t], before = b.pos[t] == 0 ? -1 : i ? token(t - 1) : b.prev[b.seq[t]];
        row = before < 0 ? a.buckets : (before * a.mul_prev + tok * a.mul_cur) % a.buckets;
        __syncthreads();                                   // (every wave has read prev)
        if (i == 0 && threadIdx.x == 0) b.prev[b.seq[t]] = token(t + b.left[t]);
    }
    float v[EMBED_ROUNDS][8], s = 0.0f;
#pragma unroll
    for (int i = 0; i < EMBED_ROUNDS; ++i) {
        const int c = (i * (int) blockDim.x + (int) threadIdx.x) * 8;
        if (c >= a.Kp) continue;
        ld8(a.embed, (size_t) tok * a.Kp + c, a.type, v[i]);
        if (row >= 0) {
            float g[8];
            ld8(a.bigram, (size_t) row * a.Kp + c, a.type, g);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[i][e] += g[e];
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf(v[i][e], v[i][e], s);                       // (padding columns are zero)
    }
    const float rs = a.out && a.w2 ? 1.0f / sqrtf(block_sum(s, red) / (float) a.width + a.eps) : 1.0f;
#pragma unroll
    for (int i = 0; i < EMBED_ROUNDS; ++i) {
        const int c = (i * (int) blockDim.x + (int) threadIdx.x) * 8;
        if (c >= a.Kp) continue;
        st8(a.x, (size_t) t * a.Kp + c, PM_F32, v[i]);
        if (!a.out) continue;
        if (a.w2) {
            float w[8];
            ld8(a.w2, c, PM_F32, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[i][e] *= rs * w[e];
        }
        st8(a.out, (size_t) t * a.Kp + c, a.type, v[i]);
    }
}
__global__ void rope_table_kernel(const int32_t * pos, float base, int dims, float * cs) {
    const int half = dims / 2;
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
        double sn, cn;                                     // (once per token and step: far positions keep the angle's low bits)
        sincos((double) pos[blockIdx.x] * pow((double) base, -2.0 * i / dims), &sn, &cn);
        float * o = cs + ((size_t) blockIdx.x * half + i) * 2;
        o[0] = (float) cn; o[1] = (float) sn;
    }
}

// one row per workgroup. RES: x[row] += norm(y[row]) and out = the sum (or its RMS norm with weight w2) in T; else out[row] = norm(x[rows[row]]) in T. VP > 0: the row and
// everything that joins it are requested at once, VP values per lane; 0: any width, row in LDS
template <bool RES, int NTH, int VP> __global__ __launch_bounds__(NTH) void norm_kernel(int type, pm_norm_args q, float * x, const void * y, int ldx, int ldy, const int32_t * rows, void * out,
                                                                                       int ldo) {
    extern __shared__ __attribute__((aligned(16))) float row[];
    __shared__ float red[NTH / 64];
    constexpr int N = VP ? VP : 1;
    const int r = blockIdx.x, width = q.width;
    float * xr = x + (size_t) (!RES && rows ? rows[r] : r) * ldx;
    auto value = [&](int c) __attribute__((always_inline)) -> float {        // what is normed
        if (!RES) return ld_g(xr + c);
        if (!q.parts) return q.y_type == PM_F32 ? ld_g((const float *) y + (size_t) r * ldy + c) : ld_any(y, (size_t) r * ldy + c, q.y_type);
        float s = 0.0f;
        for (int k = 0; k < q.parts; ++k) s += ld_any(y, ((size_t) r * q.parts + k) * ldy + c, q.y_type);
        return s;
    };
    float v[N], xv[N], wv[N], bv[N], w2v[N], s = 0.0f;
    if (VP) {
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const int c = i * NTH + threadIdx.x, cc = c < width ? c : width - 1;
            v[i] = value(cc); wv[i] = ld_g(q.w + cc); bv[i] = q.b ? ld_g(q.b + cc) : 0.0f;
            xv[i] = RES ? ld_g(xr + cc) : 0.0f;
            w2v[i] = RES && q.w2 ? ld_g(q.w2 + cc) : 1.0f;
        }
#pragma unroll
        for (int i = 0; i < N; ++i) s += i * NTH + (int) threadIdx.x < width ? v[i] : 0.0f;
    } else for (int c = threadIdx.x; c < width; c += NTH) { const float f = value(c); row[c] = f; s += f; }
    const float mean = q.rms ? 0.0f : block_sum(s, red) / (float) width;
    float s2 = 0.0f;
    if (VP) {
#pragma unroll
        for (int i = 0; i < N; ++i) { const float d = i * NTH + (int) threadIdx.x < width ? v[i] - mean : 0.0f; s2 = fmaf(d, d, s2); }
    } else for (int c = threadIdx.x; c < width; c += NTH) { const float d = row[c] - mean; s2 = fmaf(d, d, s2); }
    const float rs = 1.0f / sqrtf(block_sum(s2, red) / (float) width + q.eps);
    float s3 = 0.0f;
    auto sum = [&](int c, float f, float xo, float wo, float bo) __attribute__((always_inline)) -> float {
        float o = (f - mean) * rs * wo + bo;
        if (RES) { o = xo + o; xr[c] = o; }
        s3 = fmaf(o, o, s3);
        return o;
    };
    if (VP) {
#pragma unroll
        for (int i = 0; i < N; ++i) { const int c = i * NTH + threadIdx.x; if (c < width) v[i] = sum(c, v[i], xv[i], wv[i], bv[i]); }
    } else for (int c = threadIdx.x; c < width; c += NTH) row[c] = sum(c, row[c], RES ? xr[c] : 0.0f, q.w[c], q.b ? q.b[c] : 0.0f);
    if (!out) return;
    const float r2 = RES && q.w2 ? 1.0f / sqrtf(block_sum(s3, red) / (float) width + q.eps) : 1.0f;
    if (VP) {
#pragma unroll
        for (int i = 0; i < N; ++i) { const int c = i * NTH + threadIdx.x; if (c < width) st_type(out, (size_t) r * ldo + c, type, v[i] * (r2 * w2v[i])); }
    } else for (int c = threadIdx.x; c < width; c += NTH) st_type(out, (size_t) r * ldo + c, type, row[c] * (r2 * (RES && q.w2 ? q.w2[c] : 1.0f)));
}

// x[row] += norm(y[row]), out = the sum or its RMS norm with weight w2, four consecutive columns per thread and round: rows that are padded to multiples of 4
template <int NTH, int VP> __global__ __launch_bounds__(NTH) void norm4_kernel(int type, pm_norm_args q, float * x, const void * y, int ldx, int ldy, void * out, int ldo) {
    __shared__ float red[NTH / 64];
    const int r = blockIdx.x, width = q.width;
    float * xr = x + (size_t) r * ldx;
    const int parts = q.parts ? q.parts : 1;
    f32x4 v[VP], xv[VP];
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < VP; ++i) {
        const int c = (i * NTH + threadIdx.x) * 4;
        v[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        xv[i] = v[i];
        if (c >= width) continue;
        xv[i] = *(const PM_G f32x4 *) (xr + c);
        for (int k = 0; k < parts; ++k) {
            const size_t at = ((size_t) r * parts + k) * ldy + c;
            if (q.y_type == PM_F32) v[i] += *(const PM_G f32x4 *) ((const float *) y + at);
            else {
                const u32x2 b = *(const PM_G u32x2 *) ((const uint16_t *) y + at);
                v[i] += f32x4{bf2f((uint16_t) b[0]), bf2f((uint16_t) (b[0] >> 16)), bf2f((uint16_t) b[1]), bf2f((uint16_t) (b[1] >> 16))};
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) { if (c + e >= width) v[i][e] = 0.0f; s += v[i][e]; }
    }
    const float mean = q.rms ? 0.0f : block_sum(s, red) / (float) width;
    float s2 = 0.0f;
#pragma unroll
    for (int i = 0; i < VP; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) { const float d = (i * NTH + (int) threadIdx.x) * 4 + e < width ? v[i][e] - mean : 0.0f; s2 = fmaf(d, d, s2); }
    const float rs = 1.0f / sqrtf(block_sum(s2, red) / (float) width + q.eps);
    float s3 = 0.0f;
#pragma unroll
    for (int i = 0; i < VP; ++i) {
        const int c = (i * NTH + threadIdx.x) * 4;
        if (c >= width) continue;
        const f32x4 w = *(const PM_G f32x4 *) (q.w + c);
        f32x4 bias = {0.0f, 0.0f, 0.0f, 0.0f};
        if (q.b) bias = *(const PM_G f32x4 *) (q.b + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) { const float o = xv[i][e] + ((v[i][e] - mean) * rs * w[e] + bias[e]); v[i][e] = c + e < width ? o : 0.0f; s3 = fmaf(v[i][e], v[i][e], s3); }
        *(PM_G f32x4 *) (xr + c) = v[i];
    }
    const float r2 = q.w2 ? 1.0f / sqrtf(block_sum(s3, red) / (float) width + q.eps) : 1.0f;
#pragma unroll
    for (int i = 0; i < VP; ++i) {
        const int c = (i * NTH + threadIdx.x) * 4;
        if (c >= width) continue;
        f32x4 o = v[i];
        if (q.w2) {
            const f32x4 w2 = *(const PM_G f32x4 *) (q.w2 + c);
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] *= r2 * w2[e];
        }
        if (type == PM_F32) *(PM_G f32x4 *) ((float *) out + (size_t) r * ldo + c) = o;
        else *(PM_G u32x2 *) ((uint16_t *) out + (size_t) r * ldo + c) = u32x2{(uint32_t) f2bf(o[0]) | (uint32_t) f2bf(o[1]) << 16, (uint32_t) f2bf(o[2]) | (uint32_t) f2bf(o[3]) << 16};
    }
}

// index of the first maximum of every row (src/llama-sampling.cpp:390-397), also kept per sequence for the next step
__global__ __launch_bounds__(1024) void argmax_rows_kernel(const float * x, int n, int32_t * out, const int32_t * seq_of_row, int32_t * last) {
    __shared__ float bv[16]; __shared__ int bi[16];
    const float * r = x + (size_t) blockIdx.x * n;
    float v = -INFINITY; int idx = 0x7fffffff;
    for (int i = threadIdx.x; i < n; i += 1024) { const float f = r[i]; if (f > v || (f == v && i < idx)) { v = f; idx = i; } }
    for (int o = 32; o; o >>= 1) {
        const float v2 = __shfl_xor(v, o); const int i2 = __shfl_xor(idx, o);
        if (v2 > v || (v2 == v && i2 < idx)) { v = v2; idx = i2; }
    }
    if ((threadIdx.x & 63) == 0) { bv[threadIdx.x >> 6] = v; bi[threadIdx.x >> 6] = idx; }
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w = 1; w < 16; ++w) if (bv[w] > v || (bv[w] == v && bi[w] < idx)) { v = bv[w]; idx = bi[w]; }
        if (idx >= n) idx = 0;                             // (a row of NaNs)
        if (out) out[blockIdx.x] = idx;
        if (last && seq_of_row[blockIdx.x] >= 0) last[seq_of_row[blockIdx.x]] = idx;       // (the last wanted row of an entry)
    }
}

} // namespace

void pm_launch_dense_convert(int src_type, const void * src, int type, void * dst, int K, int64_t N, int Kp, hipStream_t st, int group, int gstride, int transpose) {
    const long n = (long) N * K, g = (n + 255) / 256;
    hipLaunchKernelGGL(convert_kernel, dim3((unsigned) (g < 65536 ? g : 65536)), dim3(256), 0, st, src_type, src, type, dst, K, n, Kp, group, gstride, transpose);
}
void pm_launch_ssm_decay(float * a, int64_t n, hipStream_t st) {
    const long g = (n + 255) / 256;
    hipLaunchKernelGGL(ssm_decay_kernel, dim3((unsigned) (g < 65536 ? g : 65536)), dim3(256), 0, st, a, (long) n);
}
void pm_launch_dense_fill(int type, void * dst, int K, int64_t N, int Kp, uint64_t seed, float mean, float amp, hipStream_t st) {
    const long n = (long) N * K, g = (n + 255) / 256;
    hipLaunchKernelGGL(fill_kernel, dim3((unsigned) (g < 65536 ? g : 65536)), dim3(256), 0, st, type, dst, K, n, Kp, seed, mean, amp);
}
int pm_launch_stack_embed(const pm_embed_args & a, const pm_batch_dev & b, int T, hipStream_t st) {
    const int threads = a.Kp / 8 >= 1024 ? 1024 : (a.Kp / 8 + 63) / 64 * 64;
    if (a.Kp % 64 || a.Kp > threads * 8 * EMBED_ROUNDS) return PM355_E_SHAPE;
    hipLaunchKernelGGL(embed_kernel, dim3(T), dim3(threads), 0, st, a, b);
    return 0;
}
void pm_launch_rope_table(const int32_t * pos, int T, float base, int dims, float * cs, hipStream_t st) {
    hipLaunchKernelGGL(rope_table_kernel, dim3(T), dim3(64), 0, st, pos, base, dims, cs);
}
template <bool RES> static void launch_norm(int type, const pm_norm_args & q, float * x, const void * y, int ldx, int ldy, const int32_t * rows, int n_rows, void * out, int ldo,
                                            hipStream_t st) {
    auto go = [&](auto kern, int threads, size_t lds) {
        pm_allow_big_lds((const void *) kern, lds);
        hipLaunchKernelGGL(kern, dim3(n_rows), dim3(threads), lds, st, type, q, x, y, ldx, ldy, rows, out, ldo);
    };
    if (q.width <= 1024) go(norm_kernel<RES, 256, 4>, 256, 0);
    else if (q.width <= 4096 && n_rows > 512) go(norm_kernel<RES, 256, 16>, 256, 0);
    else if (q.width <= 4096) go(norm_kernel<RES, 1024, 4>, 1024, 0);
    else if (q.width <= 8192) go(norm_kernel<RES, 1024, 8>, 1024, 0);
    else go(norm_kernel<RES, 1024, 0>, 1024, (size_t) q.width * 4);
}
void pm_launch_add_norm(int type, const pm_norm_args & q, float * x, const void * y, int ldx, int ldy, int n_rows, void * out, int ldo, hipStream_t st) {
    if (q.padded && out && n_rows > 16 && q.width <= 8192 && ldx % 4 == 0 && ldy % 4 == 0 && ldo % 4 == 0) {
        auto go = [&](auto kern, int threads) { hipLaunchKernelGGL(kern, dim3(n_rows), dim3(threads), 0, st, type, q, x, y, ldx, ldy, out, ldo); };
        if (q.width <= 1024) go(norm4_kernel<256, 1>, 256);
        else if (q.width <= 2048) go(norm4_kernel<256, 2>, 256);
        else if (q.width <= 4096) go(norm4_kernel<256, 4>, 256);
        else go(norm4_kernel<512, 4>, 512);
        return;
    }
    launch_norm<true>(type, q, x, y, ldx, ldy, nullptr, n_rows, out, ldo, st);
}
void pm_launch_norm_rows(int type, const pm_norm_args & q, const float * x, int ldx, const int32_t * rows, int n_rows, void * out, int ldo, hipStream_t st) {
    launch_norm<false>(type, q, (float *) x, nullptr, ldx, 0, rows, n_rows, out, ldo, st);
}
void pm_launch_argmax_rows(const float * logits, int n, int n_rows, int32_t * out, const int32_t * seq_of_row, int32_t * last, hipStream_t st) {
    hipLaunchKernelGGL(argmax_rows_kernel, dim3(n_rows), dim3(1024), 0, st, logits, n, out, seq_of_row, last);
}
