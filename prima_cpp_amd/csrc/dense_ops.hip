// dense_ops.hip — what surrounds the matrix products of a layer-described model: weight conversion, embedding, layer norms (f32), greedy tokens.
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"

namespace {

__global__ void convert_kernel(int src_type, const void * src, int type, void * dst, int K, long n, int Kp) {
    for (long i = (long) blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long) gridDim.x * blockDim.x) st_type(dst, (size_t) (i / K) * Kp + i % K, type, ld_any(src, i, src_type));
}

__device__ __forceinline__ uint32_t hash32(uint64_t x) {
    x ^= x >> 33; x *= 0xff51afd7ed558ccdULL; x ^= x >> 33; x *= 0xc4ceb9fe1a85ec53ULL; x ^= x >> 33;
    return (uint32_t) x;
}
__global__ void fill_kernel(int type, void * dst, int K, long n, int Kp, uint64_t seed, float mean, float amp) {
    for (long i = (long) blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long) gridDim.x * blockDim.x)
        st_type(dst, (size_t) (i / K) * Kp + i % K, type, mean + amp * ((float) (hash32(seed * 0x9E3779B97F4A7C15ULL + (uint64_t) i) & 0xFFFFFF) / 8388608.0f - 1.0f));
}

// x[t] = embedding row (f32), xb[t] = the same in T; workgroup (0, 0) brings the device page tables up to date (their readers are later launches)
__global__ void embed_kernel(int type, const void * embed, int Kp, int width, pm_batch_dev b, float * x, void * xb) {
    const int t = blockIdx.x;
    if (t == 0) for (int i = threadIdx.x; i < b.n_upd[0]; i += blockDim.x) b.table[b.upd[2 * i]] = b.upd[2 * i + 1];
    int tok = b.tok[t];
    if (tok < 0) tok = b.last[b.seq[t]];
    for (int c = threadIdx.x; c < Kp; c += blockDim.x) {
        const float v = c < width ? ld_any(embed, (size_t) tok * Kp + c, type) : 0.0f;
        x[(size_t) t * Kp + c] = v;
        if (xb) st_type(xb, (size_t) t * Kp + c, type, v);
    }
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

// one row per workgroup. RES: x[row] += layer_norm(y[row]) and out = the sum in T; else out[row] = layer_norm(x[rows[row]]) in T. VP > 0: the row and everything that joins
// it are requested at once, VP values per lane; 0: any width, row in LDS
template <bool RES, int NTH, int VP> __global__ __launch_bounds__(NTH) void layer_norm_kernel(int type, float * x, const float * y, int ldx, int ldy, const int32_t * rows, const float * w,
                                                                                             const float * b, float eps, int width, void * out, int ldo) {
    extern __shared__ __attribute__((aligned(16))) float row[];
    __shared__ float red[NTH / 64];
    constexpr int N = VP ? VP : 1;
    const int r = blockIdx.x;
    const float * src = RES ? y + (size_t) r * ldy : x + (size_t) (rows ? rows[r] : r) * ldx;
    float v[N], xv[N], wv[N], bv[N], s = 0.0f;
    if (VP) {
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const int c = i * NTH + threadIdx.x, cc = c < width ? c : width - 1;
            v[i] = ld_g(src + cc); wv[i] = ld_g(w + cc); bv[i] = ld_g(b + cc);
            xv[i] = RES ? ld_g(x + (size_t) r * ldx + cc) : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < N; ++i) s += i * NTH + (int) threadIdx.x < width ? v[i] : 0.0f;
    } else for (int c = threadIdx.x; c < width; c += NTH) { const float f = src[c]; row[c] = f; s += f; }
    const float mean = block_sum(s, red) / (float) width;
    float s2 = 0.0f;
    if (VP) {
#pragma unroll
        for (int i = 0; i < N; ++i) { const float d = i * NTH + (int) threadIdx.x < width ? v[i] - mean : 0.0f; s2 = fmaf(d, d, s2); }
    } else for (int c = threadIdx.x; c < width; c += NTH) { const float d = row[c] - mean; s2 = fmaf(d, d, s2); }
    const float rs = 1.0f / sqrtf(block_sum(s2, red) / (float) width + eps);
    auto put = [&](int c, float f, float xo, float wo, float bo) __attribute__((always_inline)) {
        float o = (f - mean) * rs * wo + bo;
        if (RES) { o = xo + o; x[(size_t) r * ldx + c] = o; }
        if (out) st_type(out, (size_t) r * ldo + c, type, o);
    };
    if (VP) {
#pragma unroll
        for (int i = 0; i < N; ++i) { const int c = i * NTH + threadIdx.x; if (c < width) put(c, v[i], xv[i], wv[i], bv[i]); }
    } else for (int c = threadIdx.x; c < width; c += NTH) put(c, row[c], RES ? x[(size_t) r * ldx + c] : 0.0f, w[c], b[c]);
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

void pm_launch_dense_convert(int src_type, const void * src, int type, void * dst, int K, int64_t N, int Kp, hipStream_t st) {
    const long n = (long) N * K, g = (n + 255) / 256;
    hipLaunchKernelGGL(convert_kernel, dim3((unsigned) (g < 65536 ? g : 65536)), dim3(256), 0, st, src_type, src, type, dst, K, n, Kp);
}
void pm_launch_dense_fill(int type, void * dst, int K, int64_t N, int Kp, uint64_t seed, float mean, float amp, hipStream_t st) {
    const long n = (long) N * K, g = (n + 255) / 256;
    hipLaunchKernelGGL(fill_kernel, dim3((unsigned) (g < 65536 ? g : 65536)), dim3(256), 0, st, type, dst, K, n, Kp, seed, mean, amp);
}
void pm_launch_stack_embed(int type, const void * embed, int Kp, int width, const pm_batch_dev & b, int T, float * x, void * xb, hipStream_t st) {
    hipLaunchKernelGGL(embed_kernel, dim3(T), dim3(256), 0, st, type, embed, Kp, width, b, x, xb);
}
template <bool RES> static void launch_norm(int type, float * x, const float * y, int ldx, int ldy, const int32_t * rows, const float * w, const float * b, float eps, int width, int n_rows,
                                            void * out, int ldo, hipStream_t st) {
    auto go = [&](auto kern, int threads, size_t lds) {
        pm_allow_big_lds((const void *) kern, lds);
        hipLaunchKernelGGL(kern, dim3(n_rows), dim3(threads), lds, st, type, x, y, ldx, ldy, rows, w, b, eps, width, out, ldo);
    };
    if (width <= 1024) go(layer_norm_kernel<RES, 256, 4>, 256, 0);
    else if (width <= 4096 && n_rows > 512) go(layer_norm_kernel<RES, 256, 16>, 256, 0);
    else if (width <= 4096) go(layer_norm_kernel<RES, 1024, 4>, 1024, 0);
    else if (width <= 8192) go(layer_norm_kernel<RES, 1024, 8>, 1024, 0);
    else go(layer_norm_kernel<RES, 1024, 0>, 1024, (size_t) width * 4);
}
void pm_launch_add_layer_norm(int type, float * x, const float * y, int ldx, int ldy, const float * w, const float * b, float eps, int width, int n_rows, void * xb, hipStream_t st) {
    launch_norm<true>(type, x, y, ldx, ldy, nullptr, w, b, eps, width, n_rows, xb, ldx, st);
}
void pm_launch_layer_norm_rows(int type, const float * x, int ldx, const int32_t * rows, const float * w, const float * b, float eps, int width, int n_rows, void * out, int ldo,
                               hipStream_t st) {
    launch_norm<false>(type, (float *) x, nullptr, ldx, 0, rows, w, b, eps, width, n_rows, out, ldo, st);
}
void pm_launch_argmax_rows(const float * logits, int n, int n_rows, int32_t * out, const int32_t * seq_of_row, int32_t * last, hipStream_t st) {
    hipLaunchKernelGGL(argmax_rows_kernel, dim3(n_rows), dim3(1024), 0, st, logits, n, out, seq_of_row, last);
}
