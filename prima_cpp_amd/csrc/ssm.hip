// ssm.hip — selective scan layers: causal convolution + silu, the recurrence S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n with y_c = sum_n S[c, n] C_n + D_c x_c, and the
// gate silu(z). State, step sizes and decays are f32; a sequence's state lies in its slot and counts as zero at position 0, so that slots need no clearing.
//   conv    a thread per channel walks 16 tokens; the inputs in front of a portion come from the slot
//   step    decoded tokens: the step-size product, softplus, update, gate and the convolution's state in one launch; 4 states per lane, lanes of a channel add up by shuffles
//   scan    portions in chunks of up to 128 tokens: end states of all chunks but the last from zero, a pass over the chunks that turns them into start states, then every
//           chunk from its start state. Portions of one chunk take the last pass only
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "../../include/prima_mi355.h"

namespace {

constexpr int CONV_TOK = 16, TT = 16;                      // tokens a thread of the convolution walks through in prompts; tokens whose scan inputs lie in LDS at a time

// input `back` tokens before token t of the step, x half of the projections; place i in its portion, position pos
__device__ __forceinline__ float conv_input(const pm_ssm_layer & a, int t, int c, int back, int i, int pos, int seq) {
    if (pos < back) return 0.0f;
    if (i >= back) return ld_any(a.raw, (size_t) (t - back) * a.ldraw + c, a.raw_type);
    return a.cstate[((size_t) seq * (a.conv - 1) + a.conv - 1 + i - back) * a.innerp + c];
}
template <typename T, int TAPS> __global__ __launch_bounds__(256) void conv_kernel(pm_ssm_layer a, pm_batch_dev b, int n_tok, int per) {
    const int c = blockIdx.y * 256 + threadIdx.x, t0 = blockIdx.x * per;
    if (c >= a.innerp) return;
    const bool real = c < a.inner;
    const int taps = TAPS ? TAPS : a.conv;
    constexpr int N = TAPS ? TAPS : 1;
    float in[N], w[N];
    const float bias = real ? a.conv_b[c] : 0.0f;
    if (TAPS && real) {
#pragma unroll
        for (int j = 0; j < N; ++j) w[j] = a.conv_w[(size_t) c * taps + j];
    }
    for (int k = 0; k < per && t0 + k < n_tok; ++k) {
        const int t = t0 + k;
        float v = bias;
        if (real) {
            const int i = b.idx[t], pos = b.pos[t], seq = b.seq[t];
            if (TAPS) {                                    // in[j]: the input j tokens back
                if (k == 0 || i == 0) {
#pragma unroll
                    for (int j = 1; j < N; ++j) in[j] = conv_input(a, t, c, j, i, pos, seq);
                } else {
#pragma unroll
                    for (int j = N - 1; j > 0; --j) in[j] = in[j - 1];
                }
                in[0] = ld_any(a.raw, (size_t) t * a.ldraw + c, a.raw_type);
#pragma unroll
                for (int j = N - 1; j >= 0; --j) v = fmaf(in[j], w[N - 1 - j], v);
            } else for (int j = taps - 1; j >= 0; --j) v = fmaf(conv_input(a, t, c, j, i, pos, seq), a.conv_w[(size_t) c * taps + taps - 1 - j], v);
        }
        ((T *) a.xc)[(size_t) t * a.innerp + c] = from_f<T>(real ? silu32(v) : 0.0f);
    }
}

// the convolution's state behind a portion of n tokens that starts at row `row`: the last conv - 1 inputs (one thread per channel: old entries are read before they go)
__device__ __forceinline__ void keep_conv_state(const pm_ssm_layer & a, int row, int n, int seq, int c) {
    float * s = a.cstate + (size_t) seq * (a.conv - 1) * a.innerp + c;
    for (int k = 0; k < a.conv - 1; ++k) {
        const int at = n - (a.conv - 1) + k;               // token of the portion, or an older input
        s[(size_t) k * a.innerp] = at >= 0 ? ld_any(a.raw, (size_t) (row + at) * a.ldraw + c, a.raw_type) : s[(size_t) (k + n) * a.innerp];
    }
}

template <int NG> struct States { f32x4 s[NG], a[NG]; };
__device__ __forceinline__ f32x4 decay4(f32x4 a, float dt) {
    return f32x4{__builtin_amdgcn_exp2f(a[0] * dt), __builtin_amdgcn_exp2f(a[1] * dt), __builtin_amdgcn_exp2f(a[2] * dt), __builtin_amdgcn_exp2f(a[3] * dt)};
}
// sum over groups of n lanes (a power of two, the same in every lane): data-parallel moves inside a row of 16 lanes
template <int CTRL> __device__ __forceinline__ float moved(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}
__device__ __forceinline__ float lanes_sum(float v, int n) {
    if (n > 1) v += moved<0xB1>(v);                        // quad_perm 1 0 3 2
    if (n > 2) v += moved<0x4E>(v);                        // quad_perm 2 3 0 1
    if (n > 4) v += moved<0x141>(v);                       // row_half_mirror: the other quad
    if (n > 8) v += moved<0x140>(v);                       // row_mirror: the other half row
    if (n > 16) v += __shfl_xor(v, 16);
    if (n > 32) v += __shfl_xor(v, 32);
    return v;
}

template <typename T, int NG> __global__ __launch_bounds__(256) void step_kernel(pm_ssm_layer a, pm_batch_dev b, int lpc) {
    const int t = blockIdx.x, sub = threadIdx.x % lpc, c = blockIdx.y * (256 / lpc) + threadIdx.x / lpc, cc = c < a.inner ? c : a.inner - 1;
    const int pos = b.pos[t], seq = b.seq[t];
    const T * f = (const T *) a.f + (size_t) t * a.ldf;
    float * sp = a.S + ((size_t) seq * a.inner + cc) * a.sp + sub * 4;
    States<NG> st;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
        st.a[g] = *(const PM_G f32x4 *) (a.A2 + (size_t) cc * a.sp + sub * 4 + g * lpc * 4);
        st.s[g] = pos ? *(const PM_G f32x4 *) (sp + g * lpc * 4) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
    const float x = to_f<T>(((const T *) a.xc)[(size_t) t * a.innerp + cc]);
    // step size: the lanes of a channel share the product over dt_rank
    constexpr int EPL = 16 / sizeof(T);
    float d = 0.0f;
    for (int k = sub * EPL; k < a.dtp; k += lpc * EPL) {
        const u32x4 wv = *(const PM_G u32x4 *) ((const T *) a.w_dt + (size_t) cc * a.dtp + k), fv = *(const PM_G u32x4 *) (f + k);
#pragma unroll
        for (int e = 0; e < EPL; ++e) d = fmaf(to_f<T>(((const T *) &wv)[e]), to_f<T>(((const T *) &fv)[e]), d);
    }
    const float dt = softplus_f(lanes_sum(d, lpc) + a.dt_b[cc]), dx = dt * x;
    float y = 0.0f;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
        const f32x4 dec = decay4(st.a[g], dt);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = g * lpc * 4 + sub * 4 + e;
            const bool on = n < a.state;
            const float B = on ? to_f<T>(f[a.dtp + n]) : 0.0f, C = on ? to_f<T>(f[a.dtp + a.state + n]) : 0.0f;
            st.s[g][e] = fmaf(dec[e], st.s[g][e], dx * B);
            y = fmaf(st.s[g][e], C, y);
        }
    }
    y = lanes_sum(y, lpc);
    if (c >= a.inner) return;
#pragma unroll
    for (int g = 0; g < NG; ++g) *(PM_G f32x4 *) (sp + g * lpc * 4) = st.s[g];
    if (sub) return;
    const float z = ld_any(a.raw, (size_t) t * a.ldraw + a.inner + c, a.raw_type);
    ((T *) a.y)[(size_t) t * a.ldy + c] = from_f<T>((y + a.D[c] * x) * silu32(z));
    keep_conv_state(a, t, 1, seq, c);
}

// PHASE 0: end state from zero and the sum of step sizes (all chunks of a portion but the last). PHASE 1: outputs from the chunk's start state
template <typename T, int NG, int PHASE> __global__ __launch_bounds__(256) void scan_kernel(pm_ssm_layer a, const pm_scan_chunk * chunks, int lpc) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const pm_scan_chunk ch = chunks[blockIdx.x];
    const bool last = ch.j == ch.n_chunks - 1;
    if (PHASE == 0 && last) return;
    const int cpb = 256 / lpc, sub = threadIdx.x % lpc, cl = threadIdx.x / lpc, c0 = blockIdx.y * cpb, c = c0 + cl, cc = c < a.inner ? c : a.inner - 1;
    float2 * s_dd = (float2 *) sm;                         // (step size, step size * input)
    float * s_y = (float *) (s_dd + TT * cpb), * s_B = s_y + TT * cpb, * s_C = s_B + TT * a.sp;
    States<NG> st;
    const size_t at = (size_t) cc * a.sp + sub * 4;
    float * E = a.E + (size_t) (ch.e_base + ch.j) * a.inner * a.sp + at, * S = a.S + (size_t) ch.seq * a.inner * a.sp + at;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
        st.a[g] = *(const PM_G f32x4 *) (a.A2 + at + g * lpc * 4);
        st.s[g] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        if (PHASE == 1) {
            if (ch.n_chunks > 1) st.s[g] = *(const PM_G f32x4 *) (E + g * lpc * 4);
            else if (ch.pos) st.s[g] = *(const PM_G f32x4 *) (S + g * lpc * 4);
        }
    }
    float sum = 0.0f;
    for (int t0 = 0; t0 < ch.n; t0 += TT) {
        const int nt = ch.n - t0 < TT ? ch.n - t0 : TT;
        __syncthreads();
        for (int i = threadIdx.x; i < TT * cpb; i += 256) {       // (tokens past the end: steps of size 0 change nothing)
            const int t = i / cpb, k = c0 + i % cpb;
            const size_t r = (size_t) (ch.row + t0 + t);
            float dt = 0.0f, x = 0.0f;
            if (k < a.inner && t < nt) { dt = softplus_f(a.dt[r * a.innerp + k]); x = to_f<T>(((const T *) a.xc)[r * a.innerp + k]); }
            s_dd[i] = make_float2(dt, dt * x);
        }
        for (int i = threadIdx.x; i < TT * a.sp; i += 256) {
            const int t = i / a.sp, n = i % a.sp;
            const T * f = (const T *) a.f + (size_t) (ch.row + t0 + t) * a.ldf + a.dtp;
            const bool on = n < a.state && t < nt;
            s_B[i] = on ? to_f<T>(f[n]) : 0.0f;
            if (PHASE == 1) s_C[i] = on ? to_f<T>(f[a.state + n]) : 0.0f;
        }
        __syncthreads();
#pragma unroll 4
        for (int t = 0; t < TT; ++t) {
            const float2 dd = s_dd[t * cpb + cl];
            if (PHASE == 0) sum += dd.x;
            float y = 0.0f;
#pragma unroll
            for (int g = 0; g < NG; ++g) {
                const f32x4 B = *(const f32x4 *) (s_B + t * a.sp + sub * 4 + g * lpc * 4), dec = decay4(st.a[g], dd.x);
#pragma unroll
                for (int e = 0; e < 4; ++e) st.s[g][e] = fmaf(dec[e], st.s[g][e], dd.y * B[e]);
                if (PHASE == 1) {
                    const f32x4 C = *(const f32x4 *) (s_C + t * a.sp + sub * 4 + g * lpc * 4);
#pragma unroll
                    for (int e = 0; e < 4; ++e) y = fmaf(st.s[g][e], C[e], y);
                }
            }
            if (PHASE == 1) {
                y = lanes_sum(y, lpc);
                if (sub == 0) s_y[t * cpb + cl] = y;
            }
        }
        if (PHASE == 0) continue;
        __syncthreads();
        for (int i = threadIdx.x; i < nt * cpb; i += 256) {
            const int k = c0 + i % cpb;
            if (k >= a.inner) continue;
            const size_t r = (size_t) (ch.row + t0 + i / cpb);
            const float x = to_f<T>(((const T *) a.xc)[r * a.innerp + k]), z = ld_any(a.raw, r * a.ldraw + a.inner + k, a.raw_type);
            ((T *) a.y)[r * a.ldy + k] = from_f<T>((s_y[i] + a.D[k] * x) * silu32(z));
        }
    }
    if (c >= a.inner) return;
    float * o = PHASE == 0 ? E : S;
    if (PHASE == 0 || last)
#pragma unroll
        for (int g = 0; g < NG; ++g) *(PM_G f32x4 *) (o + g * lpc * 4) = st.s[g];
    if (sub) return;
    if (PHASE == 0) a.dtsum[(size_t) (ch.e_base + ch.j) * a.innerp + c] = sum;
    else if (last) keep_conv_state(a, ch.row - ch.j * 128, ch.n + ch.j * 128, ch.seq, c);
}

// end states of a portion's chunks -> their start states
__global__ __launch_bounds__(256) void scan_carry_kernel(pm_ssm_layer a, const pm_scan_chunk * chunks) {
    const pm_scan_chunk ch = chunks[blockIdx.x];
    if (ch.j || ch.n_chunks < 2) return;
    const size_t i = ((size_t) blockIdx.y * 256 + threadIdx.x) * 4, n = (size_t) a.inner * a.sp;
    if (i >= n) return;
    const int c = (int) (i / a.sp);
    const f32x4 A = *(const PM_G f32x4 *) (a.A2 + i);
    f32x4 s = {0.0f, 0.0f, 0.0f, 0.0f};
    if (ch.pos) s = *(const PM_G f32x4 *) (a.S + (size_t) ch.seq * n + i);
    float * E = a.E + (size_t) ch.e_base * n + i;
    const float * dts = a.dtsum + (size_t) ch.e_base * a.innerp + c;
    for (int j0 = 0; j0 < ch.n_chunks; j0 += 8) {          // eight chunks' loads at a time
        f32x4 e[8]; float d[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) if (j0 + j < ch.n_chunks - 1) { e[j] = *(const PM_G f32x4 *) (E + (size_t) (j0 + j) * n); d[j] = dts[(size_t) (j0 + j) * a.innerp]; }
#pragma unroll
        for (int j = 0; j < 8; ++j)
            if (j0 + j < ch.n_chunks) {
                *(PM_G f32x4 *) (E + (size_t) (j0 + j) * n) = s;
                if (j0 + j < ch.n_chunks - 1) {
                    const f32x4 dec = decay4(A, d[j]);
#pragma unroll
                    for (int k = 0; k < 4; ++k) s[k] = fmaf(dec[k], s[k], e[j][k]);
                }
            }
    }
}

int lanes(const pm_ssm_layer & a) { return a.sp >= 256 ? 64 : a.sp / 4; }
template <typename T> void conv(const pm_ssm_layer & a, const pm_batch_dev & b, int T_, hipStream_t st) {
    const int per = T_ <= 64 ? 1 : CONV_TOK;
    const dim3 grid((T_ + per - 1) / per, (a.innerp + 255) / 256);
    auto go = [&](auto kern) { hipLaunchKernelGGL(kern, grid, dim3(256), 0, st, a, b, T_, per); };
    if (a.conv == 4) go(conv_kernel<T, 4>);
    else if (a.conv == 3) go(conv_kernel<T, 3>);
    else if (a.conv == 2) go(conv_kernel<T, 2>);
    else go(conv_kernel<T, 0>);
}
template <typename T> void step(const pm_ssm_layer & a, const pm_batch_dev & b, int T_, hipStream_t st) {
    const int lpc = lanes(a), cpb = 256 / lpc;
    auto go = [&](auto kern) { hipLaunchKernelGGL(kern, dim3(T_, (a.inner + cpb - 1) / cpb), dim3(256), 0, st, a, b, lpc); };
    if (a.sp <= 256) go(step_kernel<T, 1>); else if (a.sp == 512) go(step_kernel<T, 2>); else go(step_kernel<T, 4>);
}
template <typename T, int PHASE> void scan_phase(const pm_ssm_layer & a, const pm_scan_chunk * chunks, int n, hipStream_t st) {
    const int lpc = lanes(a), cpb = 256 / lpc;
    const size_t lds = (size_t) TT * (3 * cpb + 2 * a.sp) * 4;
    auto go = [&](auto kern) { pm_allow_big_lds((const void *) kern, lds); hipLaunchKernelGGL(kern, dim3(n, (a.inner + cpb - 1) / cpb), dim3(256), lds, st, a, chunks, lpc); };
    if (a.sp <= 256) go(scan_kernel<T, 1, PHASE>); else if (a.sp == 512) go(scan_kernel<T, 2, PHASE>); else go(scan_kernel<T, 4, PHASE>);
}
template <typename T> void scan(const pm_ssm_layer & a, const pm_scan_chunk * chunks, int n, int multi, hipStream_t st) {
    if (multi) {
        scan_phase<T, 0>(a, chunks, n, st);
        hipLaunchKernelGGL(scan_carry_kernel, dim3(n, (unsigned) (((size_t) a.inner * a.sp / 4 + 255) / 256)), dim3(256), 0, st, a, chunks);
    }
    scan_phase<T, 1>(a, chunks, n, st);
}

} // namespace

void pm_launch_ssm_conv(const pm_ssm_layer & a, const pm_batch_dev & b, int T, hipStream_t st) { if (a.type == PM_BF16) conv<uint16_t>(a, b, T, st); else conv<float>(a, b, T, st); }
void pm_launch_ssm_step(const pm_ssm_layer & a, const pm_batch_dev & b, int T, hipStream_t st) { if (a.type == PM_BF16) step<uint16_t>(a, b, T, st); else step<float>(a, b, T, st); }
void pm_launch_ssm_scan(const pm_ssm_layer & a, const pm_batch_dev &, const pm_scan_chunk * chunks, int n, int multi, hipStream_t st) {
    if (a.type == PM_BF16) scan<uint16_t>(a, chunks, n, multi, st); else scan<float>(a, chunks, n, multi, st);
}
