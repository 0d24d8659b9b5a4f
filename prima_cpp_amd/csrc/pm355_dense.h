// pm355_dense.h — kernels over dense (bf16 / f32) weights and paged KV caches: launch interface, and the device helpers they share.
//
// T = storage type of weights, activations and cache: bf16 (products on the bf16 matrix cores, f32 accumulation) or f32 (f32 matrix cores). Matrices are [N][K] rows,
// K padded with zeros to a multiple of 64 and N to a multiple of 64 (PM_DENSE_PAD), activations [tokens][K] with the same zero padding - padding columns multiply to 0.
#pragma once
#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

#define PM_BF16 30
#define PM_PAGE 64                       // tokens per KV page
static inline int pm_dense_pad(int n) { return (n + 63) / 64 * 64; }
static inline size_t pm_dense_bytes(int type) { return type == PM_BF16 ? 2 : 4; }

// x + layer_norm(y) in the prologue of a mat-vec (few tokens): the normed sum is the activation row of every workgroup, workgroup 0 stores it as the new residual row
struct pm_add_norm {
    const float * x; const float * y; int ldx, ldy; const float * w; const float * b; float eps; int width;
    float * x_out; int ldo;
};
struct pm_dense_args {
    int type; const void * W; int K, N;                 // N: rows of W that exist (multiple of 64)
    const void * act; int lda; int T;
    void * y; int ldy, y_type, n_store;                 // columns [0, n_store) of y are written
    const float * bias; int act_fn;                     // bias: n_store floats or null; act_fn: PM355_ACT_*
    const pm_add_norm * pro;                            // != null: the activations are x + norm(y) (pm_dense_pro_ok)
};
int pm_launch_dense(const pm_dense_args & a, hipStream_t st);                    // picks the small-batch or the prompt kernel
bool pm_dense_pro_ok(int T, int width);

// f32 / bf16 host-order matrix [N][K] -> [rows at dst_row][Kp] of `type` (columns >= K stay as they are: zero from allocation)
void pm_launch_dense_convert(int src_type, const void * src, int type, void * dst, int K, int64_t N, int Kp, hipStream_t st);
void pm_launch_dense_fill(int type, void * dst, int K, int64_t N, int Kp, uint64_t seed, float mean, float amp, hipStream_t st);

// per-step tables of a batch in device memory (one upload per step): n tokens in the order of the entries
struct pm_batch_dev {
    const int32_t * tok;            // [T] token ids; < 0: last[seq]
    const int32_t * pos;            // [T]
    const int32_t * seq;            // [T]
    const int32_t * last;           // [n_seq] last greedy token per sequence
    int32_t * table; int table_ld;  // [n_seq][table_ld] pool pages (device copy of the page tables)
    const int32_t * upd; const int32_t * n_upd;         // table updates of this step: pairs (index, page)
};
void pm_launch_stack_embed(int type, const void * embed, int Kp, int width, const pm_batch_dev & b, int T, float * x, void * xb, hipStream_t st);
// x += layer_norm(y) (y == null: x is normed in place of the sum: out = layer_norm(x)); xb = the same rows in T. rows: gather list or null
void pm_launch_add_layer_norm(int type, float * x, const float * y, int ldx, int ldy, const float * w, const float * b, float eps, int width, int n_rows, void * xb, hipStream_t st);
void pm_launch_layer_norm_rows(int type, const float * x, int ldx, const int32_t * rows, const float * w, const float * b, float eps, int width, int n_rows, void * out, int ldo,
                               hipStream_t st);
void pm_launch_argmax_rows(const float * logits, int n, int n_rows, int32_t * out, const int32_t * seq_of_row, int32_t * last, hipStream_t st);

// one attention layer over paged caches
struct pm_attn_layer {
    int type, H, G, dk, dv, dkp, dvp;       // dkp, dvp: multiples of 64 (cache and query rows; padding is zero)
    float scale, cap, eps; int flags, mask, mask_size;
    const float * sink; float lambda; int mixes;        // mixes: 1 = mix with v_first, 2 = this layer's v IS v_first
    void * kc, * vc;                        // K pages [page][G][64][dkp], V pages [page][G][dvp][64]
    float * vfirst; int ld_vfirst;          // [T][G * dv] f32
    const void * raw; int ldraw, raw_type;  // projections [T][q: H dk | k: G dk | v: G dv | gate: H dv]
    void * q;                               // [T][H][dkp] in T (written by pm_launch_attn_prepare)
    void * out; int ldo;                    // [T][H dv] in T (gate applied)
    float * part; unsigned * ticket; size_t part_floats;       // split-keys decode
};
// unit norm of q and k, value mixing, K / V into the pages
void pm_launch_attn_prepare(const pm_attn_layer & a, const pm_batch_dev & b, int T, hipStream_t st);
// a prompt tile: up to 128 consecutive tokens of one entry; {first row, tokens, position of the first, sequence}
struct pm_attn_tile { int32_t row, n, pos, seq; };
int  pm_launch_attn_tiles(const pm_attn_layer & a, const pm_batch_dev & b, const pm_attn_tile * d_tiles, int n_tiles, hipStream_t st);
// decoded tokens: rows d_rows[0 .. n) (null: rows 0 .. n - 1). fused != 0: pm_launch_attn_prepare's work for these rows happens inside. max_keys bounds the keys a token sees
int  pm_launch_attn_decode_paged(const pm_attn_layer & a, const pm_batch_dev & b, const int32_t * d_rows, int n, int fused, int max_keys, hipStream_t st);
// any sizes, either type, one token at a time on the vector pipe: the 32-bit model, and head sizes beyond 256
void pm_launch_attn_plain(const pm_attn_layer & a, const pm_batch_dev & b, int T, hipStream_t st);
size_t pm_attn_decode_part_floats(int n_tokens, int G, int H, int dvp);
int  pm_attn_decode_splits(int n_tokens, int G, int max_keys);

#ifdef __HIPCC__
#include "pm355_device.h"
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
__device__ __forceinline__ float bf2f(uint16_t v) { return __builtin_bit_cast(float, (uint32_t) v << 16); }
__device__ __forceinline__ uint16_t f2bf(float f) { return __builtin_bit_cast(uint16_t, (__bf16) f); }          // RNE
template <typename T> __device__ __forceinline__ float to_f(T v);
template <> __device__ __forceinline__ float to_f<float>(float v) { return v; }
template <> __device__ __forceinline__ float to_f<uint16_t>(uint16_t v) { return bf2f(v); }
template <typename T> __device__ __forceinline__ T from_f(float v);
template <> __device__ __forceinline__ float from_f<float>(float v) { return v; }
template <> __device__ __forceinline__ uint16_t from_f<uint16_t>(float v) { return f2bf(v); }
__device__ __forceinline__ float ld_any(const void * p, size_t i, int type) { return type == PM_BF16 ? bf2f(((const uint16_t *) p)[i]) : ((const float *) p)[i]; }
__device__ __forceinline__ void st_type(void * p, size_t i, int type, float v) { if (type == PM_BF16) ((uint16_t *) p)[i] = f2bf(v); else ((float *) p)[i] = v; }
__device__ __forceinline__ float wave_max(float v) {
    for (int o = 32; o; o >>= 1) v = fmaxf(v, __shfl_xor(v, o));
    return v;
}
// 1 KiB of LDS at byte address `dst` (wave-uniform) <- 64 x 16 bytes, lane l from base + voff (its own 32-bit offset). Inline asm for the reason given in mmq_pf.hip:
// an LDS-DMA the compiler can see turns its counted lgkmcnt waits into full drains. The caller waits with pm_vm_drain().
__device__ __forceinline__ void pm_dma16(const void * base, uint32_t voff, uint32_t dst) {
    unsigned keep;
    dst = (uint32_t) __builtin_amdgcn_readfirstlane((int) dst);
    asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                 : "=&s"(keep) : "v"(voff), "s"(uniform_ptr((char *) base)), "s"(dst) : "memory");
}
__device__ __forceinline__ void pm_vm_drain() { asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); }
// softcap * tanh(s / softcap): tanh z = 1 - 2 / (e^2z + 1), absolute error of a few ulp of softcap
__device__ __forceinline__ float cap_score(float s, float cap, float inv2cap_log2e) {
    const float e = __builtin_amdgcn_exp2f(s * inv2cap_log2e);
    return cap - 2.0f * cap * __builtin_amdgcn_rcpf(e + 1.0f);
}
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + __expf(-z)); }
// first key position the query at `pos` sees
__device__ __forceinline__ int first_key(int pos, int mask, int size) { return mask == 1 ? pos - pos % size : 0; }
#endif
