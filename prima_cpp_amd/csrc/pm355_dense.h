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

// x + norm(y) in the prologue of a mat-vec (few tokens), where norm is a layer norm (weight, bias) or, with rms, y / sqrt(mean(y^2) + eps) * w; x == null: norm(y) alone. With
// w2 the sum is RMS-normed once more on its way to the product (a norm in front of the sublayer). The result is the activation row of every workgroup; workgroup 0 stores
// the sum as the new residual row (x_out) and the activations (act_out) where these are given
struct pm_add_norm {
    const float * x; const float * y; int ldx, ldy; const float * w; const float * b; float eps; int width;
    float * x_out; int ldo;
    int rms; const float * w2; void * act_out; int ld_act;
};
// attention outputs of one head per group that are still split by keys: part [T x head tiles][splits][16 heads][K] sums, ml [..][splits][16][maximum (log2 units), sum]
struct pm_split_merge { const float * part, * ml; int splits, H; };
constexpr size_t PM_SPLIT_FLOATS = (size_t) 256 * 128 * 128;
struct pm_dense_args {
    int type; const void * W; int K, N;                 // N: rows of W that exist (multiple of 64)
    const void * act; int lda; int T;
    void * y; int ldy, y_type, n_store;                 // columns [0, n_store) of y are written
    const float * bias; int act_fn;                     // bias: n_store floats or null; act_fn: PM355_ACT_*
    const pm_add_norm * pro;                            // != null: the activations are x + norm(y) (pm_dense_pro_ok)
    // group != 0 (a multiple of 32; the small-batch kernel, any T): one matrix per group of `group` rows (attention heads): group g multiplies the K activations from column
    // g * g_act on, its first g_store rows go to the columns from g * g_out on
    int group, g_act, g_out, g_store;
    float * split; size_t split_floats;                 // != null: scratch for products whose few tiles are split over k (PM_SPLIT_FLOATS always suffices)
    const pm_split_merge * merge;                       // != null (pm_dense_merge_ok, bf16, group = a head): the activations are merged from key splits on the way in
};
int pm_launch_dense(const pm_dense_args & a, hipStream_t st);                    // picks the small-batch or the prompt kernel
bool pm_dense_merge_ok(int T, int K);
bool pm_dense_pro_ok(int T, int width);

// f32 / bf16 host-order matrix [N][K] -> [rows at dst_row][Kp] of `type` (columns >= K stay as they are: zero from allocation). group > 0: rows come in groups of `group`,
// which start every `gstride` rows of dst; transpose: group g's rows become columns, dst row g * gstride + k
void pm_launch_dense_convert(int src_type, const void * src, int type, void * dst, int K, int64_t N, int Kp, hipStream_t st, int group = 0, int gstride = 0, int transpose = 0);
void pm_launch_ssm_decay(float * a, int64_t n, hipStream_t st);                  // a <- -exp(a) * log2(e)
void pm_launch_dense_fill(int type, void * dst, int K, int64_t N, int Kp, uint64_t seed, float mean, float amp, hipStream_t st);

// per-step tables of a batch in device memory (one upload per step): n tokens in the order of the entries
struct pm_batch_dev {
    const int32_t * tok;            // [T] token ids; < 0: last[seq]
    const int32_t * pos;            // [T]
    const int32_t * seq;            // [T]
    const int32_t * last;           // [n_seq] last greedy token per sequence
    int32_t * table; int table_ld;  // [n_seq][table_ld] pool pages (device copy of the page tables)
    const int32_t * upd; const int32_t * n_upd;         // table updates of this step: pairs (index, page)
    const int32_t * idx;            // [T] place of the token in its portion
    const int32_t * left;           // [T] tokens of the portion behind it
    int32_t * prev;                 // [n_seq] token in front of the portion (bigram embeddings), kept up to date by the embedding launch
};
// what the embedding launch does: x = embed[token] + bigram[(previous token * mul_prev + token * mul_cur) mod buckets] (first token of a sequence: row `buckets`);
// out = x, or its RMS norm with weight w2. It also brings page tables and `prev` up to date and clears `clear`
struct pm_embed_args {
    int type; const void * embed; int Kp, width;
    const void * bigram; int64_t buckets, mul_prev, mul_cur;      // bigram null: none
    const float * w2; float eps; int32_t * clear; int n_clear;
    float * x; void * out;
};
int  pm_launch_stack_embed(const pm_embed_args & a, const pm_batch_dev & b, int T, hipStream_t st);
// x += norm(y); out = x (or, with w2, x / rms(x) * w2) in T. parts > 0: y is the sum of `parts` rows, y[row * parts ..]; y_type: of y
// padded: rows (and w, b, w2) may be read and x and out written up to the next multiple of 4 columns
struct pm_norm_args { int rms; const float * w, * b, * w2; float eps; int width; int y_type, parts; bool padded; };
void pm_launch_add_norm(int type, const pm_norm_args & n, float * x, const void * y, int ldx, int ldy, int n_rows, void * out, int ldo, hipStream_t st);
// out[r] = norm(x[rows[r]]) in T (rows: gather list or null)
void pm_launch_norm_rows(int type, const pm_norm_args & n, const float * x, int ldx, const int32_t * rows, int n_rows, void * out, int ldo, hipStream_t st);
// cs[t][i] = cos, sin of pos[t] * base^(-2 i / dims), i < dims / 2
void pm_launch_rope_table(const int32_t * pos, int T, float base, int dims, float * cs, hipStream_t st);
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
    int flat;                               // tiles kernel: a tile's page p is page seq + p of kc / vc (keys made for this step) instead of the sequence's pool page
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

// one latent-attention layer (attn_latent.hip): keys and values of all heads are products of one cached row per token, [normed latent: kvp | rotated key part], ld values.
// Decoded tokens attend in the latent itself (query and output matrices are applied to them instead of to every key); prompts expand the keys they see
struct pm_latent_layer {
    int type, H, dim, rot, rot_dims, kv_rank, kvp, ld; float scale, eps; int mask, mask_size;
    void * cache;                           // [page][64][ld]
    const void * raw; int ldraw, raw_type;  // projections [T][query latent: q_rank | latent: kv_rank | rot]
    int q_rank; const float * q_norm; void * cq; int ld_cq;      // [T][ld_cq] normed query latent (written by pm_launch_latent_prepare)
    const float * kv_norm;                  // null: the layer reads another layer's cache
    void * qh; int qs;                      // [T][H][qs] queries, unrotated | rotated part
    void * qa;                              // [T][H][ld] queries in the latent | rotated part
    void * out; int ldo;                    // [T][ldo]: H x kvp weighted latents
    const float * cs;                       // [T][rot_dims / 2][cos, sin]
    float * part; size_t part_floats;
};
// query latents normed (cq != null), latents normed and keys rotated into the cache (kv_norm != null)
void pm_launch_latent_prepare(const pm_latent_layer & a, const pm_batch_dev & b, int T, hipStream_t st);
// rotates the queries' rotated part: in place in qh, and into qa
void pm_launch_latent_rotate(const pm_latent_layer & a, int T, hipStream_t st);
// tokens 0 .. n - 1 of the step. fused: the cache store and the rotation of the queries happen inside (every entry is one token). Keys may be split over workgroups: with
// merge != null the sums stay split for the value product (merge->splits > 1), otherwise `out` is complete
int  pm_launch_latent_decode(const pm_latent_layer & a, const pm_batch_dev & b, int n, int fused, int max_keys, pm_split_merge * merge, hipStream_t st);
void pm_launch_latent_plain(const pm_latent_layer & a, const pm_batch_dev & b, int n, hipStream_t st);
bool pm_latent_decode_ok(int kvp, int ld);
size_t pm_latent_part_floats(int n_tokens, int H, int kvp);
// keys of n_pages cache pages for the tiles kernel: K [page][H][64][dkp] (W_uk: [H * dim][kvp] plus the shared rotated part), V [page][H][dvp][64] (W_uv: per head vrows rows)
struct pm_latent_expand { const void * cache; int ld, kvp; const int32_t * pages; int n_pages; const void * Wk, * Wv; int H, dim, rot, vdim, vrows; void * K, * V; int dkp, dvp; };
int  pm_launch_latent_expand(const pm_latent_expand & e, hipStream_t st);       // the products
void pm_launch_latent_spread(const pm_latent_expand & e, hipStream_t st);       // the rotated part, to every head

// experts (moe.hip, dense_*.hip). Routing of T tokens: softmax over E logits, the `keep` best of `groups` groups of neighbours (by their largest score), the `top` largest
// scores among these, not renormalized
struct pm_route {
    const float * logits; int ldl, E, top, groups, keep;
    int32_t * id; float * w;                // [T * top] expert and weight per (token, slot)
    int32_t * pos;                          // [T * top] place among the expert's pairs
    int32_t * count;                        // [E] cleared by the embedding launch
    int32_t * off;                          // [E + 1] first sorted pair of an expert
    int32_t * order;                        // [T * top] sorted pairs
    int32_t * active;                       // [1 + E] number of experts with pairs, and which
    int32_t * tiles;                        // [1 + 3 n] number of tiles, then {expert, first sorted pair, pairs} each
    int tile;                               // pairs per tile (pm_expert_tile)
};
// pairs per tile of the prompt kernel: large ones where an expert has pairs for more than one
static inline int pm_expert_tile(int64_t pairs, int E) { return pairs >= 384 * (int64_t) E ? 256 : 128; }
constexpr int PM_ROUTE_PAIR_MAX = 4, PM_ROUTE_ONE_MAX = 64;      // tokens up to which the pairs go one by one / one workgroup routes and sorts
void pm_launch_route(const pm_route & r, int T, int want_tiles, hipStream_t st);
struct pm_expert_args {
    int type; pm_route r; int T, width_p, ffp, width;             // width_p, ffp: padded row lengths of up and down
    const void * up, * down; int64_t up_stride, down_stride;      // values between experts: [E][ffp][width_p], [E][width_p][ffp]
    int act_fn; const void * x; int ldx;                          // input rows in T
    void * hid;                                                   // [T * top][ffp] in T: weight * act(W_up x)
    void * y; int ldy, y_type;                                    // up to PM_ROUTE_PAIR_MAX tokens: [T] sums (f32); more: [T * top] rows, slot by slot
};
int pm_launch_experts_small(const pm_expert_args & a, hipStream_t st);
int pm_launch_experts_gemm(const pm_expert_args & a, hipStream_t st);

// selective scan (ssm.hip): S[c, n] <- exp(dt A) S + dt x B, y = sum_n S C + D x, gated with silu(z); x: causal convolution + silu of the first half of the projections
struct pm_scan_chunk { int32_t row, n, pos, seq, e_base, j, n_chunks, left; };      // up to 128 tokens of one portion; its place among the portion's chunks
struct pm_ssm_layer {
    int type, inner, innerp, state, sp, dt_rank, dtp, conv;       // sp: padded state (pm_ssm_state_pad)
    const void * raw; int ldraw, raw_type;                        // [T][x: inner | z: inner]
    const float * conv_w, * conv_b;                               // [inner][conv], [inner]
    void * xc;                                                    // [T][innerp] in T
    const void * f; int ldf;                                      // [T][dt: dtp | B: state | C: state] in T
    const void * w_dt; const float * dt_b;                        // [innerp][dtp] in T
    float * dt;                                                   // [T][innerp]: W_dt dt + bias, before the softplus (chunked scan)
    const float * A2, * D;                                        // [inner][sp]: -exp(A_log) log2(e)
    float * S, * cstate;                                          // [slot][inner][sp], [slot][conv - 1][innerp]
    float * E, * dtsum;                                           // [chunk][inner][sp], [chunk][innerp]
    void * y; int ldy;                                            // [T][ldy] in T
};
static inline int pm_ssm_state_pad(int n) { int p = 4; while (p < n) p *= 2; return p; }
void pm_launch_ssm_conv(const pm_ssm_layer & a, const pm_batch_dev & b, int T, hipStream_t st);
void pm_launch_ssm_step(const pm_ssm_layer & a, const pm_batch_dev & b, int T, hipStream_t st);      // every entry is one token: dt product, update, gate
void pm_launch_ssm_scan(const pm_ssm_layer & a, const pm_batch_dev & b, const pm_scan_chunk * chunks, int n_chunks, int multi, hipStream_t st);

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
__device__ __forceinline__ int first_key(int pos, int mask, int size) { return mask == 1 ? pos - pos % size : mask == 2 && pos >= size ? pos - size + 1 : 0; }
__device__ __forceinline__ float silu32(float z) { return z / (1.0f + expf(-z)); }
// log(1 + e^z) = max(z, 0) + log(1 + u), u = e^-|z|; log(1 + u) = 2 atanh(s), s = u / (2 + u) <= 1/3, by the series of atanh (next term: 1e-9 of the sum)
__device__ __forceinline__ float softplus_f(float z) {
    const float u = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z)), s = u * __builtin_amdgcn_rcpf(2.0f + u), q = s * s;
    float p = 1.0f / 17;
    p = fmaf(p, q, 1.0f / 15); p = fmaf(p, q, 1.0f / 13); p = fmaf(p, q, 1.0f / 11); p = fmaf(p, q, 1.0f / 9); p = fmaf(p, q, 1.0f / 7); p = fmaf(p, q, 0.2f); p = fmaf(p, q, 1.0f / 3);
    return fmaxf(z, 0.0f) + 2.0f * fmaf(s * q, p, s);
}
// activation functions of the dense products (PM355_ACT_*)
__device__ __forceinline__ float act_apply(int fn, float v) {
    if (fn == 1) { v = fmaxf(v, 0.0f); v *= v; }
    return v;
}
#endif
