// dense_api.hip — extern "C" surface of the dense-weight and paged-attention kernels (part A" of include/prima_mi355.h).
#include "../../include/prima_mi355.h"
#include "pm355_dense.h"
#include "pm355_kernels.h"

static int done(int rc, const char * what) {
    if (rc) return pm_api_fail(rc, what, hipSuccess);
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? 0 : pm_api_fail(PM355_E_HIP, what, e);
}
static pm_dense_args dense_args(int type, const void * W, int64_t K, int64_t N, const void * x, int64_t ldx, int T, void * y, int64_t ldy, int y_type, int64_t n_store, const float * bias,
                                int act) {
    pm_dense_args a{};
    a.type = type; a.W = W; a.K = (int) K; a.N = (int) N; a.act = x; a.lda = (int) ldx; a.T = T; a.y = y; a.ldy = (int) ldy; a.y_type = y_type; a.n_store = (int) n_store; a.bias = bias;
    a.act_fn = act;
    return a;
}

extern "C" {

int pm355_dense_mul_mat(int type, const void * W, int64_t K, int64_t N, const void * x, int64_t ldx, int n_tokens, void * y, int64_t ldy, int y_type, int64_t n_store, const float * bias,
                        int act, pm355_stream_t st) {
    if (!W || !x || !y || K < 64 || ldx < K || ldx % 8 || ldy < n_store || n_store < 1) return pm_api_fail(PM355_E_SHAPE, "dense_mul_mat: shape", hipSuccess);
    (void) hipGetLastError();
    return done(pm_launch_dense(dense_args(type, W, K, N, x, ldx, n_tokens, y, ldy, y_type, n_store, bias, act), (hipStream_t) st), "dense_mul_mat");
}
int pm355_dense_mul_mat_norm(int type, const void * W, int64_t K, int64_t N, const float * r, const float * d, int64_t ld, const float * w, const float * b, float eps, int width,
                             float * r_out, int n_tokens, void * y, int64_t ldy, int y_type, int64_t n_store, const float * bias, int act, pm355_stream_t st) {
    if (!W || !r || !d || !w || !b || !r_out || r_out == r || !y || K < 64 || width < 1 || width > K || ld < width || ldy < n_store || n_store < 1)
        return pm_api_fail(PM355_E_SHAPE, "dense_mul_mat_norm: shape", hipSuccess);
    (void) hipGetLastError();
    const pm_add_norm pro{r, d, (int) ld, (int) ld, w, b, eps, width, r_out, (int) ld, 0, nullptr, nullptr, 0};
    pm_dense_args a = dense_args(type, W, K, N, nullptr, 0, n_tokens, y, ldy, y_type, n_store, bias, act);
    a.pro = &pro;
    return done(pm_launch_dense(a, (hipStream_t) st), "dense_mul_mat_norm");
}
int pm355_add_layer_norm(int type, float * r, const float * d, int64_t ld, const float * w, const float * b, float eps, int width, int n_rows, void * xb, pm355_stream_t st) {
    if (!r || !d || !w || !b || width < 1 || width > 32768 || ld < width || n_rows < 1) return pm_api_fail(PM355_E_SHAPE, "add_layer_norm: shape", hipSuccess);
    (void) hipGetLastError();
    pm_launch_add_norm(type, pm_norm_args{0, w, b, nullptr, eps, width, PM_F32, 0}, r, d, (int) ld, (int) ld, n_rows, xb, (int) ld, (hipStream_t) st);
    return done(0, "add_layer_norm");
}
size_t pm355_attn_paged_scratch(int n_tokens, int n_head, int n_head_kv, int v_pad) { return pm_attn_decode_part_floats(n_tokens, n_head_kv, n_head, v_pad); }
int pm355_attn_paged(const pm355_attn_paged_args * p, int mode, pm355_stream_t pst) {
    const bool prepared = mode & 16;
    mode &= 15;
    if (!p || p->n_tokens < 1 || p->n_head_kv < 1 || p->n_head % p->n_head_kv || p->k_pad % 64 || p->v_pad % 64 || p->k_dim > p->k_pad || p->v_dim > p->v_pad || mode > 3 ||
        (mode == 2 && (p->n_tiles < 1 || !p->d_tiles)) || (p->mask == PM355_MASK_CHUNK && p->mask_size < 1))
        return pm_api_fail(PM355_E_SHAPE, "attn_paged: shape", hipSuccess);
    (void) hipGetLastError();
    hipStream_t st = (hipStream_t) pst;
    pm_attn_layer a{};
    a.type = p->type; a.H = p->n_head; a.G = p->n_head_kv; a.dk = p->k_dim; a.dv = p->v_dim; a.dkp = p->k_pad; a.dvp = p->v_pad; a.scale = p->scale; a.cap = p->softcap; a.eps = p->eps;
    a.flags = p->mix_flags; a.mask = p->mask; a.mask_size = p->mask_size; a.sink = p->sink; a.lambda = p->lambda; a.mixes = p->mixes; a.kc = p->k_pages; a.vc = p->v_pages;
    a.vfirst = p->v_first; a.ld_vfirst = p->ld_v_first; a.raw = p->proj; a.ldraw = p->ld_proj; a.raw_type = p->proj_type; a.q = p->q; a.out = p->out; a.ldo = p->ldo; a.part = p->scratch;
    a.ticket = p->tickets; a.part_floats = p->scratch_floats;
    pm_batch_dev b{};
    b.pos = p->d_pos; b.seq = p->d_seq; b.table = (int32_t *) p->d_table; b.table_ld = p->table_ld;
    if (mode < 3 && !prepared) pm_launch_attn_prepare(a, b, p->n_tokens, st);
    int rc = 0;
    if (mode == 1) pm_launch_attn_plain(a, b, p->n_tokens, st);
    if (mode == 2) rc = pm_launch_attn_tiles(a, b, (const pm_attn_tile *) p->d_tiles, p->n_tiles, st);
    if (mode == 3) rc = pm_launch_attn_decode_paged(a, b, nullptr, p->n_tokens, prepared ? 0 : 1, p->max_keys, st);
    return done(rc, "attn_paged");
}

} // extern "C"
