// stack.hip — layer-described models (part B' of include/prima_mi355.h) behind the pm355_model handle: weights, page pool, and the step over a batch of unequal
// sequences. A layer is the kernels of dense_*.hip / attn_*.hip / ssm.hip / moe.hip with the constants of its descriptor; a new design is a new list of descriptors.
//
// Few tokens (decode): projections (prologue: residual + norm of the sublayer before, and the norm in front of this one), the mixer with its cache or state store inside, output
// projection, feed-forward - replayed from a hipGraph when every entry is one token. Prompts: the same products on the prompt GEMM, residual + norms and the cache store as
// launches of their own. All entries of a step share every launch; single tokens and short portions next to long ones attend through the decode kernels.
// A sequence holds pages of the cache (attention layers), a state slot per recurrent layer and its previous token; states count as zero at position 0.
#include "pm355_model.h"
#include "pm355_dense.h"
#include "pm355_kernels.h"
#include "kv_pool.h"
#include <math.h>
#include <stdlib.h>
#include <string.h>
#include <algorithm>
#include <map>
#include <vector>

namespace {

constexpr int META_BUFS = 4, GRAPH_MAX_TOKENS = 64, RAW_F32_MAX = 64, HEAD_ROWS = 256, TILE = 128;
constexpr int LATENT_ROWS = 32;                            // portions up to this long attend row by row in the latent, longer ones over expanded keys

struct Mat { void * d = nullptr; int K = 0, N = 0, Kp = 0, Np = 0; };
struct LayerState {
    pm355_layer_spec s{};
    Mat proj, out, up, down;                   // proj: q | k | v | gate rows; query latent | latent and rotated key; x | z
    float * norm1 = nullptr, * norm1_b = nullptr, * norm2 = nullptr, * norm2_b = nullptr, * up_b = nullptr, * down_b = nullptr, * sink = nullptr;
    float * pre1 = nullptr, * pre2 = nullptr;  // norms in front of the sublayers
    float lambda = 0.0f;
    int mixes = 0, dkp = 0, dvp = 0;
    void * kc = nullptr, * vc = nullptr;
    // latent attention: uk for expanded keys, uk_t per head transposed; rows of uv per head padded to vrows, rows of uq to qs
    Mat uq, uk, uk_t, uv; float * dq_norm = nullptr, * dkv_norm = nullptr;
    int kvp = 0, ld = 0, qs = 0, vrows = 0, mask_list = -1;       // mask_list: expanded keys of the step's long portions (-1: every token attends row by row)
    // selective scan
    Mat x_w, dt_w; float * conv_w = nullptr, * conv_b = nullptr, * dt_b = nullptr, * A2 = nullptr, * D = nullptr, * S = nullptr, * cstate = nullptr; int innerp = 0, sp = 0, dtp = 0;
    // experts
    Mat router, e_up, e_down; int ffp = 0, moe_index = 0; std::vector<char> have_part[2];
    uint64_t have = 0;                         // bit per tensor kind
};
uint64_t bit(int kind) { return 1ull << kind; }
static_assert(PM355_T_COUNT <= 64, "a bit per tensor kind");
// where a tensor goes: n rows of the source from src_row on, in groups of `group` rows every gstride rows of dst (pm_launch_dense_convert)
struct Dest { int64_t src_row, rows; void * dst; int Kp, type, group, gstride, transpose; };
struct Mask { int kind, size; };
int first_key_at(const Mask & m, int pos) { return m.kind == PM355_MASK_CHUNK ? pos - pos % m.size : m.kind == PM355_MASK_WINDOW ? std::max(0, pos - m.size + 1) : 0; }

struct pm_stack : pm355_model {
    pm355_stack_desc d{};
    std::vector<pm355_layer_spec> specs;
    std::vector<LayerState> layers;
    int Wp = 0;
    Mat embed, head_w, bigram;
    float * final_norm = nullptr, * final_norm_b = nullptr;
    uint64_t have = 0;
    bool any_latent = false, any_ssm = false; int n_moe = 0, max_E = 0;
    std::vector<Mask> masks;                   // of the latent layers whose long portions expand keys
    size_t n_weight_bytes = 0;
    std::vector<void *> owned;                 // device allocations of the weights
    std::vector<void *> scratch;               // of finalize
    pm355_uploader * up = nullptr; void * stage = nullptr; size_t stage_bytes = 0;

    int max_tokens = 0; pm355_page_pool * pool = nullptr; std::vector<int> len;
    float * x[2] = {}, * y = nullptr, * vfirst = nullptr, * part = nullptr, * ksplit = nullptr, * logits = nullptr; unsigned * ticket = nullptr;
    void * xb = nullptr, * raw = nullptr, * q = nullptr, * hb = nullptr, * fin = nullptr;
    std::map<int, void *> att;                 // attention outputs by width: their zero padding stays valid
    int max_raw = 0, max_q = 0, max_ff = 0, max_vf = 0; size_t part_floats = 0;
    void * cq = nullptr, * qa = nullptr, * ol = nullptr, * xK = nullptr, * xV = nullptr; int x_pages = 0;
    std::vector<std::pair<std::pair<float, int>, float *>> ropes;      // (base, dims) -> table of the step
    void * xc = nullptr, * fx = nullptr; float * dtb = nullptr, * E = nullptr, * dtsum = nullptr;
    float * rlog = nullptr, * rw = nullptr; void * hid = nullptr, * yrows = nullptr; int32_t * rid = nullptr, * rpos = nullptr, * counts = nullptr, * roff = nullptr, * rorder = nullptr, * ract = nullptr,
            * rtiles = nullptr, * prev = nullptr;
    int32_t * meta = nullptr, * table = nullptr, * last = nullptr, * last_out = nullptr; size_t meta_ints = 0;
    int32_t * h_meta[META_BUFS] = {}; hipEvent_t h_free[META_BUFS] = {}; int h_next = 0;
    bool plain = false, no_graph = false;      // PM355_STACK_PLAIN=1: unfused launches and the vector-pipe attention; PM355_STACK_GRAPH=0
    struct Key { int T, nw, keys; const void * lg, * am; bool operator==(const Key & o) const { return T == o.T && nw == o.nw && keys == o.keys && lg == o.lg && am == o.am; } };
    struct Graph { Key key; hipGraphExec_t exec; };
    std::vector<Graph> graphs; Key seen{0, 0, 0, nullptr, nullptr}; hipStream_t cap_stream = nullptr;

    explicit pm_stack(const pm355_stack_desc & desc) : d(desc), specs(desc.layers, desc.layers + desc.n_layer) { d.layers = specs.data(); }
    ~pm_stack() override {
        (void) hipDeviceSynchronize();
        drop_scratch();
        for (auto p : owned) (void) hipFree(p);
        if (stage) (void) hipFree(stage);
        pm355_uploader_free(up);
        if (cap_stream) (void) hipStreamDestroy(cap_stream);
    }
    void drop_scratch() {
        for (auto & g : graphs) (void) hipGraphExecDestroy(g.exec);
        graphs.clear(); seen = Key{0, 0, 0, nullptr, nullptr};
        for (auto p : scratch) (void) hipFree(p);
        scratch.clear(); att.clear(); ropes.clear();
        for (int i = 0; i < META_BUFS; ++i) { if (h_meta[i]) (void) hipHostFree(h_meta[i]); if (h_free[i]) (void) hipEventDestroy(h_free[i]); h_meta[i] = nullptr; h_free[i] = nullptr; }
        delete pool; pool = nullptr;
        max_tokens = 0;
    }
    // zeroed device memory
    void * zalloc(size_t n, std::vector<void *> & list) {
        void * p = nullptr;
        n = (std::max<size_t>(n, 1) + 255) / 256 * 256;
        if (hipMalloc(&p, n) != hipSuccess) { (void) hipGetLastError(); return nullptr; }
        if (hipMemset(p, 0, n) != hipSuccess) { (void) hipFree(p); (void) hipGetLastError(); return nullptr; }
        list.push_back(p);
        return p;
    }
    bool make(Mat & m, int K, int N) {
        m.K = K; m.N = N; m.Kp = pm_dense_pad(K); m.Np = pm_dense_pad(N);
        m.d = zalloc((size_t) m.Kp * m.Np * pm_dense_bytes(d.type), owned);
        n_weight_bytes += (size_t) m.Kp * m.Np * pm_dense_bytes(d.type);
        return m.d != nullptr;
    }
    bool init();
    bool wants(int kind, int layer) const;
    int locate(int kind, int layer, int part, std::vector<Dest> & to, int64_t & rows, int & K, float ** scalar);
    void have_it(int kind, int layer, int part);
    void after(int kind, int layer);
    int set_tensor(int kind, int layer, int type, const void * host, size_t nbytes) override { return set_tensor_part(kind, layer, 0, type, host, nbytes); }
    int set_tensor_part(int kind, int layer, int part, int type, const void * host, size_t nbytes) override;
    int fill_tensor(int kind, int layer, int type, uint64_t seed, float scale) override;
    void * tensor_ptr(int kind, int layer, int * type_out) override {
        std::vector<Dest> to; int64_t rows; int K; float * scalar;
        if (locate(kind, layer, 0, to, rows, K, &scalar) || scalar) return nullptr;
        if (type_out) *type_out = to[0].type;
        return to[0].dst;
    }
    int finalize(int max_tokens_, int n_seq) override { return finalize_pool(max_tokens_, n_seq, (int64_t) n_seq * 4096); }
    int finalize_pool(int max_tokens_, int n_seq, int64_t pool_tokens) override;
    size_t weight_bytes() const override { return n_weight_bytes - (size_t) embed.Kp * embed.Np * pm_dense_bytes(d.type); }
    size_t kv_bytes_per_pos() const override {
        size_t n = 0;
        for (auto & L : layers) {
            if (L.s.mixer == PM355_MIXER_ATTENTION) n += (size_t) L.s.n_head_kv * (L.dkp + L.dvp);
            if (L.s.mixer == PM355_MIXER_LATENT && L.s.kv_from < 0) n += L.ld;
        }
        return n * pm_dense_bytes(d.type);
    }
    int kv_clear(hipStream_t) override { return unsupported("kv_clear"); }       // (closed sequences leave nothing that is read)
    void * kv_ptr(int layer, int which) override { return layer < 0 || layer >= d.n_layer ? nullptr : which ? layers[layer].vc : layers[layer].kc; }
    int n_embd() const override { return d.n_embd; }
    int n_vocab() const override { return d.n_vocab; }
    int n_seqs() const override { return pool ? (int) pool->seqs.size() : 0; }
    int check() override { return hipDeviceSynchronize() == hipSuccess ? 0 : fail(PM355_E_HIP, "check"); }
    int seq_new() override {
        if (!pool) return fail(PM355_E_SHAPE, "seq_new: finalize_pool first");
        const int s = pool->open();
        if (s < 0) return fail(s, "seq_new: every sequence slot is taken");
        len[s] = 0;
        return s;
    }
    int seq_free(int s) override { return pool && pool->close(s) == 0 ? 0 : fail(PM355_E_RANGE, "seq_free: not an open sequence"); }
    int seq_len(int s) override { return pool && pool->valid(s) ? len[s] : PM355_E_RANGE; }
    int pool_info(pm355_pool_info * o) override {
        if (!pool) return fail(PM355_E_SHAPE, "pool_info: finalize_pool first");
        int fs = 0;
        for (auto & s : pool->seqs) fs += !s.open;
        *o = pm355_pool_info{PM_PAGE, pool->n_pages, (int) pool->free_list.size(), (int) pool->seqs.size(), fs, pool->max_seq_pages * PM_PAGE};
        return 0;
    }
    int batch(const pm355_batch_entry * e, int n, float * d_logits, int32_t * d_argmax, hipStream_t st) override;
    int generate(int32_t * d_io, int pos0, int n_steps, int use_graph, hipStream_t st) override;

    // one pass over T <= max_tokens tokens
    struct Piece { int seq, pos, n; const int32_t * tok; std::vector<std::pair<int, int>> want; };      // want: (token of the piece, logits row)
    int pass(const std::vector<Piece> & ps, float * d_logits, int32_t * d_argmax, hipStream_t st);
    struct Round { const int32_t * pages; int n_pages; const pm_attn_tile * tiles; int n_tiles; };      // expanded keys that fit the scratch, and the tiles that read them
    // rows [0, n_rows): single tokens and short portions; n_multi: entries of several tokens
    struct Step { pm_batch_dev b; int T, n_rows, n_multi, n_tiles, n_want; const int32_t * want, * want_seq; const pm_attn_tile * tiles; std::vector<std::vector<Round>> rounds;
                  const pm_scan_chunk * chunks; int n_chunks, multi_chunk; int keys; float * lg; int32_t * am; std::vector<int> out_row; };   // out_row: logits row of a wanted row, from lg / am on
    int launch(const Step & p, hipStream_t st);
    int first_visible(int pos) const {
        int lo = pos;
        for (auto & s : specs) if (s.mixer != PM355_MIXER_SSM) lo = std::min(lo, first_key_at({s.mask, s.mask_size}, pos));
        return lo;
    }
};

// head sizes of the matrix-core attention kernels: 64, 128 or 256 (both 256 when one exceeds 128); larger heads take the vector-pipe kernel
void head_pads(int type, int dk, int dv, int & dkp, int & dvp) {
    dkp = pm_dense_pad(dk); dvp = pm_dense_pad(dv);
    if (type != PM_BF16 || dkp > 256 || dvp > 256) return;
    if (dkp > 128 || dvp > 128) dkp = dvp = 256;
}

// the same for expanded latent keys: false where the prompt kernel has no such size
bool expanded_pads(int dk, int dv, int & dkp, int & dvp) {
    dkp = pm_dense_pad(dk); dvp = pm_dense_pad(dv);
    if (dkp > 256 || dvp > 256) return false;
    if (dkp > 192 || dvp > 128) dkp = dvp = 256;
    else if (dkp == 192) dvp = 128;
    return true;
}

bool pm_stack::init() {
    Wp = pm_dense_pad(d.n_embd);
    layers.resize(d.n_layer);
    if (!make(embed, d.n_embd, d.n_vocab) || !make(head_w, d.n_embd, d.n_vocab)) return false;
    auto vec = [&](float *& p, int n) { p = (float *) zalloc((size_t) pm_dense_pad(n) * 4, owned); return p != nullptr; };
    bool ok = vec(final_norm, d.n_embd) && vec(final_norm_b, d.n_embd) && (!d.bigram_buckets || make(bigram, d.n_embd, (int) d.bigram_buckets + 1));
    int first_mix = -1;
    for (int i = 0; i < d.n_layer; ++i) {
        LayerState & L = layers[i];
        L.s = specs[i];
        const pm355_layer_spec & s = L.s;
        if (s.mix_flags & PM355_MIX_VALUE_MIX) {
            if (first_mix < 0) first_mix = i;
            L.mixes = first_mix == i ? 2 : 1;
        }
        ok = ok && vec(L.norm1, d.n_embd) && vec(L.norm1_b, d.n_embd) && (!d.pre_norm || vec(L.pre1, d.n_embd));
        if (s.mixer == PM355_MIXER_ATTENTION) {
            head_pads(d.type, s.k_dim, s.v_dim, L.dkp, L.dvp);
            const int qk = (s.n_head + s.n_head_kv) * s.k_dim, gate = s.mix_flags & PM355_MIX_OUT_GATE ? s.n_head * s.v_dim : 0;
            ok = ok && make(L.proj, d.n_embd, qk + s.n_head_kv * s.v_dim + gate) && make(L.out, s.n_head * s.v_dim, d.n_embd) && vec(L.sink, s.n_head);
            max_q = std::max(max_q, s.n_head * L.dkp);
            if (L.mixes) max_vf = std::max(max_vf, s.n_head_kv * s.v_dim);
        } else if (s.mixer == PM355_MIXER_LATENT) {
            any_latent = true;
            L.kvp = pm_dense_pad(s.kv_rank); L.ld = L.kvp + pm_dense_pad(s.rot_dim); L.vrows = (s.v_dim + 31) / 32 * 32; L.qs = (s.k_dim + s.rot_dim + 7) / 8 * 8;
            if (d.type == PM_BF16 && pm_latent_decode_ok(L.kvp, L.ld) && expanded_pads(s.k_dim + s.rot_dim, s.v_dim, L.dkp, L.dvp)) {
                L.qs = L.dkp;
                for (size_t m = 0; m < masks.size(); ++m) if (masks[m].kind == s.mask && masks[m].size == s.mask_size) L.mask_list = (int) m;
                if (L.mask_list < 0) { L.mask_list = (int) masks.size(); masks.push_back({s.mask, s.mask_size}); }
                ok = ok && make(L.uk, s.kv_rank, s.n_head * s.k_dim);
            }
            ok = ok && make(L.proj, d.n_embd, s.q_rank + (s.kv_from < 0 ? s.kv_rank + s.rot_dim : 0)) && make(L.uq, s.q_rank, s.n_head * L.qs) && make(L.uk_t, s.k_dim, s.n_head * L.kvp) &&
                 make(L.uv, s.kv_rank, s.n_head * L.vrows) && make(L.out, s.n_head * s.v_dim, d.n_embd) && vec(L.dq_norm, s.q_rank) && vec(L.dkv_norm, s.kv_rank);
            max_q = std::max(max_q, s.n_head * L.qs);
        } else {
            any_ssm = true;
            L.innerp = pm_dense_pad(s.inner); L.sp = pm_ssm_state_pad(s.state); L.dtp = pm_dense_pad(s.dt_rank);
            L.A2 = (float *) zalloc((size_t) s.inner * L.sp * 4, owned); L.conv_w = (float *) zalloc((size_t) s.inner * s.conv * 4, owned);
            ok = ok && L.A2 && L.conv_w && make(L.proj, d.n_embd, 2 * s.inner) && make(L.x_w, s.inner, L.dtp + 2 * s.state) && make(L.dt_w, s.dt_rank, s.inner) && make(L.out, s.inner, d.n_embd) &&
                 vec(L.conv_b, s.inner) && vec(L.dt_b, s.inner) && vec(L.D, s.inner);
        }
        if (s.ff != PM355_FF_NONE) ok = ok && vec(L.norm2, d.n_embd) && vec(L.norm2_b, d.n_embd) && (!d.pre_norm || vec(L.pre2, d.n_embd));
        if (s.ff == PM355_FF_DENSE) ok = ok && make(L.up, d.n_embd, s.n_ff) && make(L.down, s.n_ff, d.n_embd) && vec(L.up_b, s.n_ff) && vec(L.down_b, d.n_embd);
        if (s.ff == PM355_FF_EXPERTS) {
            L.ffp = pm_dense_pad(s.n_ff); L.moe_index = n_moe++; max_E = std::max(max_E, s.n_expert);
            for (auto & h : L.have_part) h.assign(s.n_expert, 0);
            ok = ok && make(L.router, d.n_embd, s.n_expert) && make(L.e_up, d.n_embd, s.n_expert * L.ffp) && make(L.e_down, s.n_ff, s.n_expert * Wp);
        }
        max_raw = std::max(max_raw, L.proj.Np); max_ff = std::max(max_ff, s.ff == PM355_FF_DENSE ? L.up.Np : 0);
    }
    return ok;
}

// does the model need this tensor?
bool pm_stack::wants(int kind, int layer) const {
    const bool bias = d.norm == PM355_NORM_LAYER;
    if (layer < 0) return kind == PM355_T_TOK_EMBD || kind == PM355_T_OUTPUT || kind == PM355_T_OUT_NORM || (kind == PM355_T_OUT_NORM_B && bias) || (kind == PM355_T_BIGRAM && d.bigram_buckets);
    const pm355_layer_spec & s = specs[layer];
    const bool att = s.mixer == PM355_MIXER_ATTENTION, lat = s.mixer == PM355_MIXER_LATENT, ssm = s.mixer == PM355_MIXER_SSM;
    switch (kind) {
        case PM355_T_WQ: case PM355_T_WK: case PM355_T_WV: return att;
        case PM355_T_WO: case PM355_T_ATTN_NORM: return true;
        case PM355_T_ATTN_NORM_B: return bias;
        case PM355_T_ATTN_PRE_NORM: return d.pre_norm;
        case PM355_T_FFN_PRE_NORM: return d.pre_norm && s.ff != PM355_FF_NONE;
        case PM355_T_W_OUT_GATE: return att && (s.mix_flags & PM355_MIX_OUT_GATE);
        case PM355_T_SINK: return att && (s.mix_flags & PM355_MIX_SINK);
        case PM355_T_VALUE_MIX: return att && layers[layer].mixes == 1;
        case PM355_T_DQ: case PM355_T_DQ_NORM: case PM355_T_UQ: case PM355_T_UK: case PM355_T_UV: return lat;
        case PM355_T_DKV: case PM355_T_DKV_NORM: return lat && s.kv_from < 0;
        case PM355_T_SSM_IN: case PM355_T_SSM_CONV: case PM355_T_SSM_CONV_B: case PM355_T_SSM_X: case PM355_T_SSM_DT: case PM355_T_SSM_DT_B: case PM355_T_SSM_A_LOG: case PM355_T_SSM_D: return ssm;
        case PM355_T_FFN_NORM: return s.ff != PM355_FF_NONE;
        case PM355_T_FFN_NORM_B: return s.ff != PM355_FF_NONE && bias;
        case PM355_T_FFN_UP: case PM355_T_FFN_UP_B: case PM355_T_FFN_DOWN: case PM355_T_FFN_DOWN_B: return s.ff == PM355_FF_DENSE;
        case PM355_T_ROUTER: case PM355_T_EXP_UP: case PM355_T_EXP_DOWN: return s.ff == PM355_FF_EXPERTS;
    }
    return false;
}

// destinations of a tensor of rows x K values (vectors: one row of f32), or a host scalar
int pm_stack::locate(int kind, int layer, int part, std::vector<Dest> & to, int64_t & rows, int & K, float ** scalar) {
    if (layer >= d.n_layer || kind < 0 || kind >= PM355_T_COUNT || (layer >= 0 && kind == PM355_T_VALUE_MIX ? !(specs[layer].mix_flags & PM355_MIX_VALUE_MIX) : !wants(kind, layer < 0 ? -1 : layer)))
        return fail(PM355_E_RANGE, "tensor does not belong to this model");
    const bool parts = kind == PM355_T_EXP_UP || kind == PM355_T_EXP_DOWN;
    if (part < 0 || part >= (parts ? specs[layer].n_expert : 1)) return fail(PM355_E_RANGE, "tensor part out of range");
    *scalar = nullptr; rows = 1; K = d.n_embd; to.clear();
    const size_t eb = pm_dense_bytes(d.type);
    auto mat = [&](const Mat & m, int64_t row0, int n, int group = 0, int gstride = 0) { to.push_back({0, n, (char *) m.d + (size_t) row0 * m.Kp * eb, m.Kp, d.type, group, gstride, 0}); rows = n; K = m.K; return 0; };
    auto vec = [&](float * p, int n, int k = 1, int kp = 1) { if (k == 1 && kp == 1) { k = kp = n; n = 1; } to.push_back({0, n, p, kp, PM_F32, 0, 0, 0}); rows = n; K = k; return 0; };
    if (layer < 0) switch (kind) {
        case PM355_T_TOK_EMBD: return mat(embed, 0, d.n_vocab);
        case PM355_T_OUTPUT: return mat(head_w, 0, d.n_vocab);
        case PM355_T_BIGRAM: return mat(bigram, 0, (int) d.bigram_buckets + 1);
        case PM355_T_OUT_NORM: return vec(final_norm, d.n_embd);
        default: return vec(final_norm_b, d.n_embd);
    }
    LayerState & L = layers[layer];
    const pm355_layer_spec & s = L.s;
    const int qn = s.n_head * s.k_dim, kn = s.n_head_kv * s.k_dim, vn = s.n_head_kv * s.v_dim;
    switch (kind) {
        case PM355_T_WQ: return mat(L.proj, 0, qn);
        case PM355_T_WK: return mat(L.proj, qn, kn);
        case PM355_T_WV: return mat(L.proj, qn + kn, vn);
        case PM355_T_W_OUT_GATE: return mat(L.proj, qn + kn + vn, s.n_head * s.v_dim);
        case PM355_T_WO: return mat(L.out, 0, d.n_embd);
        case PM355_T_FFN_UP: return mat(L.up, 0, s.n_ff);
        case PM355_T_FFN_DOWN: return mat(L.down, 0, d.n_embd);
        case PM355_T_ATTN_NORM: return vec(L.norm1, d.n_embd);
        case PM355_T_ATTN_NORM_B: return vec(L.norm1_b, d.n_embd);
        case PM355_T_FFN_NORM: return vec(L.norm2, d.n_embd);
        case PM355_T_FFN_NORM_B: return vec(L.norm2_b, d.n_embd);
        case PM355_T_ATTN_PRE_NORM: return vec(L.pre1, d.n_embd);
        case PM355_T_FFN_PRE_NORM: return vec(L.pre2, d.n_embd);
        case PM355_T_FFN_UP_B: return vec(L.up_b, s.n_ff);
        case PM355_T_FFN_DOWN_B: return vec(L.down_b, d.n_embd);
        case PM355_T_SINK: return vec(L.sink, s.n_head);
        case PM355_T_DQ: return mat(L.proj, 0, s.q_rank);
        case PM355_T_DKV: return mat(L.proj, s.q_rank, s.kv_rank + s.rot_dim);
        case PM355_T_DQ_NORM: return vec(L.dq_norm, s.q_rank);
        case PM355_T_DKV_NORM: return vec(L.dkv_norm, s.kv_rank);
        case PM355_T_UQ: return mat(L.uq, 0, s.n_head * (s.k_dim + s.rot_dim), s.k_dim + s.rot_dim, L.qs);
        case PM355_T_UV: return mat(L.uv, 0, s.n_head * s.v_dim, s.v_dim, L.vrows);
        case PM355_T_UK:
            to.push_back({0, qn, L.uk_t.d, L.uk_t.Kp, d.type, s.k_dim, L.kvp, 1});
            if (L.uk.d) to.push_back({0, qn, L.uk.d, L.uk.Kp, d.type, 0, 0, 0});
            rows = qn; K = s.kv_rank;
            return 0;
        case PM355_T_SSM_IN: return mat(L.proj, 0, 2 * s.inner);
        case PM355_T_SSM_X:
            to.push_back({0, s.dt_rank, L.x_w.d, L.x_w.Kp, d.type, 0, 0, 0});
            to.push_back({s.dt_rank, 2 * s.state, (char *) L.x_w.d + (size_t) L.dtp * L.x_w.Kp * eb, L.x_w.Kp, d.type, 0, 0, 0});
            rows = s.dt_rank + 2 * s.state; K = s.inner;
            return 0;
        case PM355_T_SSM_DT: return mat(L.dt_w, 0, s.inner);
        case PM355_T_SSM_CONV: return vec(L.conv_w, s.inner * s.conv);
        case PM355_T_SSM_A_LOG: return vec(L.A2, s.inner, s.state, L.sp);
        case PM355_T_SSM_CONV_B: return vec(L.conv_b, s.inner);
        case PM355_T_SSM_DT_B: return vec(L.dt_b, s.inner);
        case PM355_T_SSM_D: return vec(L.D, s.inner);
        case PM355_T_ROUTER: return mat(L.router, 0, s.n_expert);
        case PM355_T_EXP_UP: return mat(L.e_up, (int64_t) part * L.ffp, s.n_ff);
        case PM355_T_EXP_DOWN: return mat(L.e_down, (int64_t) part * Wp, d.n_embd);
    }
    *scalar = &L.lambda; K = 1;
    return 0;
}
void pm_stack::have_it(int kind, int layer, int part) {
    if (layer < 0) { have |= bit(kind); return; }
    LayerState & L = layers[layer];
    if (kind == PM355_T_EXP_UP || kind == PM355_T_EXP_DOWN) {
        auto & h = L.have_part[kind == PM355_T_EXP_DOWN];
        h[part] = 1;
        for (char c : h) if (!c) return;
    }
    L.have |= bit(kind);
}
// what a tensor turns into once its values are in place
void pm_stack::after(int kind, int layer) {
    if (kind == PM355_T_SSM_A_LOG) pm_launch_ssm_decay(layers[layer].A2, (int64_t) specs[layer].inner * layers[layer].sp, nullptr);
}

int pm_stack::set_tensor_part(int kind, int layer, int part, int type, const void * host, size_t nbytes) {
    (void) hipGetLastError();
    std::vector<Dest> to; int64_t rows; int K; float * scalar;
    int rc = locate(kind, layer, part, to, rows, K, &scalar);
    if (rc) return rc;
    if (type != PM_BF16 && type != PM_F32) return fail(PM355_E_UNSUPPORTED, "set_tensor: dense models take BF16 or F32 data");
    if (nbytes != (size_t) rows * K * pm_dense_bytes(type)) return fail(PM355_E_SHAPE, "set_tensor: byte size does not match the shape");
    if (scalar) {
        uint32_t u = 0;
        memcpy((char *) &u + (type == PM_BF16 ? 2 : 0), host, pm_dense_bytes(type));
        memcpy(scalar, &u, 4);
        have_it(kind, layer, part);
        return 0;
    }
    if (!up && !(up = pm355_uploader_new(0, -1))) return fail(PM355_E_NOMEM, "set_tensor: uploader");
    if (hipStreamSynchronize(nullptr) != hipSuccess) return fail(PM355_E_HIP, "set_tensor");          // the stage's previous conversion
    if (nbytes > stage_bytes) {
        if (stage) (void) hipFree(stage);
        stage = nullptr; stage_bytes = 0;
        if (hipMalloc(&stage, nbytes) != hipSuccess) return fail(PM355_E_NOMEM, "set_tensor: stage");
        stage_bytes = nbytes;
    }
    rc = pm355_upload(up, PM_F32, K, host, stage, nbytes, 0);
    if (rc || pm355_uploader_sync(up)) return fail(PM355_E_HIP, "set_tensor: upload");
    for (auto & t : to)
        pm_launch_dense_convert(type, (const char *) stage + (size_t) t.src_row * K * pm_dense_bytes(type), t.type, t.dst, K, t.rows, t.Kp, nullptr, t.group, t.gstride, t.transpose);
    after(kind, layer);
    if (hipGetLastError() != hipSuccess) return fail(PM355_E_HIP, "set_tensor: conversion");
    have_it(kind, layer, part);
    return 0;
}

int pm_stack::fill_tensor(int kind, int layer, int, uint64_t seed, float scale) {
    (void) hipGetLastError();
    const int parts = layer >= 0 && layer < d.n_layer && (kind == PM355_T_EXP_UP || kind == PM355_T_EXP_DOWN) ? specs[layer].n_expert : 1;
    for (int part = 0; part < parts; ++part) {
        std::vector<Dest> to; int64_t rows; int K; float * scalar;
        const int rc = locate(kind, layer, part, to, rows, K, &scalar);
        if (rc) return rc;
        if (scalar) *scalar = 0.5f;
        else if (kind == PM355_T_UK || kind == PM355_T_UQ || kind == PM355_T_UV) {
            // (rows are placed by group: random values everywhere would put some into the padding)
            for (auto & t : to) for (int64_t g = 0; g < (t.group ? rows / t.group : 1); ++g)
                pm_launch_dense_fill(t.type, (char *) t.dst + (size_t) (t.group ? g * t.gstride * t.Kp : 0) * pm_dense_bytes(t.type), t.transpose ? t.group : K, t.transpose ? K : t.group ? t.group : rows,
                                     t.Kp, seed + g, 0.0f, scale, nullptr);
        } else {
            const bool norm = kind == PM355_T_ATTN_NORM || kind == PM355_T_FFN_NORM || kind == PM355_T_OUT_NORM || kind == PM355_T_ATTN_PRE_NORM || kind == PM355_T_FFN_PRE_NORM ||
                              kind == PM355_T_DQ_NORM || kind == PM355_T_DKV_NORM || kind == PM355_T_SSM_D;
            for (auto & t : to)
                pm_launch_dense_fill(t.type, t.dst, K, t.rows, t.Kp, seed + part * 1000, norm ? 1.0f : kind == PM355_T_SSM_DT_B ? -3.0f : kind == PM355_T_SSM_A_LOG ? 1.0f : 0.0f, norm ? 0.05f : scale, nullptr);
        }
        after(kind, layer);
        have_it(kind, layer, part);
    }
    return hipGetLastError() == hipSuccess ? 0 : fail(PM355_E_HIP, "fill_tensor");
}

int pm_stack::finalize_pool(int max_tokens_, int n_seq, int64_t pool_tokens) {
    (void) hipGetLastError();
    if (n_seq < 1 || n_seq > 1024 || max_tokens_ < 1 || pool_tokens < 1 || pool_tokens > (1ll << 30)) return fail(PM355_E_RANGE, "finalize: n_seq 1..1024, tokens >= 1");
    for (int i = -1; i < d.n_layer; ++i)
        for (int k = 0; k < PM355_T_COUNT; ++k)
            if (wants(k, i) && !((i < 0 ? have : layers[i].have) & bit(k))) { snprintf(err, sizeof(err), "finalize: tensor kind %d of layer %d is missing", k, i); return PM355_E_SHAPE; }
    (void) hipDeviceSynchronize();
    drop_scratch();
    if (stage) { (void) hipFree(stage); stage = nullptr; stage_bytes = 0; }
    { const char * e = getenv("PM355_STACK_PLAIN"); plain = e && e[0] == '1'; }
    { const char * e = getenv("PM355_STACK_GRAPH"); no_graph = e && e[0] == '0'; }
    const size_t T = (size_t) max_tokens_, eb = pm_dense_bytes(d.type);
    const int pages = (int) ((pool_tokens + PM_PAGE - 1) / PM_PAGE), seq_pages = std::max(pages, 16384);      // (a sequence whose layers all forget may outgrow the pool)
    bool ok = true;
    auto Z = [&](auto *& p, size_t bytes) { p = (std::remove_reference_t<decltype(p)>) zalloc(bytes, scratch); ok = ok && p; };
    const int nd = (int) std::min<size_t>(T, GRAPH_MAX_TOKENS);      // (one allocation serves every decode size of every layer: rows of partials grow with the tokens of a batch)
    for (auto & L : layers) {
        const pm355_layer_spec & s = L.s;
        if (s.mixer == PM355_MIXER_ATTENTION) {
            Z(L.kc, (size_t) pages * s.n_head_kv * PM_PAGE * L.dkp * eb);
            Z(L.vc, (size_t) pages * s.n_head_kv * PM_PAGE * L.dvp * eb);
            if (d.type == PM_BF16) part_floats = std::max(part_floats, pm_attn_decode_part_floats(nd, s.n_head_kv, s.n_head, L.dvp));
        } else if (s.mixer == PM355_MIXER_LATENT) {
            if (s.kv_from < 0) Z(L.kc, (size_t) pages * PM_PAGE * L.ld * eb);
            else L.kc = layers[s.kv_from].kc;
            if (d.type == PM_BF16) part_floats = std::max(part_floats, pm_latent_part_floats(nd, s.n_head, L.kvp));
        } else {
            Z(L.S, (size_t) n_seq * s.inner * L.sp * 4);
            Z(L.cstate, (size_t) n_seq * (s.conv - 1) * L.innerp * 4);
        }
        const int w = s.mixer == PM355_MIXER_SSM ? s.inner : s.n_head * s.v_dim;
        if (!att.count(w)) Z(att[w], T * L.out.Kp * eb);
    }
    if (!ok) return fail(PM355_E_NOMEM, "finalize: cache pages");
    int groups = 1;
    size_t n_cq = 0, n_qa = 0, n_ol = 0, n_xk = 0, n_xv = 0, n_xc = 0, n_fx = 0, n_E = 0, n_hid = 0, n_top = 0;
    for (auto & L : layers) {
        const pm355_layer_spec & s = L.s;
        if (s.mixer == PM355_MIXER_ATTENTION) groups = std::max(groups, s.n_head_kv * ((s.n_head / s.n_head_kv + 15) / 16));
        if (s.mixer == PM355_MIXER_LATENT) {
            n_cq = std::max(n_cq, (size_t) L.uq.Kp); n_qa = std::max(n_qa, (size_t) s.n_head * L.ld); n_ol = std::max(n_ol, (size_t) s.n_head * L.kvp);
            if (L.mask_list >= 0) { n_xk = std::max(n_xk, (size_t) s.n_head * PM_PAGE * L.dkp); n_xv = std::max(n_xv, (size_t) s.n_head * PM_PAGE * L.dvp); }
            bool known = false;
            for (auto & r : ropes) known = known || r.first == std::make_pair(s.rot_base, s.rot_dims);
            if (!known) { float * t = nullptr; Z(t, T * std::max(s.rot_dims, 2) * 4); ropes.push_back({{s.rot_base, s.rot_dims}, t}); }
        }
        if (s.mixer == PM355_MIXER_SSM) { n_xc = std::max(n_xc, (size_t) L.innerp); n_fx = std::max(n_fx, (size_t) L.x_w.Np); n_E = std::max(n_E, (size_t) s.inner * L.sp); }
        if (s.ff == PM355_FF_EXPERTS) { n_hid = std::max(n_hid, (size_t) s.n_expert_used * L.ffp); n_top = std::max(n_top, (size_t) s.n_expert_used); }
    }
    const size_t slack = 4096;                             // (products over padded k read a little beyond the last row)
    if (n_cq) { Z(cq, T * n_cq * eb); Z(qa, T * n_qa * eb + slack); Z(ol, (T * n_ol + n_ol) * eb + slack); }
    if (n_xk) {
        x_pages = std::min(pages, (int) std::max<size_t>(512, T * 4 / PM_PAGE));
        Z(xK, x_pages * n_xk * eb); Z(xV, x_pages * n_xv * eb);
    }
    if (n_xc) { Z(xc, T * n_xc * eb); Z(fx, T * n_fx * eb); Z(dtb, T * n_xc * 4); Z(E, (2 * T / TILE + 2) * n_E * 4); Z(dtsum, (2 * T / TILE + 2) * n_xc * 4); }
    if (n_moe) {
        const size_t rows = T * n_top, Ep = pm_dense_pad(max_E);
        Z(rlog, T * Ep * 4); Z(rw, rows * 4); Z(rid, rows * 4); Z(rpos, rows * 4); Z(counts, (size_t) n_moe * max_E * 4); Z(roff, (max_E + 1) * 4); Z(rorder, rows * 4); Z(ract, (max_E + 1) * 4);
        Z(rtiles, (1 + 3 * (rows / 128 + std::min<size_t>(max_E, rows) + 1)) * 4);
        Z(hid, T * n_hid * eb); Z(yrows, std::max(rows * eb, std::min<size_t>(T, RAW_F32_MAX) * n_top * 4) * Wp);
    }
    Z(x[0], T * Wp * 4); Z(x[1], T * Wp * 4); Z(y, T * Wp * 4); Z(xb, T * Wp * eb); Z(fin, T * Wp * eb);
    Z(raw, T * max_raw * (d.type == PM_BF16 ? 2 : 4) + (size_t) RAW_F32_MAX * max_raw * 4);
    Z(q, T * max_q * eb + slack); Z(hb, T * std::max(max_ff, 64) * eb); Z(vfirst, T * std::max(max_vf, 1) * 4);
    Z(part, part_floats * 4); if (T > RAW_F32_MAX && d.type == PM_BF16) Z(ksplit, PM_SPLIT_FLOATS * 4); else ksplit = nullptr; Z(ticket, (size_t) GRAPH_MAX_TOKENS * groups * 4 + 64);
    Z(logits, (size_t) HEAD_ROWS * d.n_vocab * 4);
    meta_ints = 16 + 19 * std::max<size_t>(T, 16) + (size_t) pages * 2 + masks.size() * (4 * (T / 16 + 2) + 2 * (size_t) x_pages);
    Z(meta, meta_ints * 4); Z(table, (size_t) n_seq * seq_pages * 4); Z(last, (size_t) n_seq * 4); Z(prev, (size_t) n_seq * 4); Z(last_out, 64);
    if (!ok) return fail(PM355_E_NOMEM, "finalize: scratch");
    for (int i = 0; i < META_BUFS; ++i)
        if (hipHostMalloc((void **) &h_meta[i], meta_ints * 4, hipHostMallocDefault) != hipSuccess || hipEventCreateWithFlags(&h_free[i], hipEventDisableTiming) != hipSuccess)
            return fail(PM355_E_NOMEM, "finalize: pinned step tables");
    if (!cap_stream && hipStreamCreateWithFlags(&cap_stream, hipStreamNonBlocking) != hipSuccess) return fail(PM355_E_HIP, "finalize: capture stream");
    pool = new pm355_page_pool(pages, n_seq, seq_pages);
    len.assign(n_seq, 0);
    max_tokens = max_tokens_;
    return hipDeviceSynchronize() == hipSuccess ? 0 : fail(PM355_E_HIP, "finalize");
}

int pm_stack::batch(const pm355_batch_entry * e, int n, float * d_logits, int32_t * d_argmax, hipStream_t st) {
    (void) hipGetLastError();
    if (!pool) return fail(PM355_E_SHAPE, "batch: finalize_pool first");
    if (n < 1) return 0;
    // everything that can be wrong with the request, before anything changes
    std::vector<char> used(pool->seqs.size(), 0);
    for (int i = 0; i < n; ++i) {
        if (!pool->valid(e[i].seq) || e[i].n_tokens < 1) return fail(PM355_E_RANGE, "batch: not an open sequence, or no tokens");
        if (used[e[i].seq]++) return fail(PM355_E_SHAPE, "batch: a sequence appears twice");
        if (!e[i].tokens && e[i].n_tokens != 1) return fail(PM355_E_SHAPE, "batch: the device-side token is one token");
        for (int j = 0; e[i].tokens && j < e[i].n_tokens; ++j) if (e[i].tokens[j] < 0 || e[i].tokens[j] >= d.n_vocab) return fail(PM355_E_RANGE, "batch: token id outside the vocabulary");
        for (int j = 0; j < e[i].n_want; ++j) if (e[i].want[j] < 0 || e[i].want[j] >= e[i].n_tokens) return fail(PM355_E_RANGE, "batch: want outside the portion");
        if ((int64_t) len[e[i].seq] + e[i].n_tokens > (int64_t) pool->max_seq_pages * PM_PAGE) return fail(PM355_E_RANGE, "batch: the sequence is too long");
    }
    int64_t need = 0;
    for (int i = 0; i < n; ++i) need += pool->missing(e[i].seq, len[e[i].seq] + e[i].n_tokens);
    if (need > (int64_t) pool->free_list.size()) return fail(PM355_E_NOMEM, "batch: the page pool is exhausted");
    for (int i = 0; i < n; ++i) (void) pool->grow(e[i].seq, len[e[i].seq] + e[i].n_tokens);

    std::vector<Piece> ps;
    int T = 0, row0 = 0;
    auto flush = [&]() {
        if (ps.empty()) return 0;
        const int rc = pass(ps, d_logits, d_argmax, st);
        ps.clear(); T = 0;
        return rc;
    };
    for (int i = 0; i < n; ++i) {
        for (int off = 0; off < e[i].n_tokens;) {
            if (T == max_tokens) { const int rc = flush(); if (rc) return rc; }
            Piece p{e[i].seq, len[e[i].seq], std::min(e[i].n_tokens - off, max_tokens - T), e[i].tokens ? e[i].tokens + off : nullptr, {}};
            for (int j = 0; j < e[i].n_want; ++j) if (e[i].want[j] >= off && e[i].want[j] < off + p.n) p.want.push_back({e[i].want[j] - off, row0 + j});
            off += p.n; T += p.n; len[e[i].seq] += p.n;
            ps.push_back(std::move(p));
        }
        row0 += e[i].n_want;
    }
    const int rc = flush();
    // pages that no layer can see from the next position on
    for (int i = 0; i < n; ++i) (void) pool->drop_before(e[i].seq, first_visible(len[e[i].seq]));
    return rc;
}

int pm_stack::pass(const std::vector<Piece> & entries, float * d_logits, int32_t * d_argmax, hipStream_t st) {
    Step p{};
    int longest = 0;
    // rows first: single tokens, portions short enough to attend row by row, and those whose keys would not fit the scratch
    auto pages_of = [&](const Piece & q, const Mask & m) { return (q.pos + q.n - 1) / PM_PAGE - first_key_at(m, q.pos) / PM_PAGE + 1; };
    auto is_row = [&](const Piece & q) {
        if (q.n <= (any_latent ? LATENT_ROWS : 1)) return true;
        for (auto & m : masks) if (pages_of(q, m) > x_pages) return true;
        return false;
    };
    std::vector<Piece> ps(entries);
    const size_t n_row_ps = std::stable_partition(ps.begin(), ps.end(), is_row) - ps.begin();
    std::vector<std::pair<int, std::pair<int, int>>> want;      // logits row, (batch row, sequence or -1)
    for (auto & q : ps) {
        for (auto & w : q.want) want.push_back({w.second, {p.T + w.first, &w == &q.want.back() ? q.seq : -1}});
        p.T += q.n; longest = std::max(longest, q.pos + q.n); p.n_multi += q.n > 1;
    }
    if (!d_logits && !d_argmax) want.clear();
    std::sort(want.begin(), want.end());
    int cap = 16;                                               // offsets depend on the size class only: a captured graph finds its tables where they were
    while (cap < p.T) cap *= 2;
    cap = std::min(cap, std::max(max_tokens, 16));
    const int upd_at = 16 + 19 * cap, n_upd = (int) pool->changes.size();
    if ((size_t) upd_at + 2 * n_upd > meta_ints) return fail(PM355_E_SHAPE, "batch: step tables");
    const int hbuf = h_next;
    h_next = (h_next + 1) % META_BUFS;
    if (hipEventSynchronize(h_free[hbuf]) != hipSuccess) return fail(PM355_E_HIP, "batch: step tables");
    int32_t * h = h_meta[hbuf], * chk = h + 16, * til = chk + 8 * cap, * tok = til + 4 * cap, * pos = tok + cap, * seq = pos + cap, * idx = seq + cap, * left = idx + cap, * wr = left + cap,
            * ws = wr + cap;
    h[0] = n_upd;
    int r = 0, n_e = 0;
    for (size_t k = 0; k < ps.size(); ++k) {
        const Piece & q = ps[k];
        for (int i = 0; i < q.n; ++i) { tok[r + i] = q.tok ? q.tok[i] : -1; pos[r + i] = q.pos + i; seq[r + i] = q.seq; idx[r + i] = i; left[r + i] = q.n - 1 - i; }
        if (k < n_row_ps) p.n_rows += q.n;
        else for (int i = 0; i < q.n; i += TILE) { int32_t * t = til + 4 * p.n_tiles++; t[0] = r + i; t[1] = std::min(TILE, q.n - i); t[2] = q.pos + i; t[3] = q.seq; }
        const int nc = (q.n + TILE - 1) / TILE;
        for (int j = 0; j < nc && any_ssm; ++j) {
            int32_t * c = chk + 8 * p.n_chunks++;
            c[0] = r + j * TILE; c[1] = std::min(TILE, q.n - j * TILE); c[2] = q.pos; c[3] = q.seq; c[4] = nc > 1 ? n_e : 0; c[5] = j; c[6] = nc; c[7] = 0;
        }
        if (nc > 1) { n_e += nc; p.multi_chunk = 1; }
        r += q.n;
    }
    // expanded keys of the long portions, by mask: as many portions per round as the scratch holds
    int end = upd_at + 2 * n_upd;
    auto D = [&](const int32_t * host) { return meta + (host - h); };
    for (auto & m : masks) {
        std::vector<Round> rounds;
        int row = p.n_rows, used = 0, at = end;                 // (tiles of this mask from `at` on, then its pages)
        int32_t * lt = h + at, * lp = lt + 4 * (p.T / 16 + 2);
        int n_t = 0, n_p = 0;
        for (size_t k = n_row_ps; k < ps.size(); ++k) {
            const Piece & q = ps[k];
            const int p0 = first_key_at(m, q.pos) / PM_PAGE, np = pages_of(q, m);
            if (rounds.empty() || used + np > x_pages) { rounds.push_back({D(lp + n_p), 0, (const pm_attn_tile *) D(lt + 4 * n_t), 0}); used = 0; }
            for (int i = 0; i < np; ++i) {
                if ((size_t) (lp - h) + n_p >= meta_ints) return fail(PM355_E_SHAPE, "batch: step tables");
                lp[n_p++] = pool->page(q.seq, p0 + i);
            }
            for (int i = 0; i < q.n; i += TILE) { int32_t * t = lt + 4 * n_t++; t[0] = row + i; t[1] = std::min(TILE, q.n - i); t[2] = q.pos + i; t[3] = used - p0; }
            rounds.back().n_pages += np; rounds.back().n_tiles += (q.n + TILE - 1) / TILE;
            used += np; row += q.n;
        }
        end = (int) (lp - h) + n_p;
        p.rounds.push_back(std::move(rounds));
    }
    p.n_want = (int) want.size();
    for (int i = 0; i < p.n_want; ++i) { wr[i] = want[i].second.first; ws[i] = want[i].second.second; }
    for (int i = 0; i < n_upd; ++i) { h[upd_at + 2 * i] = pool->changes[i].first; h[upd_at + 2 * i + 1] = pool->changes[i].second; }
    pool->changes.clear();
    if (hipMemcpyAsync(meta, h, (size_t) end * 4, hipMemcpyHostToDevice, st) != hipSuccess || hipEventRecord(h_free[hbuf], st) != hipSuccess)
        return fail(PM355_E_HIP, "batch: step tables");
    p.b = pm_batch_dev{D(tok), D(pos), D(seq), last, table, pool->max_seq_pages, meta + upd_at, meta, D(idx), D(left), prev};
    p.tiles = (const pm_attn_tile *) D(til); p.want = D(wr); p.want_seq = D(ws); p.chunks = (const pm_scan_chunk *) D(chk);
    p.keys = 256;
    while (p.keys < longest) p.keys *= 2;
    const int base = p.n_want ? want[0].first : 0;
    for (auto & w : want) p.out_row.push_back(w.first - base);
    p.lg = d_logits ? d_logits + (size_t) base * d.n_vocab : nullptr; p.am = d_argmax ? d_argmax + base : nullptr;

    const Key key{p.T, p.n_want, p.keys, p.lg, p.am};
    if (no_graph || plain || p.n_multi || p.T > GRAPH_MAX_TOKENS || p.n_want > GRAPH_MAX_TOKENS) return launch(p, st);
    for (auto & g : graphs) if (g.key == key) return hipGraphLaunch(g.exec, st) == hipSuccess ? 0 : fail(PM355_E_HIP, "batch: graph launch");
    if (!(seen == key)) { seen = key; return launch(p, st); }  // worth a graph once it repeats
    hipGraph_t g = nullptr; hipGraphExec_t exec = nullptr;
    if (hipStreamBeginCapture(cap_stream, hipStreamCaptureModeRelaxed) != hipSuccess) return fail(PM355_E_HIP, "batch: begin capture");
    const int rc = launch(p, cap_stream);
    const hipError_t he = hipStreamEndCapture(cap_stream, &g);
    if (rc || he != hipSuccess || !g) { if (g) (void) hipGraphDestroy(g); return rc ? rc : fail(PM355_E_HIP, "batch: end capture"); }
    const hipError_t hi = hipGraphInstantiate(&exec, g, nullptr, nullptr, 0);
    (void) hipGraphDestroy(g);
    if (hi != hipSuccess) return fail(PM355_E_HIP, "batch: graph instantiate");
    if (graphs.size() >= 32) { (void) hipDeviceSynchronize(); (void) hipGraphExecDestroy(graphs.front().exec); graphs.erase(graphs.begin()); }
    graphs.push_back({key, exec});
    return hipGraphLaunch(exec, st) == hipSuccess ? 0 : fail(PM355_E_HIP, "batch: graph launch");
}

int pm_stack::launch(const Step & p, hipStream_t st) {
    const int T = p.T, ty = d.type;
    const bool fuse = !plain && pm_dense_pro_ok(T, d.n_embd), raw32 = ty == PM_F32 || T <= RAW_F32_MAX, single = !p.n_multi;
    const int raw_type = raw32 ? PM_F32 : PM_BF16;
    int cur = 0;
    // a sublayer's output whose norm has not joined the residual stream yet: y, or the sum of `parts` rows of yrows per token
    struct { const float * w, * b; int parts, type; bool on; } pend = {nullptr, nullptr, 0, PM_F32, false};
    const int rms = d.norm == PM355_NORM_RMS;
    auto norm_b = [&](float * b) -> const float * { return rms ? nullptr : b; };
    auto settle = [&](const float * pre) {
        if (pend.on) pm_launch_add_norm(ty, pm_norm_args{rms, pend.w, pend.b, pre, d.norm_eps, d.n_embd, pend.type, pend.parts, true}, x[cur], pend.parts ? yrows : (void *) y, Wp, Wp, T, xb, Wp, st);
        pend.on = false;
    };
    // W . (residual stream, normed by `pre` where the design norms in front of a sublayer); keep: the activations are read again from xb
    auto from_stream = [&](const Mat & m, const float * pre, bool keep, void * out, int ldo, int otype, int n_store, const float * bias, int act) {
        pm_dense_args a{};
        a.type = ty; a.W = m.d; a.K = m.Kp; a.N = m.Np; a.T = T; a.y = out; a.ldy = ldo; a.y_type = otype; a.n_store = n_store; a.bias = bias; a.act_fn = act; a.split = ksplit; a.split_floats = PM_SPLIT_FLOATS;
        if (pend.on && fuse && !pend.parts) {
            const pm_add_norm pro{x[cur], y, Wp, Wp, pend.w, pend.b, d.norm_eps, d.n_embd, x[cur ^ 1], Wp, rms, pre, keep ? xb : nullptr, Wp};
            a.pro = &pro;
            const int rc = pm_launch_dense(a, st);
            cur ^= 1; pend.on = false;
            return rc;
        }
        settle(pre);
        a.act = xb; a.lda = Wp;
        return pm_launch_dense(a, st);
    };
    auto product = [&](const Mat & m, const void * act, int lda, void * out, int ldo, int otype, int n_store, const float * bias, int rows) {
        pm_dense_args a{};
        a.type = ty; a.W = m.d; a.K = m.Kp; a.N = m.Np; a.act = act; a.lda = lda; a.T = rows; a.y = out; a.ldy = ldo; a.y_type = otype; a.n_store = n_store; a.bias = bias;
        a.split = ksplit; a.split_floats = PM_SPLIT_FLOATS;
        return pm_launch_dense(a, st);
    };
    auto dense = [&](const Mat & m, const void * act, void * out, int ldo, int otype, int n_store, const float * bias, int rows) { return product(m, act, m.Kp, out, ldo, otype, n_store, bias, rows); };
    auto seen_keys = [&](const pm355_layer_spec & s) { return s.mask == PM355_MASK_CAUSAL ? p.keys : std::min(p.keys, s.mask_size + 2 * PM_PAGE); };

    auto attention = [&](LayerState & L) -> int {
        const pm355_layer_spec & s = L.s;
        pm_attn_layer a{};
        a.type = ty; a.H = s.n_head; a.G = s.n_head_kv; a.dk = s.k_dim; a.dv = s.v_dim; a.dkp = L.dkp; a.dvp = L.dvp; a.scale = s.scale; a.cap = s.softcap; a.eps = d.norm_eps;
        a.flags = s.mix_flags; a.mask = s.mask; a.mask_size = s.mask_size; a.sink = L.sink; a.lambda = L.lambda; a.mixes = L.mixes; a.kc = L.kc; a.vc = L.vc;
        a.vfirst = vfirst; a.ld_vfirst = std::max(max_vf, 1); a.raw = raw; a.ldraw = L.proj.Np; a.raw_type = raw_type; a.q = q; a.out = att[s.n_head * s.v_dim];
        a.ldo = L.out.Kp; a.part = part; a.ticket = ticket; a.part_floats = part_floats;
        int rc = from_stream(L.proj, L.pre1, false, raw, L.proj.Np, raw_type, L.proj.N, nullptr, PM355_ACT_NONE);
        if (rc) return rc;
        const bool mfma = ty == PM_BF16 && !plain && L.dkp <= 256 && L.dvp <= 256;
        if (mfma && single) rc = pm_launch_attn_decode_paged(a, p.b, nullptr, T, 1, seen_keys(s), st);
        else {
            pm_launch_attn_prepare(a, p.b, T, st);
            if (!mfma) pm_launch_attn_plain(a, p.b, T, st);
            else {
                if (p.n_tiles) rc = pm_launch_attn_tiles(a, p.b, p.tiles, p.n_tiles, st);
                if (!rc && p.n_rows) rc = pm_launch_attn_decode_paged(a, p.b, nullptr, p.n_rows, 0, seen_keys(s), st);
            }
        }
        return rc ? rc : dense(L.out, a.out, y, Wp, PM_F32, d.n_embd, nullptr, T);
    };

    auto latent = [&](LayerState & L) -> int {
        const pm355_layer_spec & s = L.s;
        pm_latent_layer a{};
        a.type = ty; a.H = s.n_head; a.dim = s.k_dim; a.rot = s.rot_dim; a.rot_dims = s.rot_dims; a.kv_rank = s.kv_rank; a.kvp = L.kvp; a.ld = L.ld; a.scale = s.scale; a.eps = d.norm_eps;
        a.mask = s.mask; a.mask_size = s.mask_size; a.cache = L.kc; a.raw = raw; a.ldraw = L.proj.Np; a.raw_type = raw_type; a.q_rank = s.q_rank; a.q_norm = L.dq_norm;
        a.ld_cq = L.uq.Kp; a.kv_norm = s.kv_from < 0 ? L.dkv_norm : nullptr; a.qh = q; a.qs = L.qs; a.qa = qa; a.out = ol; a.ldo = s.n_head * L.kvp; a.part = part; a.part_floats = part_floats;
        for (auto & r : ropes) if (r.first == std::make_pair(s.rot_base, s.rot_dims)) a.cs = r.second;
        void * out = att[s.n_head * s.v_dim];
        const int hq = s.n_head * L.qs;
        const bool mfma = ty == PM_BF16 && !plain && pm_latent_decode_ok(L.kvp, L.ld), inside = mfma && single;
        const bool pro = inside && raw32 && pm_dense_pro_ok(T, s.q_rank);      // the query latent's norm in its product's prologue, the cache store in the attention launch
        int rc = from_stream(L.proj, L.pre1, false, raw, L.proj.Np, raw_type, L.proj.N, nullptr, PM355_ACT_NONE);
        if (rc) return rc;
        if (pro) {
            const pm_add_norm n{nullptr, (const float *) raw, 0, L.proj.Np, L.dq_norm, nullptr, d.norm_eps, s.q_rank, nullptr, 0, 1, nullptr, nullptr, 0};
            pm_dense_args g{};
            g.type = ty; g.W = L.uq.d; g.K = L.uq.Kp; g.N = L.uq.Np; g.T = T; g.y = q; g.ldy = hq; g.y_type = ty; g.n_store = hq; g.pro = &n;
            rc = pm_launch_dense(g, st);
        } else {
            a.cq = cq;
            pm_launch_latent_prepare(a, p.b, T, st);
            a.kv_norm = nullptr;
            rc = dense(L.uq, cq, q, hq, ty, hq, nullptr, T);
        }
        if (rc) return rc;
        if (!inside) pm_launch_latent_rotate(a, T, st);
        const int rows = mfma && L.mask_list >= 0 ? p.n_rows : T;
        if (rows) {
            pm_dense_args g{};
            g.type = ty; g.W = L.uk_t.d; g.K = L.uk_t.Kp; g.N = L.uk_t.Np; g.act = q; g.lda = hq; g.T = rows; g.y = qa; g.ldy = s.n_head * L.ld; g.y_type = ty; g.n_store = s.n_head * L.ld;
            g.group = L.kvp; g.g_act = L.qs; g.g_out = L.ld; g.g_store = L.kvp;
            rc = pm_launch_dense(g, st);
            if (rc) return rc;
            pm_split_merge split{nullptr, nullptr, 1, 0};
            if (mfma) rc = pm_launch_latent_decode(a, p.b, rows, inside, seen_keys(s), pm_dense_merge_ok(rows, L.uv.Kp) ? &split : nullptr, st);
            else pm_launch_latent_plain(a, p.b, rows, st);
            if (rc) return rc;
            if (split.splits > 1) g.merge = &split;
            g.W = L.uv.d; g.K = L.uv.Kp; g.N = L.uv.Np; g.act = ol; g.lda = a.ldo; g.y = out; g.ldy = L.out.Kp; g.n_store = s.n_head * s.v_dim;
            g.group = L.vrows; g.g_act = L.kvp; g.g_out = s.v_dim; g.g_store = s.v_dim;
            rc = pm_launch_dense(g, st);
            if (rc) return rc;
        }
        if (rows < T) for (auto & r : p.rounds[L.mask_list]) {
            const pm_latent_expand x{L.kc, L.ld, L.kvp, r.pages, r.n_pages, L.uk.d, L.uv.d, s.n_head, s.k_dim, s.rot_dim, s.v_dim, L.vrows, xK, xV, L.dkp, L.dvp};
            rc = pm_launch_latent_expand(x, st);
            if (rc) return rc;
            pm_launch_latent_spread(x, st);
            pm_attn_layer t{};
            t.type = ty; t.H = t.G = s.n_head; t.dk = s.k_dim + s.rot_dim; t.dv = s.v_dim; t.dkp = L.dkp; t.dvp = L.dvp; t.scale = s.scale; t.eps = d.norm_eps; t.mask = s.mask;
            t.mask_size = s.mask_size; t.kc = xK; t.vc = xV; t.q = q; t.out = out; t.ldo = L.out.Kp; t.raw_type = raw_type; t.flat = 1;
            rc = pm_launch_attn_tiles(t, p.b, r.tiles, r.n_tiles, st);
            if (rc) return rc;
        }
        return dense(L.out, out, y, Wp, PM_F32, d.n_embd, nullptr, T);
    };

    auto ssm = [&](LayerState & L) -> int {
        const pm355_layer_spec & s = L.s;
        pm_ssm_layer a{};
        a.type = ty; a.inner = s.inner; a.innerp = L.innerp; a.state = s.state; a.sp = L.sp; a.dt_rank = s.dt_rank; a.dtp = L.dtp; a.conv = s.conv; a.raw = raw; a.ldraw = L.proj.Np;
        a.raw_type = raw_type; a.conv_w = L.conv_w; a.conv_b = L.conv_b; a.xc = xc; a.f = fx; a.ldf = L.x_w.Np; a.w_dt = L.dt_w.d; a.dt_b = L.dt_b; a.dt = dtb; a.A2 = L.A2; a.D = L.D; a.S = L.S;
        a.cstate = L.cstate; a.E = E; a.dtsum = dtsum; a.y = att[s.inner]; a.ldy = L.out.Kp;
        int rc = from_stream(L.proj, L.pre1, false, raw, L.proj.Np, raw_type, L.proj.N, nullptr, PM355_ACT_NONE);
        if (rc) return rc;
        pm_launch_ssm_conv(a, p.b, T, st);
        rc = dense(L.x_w, xc, fx, L.x_w.Np, ty, L.x_w.N, nullptr, T);
        if (rc) return rc;
        if (single && !plain) pm_launch_ssm_step(a, p.b, T, st);
        else {
            rc = product(L.dt_w, fx, L.x_w.Np, dtb, L.innerp, PM_F32, s.inner, L.dt_b, T);
            if (rc) return rc;
            pm_launch_ssm_scan(a, p.b, p.chunks, p.n_chunks, p.multi_chunk, st);
        }
        return dense(L.out, a.y, y, Wp, PM_F32, d.n_embd, nullptr, T);
    };

    auto experts = [&](LayerState & L, int & parts, int & y_type) -> int {
        const pm355_layer_spec & s = L.s;
        const int Ep = L.router.Np, small = ty == PM_F32 || T <= PM_ROUTE_ONE_MAX;
        int rc = from_stream(L.router, L.pre2, true, rlog, Ep, PM_F32, s.n_expert, nullptr, PM355_ACT_NONE);
        if (rc) return rc;
        pm_expert_args a{};
        a.type = ty; a.T = T; a.width_p = Wp; a.ffp = L.ffp; a.width = d.n_embd; a.up = L.e_up.d; a.down = L.e_down.d; a.up_stride = (int64_t) L.ffp * Wp; a.down_stride = (int64_t) Wp * L.ffp;
        a.act_fn = s.act; a.x = xb; a.ldx = Wp; a.hid = hid;
        a.r = pm_route{rlog, Ep, s.n_expert, s.n_expert_used, s.n_group, s.n_group_keep, rid, rw, rpos, counts + (size_t) L.moe_index * max_E, roff, rorder, ract, rtiles, pm_expert_tile((int64_t) T * s.n_expert_used, s.n_expert)};
        const bool pairs = T <= PM_ROUTE_PAIR_MAX;
        parts = pairs ? 0 : s.n_expert_used; y_type = small ? PM_F32 : PM_BF16;
        a.y = pairs ? (void *) y : yrows; a.ldy = Wp; a.y_type = y_type;
        if (!pairs) pm_launch_route(a.r, T, !small, st);
        return small ? pm_launch_experts_small(a, st) : pm_launch_experts_gemm(a, st);
    };

    pm_embed_args em{};
    em.type = ty; em.embed = embed.d; em.Kp = Wp; em.width = d.n_embd; em.bigram = bigram.d; em.buckets = d.bigram_buckets; em.mul_prev = d.bigram_mul_prev; em.mul_cur = d.bigram_mul_cur;
    em.w2 = layers[0].pre1; em.eps = d.norm_eps; em.clear = counts; em.n_clear = T > PM_ROUTE_PAIR_MAX ? n_moe * max_E : 0; em.x = x[0]; em.out = xb;
    if (const int rc = pm_launch_stack_embed(em, p.b, T, st)) return fail(rc, "batch: embedding");
    for (auto & r : ropes) pm_launch_rope_table(p.b.pos, T, r.first.first, r.first.second, r.second, st);
    for (auto & L : layers) {
        const pm355_layer_spec & s = L.s;
        int rc = s.mixer == PM355_MIXER_LATENT ? latent(L) : s.mixer == PM355_MIXER_SSM ? ssm(L) : attention(L);
        if (rc) return fail(rc, "batch: mixer");
        pend = {L.norm1, norm_b(L.norm1_b), 0, PM_F32, true};
        int parts = 0, y_type = PM_F32;
        if (s.ff == PM355_FF_NONE) continue;
        if (s.ff == PM355_FF_DENSE) {
            rc = from_stream(L.up, L.pre2, false, hb, L.up.Np, ty, L.up.Np, L.up_b, s.act);       // (padding columns: zero weights and bias)
            if (!rc) rc = dense(L.down, hb, y, Wp, PM_F32, d.n_embd, L.down_b, T);
        } else rc = experts(L, parts, y_type);
        if (rc) return fail(rc, "batch: feed-forward");
        pend = {L.norm2, norm_b(L.norm2_b), parts, y_type, true};
    }
    if (p.n_want) {
        settle(nullptr);
        pm_launch_norm_rows(ty, pm_norm_args{rms, final_norm, norm_b(final_norm_b), nullptr, d.norm_eps, d.n_embd, PM_F32, 0}, x[cur], Wp, p.want, p.n_want, fin, Wp, st);
        for (int r = 0, nr; r < p.n_want; r += nr) {       // rows that are neighbours in the output go together (all of them, unless a step ran in pieces)
            for (nr = 1; r + nr < p.n_want && p.out_row[r + nr] == p.out_row[r] + nr && (p.lg || nr < HEAD_ROWS); ++nr) {}
            float * lg = p.lg ? p.lg + (size_t) p.out_row[r] * d.n_vocab : logits;
            const int rc = dense(head_w, (char *) fin + (size_t) r * Wp * pm_dense_bytes(ty), lg, d.n_vocab, PM_F32, d.n_vocab, nullptr, nr);
            if (rc) return fail(rc, "batch: head");
            if (p.am) pm_launch_argmax_rows(lg, d.n_vocab, nr, p.am + p.out_row[r], p.want_seq + r, last, st);
        }
    }
    return hipGetLastError() == hipSuccess ? 0 : fail(PM355_E_HIP, "batch: kernel launch");
}

// greedy continuation of sequence 0, which stands at pos0: d_io[i] -> d_io[i + 1], tokens stay on the device
int pm_stack::generate(int32_t * d_io, int pos0, int n_steps, int, hipStream_t st) {
    if (!pool) return fail(PM355_E_SHAPE, "generate: finalize first");
    if (!pool->valid(0) && seq_new() != 0) return fail(PM355_E_SHAPE, "generate: sequence 0");
    if (len[0] != pos0) return fail(PM355_E_RANGE, "generate: sequence 0 does not stand at pos0");
    if (n_steps > 0 && hipMemcpyAsync(last, d_io, 4, hipMemcpyDeviceToDevice, st) != hipSuccess) return fail(PM355_E_HIP, "generate");
    const int32_t w = 0;
    for (int i = 0; i < n_steps; ++i) {
        const pm355_batch_entry e{0, 1, nullptr, 1, &w};
        const int rc = batch(&e, 1, nullptr, last_out, st);
        if (rc) return rc;
        if (hipMemcpyAsync(d_io + i + 1, last_out, 4, hipMemcpyDeviceToDevice, st) != hipSuccess) return fail(PM355_E_HIP, "generate");
    }
    return 0;
}

pm355_model * stack_new(const pm355_stack_desc * d) {
    if (d->n_layer < 1 || d->n_layer > 1024 || d->n_embd < 1 || d->n_embd > 32768 || d->n_vocab < 1 || !d->layers || (d->type != PM_BF16 && d->type != PM_F32)) return nullptr;
    int vf = -1;
    if (d->bigram_buckets < 0 || d->bigram_buckets >= 1ll << 31 || d->bigram_mul_prev < 0 || d->bigram_mul_cur < 0 || d->bigram_mul_prev >= 1ll << 31 || d->bigram_mul_cur >= 1ll << 31) return nullptr;
    if ((d->norm != PM355_NORM_LAYER && d->norm != PM355_NORM_RMS) || (d->pre_norm && d->norm != PM355_NORM_RMS)) return nullptr;
    for (int i = 0; i < d->n_layer; ++i) {
        const pm355_layer_spec & s = d->layers[i];
        const bool heads = s.n_head >= 1 && s.n_head <= 4096 && s.k_dim >= 1 && s.v_dim >= 1 && s.k_dim <= 4096 && s.v_dim <= 4096 &&
                           (s.mask == PM355_MASK_CAUSAL || ((s.mask == PM355_MASK_CHUNK || s.mask == PM355_MASK_WINDOW) && s.mask_size >= 1));
        if (s.mixer == PM355_MIXER_ATTENTION) {
            if (!heads || s.n_head_kv < 1 || s.n_head % s.n_head_kv) return nullptr;
        } else if (s.mixer == PM355_MIXER_LATENT) {
            if (!heads || s.mix_flags || s.q_rank < 1 || s.kv_rank < 1 || s.q_rank > 32768 || s.kv_rank > 4096 || s.rot_dim < 1 || s.rot_dim > 1024 || s.rot_dims < 2 || s.rot_dims % 2 ||
                s.rot_dims > s.rot_dim || s.kv_from >= i || !(s.rot_base > 0.0f)) return nullptr;
            if (s.kv_from >= 0) {                          // the layer whose rows are read has rows of its own, of the same shape
                const pm355_layer_spec & o = d->layers[s.kv_from];
                if (o.mixer != PM355_MIXER_LATENT || o.kv_from >= 0 || o.kv_rank != s.kv_rank || o.rot_dim != s.rot_dim || o.rot_dims != s.rot_dims || o.rot_base != s.rot_base) return nullptr;
            }
        } else if (s.mixer == PM355_MIXER_SSM) {
            if (s.inner < 1 || s.inner > 131072 || s.state < 1 || s.state > 1024 || s.dt_rank < 1 || s.dt_rank > 16384 || s.conv < 1 || s.conv > 64) return nullptr;
        } else return nullptr;
        if (s.ff < PM355_FF_NONE || s.ff > PM355_FF_EXPERTS || (s.ff != PM355_FF_NONE && (s.n_ff < 1 || (s.act != PM355_ACT_NONE && s.act != PM355_ACT_RELU2)))) return nullptr;
        if (s.ff == PM355_FF_EXPERTS && (s.n_expert < 1 || s.n_expert > 1024 || s.n_group < 1 || s.n_expert % s.n_group || s.n_group_keep < 1 || s.n_group_keep > s.n_group ||
                                         s.n_expert_used < 1 || s.n_expert_used > 64 || s.n_expert_used > s.n_group_keep * (s.n_expert / s.n_group))) return nullptr;
        if (s.mix_flags & PM355_MIX_VALUE_MIX) {           // values of different layers are mixed: one shape
            if (vf >= 0 && vf != s.n_head_kv * s.v_dim) return nullptr;
            vf = s.n_head_kv * s.v_dim;
        }
    }
    pm_stack * m = new pm_stack(*d);
    if (!m->init()) { delete m; return nullptr; }
    return m;
}

const pm_arch_registrar reg_kudirax({2, "kudirax", nullptr, stack_new}), reg_keranex({3, "keranex", nullptr, stack_new});

} // namespace
