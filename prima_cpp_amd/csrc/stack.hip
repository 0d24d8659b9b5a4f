// stack.hip — layer-described models (part B' of include/prima_mi355.h) behind the pm355_model handle: weights, page pool, and the step over a batch of unequal
// sequences. A layer is the kernels of dense_*.hip / attn_paged.hip with the constants of its descriptor; a new design is a new list of descriptors.
//
// Few tokens (decode): five launches per layer - projections (prologue: residual + norm of the sublayer before), attention (unit norm, value mixing, K / V store, gate),
// output projection, up, down - replayed from a hipGraph when every entry is one token. Prompts: the same products on the prompt GEMM, residual + norm and the cache
// store as launches of their own. All entries of a step share every launch; single tokens next to prompt portions attend through the decode kernel.
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

struct Mat { void * d = nullptr; int K = 0, N = 0, Kp = 0, Np = 0; };
struct LayerState {
    pm355_layer_spec s{};
    Mat proj, out, up, down;                   // proj: q | k | v | gate rows
    float * norm1 = nullptr, * norm1_b = nullptr, * norm2 = nullptr, * norm2_b = nullptr, * up_b = nullptr, * down_b = nullptr, * sink = nullptr;
    float lambda = 0.0f;
    int mixes = 0, dkp = 0, dvp = 0;
    void * kc = nullptr, * vc = nullptr;
    uint32_t have = 0;                         // bit per tensor kind
};
uint32_t bit(int kind) { return 1u << kind; }

struct pm_stack : pm355_model {
    pm355_stack_desc d{};
    std::vector<pm355_layer_spec> specs;
    std::vector<LayerState> layers;
    int Wp = 0;
    Mat embed, head_w;
    float * final_norm = nullptr, * final_norm_b = nullptr;
    uint32_t have = 0;
    size_t n_weight_bytes = 0;
    std::vector<void *> owned;                 // device allocations of the weights
    std::vector<void *> scratch;               // of finalize
    pm355_uploader * up = nullptr; void * stage = nullptr; size_t stage_bytes = 0;

    int max_tokens = 0; pm355_page_pool * pool = nullptr; std::vector<int> len;
    float * x[2] = {}, * y = nullptr, * vfirst = nullptr, * part = nullptr, * logits = nullptr; unsigned * ticket = nullptr;
    void * xb = nullptr, * raw = nullptr, * q = nullptr, * hb = nullptr, * fin = nullptr;
    std::map<int, void *> att;                 // attention outputs by width: their zero padding stays valid
    int max_raw = 0, max_q = 0, max_ff = 0, max_vf = 0; size_t part_floats = 0;
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
        scratch.clear(); att.clear();
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
    int locate(int kind, int layer, void ** dst, int64_t & rows, int & K, int & Kp, int & type, float ** scalar);
    int set_tensor(int kind, int layer, int type, const void * host, size_t nbytes) override;
    int fill_tensor(int kind, int layer, int type, uint64_t seed, float scale) override;
    void * tensor_ptr(int kind, int layer, int * type_out) override {
        void * dst = nullptr; int64_t rows; int K, Kp, dt; float * scalar;
        if (locate(kind, layer, &dst, rows, K, Kp, dt, &scalar) || scalar) return nullptr;
        if (type_out) *type_out = dt;
        return dst;
    }
    int finalize(int max_tokens_, int n_seq) override { return finalize_pool(max_tokens_, n_seq, (int64_t) n_seq * 4096); }
    int finalize_pool(int max_tokens_, int n_seq, int64_t pool_tokens) override;
    size_t weight_bytes() const override { return n_weight_bytes - (size_t) embed.Kp * embed.Np * pm_dense_bytes(d.type); }
    size_t kv_bytes_per_pos() const override { size_t n = 0; for (auto & L : layers) n += (size_t) L.s.n_head_kv * (L.dkp + L.dvp) * pm_dense_bytes(d.type); return n; }
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
    struct Step { pm_batch_dev b; int T, n_dec, n_tiles, n_want; const int32_t * dec, * want, * want_seq; const pm_attn_tile * tiles; int keys; float * lg; int32_t * am; std::vector<int> out_row; };   // out_row: logits row of a wanted row, from lg / am on
    int launch(const Step & p, hipStream_t st);
    int first_visible(int pos) const {
        int lo = pos;
        for (auto & s : specs) lo = std::min(lo, s.mask == PM355_MASK_CHUNK ? pos - pos % s.mask_size : 0);
        return lo;
    }
};

// head sizes of the matrix-core attention kernels: 64, 128 or 256 (both 256 when one exceeds 128); larger heads take the vector-pipe kernel
void head_pads(int type, int dk, int dv, int & dkp, int & dvp) {
    dkp = pm_dense_pad(dk); dvp = pm_dense_pad(dv);
    if (type != PM_BF16 || dkp > 256 || dvp > 256) return;
    if (dkp > 128 || dvp > 128) dkp = dvp = 256;
}

bool pm_stack::init() {
    Wp = pm_dense_pad(d.n_embd);
    layers.resize(d.n_layer);
    if (!make(embed, d.n_embd, d.n_vocab) || !make(head_w, d.n_embd, d.n_vocab)) return false;
    auto vec = [&](float *& p, int n) { p = (float *) zalloc((size_t) pm_dense_pad(n) * 4, owned); return p != nullptr; };
    bool ok = vec(final_norm, d.n_embd) && vec(final_norm_b, d.n_embd);
    int first_mix = -1;
    for (int i = 0; i < d.n_layer; ++i) {
        LayerState & L = layers[i];
        L.s = specs[i];
        const pm355_layer_spec & s = L.s;
        if (s.mix_flags & PM355_MIX_VALUE_MIX) {
            if (first_mix < 0) first_mix = i;
            L.mixes = first_mix == i ? 2 : 1;
        }
        head_pads(d.type, s.k_dim, s.v_dim, L.dkp, L.dvp);
        const int qk = (s.n_head + s.n_head_kv) * s.k_dim, gate = s.mix_flags & PM355_MIX_OUT_GATE ? s.n_head * s.v_dim : 0;
        ok = ok && make(L.proj, d.n_embd, qk + s.n_head_kv * s.v_dim + gate) && make(L.out, s.n_head * s.v_dim, d.n_embd) && vec(L.norm1, d.n_embd) && vec(L.norm1_b, d.n_embd) &&
             vec(L.sink, s.n_head);
        if (s.ff == PM355_FF_DENSE)
            ok = ok && make(L.up, d.n_embd, s.n_ff) && make(L.down, s.n_ff, d.n_embd) && vec(L.up_b, s.n_ff) && vec(L.down_b, d.n_embd) && vec(L.norm2, d.n_embd) && vec(L.norm2_b, d.n_embd);
        max_raw = std::max(max_raw, L.proj.Np); max_q = std::max(max_q, s.n_head * L.dkp); max_ff = std::max(max_ff, s.ff == PM355_FF_DENSE ? L.up.Np : 0);
        if (L.mixes) max_vf = std::max(max_vf, s.n_head_kv * s.v_dim);
    }
    return ok;
}

// does the model need this tensor?
bool pm_stack::wants(int kind, int layer) const {
    if (layer < 0) return kind == PM355_T_TOK_EMBD || kind == PM355_T_OUTPUT || kind == PM355_T_OUT_NORM || kind == PM355_T_OUT_NORM_B;
    const pm355_layer_spec & s = specs[layer];
    switch (kind) {
        case PM355_T_WQ: case PM355_T_WK: case PM355_T_WV: case PM355_T_WO: case PM355_T_ATTN_NORM: case PM355_T_ATTN_NORM_B: return true;
        case PM355_T_W_OUT_GATE: return s.mix_flags & PM355_MIX_OUT_GATE;
        case PM355_T_SINK: return s.mix_flags & PM355_MIX_SINK;
        case PM355_T_VALUE_MIX: return layers[layer].mixes == 1;
        case PM355_T_FFN_UP: case PM355_T_FFN_UP_B: case PM355_T_FFN_DOWN: case PM355_T_FFN_DOWN_B: case PM355_T_FFN_NORM: case PM355_T_FFN_NORM_B: return s.ff == PM355_FF_DENSE;
    }
    return false;
}

// destination of a tensor: rows x K values at *dst with row stride Kp (vectors: one row of f32), or a host scalar
int pm_stack::locate(int kind, int layer, void ** dst, int64_t & rows, int & K, int & Kp, int & type, float ** scalar) {
    if (layer >= d.n_layer || (layer >= 0 && kind == PM355_T_VALUE_MIX ? !(specs[layer].mix_flags & PM355_MIX_VALUE_MIX) : !wants(kind, layer < 0 ? -1 : layer)))
        return fail(PM355_E_RANGE, "tensor does not belong to this model");
    *scalar = nullptr; type = PM_F32; rows = 1; K = Kp = d.n_embd;
    auto mat = [&](const Mat & m, int row0, int n) { *dst = (char *) m.d + (size_t) row0 * m.Kp * pm_dense_bytes(d.type); rows = n; K = m.K; Kp = m.Kp; type = d.type; return 0; };
    auto vec = [&](float * p, int n) { *dst = p; K = Kp = n; return 0; };
    if (layer < 0) switch (kind) {
        case PM355_T_TOK_EMBD: return mat(embed, 0, d.n_vocab);
        case PM355_T_OUTPUT: return mat(head_w, 0, d.n_vocab);
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
        case PM355_T_FFN_UP_B: return vec(L.up_b, s.n_ff);
        case PM355_T_FFN_DOWN_B: return vec(L.down_b, d.n_embd);
        case PM355_T_SINK: return vec(L.sink, s.n_head);
    }
    *scalar = &L.lambda; K = Kp = 1;
    return 0;
}

int pm_stack::set_tensor(int kind, int layer, int type, const void * host, size_t nbytes) {
    (void) hipGetLastError();
    void * dst = nullptr; int64_t rows; int K, Kp, dt; float * scalar;
    int rc = locate(kind, layer, &dst, rows, K, Kp, dt, &scalar);
    if (rc) return rc;
    if (type != PM_BF16 && type != PM_F32) return fail(PM355_E_UNSUPPORTED, "set_tensor: dense models take BF16 or F32 data");
    if (nbytes != (size_t) rows * K * pm_dense_bytes(type)) return fail(PM355_E_SHAPE, "set_tensor: byte size does not match the shape");
    uint32_t & mark = layer < 0 ? have : layers[layer].have;
    if (scalar) {
        uint32_t u = 0;
        memcpy((char *) &u + (type == PM_BF16 ? 2 : 0), host, pm_dense_bytes(type));
        memcpy(scalar, &u, 4);
        mark |= bit(kind);
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
    pm_launch_dense_convert(type, stage, dt, dst, K, rows, Kp, nullptr);
    if (hipGetLastError() != hipSuccess) return fail(PM355_E_HIP, "set_tensor: conversion");
    mark |= bit(kind);
    return 0;
}

int pm_stack::fill_tensor(int kind, int layer, int, uint64_t seed, float scale) {
    (void) hipGetLastError();
    void * dst = nullptr; int64_t rows; int K, Kp, dt; float * scalar;
    const int rc = locate(kind, layer, &dst, rows, K, Kp, dt, &scalar);
    if (rc) return rc;
    if (scalar) *scalar = 0.5f;
    else {
        const bool norm = kind == PM355_T_ATTN_NORM || kind == PM355_T_FFN_NORM || kind == PM355_T_OUT_NORM;
        pm_launch_dense_fill(dt, dst, K, rows, Kp, seed, norm ? 1.0f : 0.0f, norm ? 0.05f : scale, nullptr);
    }
    (layer < 0 ? have : layers[layer].have) |= bit(kind);
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
    for (auto & L : layers) {
        Z(L.kc, (size_t) pages * L.s.n_head_kv * PM_PAGE * L.dkp * eb);
        Z(L.vc, (size_t) pages * L.s.n_head_kv * PM_PAGE * L.dvp * eb);
        const int w = L.s.n_head * L.s.v_dim;
        if (!att.count(w)) Z(att[w], T * L.out.Kp * eb);
        if (d.type == PM_BF16) {
            // (one allocation serves every decode size of every layer: rows of partials grow with the tokens of a batch)
            const int nd = (int) std::min<size_t>(T, GRAPH_MAX_TOKENS);
            part_floats = std::max(part_floats, pm_attn_decode_part_floats(nd, L.s.n_head_kv, L.s.n_head, L.dvp));
        }
    }
    if (!ok) return fail(PM355_E_NOMEM, "finalize: cache pages");
    int groups = 1;
    for (auto & L : layers) groups = std::max(groups, L.s.n_head_kv * ((L.s.n_head / L.s.n_head_kv + 15) / 16));
    Z(x[0], T * Wp * 4); Z(x[1], T * Wp * 4); Z(y, T * Wp * 4); Z(xb, T * Wp * eb); Z(fin, T * Wp * eb);
    Z(raw, T * max_raw * (d.type == PM_BF16 ? 2 : 4) + (size_t) RAW_F32_MAX * max_raw * 4);
    Z(q, T * max_q * eb); Z(hb, T * std::max(max_ff, 64) * eb); Z(vfirst, T * std::max(max_vf, 1) * 4);
    Z(part, part_floats * 4); Z(ticket, (size_t) GRAPH_MAX_TOKENS * groups * 4 + 64);
    Z(logits, (size_t) HEAD_ROWS * d.n_vocab * 4);
    meta_ints = 16 + 10 * std::max<size_t>(T, 16) + (size_t) pages * 2;
    Z(meta, meta_ints * 4); Z(table, (size_t) n_seq * seq_pages * 4); Z(last, (size_t) n_seq * 4); Z(last_out, 64);
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

int pm_stack::pass(const std::vector<Piece> & ps, float * d_logits, int32_t * d_argmax, hipStream_t st) {
    Step p{};
    int longest = 0, n_multi = 0;
    std::vector<std::pair<int, std::pair<int, int>>> want;      // logits row, (batch row, sequence or -1)
    for (auto & q : ps) {
        for (auto & w : q.want) want.push_back({w.second, {p.T + w.first, &w == &q.want.back() ? q.seq : -1}});
        p.T += q.n; longest = std::max(longest, q.pos + q.n); n_multi += q.n > 1;
    }
    if (!d_logits && !d_argmax) want.clear();
    std::sort(want.begin(), want.end());
    int cap = 16;                                               // offsets depend on the size class only: a captured graph finds its tables where they were
    while (cap < p.T) cap *= 2;
    cap = std::min(cap, std::max(max_tokens, 16));
    const int upd_at = 16 + 10 * cap, n_upd = (int) pool->changes.size();
    if ((size_t) upd_at + 2 * n_upd > meta_ints) return fail(PM355_E_SHAPE, "batch: step tables");
    const int hbuf = h_next;
    h_next = (h_next + 1) % META_BUFS;
    if (hipEventSynchronize(h_free[hbuf]) != hipSuccess) return fail(PM355_E_HIP, "batch: step tables");
    int32_t * h = h_meta[hbuf], * tok = h + 16, * pos = tok + cap, * seq = pos + cap, * dec = seq + cap, * til = dec + cap, * wr = til + 4 * cap, * ws = wr + cap;
    h[0] = n_upd;
    int r = 0;
    for (auto & q : ps) {
        for (int i = 0; i < q.n; ++i) { tok[r + i] = q.tok ? q.tok[i] : -1; pos[r + i] = q.pos + i; seq[r + i] = q.seq; }
        if (q.n == 1) dec[p.n_dec++] = r;
        else for (int i = 0; i < q.n; i += TILE) { int32_t * t = til + 4 * p.n_tiles++; t[0] = r + i; t[1] = std::min(TILE, q.n - i); t[2] = q.pos + i; t[3] = q.seq; }
        r += q.n;
    }
    p.n_want = (int) want.size();
    for (int i = 0; i < p.n_want; ++i) { wr[i] = want[i].second.first; ws[i] = want[i].second.second; }
    for (int i = 0; i < n_upd; ++i) { h[upd_at + 2 * i] = pool->changes[i].first; h[upd_at + 2 * i + 1] = pool->changes[i].second; }
    pool->changes.clear();
    if (hipMemcpyAsync(meta, h, (size_t) (upd_at + 2 * n_upd) * 4, hipMemcpyHostToDevice, st) != hipSuccess || hipEventRecord(h_free[hbuf], st) != hipSuccess)
        return fail(PM355_E_HIP, "batch: step tables");
    auto D = [&](const int32_t * host) { return meta + (host - h); };
    p.b = pm_batch_dev{D(tok), D(pos), D(seq), last, table, pool->max_seq_pages, meta + upd_at, meta};
    p.dec = n_multi ? D(dec) : nullptr; p.tiles = (const pm_attn_tile *) D(til); p.want = D(wr); p.want_seq = D(ws);
    p.keys = 256;
    while (p.keys < longest) p.keys *= 2;
    const int base = p.n_want ? want[0].first : 0;
    for (auto & w : want) p.out_row.push_back(w.first - base);
    p.lg = d_logits ? d_logits + (size_t) base * d.n_vocab : nullptr; p.am = d_argmax ? d_argmax + base : nullptr;

    const Key key{p.T, p.n_want, p.keys, p.lg, p.am};
    if (no_graph || plain || n_multi || p.T > GRAPH_MAX_TOKENS || p.n_want > GRAPH_MAX_TOKENS) return launch(p, st);
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
    const bool fuse = !plain && pm_dense_pro_ok(T, d.n_embd), raw32 = ty == PM_F32 || T <= RAW_F32_MAX;
    int cur = 0;
    struct { const float * w, * b; bool on; } pend = {nullptr, nullptr, false};      // y holds a sublayer's output whose norm has not joined the residual stream yet
    auto settle = [&]() {
        if (pend.on) pm_launch_add_layer_norm(ty, x[cur], y, Wp, Wp, pend.w, pend.b, d.norm_eps, d.n_embd, T, xb, st);
        pend.on = false;
    };
    // W . (residual stream)
    auto from_stream = [&](const Mat & m, void * out, int ldo, int otype, int n_store, const float * bias, int act) {
        pm_dense_args a{};
        a.type = ty; a.W = m.d; a.K = m.Kp; a.N = m.Np; a.T = T; a.y = out; a.ldy = ldo; a.y_type = otype; a.n_store = n_store; a.bias = bias; a.act_fn = act;
        if (pend.on && fuse) {
            const pm_add_norm pro{x[cur], y, Wp, Wp, pend.w, pend.b, d.norm_eps, d.n_embd, x[cur ^ 1], Wp};
            a.pro = &pro;
            const int rc = pm_launch_dense(a, st);
            cur ^= 1; pend.on = false;
            return rc;
        }
        settle();
        a.act = xb; a.lda = Wp;
        return pm_launch_dense(a, st);
    };
    auto dense = [&](const Mat & m, const void * act, void * out, int ldo, int otype, int n_store, const float * bias, int rows) {
        pm_dense_args a{};
        a.type = ty; a.W = m.d; a.K = m.Kp; a.N = m.Np; a.act = act; a.lda = m.Kp; a.T = rows; a.y = out; a.ldy = ldo; a.y_type = otype; a.n_store = n_store; a.bias = bias;
        return pm_launch_dense(a, st);
    };
    pm_launch_stack_embed(ty, embed.d, Wp, d.n_embd, p.b, T, x[0], xb, st);
    for (auto & L : layers) {
        const pm355_layer_spec & s = L.s;
        pm_attn_layer a{};
        a.type = ty; a.H = s.n_head; a.G = s.n_head_kv; a.dk = s.k_dim; a.dv = s.v_dim; a.dkp = L.dkp; a.dvp = L.dvp; a.scale = s.scale; a.cap = s.softcap; a.eps = d.norm_eps;
        a.flags = s.mix_flags; a.mask = s.mask; a.mask_size = s.mask_size; a.sink = L.sink; a.lambda = L.lambda; a.mixes = L.mixes; a.kc = L.kc; a.vc = L.vc;
        a.vfirst = vfirst; a.ld_vfirst = std::max(max_vf, 1); a.raw = raw; a.ldraw = L.proj.Np; a.raw_type = raw32 ? PM_F32 : PM_BF16; a.q = q; a.out = att[s.n_head * s.v_dim];
        a.ldo = L.out.Kp; a.part = part; a.ticket = ticket; a.part_floats = part_floats;
        int rc = from_stream(L.proj, raw, L.proj.Np, a.raw_type, L.proj.N, nullptr, PM355_ACT_NONE);
        if (rc) return fail(rc, "batch: projections");
        const bool mfma = ty == PM_BF16 && !plain && L.dkp <= 256 && L.dvp <= 256;
        const int keys = s.mask == PM355_MASK_CHUNK ? std::min(p.keys, s.mask_size + 2 * PM_PAGE) : p.keys;
        if (mfma && p.n_dec == T) rc = pm_launch_attn_decode_paged(a, p.b, nullptr, T, 1, keys, st);
        else {
            pm_launch_attn_prepare(a, p.b, T, st);
            if (!mfma) pm_launch_attn_plain(a, p.b, T, st);
            else {
                if (p.n_tiles) rc = pm_launch_attn_tiles(a, p.b, p.tiles, p.n_tiles, st);
                if (!rc && p.n_dec) rc = pm_launch_attn_decode_paged(a, p.b, p.dec, p.n_dec, 0, keys, st);
            }
        }
        if (!rc) rc = dense(L.out, a.out, y, Wp, PM_F32, d.n_embd, nullptr, T);
        if (rc) return fail(rc, "batch: attention");
        pend = {L.norm1, L.norm1_b, true};
        if (s.ff == PM355_FF_DENSE) {
            rc = from_stream(L.up, hb, L.up.Np, ty, L.up.Np, L.up_b, s.act);       // (padding columns: zero weights and bias)
            if (!rc) rc = dense(L.down, hb, y, Wp, PM_F32, d.n_embd, L.down_b, T);
            if (rc) return fail(rc, "batch: feed-forward");
            pend = {L.norm2, L.norm2_b, true};
        }
    }
    if (p.n_want) {
        settle();
        pm_launch_layer_norm_rows(ty, x[cur], Wp, p.want, final_norm, final_norm_b, d.norm_eps, d.n_embd, p.n_want, fin, Wp, st);
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
    for (int i = 0; i < d->n_layer; ++i) {
        const pm355_layer_spec & s = d->layers[i];
        if (s.n_head < 1 || s.n_head_kv < 1 || s.n_head % s.n_head_kv || s.k_dim < 1 || s.v_dim < 1 || s.k_dim > 4096 || s.v_dim > 4096) return nullptr;
        if ((s.mask != PM355_MASK_CAUSAL && s.mask != PM355_MASK_CHUNK) || (s.mask == PM355_MASK_CHUNK && s.mask_size < 1)) return nullptr;
        if (s.ff != PM355_FF_NONE && (s.ff != PM355_FF_DENSE || s.n_ff < 1 || (s.act != PM355_ACT_NONE && s.act != PM355_ACT_RELU2))) return nullptr;
        if (s.mix_flags & PM355_MIX_VALUE_MIX) {           // values of different layers are mixed: one shape
            if (vf >= 0 && vf != s.n_head_kv * s.v_dim) return nullptr;
            vf = s.n_head_kv * s.v_dim;
        }
    }
    pm_stack * m = new pm_stack(*d);
    if (!m->init()) { delete m; return nullptr; }
    return m;
}

const pm_arch_registrar reg_kudirax({2, "kudirax", nullptr, stack_new});

} // namespace
