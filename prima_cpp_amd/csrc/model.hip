// model.hip — the C entry points of part (B) of include/prima_mi355.h: architecture registry and dispatch to the implementation behind a handle (pm355_model.h).
#include "pm355_model.h"
#include <string.h>
#include <vector>

namespace {
std::vector<pm_arch_entry> & archs() { static std::vector<pm_arch_entry> v; return v; }     // (function-local: registrars of other files run before this file's statics)
hipStream_t S(pm355_stream_t s) { return (hipStream_t) s; }
}

pm_arch_registrar::pm_arch_registrar(const pm_arch_entry & e) { archs().push_back(e); }

extern "C" {

int pm355_arch_id(const char * name) {
    if (name) for (auto & e : archs()) if (!strcmp(e.name, name)) return e.arch;
    return PM355_E_UNSUPPORTED;
}
pm355_model * pm355_model_new(const pm355_hparams * hp, int lo, int hi, int flags) {
    if (hp) for (auto & e : archs()) if (e.arch == hp->arch && e.window) return e.window(hp, lo, hi, flags);
    return nullptr;
}
pm355_model * pm355_model_new_stack(const pm355_stack_desc * d) {
    if (d) for (auto & e : archs()) if (e.arch == d->arch && e.stack) return e.stack(d);
    return nullptr;
}
void pm355_model_free(pm355_model * m) { delete m; }
const char * pm355_model_error(pm355_model * m) { return m ? m->err : ""; }

int pm355_model_set_tensor(pm355_model * m, int kind, int layer, int type, const void * host, size_t nbytes) { return m->set_tensor(kind, layer, type, host, nbytes); }
int pm355_model_set_tensor_part(pm355_model * m, int kind, int layer, int part, int type, const void * host, size_t nbytes) { return m->set_tensor_part(kind, layer, part, type, host, nbytes); }
int pm355_model_fill_tensor(pm355_model * m, int kind, int layer, int type, uint64_t seed, float scale) { return m->fill_tensor(kind, layer, type, seed, scale); }
void * pm355_model_tensor_ptr(pm355_model * m, int kind, int layer, int * type_out) { return m->tensor_ptr(kind, layer, type_out); }
int pm355_model_set_streaming(pm355_model * m, int n_slots) { return m ? m->set_streaming(n_slots) : PM355_E_SHAPE; }
uint64_t pm355_model_streamed_bytes(const pm355_model * m) { return m ? m->streamed() : 0; }
int pm355_model_finalize(pm355_model * m, int max_tokens) { return m->finalize(max_tokens, 1); }
int pm355_model_finalize_seqs(pm355_model * m, int max_tokens, int n_seq) { return m->finalize(max_tokens, n_seq); }
int pm355_model_finalize_pool(pm355_model * m, int max_tokens, int n_seq, int64_t pool_tokens) { return m->finalize_pool(max_tokens, n_seq, pool_tokens); }
size_t pm355_model_weight_bytes(const pm355_model * m) { return m->weight_bytes(); }
size_t pm355_model_kv_bytes_per_pos(const pm355_model * m) { return m->kv_bytes_per_pos(); }
int pm355_model_kv_clear(pm355_model * m, pm355_stream_t st) { return m->kv_clear(S(st)); }
void * pm355_model_kv_ptr(pm355_model * m, int layer, int which) { return m->kv_ptr(layer, which); }
int pm355_model_n_embd(const pm355_model * m) { return m ? m->n_embd() : 0; }
int pm355_model_n_vocab(const pm355_model * m) { return m ? m->n_vocab() : 0; }
int pm355_model_n_seq(const pm355_model * m) { return m ? m->n_seqs() : 0; }
int pm355_model_check(pm355_model * m) { return m ? m->check() : PM355_E_SHAPE; }

int pm355_model_seq_new(pm355_model * m) { return m->seq_new(); }
int pm355_model_seq_free(pm355_model * m, int seq) { return m->seq_free(seq); }
int pm355_model_seq_len(pm355_model * m, int seq) { return m->seq_len(seq); }
int pm355_model_pool_info(pm355_model * m, pm355_pool_info * out) { return m->pool_info(out); }
int pm355_model_batch(pm355_model * m, const pm355_batch_entry * e, int n, float * d_logits, int32_t * d_argmax, pm355_stream_t st) { return m->batch(e, n, d_logits, d_argmax, S(st)); }

int pm355_model_set_pos(pm355_model * m, int pos, pm355_stream_t st) { return m->set_seq_pos(-1, pos, S(st)); }
int pm355_model_set_seq_pos(pm355_model * m, int seq, int pos, pm355_stream_t st) { return m->set_seq_pos(seq, pos, S(st)); }
int pm355_model_set_seq(pm355_model * m, int seq, pm355_stream_t st) { return m->set_seq(seq, S(st)); }
int pm355_model_head(pm355_model * m, const float * d_x_row, float * d_logits, int32_t * d_argmax, pm355_stream_t st) { return m->head(d_x_row, d_logits, d_argmax, S(st)); }
int pm355_model_decode(pm355_model * m, const int32_t * d_tokens, const float * d_x_in, int T, int pos0, float * d_x_out, float * d_logits, int32_t * d_argmax, pm355_stream_t st) {
    return m->decode(-1, d_tokens, d_x_in, T, pos0, d_x_out, d_logits, d_argmax, S(st));
}
int pm355_model_decode_seq(pm355_model * m, int seq, const int32_t * d_tokens, const float * d_x_in, int T, int pos0, float * d_x_out, float * d_logits, int32_t * d_argmax,
                           pm355_stream_t st) {
    if (seq < 0 || seq >= m->n_seqs()) return m->fail(PM355_E_RANGE, "decode_seq: seq >= n_seq");
    return m->decode(seq, d_tokens, d_x_in, T, pos0, d_x_out, d_logits, d_argmax, S(st));
}
int pm355_model_step_ex(pm355_model * m, const int32_t * d_token, const float * d_x_in, float * d_x_out, float * d_logits, int32_t * d_argmax, int advance, int rotate,
                        int head_first, int use_graph, pm355_stream_t st) {
    return m->step_ex(d_token, d_x_in, d_x_out, d_logits, d_argmax, advance, rotate, head_first, use_graph, S(st));
}
int pm355_model_step(pm355_model * m, const int32_t * d_token, const float * d_x_in, float * d_x_out, float * d_logits, int32_t * d_argmax, int advance, int use_graph,
                     pm355_stream_t st) {
    return m->step_ex(d_token, d_x_in, d_x_out, d_logits, d_argmax, advance, 0, 0, use_graph, S(st));
}
int pm355_model_generate(pm355_model * m, int32_t * d_io, int pos0, int n_steps, int use_graph, pm355_stream_t st) { return m->generate(d_io, pos0, n_steps, use_graph, S(st)); }

} // extern "C"
