// pm355_model.h — what stands behind the C handle pm355_model: the interface every model implementation provides, and the registry that picks one by architecture.
// engine.hip registers the quantized Llama / Qwen2 layer windows, stack.hip the layer-described models; model.hip turns the C entry points into these calls. A build
// that links only some of the implementations serves only their architectures (build.py: build_dense()).
#pragma once
#include "../../include/prima_mi355.h"
#include <hip/hip_runtime.h>
#include <stdio.h>

struct pm355_model {
    char err[256] = "";
    virtual ~pm355_model() {}

    virtual int set_tensor(int kind, int layer, int type, const void * host, size_t nbytes) = 0;
    virtual int set_tensor_part(int kind, int layer, int part, int type, const void * host, size_t nbytes) {      // part: expert
        return part ? unsupported("set_tensor_part") : set_tensor(kind, layer, type, host, nbytes);
    }
    virtual int fill_tensor(int kind, int layer, int type, uint64_t seed, float scale) = 0;
    virtual void * tensor_ptr(int, int, int *) { return nullptr; }
    virtual int set_streaming(int) { return unsupported("set_streaming"); }
    virtual uint64_t streamed() const { return 0; }
    virtual int finalize(int max_tokens, int n_seq) = 0;
    virtual int finalize_pool(int max_tokens, int n_seq, int64_t pool_tokens) = 0;
    virtual size_t weight_bytes() const = 0;
    virtual size_t kv_bytes_per_pos() const = 0;
    virtual int kv_clear(hipStream_t) = 0;
    virtual void * kv_ptr(int, int) { return nullptr; }
    virtual int n_embd() const = 0;
    virtual int n_vocab() const = 0;
    virtual int n_seqs() const = 0;
    virtual int check() = 0;

    // batches of unequal sequences (scheduler, trace replay)
    virtual int seq_new() = 0;
    virtual int seq_free(int seq) = 0;
    virtual int seq_len(int seq) = 0;
    virtual int pool_info(pm355_pool_info * out) = 0;
    virtual int batch(const pm355_batch_entry * e, int n, float * d_logits, int32_t * d_argmax, hipStream_t st) = 0;

    // one sequence at a time (layer windows of the ring)
    virtual int decode(int /*seq, -1: sequence 0*/, const int32_t *, const float *, int, int, float *, float *, int32_t *, hipStream_t) { return unsupported("decode"); }
    virtual int set_seq_pos(int, int, hipStream_t) { return unsupported("set_seq_pos"); }
    virtual int set_seq(int, hipStream_t) { return unsupported("set_seq"); }
    virtual int head(const float *, float *, int32_t *, hipStream_t) { return unsupported("head"); }
    virtual int step_ex(const int32_t *, const float *, float *, float *, int32_t *, int, int, int, int, hipStream_t) { return unsupported("step"); }
    virtual int generate(int32_t * d_io, int pos0, int n_steps, int use_graph, hipStream_t st) = 0;

    int fail(int code, const char * msg) {
        const hipError_t e = hipGetLastError();        // also clears the sticky error
        if (code == PM355_E_HIP) snprintf(err, sizeof(err), "%s: %s", msg, hipGetErrorString(e));
        else snprintf(err, sizeof(err), "%s", msg);
        return code;
    }
    int unsupported(const char * what) { snprintf(err, sizeof(err), "%s: not available for this architecture", what); return PM355_E_UNSUPPORTED; }
};

// architecture registry: a factory per architecture id, registered by the implementation's translation unit
typedef pm355_model * (*pm_window_factory)(const pm355_hparams * hp, int lo, int hi, int flags);
typedef pm355_model * (*pm_stack_factory)(const pm355_stack_desc * d);
struct pm_arch_entry { int arch; const char * name; pm_window_factory window; pm_stack_factory stack; };
struct pm_arch_registrar { explicit pm_arch_registrar(const pm_arch_entry & e); };
