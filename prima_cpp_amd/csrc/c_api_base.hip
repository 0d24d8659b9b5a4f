// c_api_base.hip — the part of the extern "C" surface that every build of the library has: errors, devices, streams, events, memory.
#include "../../include/prima_mi355.h"
#include "pm355_device.h"
#include "pm355_kernels.h"
#include <stdio.h>
#include <string.h>
#include <atomic>
#include <mutex>

static thread_local char g_err[256] = "";
int pm_api_fail(int code, const char * what, hipError_t e) {
    snprintf(g_err, sizeof(g_err), "%s%s%s", what, e != hipSuccess ? ": " : "", e != hipSuccess ? hipGetErrorString(e) : "");
    return code;
}
#define HIP_TRY(expr) do { hipError_t e_ = (expr); if (e_ != hipSuccess) return pm_api_fail(PM355_E_HIP, #expr, e_); } while (0)
static inline hipStream_t S(pm355_stream_t s) { return (hipStream_t) s; }

extern "C" {

const char * pm355_version(void) { return "prima_mi355 0.1 (gfx950)"; }
const char * pm355_last_error(void) { return g_err; }

int pm355_device_count(void) { int n = 0; return hipGetDeviceCount(&n) == hipSuccess ? n : 0; }
int pm355_set_device(int d) { HIP_TRY(hipSetDevice(d)); return 0; }
int pm355_device_info(int d, char * name, size_t name_len, size_t * free_b, size_t * total_b, int * cus) {
    hipDeviceProp_t p;
    HIP_TRY(hipGetDeviceProperties(&p, d));
    if (name && name_len) { strncpy(name, p.name, name_len - 1); name[name_len - 1] = 0; }
    if (cus) *cus = p.multiProcessorCount;
    if (free_b || total_b) {
        int cur = 0; hipGetDevice(&cur); hipSetDevice(d);
        size_t f = 0, t = 0; hipError_t e = hipMemGetInfo(&f, &t); hipSetDevice(cur);
        if (e != hipSuccess) return pm_api_fail(PM355_E_HIP, "hipMemGetInfo", e);
        if (free_b) *free_b = f;
        if (total_b) *total_b = t;
    }
    return 0;
}
// Is `p` page-locked host memory? Asked for every small upload of a token (positions, mask, ...). Only POSITIVE verdicts are cached (per 4 KiB page,
// direct-mapped, flushed whenever this library allocates or frees pinned memory itself - pm355_host_malloc / pm355_host_free, the plug-in's host
// buffer type): a stale "pinned" costs one wait, but a cached "pageable" for a page somebody pins later (hipHostRegister, another library's pinned
// allocator) would let set_tensor return while the DMA still reads the source - pageable pages ask the runtime every time.
namespace { struct PinE { uintptr_t page; }; PinE g_pin[256] = {}; std::atomic<unsigned> g_pin_gen{1}; unsigned g_pin_seen = 0; std::mutex g_pin_mu; }
int pm355_host_is_pinned(const void * p) {
    const uintptr_t page = ((uintptr_t) p >> 12) + 1;                 // (+1: 0 marks an empty slot)
    {
        std::lock_guard<std::mutex> lk(g_pin_mu);
        const unsigned gen = g_pin_gen.load(std::memory_order_acquire);
        if (gen != g_pin_seen) { memset(g_pin, 0, sizeof(g_pin)); g_pin_seen = gen; }
        if (g_pin[page & 255].page == page) return 1;
    }
    const unsigned gen0 = g_pin_gen.load(std::memory_order_acquire);
    hipPointerAttribute_t a;
    int pinned = 0;
    if (hipPointerGetAttributes(&a, p) != hipSuccess) (void) hipGetLastError();                   // unknown to the runtime: pageable
    else pinned = a.type == hipMemoryTypeHost ? 1 : 0;
    if (pinned) {
        std::lock_guard<std::mutex> lk(g_pin_mu);
        if (g_pin_gen.load(std::memory_order_acquire) == gen0 && g_pin_seen == gen0) g_pin[page & 255].page = page;   // (an allocation raced the query: do not cache)
    }
    return pinned;
}
int pm355_sync_null_stream(void) { HIP_TRY(hipStreamSynchronize(nullptr)); return 0; }
int pm355_sync(pm355_stream_t s) { HIP_TRY(s ? hipStreamSynchronize(S(s)) : hipDeviceSynchronize()); return 0; }

pm355_stream_t pm355_stream_create(void) { hipStream_t s = nullptr; return hipStreamCreateWithFlags(&s, hipStreamNonBlocking) == hipSuccess ? (pm355_stream_t) s : nullptr; }
void pm355_stream_destroy(pm355_stream_t s) { if (s) (void) hipStreamDestroy(S(s)); }
pm355_event_t pm355_event_create(void) { hipEvent_t e = nullptr; return hipEventCreateWithFlags(&e, hipEventDisableTiming) == hipSuccess ? (pm355_event_t) e : nullptr; }
void pm355_event_destroy(pm355_event_t e) { if (e) (void) hipEventDestroy((hipEvent_t) e); }
int pm355_event_record(pm355_event_t e, pm355_stream_t s) { HIP_TRY(hipEventRecord((hipEvent_t) e, S(s))); return 0; }
int pm355_event_wait(pm355_stream_t s, pm355_event_t e) { HIP_TRY(hipStreamWaitEvent(S(s), (hipEvent_t) e, 0)); return 0; }
int pm355_event_sync(pm355_event_t e) { HIP_TRY(hipEventSynchronize((hipEvent_t) e)); return 0; }

void * pm355_malloc(size_t n) { void * p = nullptr; return hipMalloc(&p, n) == hipSuccess ? p : nullptr; }
void   pm355_free(void * p) { if (p) (void) hipFree(p); }
// (the generation moves AFTER the runtime has changed the status of the pages: a query that overlaps the call re-asks the runtime next time)
void * pm355_host_malloc(size_t n) { void * p = nullptr; const bool ok = hipHostMalloc(&p, n, hipHostMallocDefault) == hipSuccess; g_pin_gen.fetch_add(1, std::memory_order_release); return ok ? p : nullptr; }
void   pm355_host_free(void * p) { if (p) (void) hipHostFree(p); g_pin_gen.fetch_add(1, std::memory_order_release); }
int pm355_memcpy_h2d(void * d, const void * s, size_t n, pm355_stream_t st) { HIP_TRY(hipMemcpyAsync(d, s, n, hipMemcpyHostToDevice, S(st))); return 0; }
int pm355_memcpy_d2h(void * d, const void * s, size_t n, pm355_stream_t st) { HIP_TRY(hipMemcpyAsync(d, s, n, hipMemcpyDeviceToHost, S(st))); return 0; }
int pm355_memcpy_d2d(void * d, const void * s, size_t n, pm355_stream_t st) { HIP_TRY(hipMemcpyAsync(d, s, n, hipMemcpyDeviceToDevice, S(st))); return 0; }
int pm355_memset(void * d, int v, size_t n, pm355_stream_t st) { HIP_TRY(hipMemsetAsync(d, v, n, S(st))); return 0; }

} // extern "C"
