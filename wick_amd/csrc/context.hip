// Context, device buffers, graph capture / replay, events and per-dispatch timing of the C ABI (include/wick_rocm.h): what every
// model and every operation of the library needs, whatever its weights look like.  Host code only.
#include "../../include/wick_rocm.h"

#include <hip/hip_runtime.h>

#include <cstdio>
#include <cstring>
#include <mutex>
#include <new>
#include <string>

#include "wick_rocm_ctx.h"

// Scratch of wick_rocm_matmul_f32_noalloc: the Q8_0-quantized activations (quants, then scales) of one call, in
// device memory that exists from load time on, one copy per GPU.  `scratch` is a host-side stand-in for the symbol, not a
// device address: host code only ever uses the address hipGetSymbolAddress returns for the current device
// (wick_rocm_ctx::noalloc_scratch, looked up in wick_rocm_ctx_create).
static __device__ __align__(256) unsigned char scratch[kNoallocScratchBytes];

namespace {

// Every context on a GPU shares that GPU's one array, and nothing orders the streams of two contexts.  The host therefore
// keeps, per device, the context whose calls (or graph replays of them) may still be using the array: a call from another
// context is refused until the owner has synchronised (wick_rocm_sync, a download, destruction), which is when its work on
// the array is known to have finished.
constexpr int kNoallocMaxDevices = 64;
std::mutex g_noalloc_mu;
wick_rocm_ctx* g_noalloc_owner[kNoallocMaxDevices] = {};

}  // namespace

int noalloc_claim(wick_rocm_ctx* ctx) {
    if (ctx->device < 0 || ctx->device >= kNoallocMaxDevices) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "matmul_f32_noalloc: device index out of range");
    std::lock_guard<std::mutex> lk(g_noalloc_mu);
    wick_rocm_ctx*& owner = g_noalloc_owner[ctx->device];
    if (owner && owner != ctx)
        return fail(ctx, WICK_ROCM_ERR_STATE, "matmul_f32_noalloc: another context's work on this GPU's static scratch may still be in flight; "
                                              "wick_rocm_sync that context first");
    owner = ctx;
    return WICK_ROCM_OK;
}

// The context's stream has drained (or the context goes away): whatever it enqueued on the array has finished.
void noalloc_release(wick_rocm_ctx* ctx) {
    if (ctx->device < 0 || ctx->device >= kNoallocMaxDevices) return;
    std::lock_guard<std::mutex> lk(g_noalloc_mu);
    if (g_noalloc_owner[ctx->device] == ctx) g_noalloc_owner[ctx->device] = nullptr;
}

extern "C" {

const char* wick_rocm_version(void) { return "wick-rocm 0.1 (gfx950)"; }

int wick_rocm_device_count(int* count) {
    if (!count) return WICK_ROCM_ERR_INVALID_ARG;
    int c = 0;
    hipError_t e = hipGetDeviceCount(&c);
    if (e != hipSuccess) {
        *count = 0;
        return e == hipErrorNoDevice ? WICK_ROCM_OK : WICK_ROCM_ERR_HIP;
    }
    *count = c;
    return WICK_ROCM_OK;
}

int wick_rocm_ctx_create(int device_id, wick_rocm_ctx** out) {
    if (!out) return WICK_ROCM_ERR_INVALID_ARG;
    *out = nullptr;
    int count = 0;
    if (hipGetDeviceCount(&count) != hipSuccess || device_id < 0 || device_id >= count) return WICK_ROCM_ERR_NO_DEVICE;
    hipDeviceProp_t prop;
    if (hipGetDeviceProperties(&prop, device_id) != hipSuccess) return WICK_ROCM_ERR_HIP;
    // The kernels are built for gfx950 only; refuse anything else up front instead
    // of failing at the first launch.
    if (std::strncmp(prop.gcnArchName, "gfx950", 6) != 0) return WICK_ROCM_ERR_NO_DEVICE;
    wick_rocm_ctx* ctx = new (std::nothrow) wick_rocm_ctx();
    if (!ctx) return WICK_ROCM_ERR_HIP;
    ctx->device = device_id;
    ctx->name = std::string(prop.gcnArchName) + " " + prop.name;
    ctx->num_cus = prop.multiProcessorCount;
    ctx->hbm_bytes = prop.totalGlobalMem;
    if (hipSetDevice(device_id) != hipSuccess || hipStreamCreateWithFlags(&ctx->stream, hipStreamNonBlocking) != hipSuccess) {
        delete ctx;
        return WICK_ROCM_ERR_HIP;
    }
    // This device's copy of the static scratch array (every GPU has its own, at its own address); the device is current.
    void* sym = nullptr;
    if (hipGetSymbolAddress(&sym, HIP_SYMBOL(scratch)) != hipSuccess || !sym) {
        (void)hipStreamDestroy(ctx->stream);
        delete ctx;
        return WICK_ROCM_ERR_HIP;
    }
    ctx->noalloc_scratch = static_cast<unsigned char*>(sym);
    *out = ctx;
    return WICK_ROCM_OK;
}

void wick_rocm_ctx_destroy(wick_rocm_ctx* ctx) {
    if (!ctx) return;
    {
        Guard g(ctx);
        if (ctx->stream) {
            (void)hipStreamSynchronize(ctx->stream);
            (void)hipStreamDestroy(ctx->stream);
        }
        noalloc_release(ctx);
        if (ctx->scratch_q) (void)hipFree(ctx->scratch_q);
        if (ctx->scratch_s) (void)hipFree(ctx->scratch_s);
        if (ctx->scratch_f) (void)hipFree(ctx->scratch_f);
        if (ctx->argmax_partial) (void)hipFree(ctx->argmax_partial);
        for (auto* v : {&ctx->timer.recs, &ctx->timer.spares})
            for (KernelTimer::Rec& r : *v) {
                (void)hipEventDestroy(r.start);
                (void)hipEventDestroy(r.stop);
            }
    }
    delete ctx;
}

int wick_rocm_last_error(wick_rocm_ctx* ctx, char* buf, size_t buf_len) {
    if (!ctx || !buf || buf_len == 0) return WICK_ROCM_ERR_INVALID_ARG;
    std::lock_guard<std::recursive_mutex> lk(ctx->mu);
    std::snprintf(buf, buf_len, "%s", ctx->err.c_str());
    return WICK_ROCM_OK;
}

int wick_rocm_device_info(wick_rocm_ctx* ctx, char* name_buf, size_t name_len, int* compute_units, size_t* hbm_bytes) {
    if (!ctx) return WICK_ROCM_ERR_INVALID_ARG;
    std::lock_guard<std::recursive_mutex> lk(ctx->mu);
    if (name_buf && name_len) std::snprintf(name_buf, name_len, "%s", ctx->name.c_str());
    if (compute_units) *compute_units = ctx->num_cus;
    if (hbm_bytes) *hbm_bytes = ctx->hbm_bytes;
    return WICK_ROCM_OK;
}

void* wick_rocm_ctx_stream(wick_rocm_ctx* ctx) { return ctx ? static_cast<void*>(ctx->stream) : nullptr; }

int wick_rocm_buffer_alloc(wick_rocm_ctx* ctx, size_t nbytes, void** d_ptr) {
    WR_ENTER(ctx);
    if (!d_ptr || nbytes == 0) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "buffer_alloc: null out pointer or zero size");
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "buffer_alloc during graph capture");
    *d_ptr = nullptr;
    WR_HIP(ctx, hipMalloc(d_ptr, nbytes));
    return WICK_ROCM_OK;
}

int wick_rocm_buffer_free(wick_rocm_ctx* ctx, void* d_ptr) {
    WR_ENTER(ctx);
    if (!d_ptr) return WICK_ROCM_OK;
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "buffer_free during graph capture");
    WR_HIP(ctx, hipStreamSynchronize(ctx->stream));
    WR_HIP(ctx, hipFree(d_ptr));
    return WICK_ROCM_OK;
}

int wick_rocm_upload(wick_rocm_ctx* ctx, void* d_dst, const void* src, size_t nbytes) {
    WR_ENTER(ctx);
    if (nbytes == 0) return WICK_ROCM_OK;
    if (!d_dst || !src) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "upload: null pointer");
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "upload during graph capture");
    WR_HIP(ctx, hipMemcpyAsync(d_dst, src, nbytes, hipMemcpyHostToDevice, ctx->stream));
    WR_HIP(ctx, hipStreamSynchronize(ctx->stream));  // the host buffer may be reused on return
    return WICK_ROCM_OK;
}

int wick_rocm_download(wick_rocm_ctx* ctx, void* dst, const void* d_src, size_t nbytes) {
    WR_ENTER(ctx);
    if (nbytes == 0) return WICK_ROCM_OK;
    if (!dst || !d_src) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "download: null pointer");
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "download during graph capture");
    WR_HIP(ctx, hipMemcpyAsync(dst, d_src, nbytes, hipMemcpyDeviceToHost, ctx->stream));
    WR_HIP(ctx, hipStreamSynchronize(ctx->stream));
    noalloc_release(ctx);
    return WICK_ROCM_OK;
}

int wick_rocm_sync(wick_rocm_ctx* ctx) {
    WR_ENTER(ctx);
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "sync during graph capture");
    WR_HIP(ctx, hipStreamSynchronize(ctx->stream));
    noalloc_release(ctx);
    return WICK_ROCM_OK;
}
int wick_rocm_graph_begin(wick_rocm_ctx* ctx) {
    WR_ENTER(ctx);
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "graph_begin: capture already in progress");
    if (ctx->timer.enabled) return fail(ctx, WICK_ROCM_ERR_STATE, "graph_begin: kernel timing is on");
    WR_HIP(ctx, hipStreamBeginCapture(ctx->stream, hipStreamCaptureModeThreadLocal));
    ctx->capturing = true;
    ctx->capture_used_scratch = 0;
    ctx->capture_used_noalloc = false;
    return WICK_ROCM_OK;
}

int wick_rocm_graph_end(wick_rocm_ctx* ctx, wick_rocm_graph** out) {
    WR_ENTER(ctx);
    if (!out) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "graph_end: null out pointer");
    *out = nullptr;
    if (!ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "graph_end: no capture in progress");
    // the capture ends whatever happens next, so that no failure leaves the stream capturing
    ctx->capturing = false;
    hipGraph_t graph = nullptr;
    hipError_t e = hipStreamEndCapture(ctx->stream, &graph);
    wick_rocm_graph* g = e == hipSuccess ? new (std::nothrow) wick_rocm_graph() : nullptr;
    if (e == hipSuccess && !g) {
        (void)hipGraphDestroy(graph);
        return fail(ctx, WICK_ROCM_ERR_HIP, "out of host memory");
    }
    if (e == hipSuccess) {
        g->graph = graph;
        e = hipGraphInstantiate(&g->exec, g->graph, nullptr, nullptr, 0);
    }
    if (e != hipSuccess) {
        if (graph) (void)hipGraphDestroy(graph);
        delete g;
        return fail_hip(ctx, e, "graph_end");
    }
    g->uses_scratch = ctx->capture_used_scratch;
    for (int i = 0; i < 3; i++) g->scratch_gen[i] = ctx->scratch_gen[i];
    g->uses_noalloc = ctx->capture_used_noalloc;
    *out = g;
    return WICK_ROCM_OK;
}

int wick_rocm_graph_launch(wick_rocm_ctx* ctx, wick_rocm_graph* g) {
    WR_ENTER(ctx);
    if (!g || !g->exec) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "graph_launch: null graph");
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "graph_launch during capture");
    if (graph_is_stale(ctx, g))
        return fail(ctx, WICK_ROCM_ERR_STATE, "graph_launch: the context's scratch was regrown after this graph was captured (it holds freed addresses); "
                                              "capture it again, and size the scratch with wick_rocm_reserve_scratch before capturing");
    if (g->uses_noalloc)
        if (int rc = noalloc_claim(ctx)) return rc;
    WR_HIP(ctx, hipGraphLaunch(g->exec, ctx->stream));
    return WICK_ROCM_OK;
}

int wick_rocm_graph_destroy(wick_rocm_ctx* ctx, wick_rocm_graph* g) {
    WR_ENTER(ctx);
    if (!g) return WICK_ROCM_OK;
    WR_HIP(ctx, hipStreamSynchronize(ctx->stream));
    if (g->exec) (void)hipGraphExecDestroy(g->exec);
    if (g->graph) (void)hipGraphDestroy(g->graph);
    delete g;
    return WICK_ROCM_OK;
}

int wick_rocm_event_create(wick_rocm_ctx* ctx, wick_rocm_event** out) {
    WR_ENTER(ctx);
    if (!out) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "event_create: null out pointer");
    wick_rocm_event* e = new (std::nothrow) wick_rocm_event();
    if (!e) return fail(ctx, WICK_ROCM_ERR_HIP, "out of host memory");
    hipError_t he = hipEventCreate(&e->ev);
    if (he != hipSuccess) {
        delete e;
        return fail_hip(ctx, he, "hipEventCreate");
    }
    *out = e;
    return WICK_ROCM_OK;
}

int wick_rocm_event_record(wick_rocm_ctx* ctx, wick_rocm_event* e) {
    WR_ENTER(ctx);
    if (!e) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "event_record: null event");
    WR_HIP(ctx, hipEventRecord(e->ev, ctx->stream));
    return WICK_ROCM_OK;
}

int wick_rocm_event_elapsed_ms(wick_rocm_ctx* ctx, wick_rocm_event* start, wick_rocm_event* stop, float* ms) {
    WR_ENTER(ctx);
    if (!start || !stop || !ms) return fail(ctx, WICK_ROCM_ERR_INVALID_ARG, "event_elapsed_ms: null argument");
    WR_HIP(ctx, hipEventSynchronize(stop->ev));
    WR_HIP(ctx, hipEventElapsedTime(ms, start->ev, stop->ev));
    return WICK_ROCM_OK;
}

int wick_rocm_kernel_timing_begin(wick_rocm_ctx* ctx) {
    WR_ENTER(ctx);
    if (ctx->capturing) return fail(ctx, WICK_ROCM_ERR_STATE, "kernel_timing_begin during graph capture");
    if (ctx->timer.enabled) return fail(ctx, WICK_ROCM_ERR_STATE, "kernel timing already on");
    ctx->timer.enabled = true;
    return WICK_ROCM_OK;
}

int wick_rocm_kernel_timing_end(wick_rocm_ctx* ctx, double* total_ms, uint64_t* launches, int n_families) {
    WR_ENTER(ctx);
    if (!ctx->timer.enabled) return fail(ctx, WICK_ROCM_ERR_STATE, "kernel timing is not on");
    ctx->timer.enabled = false;
    for (int f = 0; f < n_families; f++) {
        if (total_ms) total_ms[f] = 0.0;
        if (launches) launches[f] = 0;
    }
    hipError_t first = hipStreamSynchronize(ctx->stream);
    for (KernelTimer::Rec& r : ctx->timer.recs) {
        float ms = 0.f;
        hipError_t e = hipEventElapsedTime(&ms, r.start, r.stop);
        if (e != hipSuccess && first == hipSuccess) first = e;
        if (e == hipSuccess && r.family < n_families) {
            if (total_ms) total_ms[r.family] += (double)ms;
            if (launches) launches[r.family] += 1;
        }
        ctx->timer.spares.push_back(r);
    }
    ctx->timer.recs.clear();
    if (first != hipSuccess) return fail_hip(ctx, first, "kernel_timing_end");
    return WICK_ROCM_OK;
}

int wick_rocm_event_destroy(wick_rocm_ctx* ctx, wick_rocm_event* e) {
    WR_ENTER(ctx);
    if (!e) return WICK_ROCM_OK;
    (void)hipEventDestroy(e->ev);
    delete e;
    return WICK_ROCM_OK;
}

}  // extern "C"
