// Context, error reporting, per-thread staging.
#include <atomic>
#include <mutex>
#include <vector>

#include "rmi_internal.h"

namespace {

thread_local char t_error[512] = "";
int g_device = -1;
int g_cus = 0;
size_t g_hbm = 0;
char g_name[128] = "";
std::mutex g_mutex;
// Every context ever made; shutdown empties them (stream and buffers) and leaves the objects, whose owning
// threads may still hold the pointer.  g_generation counts shutdowns: a context of an older generation has no
// stream any more and is rebuilt on its owner's next call.
std::vector<RmiThreadCtx *> g_ctxs;
std::vector<RmiThreadCtx *> g_idle;  // contexts of threads that have exited, handed to the next new thread
std::atomic<uint64_t> g_generation{1};

// The calling thread's context.  When the thread exits its context goes to the idle list, buffers and all, for
// the next thread that needs one: no HIP call runs inside a thread-exit destructor, and a pool that keeps
// starting and ending threads holds as many contexts as it has threads at once, not as many as it ever had.
struct ThreadSlot {
    RmiThreadCtx *c = nullptr;
    ~ThreadSlot() {
        if (!c) return;
        std::lock_guard<std::mutex> lock(g_mutex);
        g_idle.push_back(c);
    }
};
thread_local ThreadSlot t_slot;

}  // namespace

void rmi_set_error(const char *fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(t_error, sizeof(t_error), fmt, ap);
    va_end(ap);
}

int rmi_fail(int code, const char *fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(t_error, sizeof(t_error), fmt, ap);
    va_end(ap);
    return code;
}

bool rmi_ready() { return g_device >= 0; }
int rmi_device_cus() { return g_cus; }
int rmi_device() { return g_device; }

RmiThreadCtx *rmi_thread_ctx() {
    const uint64_t generation = g_generation.load(std::memory_order_acquire);
    RmiThreadCtx *c = t_slot.c;
    if (c && c->generation == generation && c->stream) return c;
    if (hipSetDevice(g_device) != hipSuccess) {
        rmi_set_error("hipSetDevice(%d) failed", g_device);
        return nullptr;
    }
    bool fresh = false;
    if (!c) {
        std::lock_guard<std::mutex> lock(g_mutex);
        if (!g_idle.empty()) {
            c = g_idle.back();
            g_idle.pop_back();
        }
    }
    if (!c) {
        c = new RmiThreadCtx();
        fresh = true;
    }
    if (c->generation != generation || !c->stream) {
        // new, or emptied by a shutdown since its last use: shutdown left no stream and no buffers behind
        c->stream = nullptr;
        // default priority: mixed-priority streams are not used anywhere
        if (hipStreamCreateWithFlags(&c->stream, hipStreamNonBlocking) != hipSuccess) {
            rmi_set_error("hipStreamCreate failed");
            c->stream = nullptr;
            if (fresh) delete c;
            else {
                std::lock_guard<std::mutex> lock(g_mutex);
                g_idle.push_back(c);
            }
            t_slot.c = nullptr;
            return nullptr;
        }
        c->generation = generation;
    }
    if (fresh) {
        std::lock_guard<std::mutex> lock(g_mutex);
        g_ctxs.push_back(c);
    }
    t_slot.c = c;
    return c;
}

void *rmi_dev_buf(RmiThreadCtx *c, int slot, size_t nbytes) {
    if (nbytes == 0) nbytes = 16;
    if (c->dev_cap[slot] >= nbytes) return c->dev[slot];
    if (c->dev[slot]) {
        // the stream may still read the old buffer
        (void)hipStreamSynchronize(c->stream);
        (void)hipFree(c->dev[slot]);
        c->dev[slot] = nullptr;
        c->dev_cap[slot] = 0;
    }
    size_t cap = (nbytes + 4095) & ~size_t(4095);
    if (hipMalloc(&c->dev[slot], cap) != hipSuccess) {
        rmi_set_error("hipMalloc(%zu) for staging failed", cap);
        return nullptr;
    }
    c->dev_cap[slot] = cap;
    return c->dev[slot];
}

void *rmi_pin_buf(RmiThreadCtx *c, int slot, size_t nbytes) {
    if (nbytes == 0) nbytes = 16;
    if (c->pin_cap[slot] >= nbytes) return c->pin[slot];
    if (c->pin[slot]) {
        (void)hipStreamSynchronize(c->stream);
        (void)hipHostFree(c->pin[slot]);
        c->pin[slot] = nullptr;
        c->pin_cap[slot] = 0;
    }
    size_t cap = (nbytes + 4095) & ~size_t(4095);
    if (hipHostMalloc(&c->pin[slot], cap, hipHostMallocDefault) != hipSuccess) {
        rmi_set_error("hipHostMalloc(%zu) for staging failed", cap);
        return nullptr;
    }
    c->pin_cap[slot] = cap;
    return c->pin[slot];
}

// How the forward_batched entry points of the Kernel trait multiply more than one token; process-wide, read at each call.
static std::atomic<int> g_batched_mode{RMI_HIP_BATCHED_X86_ORDER};
int rmi_batched_mode() { return g_batched_mode.load(std::memory_order_relaxed); }

extern "C" {

const char *rmi_hip_last_error(void) { return t_error; }

int rmi_hip_init(int device) {
    std::lock_guard<std::mutex> lock(g_mutex);
    if (g_device >= 0) {
        if (g_device == device) return RMI_HIP_OK;
        return rmi_fail(RMI_HIP_E_INVALID, "already initialised on device %d", g_device);
    }
    int count = 0;
    hipError_t e = hipGetDeviceCount(&count);
    if (e != hipSuccess || count == 0)
        return rmi_fail(RMI_HIP_E_NO_DEVICE, "no HIP device visible (%s)", e == hipSuccess ? "count is 0" : hipGetErrorString(e));
    if (device < 0 || device >= count) return rmi_fail(RMI_HIP_E_INVALID, "device %d out of range (have %d)", device, count);
    hipDeviceProp_t prop;
    RMI_HIP_CHECK(hipGetDeviceProperties(&prop, device));
    if (strncmp(prop.gcnArchName, "gfx950", 6) != 0)
        return rmi_fail(RMI_HIP_E_NO_DEVICE, "device %d is %s; this library holds gfx950 code only", device, prop.gcnArchName);
    RMI_HIP_CHECK(hipSetDevice(device));
    if (rmi_noalloc_setup) {  // absent from a library without the no-allocation entry points
        const int rc = rmi_noalloc_setup(device);
        if (rc != RMI_HIP_OK) return rc;
    }
    g_cus = prop.multiProcessorCount;
    g_hbm = prop.totalGlobalMem;
    snprintf(g_name, sizeof(g_name), "%s (%s)", prop.name, prop.gcnArchName);
    g_device = device;
    return RMI_HIP_OK;
}

void rmi_hip_shutdown(void) {
    std::lock_guard<std::mutex> lock(g_mutex);
    if (g_device < 0) return;
    (void)hipDeviceSynchronize();
    for (RmiThreadCtx *c : g_ctxs) {
        for (int i = 0; i < 6; i++) {
            if (c->dev[i]) (void)hipFree(c->dev[i]);
            if (c->pin[i]) (void)hipHostFree(c->pin[i]);
            c->dev[i] = nullptr;
            c->pin[i] = nullptr;
            c->dev_cap[i] = c->pin_cap[i] = 0;
        }
        for (int i = 0; i < 2; i++) {
            if (c->up_pin[i]) (void)hipHostFree(c->up_pin[i]);
            if (c->up_dev[i]) (void)hipFree(c->up_dev[i]);
            if (c->up_done[i]) (void)hipEventDestroy(c->up_done[i]);
            c->up_pin[i] = c->up_dev[i] = nullptr;
            c->up_done[i] = nullptr;
        }
        c->up_cap = 0;
        if (c->stream) (void)hipStreamDestroy(c->stream);
        c->stream = nullptr;
    }
    // contexts stay allocated: their owning threads may still hold the pointer; the new generation tells them
    // that stream and buffers are gone
    g_generation.fetch_add(1, std::memory_order_acq_rel);
    g_device = -1;
}

int rmi_hip_set_forward_batched_mode(int mode) {
    if (mode != RMI_HIP_BATCHED_X86_ORDER && mode != RMI_HIP_BATCHED_AARCH64_ORDER && mode != RMI_HIP_BATCHED_FAST)
        return rmi_fail(RMI_HIP_E_INVALID, "unknown forward_batched mode %d", mode);
    g_batched_mode.store(mode, std::memory_order_relaxed);
    return RMI_HIP_OK;
}

int rmi_hip_get_forward_batched_mode(void) { return rmi_batched_mode(); }

size_t rmi_hip_thread_context_count(void) {
    std::lock_guard<std::mutex> lock(g_mutex);
    return g_ctxs.size();
}

int rmi_hip_device_info(char *name, size_t name_len, int *compute_units, size_t *hbm_bytes) {
    RMI_REQUIRE_INIT();
    if (name && name_len) snprintf(name, name_len, "%s", g_name);
    if (compute_units) *compute_units = g_cus;
    if (hbm_bytes) *hbm_bytes = g_hbm;
    return RMI_HIP_OK;
}

void *rmi_hip_malloc(size_t nbytes) {
    if (!rmi_ready()) {
        rmi_set_error("rmi_hip_init has not succeeded");
        return nullptr;
    }
    if (!rmi_thread_ctx()) return nullptr;
    void *p = nullptr;
    hipError_t e = hipMalloc(&p, nbytes ? nbytes : 16);
    if (e != hipSuccess) {
        rmi_set_error("hipMalloc(%zu) failed: %s", nbytes, hipGetErrorString(e));
        return nullptr;
    }
    return p;
}

void rmi_hip_free(void *dptr) {
    if (dptr) (void)hipFree(dptr);
}

int rmi_hip_memcpy_h2d(void *dst, const void *src, size_t nbytes) {
    RMI_REQUIRE_INIT();
    if (!rmi_thread_ctx()) return RMI_HIP_E_RUNTIME;
    RMI_HIP_CHECK(hipMemcpy(dst, src, nbytes, hipMemcpyHostToDevice));
    return RMI_HIP_OK;
}

int rmi_hip_memcpy_d2h(void *dst, const void *src, size_t nbytes) {
    RMI_REQUIRE_INIT();
    if (!rmi_thread_ctx()) return RMI_HIP_E_RUNTIME;
    RMI_HIP_CHECK(hipMemcpy(dst, src, nbytes, hipMemcpyDeviceToHost));
    return RMI_HIP_OK;
}

int rmi_hip_synchronize(void) {
    RMI_REQUIRE_INIT();
    if (!rmi_thread_ctx()) return RMI_HIP_E_RUNTIME;
    RMI_HIP_CHECK(hipDeviceSynchronize());
    return RMI_HIP_OK;
}

}  // extern "C"
