// The library's per-device state, its error reporting, and the entry points of the C ABI that concern memory and
// streams alone (argument checks and status codes as in capi.hip).
#include "runtime.h"

#include <cstdarg>
#include <cstdio>
#include <cstring>

#include "kernels.h"

namespace mimir {

namespace {
thread_local std::string g_last_error;
// In host code the array's name is only a handle for the lookup in current_state, never an address.
static __device__ __align__(256) unsigned char g_noalloc_scratch[kNoallocScratchBytes];
}  // namespace

std::mutex g_mu;
DeviceState g_dev[kMaxDevices];
thread_local char t_last_kernel[160] = "";
thread_local std::vector<hipEvent_t> t_events;
thread_local size_t t_events_used = 0;

mi355x_status capi_fail(mi355x_status code, const char* fmt, ...) {
    char buf[512];
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(buf, sizeof buf, fmt, ap);
    va_end(ap);
    g_last_error = buf;
    return code;
}

mi355x_status hip_fail(hipError_t e, const char* what) {
    return capi_fail((mi355x_status)e, "mi355x: %s: %s", what, hipGetErrorName(e));
}

void note_kernel(const char* fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(t_last_kernel, sizeof t_last_kernel, fmt, ap);
    va_end(ap);
}
bool next_timing_events(hipEvent_t* start, hipEvent_t* stop) {
    if (t_events_used + 2 > t_events.size()) return false;
    *start = t_events[t_events_used];
    *stop = t_events[t_events_used + 1];
    t_events_used += 2;
    return true;
}

mi355x_status current_state(DeviceState** out) {
    int dev = 0;
    HIP_TRY(hipGetDevice(&dev), "hipGetDevice");
    if (dev < 0 || dev >= kMaxDevices) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: device %d out of range", dev);
    std::lock_guard<std::mutex> lock(g_mu);
    DeviceState& s = g_dev[dev];
    if (!s.ready) {
        hipDeviceProp_t prop;
        HIP_TRY(hipGetDeviceProperties(&prop, dev), "hipGetDeviceProperties");
        if (strncmp(prop.gcnArchName, "gfx950", 6) != 0)
            return capi_fail(MI355X_ERR_INTERNAL, "mi355x: device %d is %s; this library holds gfx950 code only", dev, prop.gcnArchName);
        // the lookup first: if it fails nothing has been allocated that a later call would allocate again
        HIP_TRY(hipGetSymbolAddress(&s.fixed, HIP_SYMBOL(g_noalloc_scratch)), "hipGetSymbolAddress(fixed scratch)");
        if (!s.err_dev) {
            HIP_TRY(hipMalloc((void**)&s.err_dev, 256), "hipMalloc(error word)");
            HIP_TRY(hipMemset(s.err_dev, 0, 256), "hipMemset(error word)");
        }
        if (!s.err_host) HIP_TRY(hipHostMalloc((void**)&s.err_host, 256, hipHostMallocDefault), "hipHostMalloc(error word)");
        s.ready = true;
    }
    *out = &s;
    return MI355X_OK;
}

uint32_t* device_error_word() {
    DeviceState* s;
    return current_state(&s) == MI355X_OK ? s->err_dev : nullptr;
}

}  // namespace mimir

using namespace mimir;

extern "C" {

mi355x_status mi355x_init(int device) {
    int n = 0;
    HIP_TRY(hipGetDeviceCount(&n), "hipGetDeviceCount");
    if (device < 0 || device >= n) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: device %d of %d", device, n);
    HIP_TRY(hipSetDevice(device), "hipSetDevice");
    DeviceState* s;
    return current_state(&s);
}

size_t mi355x_last_error(char* buf, size_t n) {
    if (buf && n) {
        size_t c = g_last_error.size() < n - 1 ? g_last_error.size() : n - 1;
        memcpy(buf, g_last_error.data(), c);
        buf[c] = 0;
    }
    return g_last_error.size();
}

int mi355x_block_size(int dtype) { return block_size(dtype); }
int mi355x_block_bytes(int dtype) { return block_bytes(dtype); }

int64_t mi355x_bytes(int dtype, int64_t n) {
    int bs = block_size(dtype), bb = block_bytes(dtype);
    if (bb == 0 || n < 0 || n % bs != 0 || n / bs > INT64_MAX / bb) return -1;
    return n / bs * bb;
}

mi355x_status mi355x_alloc(void** out, size_t bytes) {
    if (!out) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: alloc: null result pointer");
    *out = nullptr;
    // at least 4 bytes, as the reference's Alloc (backend/rocm/rocm_linux.go:220-240)
    hipError_t e = hipMalloc(out, bytes < 4 ? 4 : bytes);
    if (e != hipSuccess) return hip_fail(e, "hipMalloc");
    return MI355X_OK;
}

mi355x_status mi355x_free(void* ptr) {
    if (!ptr) return MI355X_OK;
    HIP_TRY(hipFree(ptr), "hipFree");
    return MI355X_OK;
}

mi355x_status mi355x_upload(void* dst, const void* src, size_t bytes, void* stream) {
    if (bytes == 0) return MI355X_OK;
    if (!dst || !src) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: upload: null pointer");
    HIP_TRY(hipMemcpyAsync(dst, src, bytes, hipMemcpyHostToDevice, (hipStream_t)stream), "hipMemcpyAsync(H2D)");
    return MI355X_OK;
}

mi355x_status mi355x_download(void* dst, const void* src, size_t bytes, void* stream) {
    if (bytes == 0) return MI355X_OK;
    if (!dst || !src) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: download: null pointer");
    HIP_TRY(hipMemcpyAsync(dst, src, bytes, hipMemcpyDeviceToHost, (hipStream_t)stream), "hipMemcpyAsync(D2H)");
    HIP_TRY(hipStreamSynchronize((hipStream_t)stream), "hipStreamSynchronize");
    return MI355X_OK;
}

mi355x_status mi355x_sync(void* stream) {
    DeviceState* s;
    if (mi355x_status st = current_state(&s)) return st;
    HIP_TRY(hipMemcpyAsync(s->err_host, s->err_dev, 4, hipMemcpyDeviceToHost, (hipStream_t)stream), "hipMemcpyAsync(error word)");
    HIP_TRY(hipStreamSynchronize((hipStream_t)stream), "hipStreamSynchronize");
    uint32_t bits = *s->err_host;
    if (bits) {
        HIP_TRY(hipMemsetAsync(s->err_dev, 0, 4, (hipStream_t)stream), "hipMemsetAsync(error word)");
        HIP_TRY(hipStreamSynchronize((hipStream_t)stream), "hipStreamSynchronize");
        if (bits & kErrIndex) return capi_fail(MI355X_ERR_INDEX, "mi355x: a gather read an index out of range");
        return capi_fail(MI355X_ERR_INTERNAL, "mi355x: device error bits %#x", bits);
    }
    return MI355X_OK;
}

}  // extern "C"
