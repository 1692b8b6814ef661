// The library's per-device state and its error reporting: what every host file above the kernels' launchers shares.
#pragma once

#include "../../include/mimir_mi355x.h"

#include <hip/hip_runtime.h>

#include <map>
#include <mutex>
#include <string>
#include <vector>

namespace mimir {

// Sets the calling thread's message (mi355x_last_error) and returns the status.
mi355x_status capi_fail(mi355x_status code, const char* fmt, ...);
mi355x_status hip_fail(hipError_t e, const char* what);

#define HIP_TRY(expr, what)                         \
    do {                                            \
        hipError_t e_ = (expr);                     \
        if (e_ != hipSuccess) return mimir::hip_fail(e_, what); \
    } while (0)

constexpr int kMaxDevices = 16;

// The converted activations of mi355x_qgemv_noalloc: a fixed block in the code object's own
// device memory, so that the entry point allocates nothing. Every device the library runs on
// holds its own copy at its own address (DeviceState::fixed, looked up when the device's state
// is created).
constexpr size_t kNoallocScratchBytes = (size_t)1 << 20;

// Scratch memory of the entry points that need some beyond their arguments (converted activations,
// partial results and tickets of split attention and argmax, float32 copies of qgemm_bf16's general
// route). One set per device and stream: calls on different streams never share a block, calls on one
// stream are ordered by it. A block that has become too small is replaced by a larger one and kept
// aside: work already queued, and HIP graphs a caller has instantiated over an entry point, may still
// read and write it, tickets included (a graph keeps the block it was recorded with and stays valid).
// Growth at least doubles a block, so what is kept aside stays below the size of the live block.
// mi355x_stream_release frees everything a stream holds, live and kept aside.
struct ScratchBlock {
    void* p = nullptr;
    size_t bytes = 0;
};
struct StreamScratch {
    ScratchBlock act, attn, attn_flags, gemm, argmax;
    std::vector<void*> retired;  // outgrown blocks
};

// Per-device state: the error word kernels OR bits into, read back at sync.
struct DeviceState {
    bool ready = false;
    uint32_t* err_dev = nullptr;
    uint32_t* err_host = nullptr;  // pinned
    std::map<void*, StreamScratch> scratch;  // by stream handle
    void* fixed = nullptr;                   // this device's copy of the fixed block
};
extern std::mutex g_mu;
extern DeviceState g_dev[kMaxDevices];
mi355x_status current_state(DeviceState** out);

// The device error word of the current device (null if its state cannot be made).
uint32_t* device_error_word();

// Which kernel the calling thread launched last (mi355x_last_kernel), and the events of mi355x_timed_begin.
extern thread_local char t_last_kernel[160];
extern thread_local std::vector<hipEvent_t> t_events;
extern thread_local size_t t_events_used;

}  // namespace mimir
