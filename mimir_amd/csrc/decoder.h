// What the decoders behind a model handle (mi355x_model_*) have in common: device buffers and weights, the sequence
// position, the logits of a call, the greedy loop and its recorded step. A decoder brings its own layers: forward() for
// tokens the host supplies, step() for one position read from the device, and what they keep between calls.
#pragma once

#include "../../include/mimir_mi355x.h"

#include <hip/hip_runtime.h>

#include <cstdint>
#include <vector>

#include "kernels.h"
#include "runtime.h"

namespace mimir {

// `who` (a string) names the decoder in the message.
#define DECODER_HIP(expr, who, what)                                                 \
    do {                                                                             \
        hipError_t e_ = (expr);                                                      \
        if (e_ != hipSuccess) return capi_fail((mi355x_status)e_, "mi355x: %s: %s: %s", who, what, hipGetErrorName(e_)); \
    } while (0)

struct DevBuf {
    void* p = nullptr;
    size_t bytes = 0;
    bool view = false;  // p points into another buffer's memory
    DevBuf() = default;
    DevBuf(DevBuf&& o) noexcept : p(o.p), bytes(o.bytes), view(o.view) { o.p = nullptr; o.bytes = 0; o.view = false; }
    ~DevBuf() { release(); }
    void release() {
        if (p && !view) (void)hipFree(p);
        p = nullptr;
        view = false;
    }
    hipError_t alloc(size_t n) {
        release();
        bytes = n;
        return hipMalloc(&p, n < 4 ? 4 : n);
    }
    void point_at(void* q, size_t n) {
        release();
        p = q;
        bytes = n;
        view = true;
    }
    template <typename T>
    T* as() const { return (T*)p; }
};

struct Weight {
    int dtype = 0;
    int64_t n = 0, k = 0;
    DevBuf buf;
    bool set() const { return buf.p != nullptr; }
};

struct Decoder {
    // fixed when the handle is created
    const char* name = "model";  // in messages
    int vocab = 0, context = 0, batch = 1;

    bool ready = false;
    int64_t cache_len = 0;   // positions every sequence holds
    int64_t max_rows = 0;    // rows (batch x tokens) of one pass over the layers
    int64_t logit_rows = 0;  // rows of `logits`
    DevBuf tokens_dev, next_tok, logits, argmax_ws;
    // The decoding step as a fixed run of launches that read the position from the device: state = {position, steps
    // taken}; record holds the tokens chosen so far, [context + 1, batch]. step_graph replays the run.
    DevBuf state, record;
    hipStream_t stream = nullptr;
    hipGraphExec_t step_graph = nullptr;
    int graph_variant = 0;  // which step the graph holds (step_variant)

    virtual ~Decoder();

    // One tensor from host bytes, by the name it has in the model's file.
    virtual mi355x_status set_tensor(const char* tensor, int dtype, const void* host, int64_t n_elems) = 0;
    // Checks that every tensor is there and allocates what calls of up to max_tokens tokens a sequence need.
    virtual mi355x_status finalize(int64_t max_tokens) = 0;
    // One pass of s tokens per sequence over the layers, tokens on the device at tokens_dev [batch, s], after the
    // positions that the caches and states hold.
    virtual mi355x_status forward(int64_t s) = 0;
    // The logits of n rows (index into batch x s, ascending or not) of the last pass, into `logits` [n, vocab].
    virtual mi355x_status head(const int64_t* rows, int64_t n) = 0;
    // One decoding position of every sequence: the tokens from next_tok, the position from `state`, the logits into
    // `logits` [batch, vocab]. Host-visible state (cache_len) is the caller's.
    virtual mi355x_status step() = 0;
    virtual int step_variant() const { return 0; }
    // Whether calls longer than max_rows may be run in several passes.
    virtual bool runs_in_portions() const { return false; }
    // Empties what the sequences hold.
    virtual mi355x_status reset() {
        cache_len = 0;
        return MI355X_OK;
    }

    // The buffers above, for max_rows rows and logit_rows rows of logits; drops a recorded step.
    mi355x_status alloc_common(int64_t rows, int64_t n_logit_rows);
    mi355x_status check_tokens(const int32_t* tokens, int64_t n) const;
    // tokens [batch, n] -> logits of the wanted rows (b * n + t) to the host, in the order asked for.
    mi355x_status logits_at(const int32_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* logits_host);
    mi355x_status generate(const int32_t* prompt, int64_t n_prompt, int64_t n_new, int32_t* out_tokens, double* seconds);
};

}  // namespace mimir
