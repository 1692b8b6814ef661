// The part of a decoder that is the same whatever its layers are (decoder.h): calls of the host's tokens, the logits a
// caller asks for, and the greedy loop (llm/model.go:391-437; examples/llama/generate.go:44-53,162-202), behind the
// mi355x_model_* entry points.
#include "decoder.h"

#include <atomic>
#include <cstring>

namespace mimir {

// How generate runs its decoding steps: 0 the step's launches replayed as a graph, 1 the same launches issued one
// by one, 2 forward() with the position from the host.
static std::atomic<int> g_llama_step_mode{0};
void set_llama_step_mode(int mode) { g_llama_step_mode = mode; }

Decoder::~Decoder() {
    if (step_graph) (void)hipGraphExecDestroy(step_graph);
    if (stream) (void)hipStreamDestroy(stream);
}

mi355x_status Decoder::alloc_common(int64_t rows, int64_t n_logit_rows) {
    max_rows = rows;
    logit_rows = n_logit_rows;
    DECODER_HIP(logits.alloc((size_t)n_logit_rows * vocab * 4), name, "hipMalloc(logits)");
    DECODER_HIP(tokens_dev.alloc(rows * 4), name, "hipMalloc");
    DECODER_HIP(next_tok.alloc((size_t)batch * 4), name, "hipMalloc");
    if (!stream) DECODER_HIP(hipStreamCreate(&stream), name, "hipStreamCreate");
    if (step_graph) {
        (void)hipGraphExecDestroy(step_graph);
        step_graph = nullptr;
    }
    DECODER_HIP(state.alloc(256), name, "hipMalloc");
    if (batch <= (int)(kArgmaxTicketBytes / 4)) {
        DECODER_HIP(argmax_ws.alloc(argmax_workspace_bytes(batch)), name, "hipMalloc");
        DECODER_HIP(hipMemset(argmax_ws.p, 0, kArgmaxTicketBytes), name, "hipMemset");
    }
    DECODER_HIP(record.alloc(((size_t)context + 1) * batch * 4), name, "hipMalloc");  // a graph keeps its address
    return MI355X_OK;
}

mi355x_status Decoder::check_tokens(const int32_t* tokens, int64_t n) const {
    if (!ready) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: %s: model is not finalized", name);
    // llm/model.go:393-400
    if (n <= 0 || (!runs_in_portions() && (int64_t)batch * n > max_rows))
        return capi_fail(MI355X_ERR_SHAPE, "mi355x: %s: %lld tokens a sequence, at most %lld a call", name, (long long)n, (long long)(max_rows / batch));
    if (cache_len + n > context)
        return capi_fail(MI355X_ERR_SHAPE, "mi355x: %s: append %lld positions to a cache holding %lld of %d", name, (long long)n, (long long)cache_len, context);
    for (int64_t i = 0; i < (int64_t)batch * n; i++)
        if (tokens[i] < 0 || tokens[i] >= vocab) return capi_fail(MI355X_ERR_INDEX, "mi355x: %s: token %d of a vocabulary of %d", name, tokens[i], vocab);
    return MI355X_OK;
}

// Model.Logits (llm/model.go:391-437) for the rows asked for; a call longer than one pass goes in portions.
mi355x_status Decoder::logits_at(const int32_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* logits_host) {
    if (mi355x_status st = check_tokens(tokens, n)) return st;
    for (int64_t i = 0; i < n_want; i++)
        if (want[i] < 0 || want[i] >= (int64_t)batch * n) return capi_fail(MI355X_ERR_INDEX, "mi355x: %s: logits of row %lld of %lld", name, (long long)want[i], (long long)((int64_t)batch * n));
    const int64_t span = max_rows / batch;
    std::vector<int32_t> part;
    std::vector<int64_t> rows, place;
    for (int64_t t0 = 0; t0 < n; t0 += span) {
        const int64_t s = n - t0 < span ? n - t0 : span;
        const int32_t* from = tokens;
        if (s != n) {  // the portion's tokens of every sequence one after the other
            part.resize((size_t)batch * s);
            for (int64_t b = 0; b < batch; b++) memcpy(part.data() + b * s, tokens + b * n + t0, s * 4);
            from = part.data();
        }
        DECODER_HIP(hipMemcpyAsync(tokens_dev.p, from, (size_t)batch * s * 4, hipMemcpyHostToDevice, stream), name, "upload tokens");
        if (mi355x_status st = forward(s)) return st;
        rows.clear();
        place.clear();
        for (int64_t i = 0; i < n_want; i++) {
            const int64_t b = want[i] / n, t = want[i] % n;
            if (t < t0 || t >= t0 + s) continue;
            rows.push_back(b * s + t - t0);
            place.push_back(i);
        }
        for (size_t at = 0; at < rows.size(); at += (size_t)logit_rows) {
            const size_t m = rows.size() - at < (size_t)logit_rows ? rows.size() - at : (size_t)logit_rows;
            if (mi355x_status st = head(rows.data() + at, (int64_t)m)) return st;
            for (size_t i = 0; i < m;) {  // runs of neighbouring places in one copy
                size_t j = i + 1;
                while (j < m && place[at + j] == place[at + j - 1] + 1) j++;
                DECODER_HIP(hipMemcpyAsync(logits_host + place[at + i] * (int64_t)vocab, logits.as<float>() + i * (size_t)vocab, (j - i) * (size_t)vocab * 4,
                                           hipMemcpyDeviceToHost, stream), name, "download logits");
                i = j;
            }
        }
        if (s != n) DECODER_HIP(hipStreamSynchronize(stream), name, "portion");  // `part` is reused
    }
    return mi355x_sync(stream);
}

// Greedy generation (examples/llama/generate.go:162-202 with Sample at :44-53):
// the prompt [batch, n_prompt], then n_new steps. Each step's token is chosen on
// the device and read by the next step's embedding lookup from device memory;
// out_tokens [batch, n_new] comes back once at the end. seconds, if not NULL,
// gets the wall time of the prompt pass and of the n_new - 1 decoding steps.
mi355x_status Decoder::generate(const int32_t* prompt, int64_t n_prompt, int64_t n_new, int32_t* out_tokens, double* seconds) {
    if (mi355x_status st = check_tokens(prompt, n_prompt)) return st;
    if (cache_len + n_prompt + n_new - 1 > context)
        return capi_fail(MI355X_ERR_SHAPE, "mi355x: %s: %lld positions for a context of %d", name, (long long)(cache_len + n_prompt + n_new - 1), context);
    const int64_t B = batch, span = max_rows / B;
    const int mode = g_llama_step_mode;
    const bool use_graph = mode == 0, use_fast = mode != 2;
    auto hip = [&](hipError_t e, const char* what) -> mi355x_status {
        return e == hipSuccess ? MI355X_OK : capi_fail((mi355x_status)e, "mi355x: %s: %s: %s", name, what, hipGetErrorName(e));
    };
    DevBuf picked;  // [n_new, batch]
    DECODER_HIP(picked.alloc((size_t)n_new * B * 4), name, "hipMalloc(tokens)");
    hipEvent_t e0, e1, e2;
    DECODER_HIP(hipEventCreate(&e0), name, "hipEventCreate");
    DECODER_HIP(hipEventCreate(&e1), name, "hipEventCreate");
    DECODER_HIP(hipEventCreate(&e2), name, "hipEventCreate");
    // the portions of a prompt that is longer than one pass, each as [batch, s]
    std::vector<int32_t> laid((size_t)B * n_prompt);
    for (int64_t t0 = 0; t0 < n_prompt; t0 += span) {
        const int64_t s = n_prompt - t0 < span ? n_prompt - t0 : span;
        for (int64_t b = 0; b < B; b++) memcpy(laid.data() + B * t0 + b * s, prompt + b * n_prompt + t0, s * 4);
    }
    DECODER_HIP(hipEventRecord(e0, stream), name, "hipEventRecord");
    mi355x_status st = MI355X_OK;
    int64_t last_s = 0;
    for (int64_t t0 = 0; t0 < n_prompt && !st; t0 += span) {
        last_s = n_prompt - t0 < span ? n_prompt - t0 : span;
        st = hip(hipMemcpyAsync(tokens_dev.p, laid.data() + B * t0, (size_t)B * last_s * 4, hipMemcpyHostToDevice, stream), "upload tokens");
        if (!st) st = forward(last_s);
    }
    std::vector<int64_t> last(B);
    auto choose = [&](int32_t* out, int64_t s) -> mi355x_status {  // from the last row of every sequence of a pass of s tokens
        for (int64_t b = 0; b < B; b++) last[b] = b * s + s - 1;
        if (mi355x_status s2 = head(last.data(), B)) return s2;
        return hip(argmax(logits.as<float>(), B, vocab, out, argmax_ws.p, stream), "argmax");
    };
    if (!st) st = choose(picked.as<int32_t>(), last_s);
    if (!st) (void)hipEventRecord(e1, stream);
    if (!st && use_fast) {
        // record[0] is the prompt's choice; each step then reads next_tok and the
        // position from the device, and leaves its own choice in both places
        st = hip(hipMemcpyAsync(next_tok.p, picked.p, B * 4, hipMemcpyDeviceToDevice, stream), "step state");
        if (!st) st = hip(set_state(state.as<int32_t>(), (int)cache_len, 0, stream), "step state");
        if (!st) st = hip(advance(state.as<int32_t>(), next_tok.as<int32_t>(), record.as<int32_t>(), (int)B, 0, stream), "step state");
        auto one_step = [&]() -> mi355x_status {
            if (mi355x_status s2 = step()) return s2;
            if (mi355x_status s2 = hip(argmax(logits.as<float>(), B, vocab, next_tok.as<int32_t>(), argmax_ws.p, stream), "argmax")) return s2;
            return hip(advance(state.as<int32_t>(), next_tok.as<int32_t>(), record.as<int32_t>(), (int)B, 1, stream), "advance");
        };
        if (step_graph && graph_variant != step_variant()) {  // a measurement aid changed which step runs
            (void)hipGraphExecDestroy(step_graph);
            step_graph = nullptr;
        }
        if (!st && n_new > 1 && !step_graph && use_graph) {
            graph_variant = step_variant();
            hipGraph_t g = nullptr;
            st = hip(hipStreamBeginCapture(stream, hipStreamCaptureModeThreadLocal), "begin capture");
            if (!st) {
                mi355x_status cst = one_step();
                hipError_t e = hipStreamEndCapture(stream, &g);
                st = cst ? cst : hip(e, "end capture");
            }
            if (!st) st = hip(hipGraphInstantiate(&step_graph, g, nullptr, nullptr, 0), "instantiate graph");
            if (g) (void)hipGraphDestroy(g);
        }
        for (int64_t t = 1; t < n_new && !st; t++) {
            st = step_graph && use_graph ? hip(hipGraphLaunch(step_graph, stream), "graph launch") : one_step();
            if (!st) cache_len += 1;
        }
        if (!st) st = hip(hipMemcpyAsync(picked.p, record.p, (size_t)n_new * B * 4, hipMemcpyDeviceToDevice, stream), "copy record");
    } else
        for (int64_t t = 1; t < n_new && !st; t++) {
            // the step reads its tokens where the last step's argmax wrote them
            st = hip(hipMemcpyAsync(tokens_dev.p, picked.as<int32_t>() + (t - 1) * B, B * 4, hipMemcpyDeviceToDevice, stream), "token copy");
            if (!st) st = forward(1);
            if (!st) st = choose(picked.as<int32_t>() + t * B, 1);
        }
    if (!st) (void)hipEventRecord(e2, stream);
    std::vector<int32_t> host((size_t)n_new * B);
    if (!st) st = hip(hipMemcpyAsync(host.data(), picked.p, host.size() * 4, hipMemcpyDeviceToHost, stream), "download tokens");
    if (!st) st = mi355x_sync(stream);
    if (!st) {
        for (int64_t t = 0; t < n_new; t++)
            for (int64_t b = 0; b < B; b++) out_tokens[b * n_new + t] = host[t * B + b];
        if (seconds) {
            float ms01 = 0, ms12 = 0;
            (void)hipEventElapsedTime(&ms01, e0, e1);
            (void)hipEventElapsedTime(&ms12, e1, e2);
            seconds[0] = ms01 * 1e-3;
            seconds[1] = ms12 * 1e-3;
        }
    } else {
        (void)hipStreamSynchronize(stream);  // nothing queued still reads this call's memory
    }
    (void)hipEventDestroy(e0); (void)hipEventDestroy(e1); (void)hipEventDestroy(e2);
    return st;
}

}  // namespace mimir

using mimir::Decoder;

extern "C" {

mi355x_status mi355x_model_destroy(void* model) {
    delete (Decoder*)model;
    return MI355X_OK;
}

mi355x_status mi355x_model_set_tensor(void* model, const char* name, int dtype, const void* host, int64_t n_elems) {
    if (!model || !name || !host) return mimir::capi_fail(MI355X_ERR_INTERNAL, "mi355x: model_set_tensor: null pointer");
    return ((Decoder*)model)->set_tensor(name, dtype, host, n_elems);
}

mi355x_status mi355x_model_finalize(void* model, int64_t max_tokens) {
    if (!model || max_tokens <= 0) return mimir::capi_fail(MI355X_ERR_INTERNAL, "mi355x: model_finalize: bad arguments");
    return ((Decoder*)model)->finalize(max_tokens);
}

mi355x_status mi355x_model_reset(void* model) {
    if (!model) return mimir::capi_fail(MI355X_ERR_INTERNAL, "mi355x: model_reset: null pointer");
    return ((Decoder*)model)->reset();
}

int64_t mi355x_model_cache_len(void* model) { return model ? ((Decoder*)model)->cache_len : -1; }

mi355x_status mi355x_model_logits_at(void* model, const int32_t* tokens, int64_t n, const int64_t* want, int64_t n_want, float* logits_host) {
    if (!model || !tokens || n_want < 0 || (n_want > 0 && (!want || !logits_host))) return mimir::capi_fail(MI355X_ERR_INTERNAL, "mi355x: model_logits_at: bad arguments");
    return ((Decoder*)model)->logits_at(tokens, n, want, n_want, logits_host);
}

mi355x_status mi355x_model_logits(void* model, const int32_t* tokens, int64_t n, int all, float* logits_host) {
    Decoder* d = (Decoder*)model;
    if (!d || !tokens || !logits_host) return mimir::capi_fail(MI355X_ERR_INTERNAL, "mi355x: model_logits: null pointer");
    if (n <= 0) return d->check_tokens(tokens, n);
    std::vector<int64_t> want;
    for (int64_t b = 0; b < d->batch; b++)
        for (int64_t t = all ? 0 : n - 1; t < n; t++) want.push_back(b * n + t);
    return d->logits_at(tokens, n, want.data(), (int64_t)want.size(), logits_host);
}

mi355x_status mi355x_model_generate(void* model, const int32_t* prompt, int64_t n_prompt, int64_t n_new, int32_t* out_tokens, double* seconds) {
    if (!model || !prompt || !out_tokens || n_new <= 0) return mimir::capi_fail(MI355X_ERR_INTERNAL, "mi355x: model_generate: bad arguments");
    return ((Decoder*)model)->generate(prompt, n_prompt, n_new, out_tokens, seconds);
}

}  // extern "C"
