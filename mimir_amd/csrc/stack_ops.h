// Kernels of the mixer stack (stack.hip): group norms with what surrounds them, short causal convolutions, the products
// of bfloat16 weights, latent attention, attention by key heads and the linear recurrences. Each launches on the given stream and returns the
// launch status. Sizes and constants are parameters; rows are sequences' positions one after the other (b * s + t).
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace mimir {

// ---- residual_ops.hip -------------------------------------------------------------------
// The steps between two products on one row of `width`, in this order, those with a null pointer left out:
//   z = group_norm(table[tokens[row]] + pair_table[pair]) * w_post            (tokens set), or
//   z = x + group_norm(y) * w_post                 (w_post null: no norm of y, or of the table's row)
//   stream_out = z;  z = sum_j dwa[j] streams[j] + dwa[n_streams] z   (the depth average: n_streams earlier results)
//   x_out = z
//   h = group_norm(z) * w_next, and with conv_w (one position a sequence): h += the causal convolution of h with the
//   taps - 1 rows of conv_state [batch, taps - 1, width], which then moves on by one
//   h_f32, h_bf16: h, rows ldh elements apart.
// group_norm: `groups` equal parts, each over sqrt(mean(part^2) + eps); all of it in float32.
// pair: (previous token * mul_prev + token * mul_cur) mod buckets, or row `buckets` for a sequence's first token. The tokens
// of every position are kept in held [batch, held_ld], where the first of a call finds the one before.
struct PairTable {
    const uint16_t* table = nullptr;  // [buckets + 1, width]; null: none
    int64_t ld = 0, buckets = 0, mul_prev = 0, mul_cur = 0;
    int32_t* held = nullptr;
    int64_t held_ld = 0, s = 1, past = 0;  // s positions a sequence in this call, after past + *past_dev
    const int32_t* past_dev = nullptr;
};
struct NormChain {
    const int32_t* tokens = nullptr;
    const uint16_t* table = nullptr;
    int64_t table_ld = 0;
    PairTable pairs;
    const float* x = nullptr;
    const float* y = nullptr;
    int64_t ldy = 0;
    const float* w_post = nullptr;
    float* stream_out = nullptr;
    const float* streams = nullptr;
    int64_t stream_stride = 0;
    int n_streams = 0;
    const float* dwa = nullptr;
    float* x_out = nullptr;
    const float* w_next = nullptr;
    float* h_f32 = nullptr;
    uint16_t* h_bf16 = nullptr;
    int64_t ldh = 0;
    const float* conv_w = nullptr;
    float* conv_state = nullptr;
    int taps = 0;
    int width = 0, groups = 1;
    float eps = 0;
};
hipError_t norm_chain(const NormChain& a, int64_t rows, hipStream_t st);
// out[i] = group_norm(x[rows[i]]) * w
hipError_t norm_rows(const float* x, const int64_t* rows, int64_t n, const float* w, int width, int groups, float eps, float* out_f32,
                     uint16_t* out_bf16, int64_t ldo, hipStream_t st);
// A prompt's causal convolution: out = h + conv(h), taps - 1 rows before the first from state, which is then brought
// forward by s positions. out_f32 and out_bf16 (either may be null) have rows ldo apart; h is [batch * s, width].
hipError_t causal_conv(const float* h, const float* w, float* state, int taps, int batch, int64_t s, int width, float* out_f32, uint16_t* out_bf16,
                       int64_t ldo, hipStream_t st);
// out = group_norm(o) * w * sigmoid(g) on rows of `width`; g float32 or (g_bf16) bfloat16, rows ldg apart.
hipError_t gated_norm(const float* o, const void* g, bool g_bf16, int64_t ldg, const float* w, int64_t rows, int width, int groups, float eps,
                      float* out_f32, uint16_t* out_bf16, int64_t ldo, hipStream_t st);

// ---- products by bfloat16 weights -----------------------------------------------------------
// y = act(x . W^T): W [N, K] bfloat16, rows ldw apart. Rows of W and of x hold zeros (x: finite values) from K to
// the next multiple of 64. act: SiLU on columns below silu_n; relu2 squares max(., 0) on all of them.
struct ProductOut {
    float* f32 = nullptr;      // exactly one of the two
    uint16_t* bf16 = nullptr;
    int64_t ld = 0;
    int64_t silu_n = 0;
    bool relu2 = false;
    // Columns from pair_from (a multiple of 4) on come in pairs (z, u), side by side, and leave one value silu(z) u a pair, in
    // one of these, rows pair_ld apart. N is even then, and there are no factors.
    int64_t pair_from = INT64_MAX;
    float* pair_f32 = nullptr;
    uint16_t* pair_bf16 = nullptr;
    int64_t pair_ld = 0;
    // y_n = scale[n] (mid[n] (the sum over k < split) + the rest of it), with null pointers for ones: two products of the same
    // row, each with factors of its own (s in front of the first: mid = s / scale), in one. split: a multiple of 64 below K.
    // Without an activation.
    const float* scale = nullptr;
    const float* mid = nullptr;
    int64_t split = 0;
    bool add = false;  // to what f32 holds
};
constexpr int64_t kGemvRows = 8;  // rows of x that gemv_bf16 takes at once (more are several passes over W)
// float32 x, few rows: W read once for up to kGemvRows of them (gemv_float.hip)
hipError_t gemv_bf16(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st);
// the same on the bfloat16 matrix cores, x as the sum of two bfloat16: at most kGemvRows rows (gemv_bf16_rows.hip)
hipError_t gemv_bf16_rows(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st);
// float32 x, many rows, on the float32 matrix cores: nothing is rounded to 16 bits (gemm_float.hip)
hipError_t gemm_f32(const uint16_t* W, int64_t ldw, const float* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st);
// bfloat16 x, many rows, on the bfloat16 matrix cores with float32 sums (gemm_bf16.hip): ldx and ldw multiples of 8
hipError_t gemm_bf16(const uint16_t* W, int64_t ldw, const uint16_t* x, int64_t ldx, int64_t M, int64_t N, int64_t K, const ProductOut& out, hipStream_t st);

// ---- linear recurrences (linear_recurrence.hip) -----------------------------------------------
// Per head, S [dim, vdim] and o = S^T q, in one of two forms:
//   gated (mLSTM): log gates i = cap tanh((gi + bias_i) / cap), f = logsigmoid(cap tanh((gf + bias_f) / cap)),
//     m' = max(f + m, i), S = exp(f + m - m') S + exp(i - m') k v^T, n likewise with k alone,
//     o = S^T q / (max(|n . q|, exp(-m')) + 1e-6), q scaled by q_scale
//   decaying (lightning): S = decay S + k v^T.
// Everything but q, k, v is float32, and so are the products with S.
struct Recurrence {
    const void *q = nullptr, *k = nullptr, *v = nullptr;  // [rows, heads * dim (vdim)], rows ld apart
    bool bf16 = false;                                    // of q, k, v
    int64_t ld = 0;
    const float* gates = nullptr;  // [rows, heads of gi | heads of gf], rows ldg apart; null: decaying
    int64_t ldg = 0;
    const float *bias_i = nullptr, *bias_f = nullptr;
    float cap = 1.f;
    const float* decay = nullptr;      // [heads]
    const float* decay_pow = nullptr;  // [heads, kRecurrenceChunk + 1]: decay^0, decay^1, ...
    float q_scale = 1.f;
    float* S = nullptr;  // [batch, heads, dim, vdim]
    float* n = nullptr;  // [batch, heads, recurrence_slices(vdim), dim]: a copy for each slice of S's columns
    float* m = nullptr;  // [batch, heads, recurrence_slices(vdim)]
    float* out = nullptr;  // [rows, heads * vdim]
    int64_t ldo = 0;
    int batch = 1, heads = 1, dim = 0, vdim = 0;
    int64_t s = 1;
    float* ws = nullptr;  // recurrence_chunk_ws_floats(...), chunked form only
};
constexpr int kRecurrenceChunk = 64;
constexpr int kRecurrenceMaxDim = 256;
int recurrence_slices(int vdim);
// Position by position (a decoding step; prompts in float32).
hipError_t recurrence_scan(const Recurrence& r, hipStream_t st);
// A prompt in chunks of kRecurrenceChunk on the matrix cores: bfloat16 q, k, v; what is rounded to 16 bits besides
// them is carried as pairs of bfloat16 (16 bits of significand).
bool recurrence_chunks_ok(const Recurrence& r);
size_t recurrence_chunk_ws_floats(int batch, int heads, int dim, int vdim, int64_t s);
hipError_t recurrence_chunks(const Recurrence& r, hipStream_t st);

// ---- latent attention (attention_latent.hip) ---------------------------------------------------
// Keys and values come from a latent c of `rank` and a rotated part of rot_dim that all heads share; a cache row is
// c | rotated part, ldc elements apart, float32 or bfloat16.
struct Latent {
    int heads = 1, dim = 0, rot_dim = 0, vdim = 0, rank = 0;
    float scale = 1.f, eps = 0.f;
    const float *cos_t = nullptr, *sin_t = nullptr;  // [context, rot_dim / 2]
    const float* norm_w = nullptr;                   // [rank]
    const uint16_t* w_uk = nullptr;                  // [heads * dim, rank], rows ldw apart
    const uint16_t* w_uv = nullptr;                  // [heads * vdim, rank]
    int64_t ldw = 0;
    void* cache = nullptr;  // [batch, context, ldc]: context is the capacity
    bool cache_bf16 = false;
    int64_t ldc = 0;
    int64_t context = 0;
    int batch = 1;
    int64_t s = 1;       // new positions a sequence
    int64_t past = 0;    // positions before them: past + *past_dev
    const int32_t* past_dev = nullptr;
};
// From projections [rows, heads * (dim + rot_dim) | rank + rot_dim] (float32, rows ldp apart), for latent_prompt: the cache
// rows of the new positions, and the queries with their rotated parts turned, as bfloat16 rows ldq apart.
hipError_t latent_prepare(const Latent& a, const float* proj, int64_t ldp, uint16_t* q_bf16, int64_t ldq, hipStream_t st);
// Few query rows, from the same projections: cache rows, then attention without ever forming keys or values: q' = W_uk^T q
// per head against the latents, and W_uv on what they sum to. ws: latent_absorbed_ws_floats floats. out
// [rows, heads * vdim] float32 or bfloat16, rows ldo apart.
int latent_splits(const Latent& a);
size_t latent_absorbed_ws_floats(const Latent& a, int64_t rows);
hipError_t latent_absorbed(const Latent& a, const float* proj, int64_t ldp, float* ws, float* out_f32, uint16_t* out_bf16, int64_t ldo, hipStream_t st);
// Many query rows (bfloat16 cache and queries), on keys and values formed beforehand for all past + s positions of every
// sequence: keys [batch * context, heads * dim], values transposed [heads * vdim, batch * context], rows ldk and ldv elements
// apart; context a multiple of 64. Products on the bfloat16 matrix cores; a weight goes to them as the sum of two bfloat16.
bool latent_prompt_ok(const Latent& a);
hipError_t latent_prompt(const Latent& a, const uint16_t* q, int64_t ldq, const uint16_t* keys, int64_t ldk, const uint16_t* values_t, int64_t ldv,
                         uint16_t* out, int64_t ldo, hipStream_t st);

// ---- attention with a key and value for every key head (attention_heads.hip) -------------------
// Query heads share key heads in neighbouring groups; causal. score = softcap tanh(scale q.k / softcap) (softcap 0: scale q.k).
struct HeadAttention {
    int heads = 1, kv_heads = 1, dim = 0, vdim = 0;
    float scale = 1.f, softcap = 0.f;
    bool unit = false;  // queries and keys over their root mean square, sqrt(mean(x^2) + eps)
    float eps = 0.f;
    int rot_dim = 0;  // the first features of queries and keys turn, feature i with feature i + rot_dim / 2
    const float *cos_t = nullptr, *sin_t = nullptr;  // [context, rot_dim / 2]
    const float* proj = nullptr;  // [rows, heads * dim of q | kv_heads * dim of k | kv_heads * vdim of v | gated: heads], rows ldp apart
    int64_t ldp = 0;
    bool gated = false;  // a head's result times the sigmoid of its gate
    // values: (1 - mix) v + mix first, where `first` is set ([rows, kv_heads * vdim]); first_out, where set, gets v
    const float* mix = nullptr;
    const float* first = nullptr;
    float* first_out = nullptr;
    void* keys = nullptr;    // [batch, kv_heads, context, ldk]
    void* values = nullptr;  // [batch, kv_heads, vdim, context], positions in the kernels' own order
    bool cache_bf16 = false;
    int64_t ldk = 0;      // a multiple of 8, zeros behind dim
    int64_t context = 0;  // the capacity, a multiple of 64
    int batch = 1;
    int64_t s = 1;     // new positions a sequence
    int64_t past = 0;  // positions before them: past + *past_dev
    const int32_t* past_dev = nullptr;
};
constexpr int kHeadAttentionMax = 1024;  // features of a head
// Cache entries of the new positions, then attention of few query rows. ws: heads_attend_ws_floats floats. out
// [rows, heads * vdim] float32 or bfloat16, rows ldo apart.
size_t heads_attend_ws_floats(const HeadAttention& a, int64_t rows);
hipError_t heads_attend(const HeadAttention& a, float* ws, float* out_f32, uint16_t* out_bf16, int64_t ldo, hipStream_t st);
// The same for many query rows on a bfloat16 cache. q: [rows, heads, ldk] of workspace.
bool heads_prompt_ok(const HeadAttention& a);
hipError_t heads_prompt(const HeadAttention& a, uint16_t* q, uint16_t* out, int64_t ldo, hipStream_t st);

}  // namespace mimir
