// A decoder whose layers are a list of mixers, each with its own sizes (mi355x_stack_create). Two arrangements of a layer:
// in turn, x += norm1b(mixer(conv(norm1(x)))), x += norm2b(mlp(norm2(x))) where it has an mlp, then the depth average over
// the embedding output and all layers' results so far (the Fuvolix design; norm1b, norm2b, conv and average can be left
// out); or in parallel, with h = norm1(x), x += s1 mixer(h) + s2 mlp(h), s1 and s2 a factor a feature (the Genetar design).
// Norms are RMS norms in groups, conv adds a short causal convolution over time. Mixers: latent attention
// (attention_latent.hip), attention by key heads (attention_heads.hip), gated and decaying linear recurrences
// (linear_recurrence.hip). What a sequence holds between calls: the last inputs of each layer's convolution, the latents
// and rotated keys of latent attention, keys and values, the recurrences' states, and its tokens where the embedding
// takes pairs of them.
//
// Weights are bfloat16 on the device; matrices that read the same input lie in one buffer and are multiplied in one
// product: a parallel layer is two, one of everything that reads h and one of the mixer's and the feed-forward's results
// side by side, which adds to the residual itself. Activations: a pass of up to kGemvRows rows, and every pass of a model
// that runs in float32, multiplies float32 activations; longer passes of a bfloat16 model round the products' inputs to
// bfloat16. The residual, norms, recurrent states, gates, scores and softmax weights are float32 either way.
#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstring>
#include <iterator>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "decoder.h"
#include "stack_ops.h"

namespace mimir {

namespace {

#define STACK_HIP(expr, what) DECODER_HIP(expr, "stack", what)

// From how many positions of a sequence in one pass a prompt's forms are taken (bfloat16, more than kGemvRows rows):
// attention on tiles of query rows (over keys and values formed beforehand for latent attention), recurrences in chunks.
constexpr int64_t kManyRows = 32, kChunked = 16;

int64_t pad64(int64_t n) { return (n + 63) / 64 * 64; }

struct Mat {  // [n, k] bfloat16, rows ld apart, zeros from k on
    int64_t n = 0, k = 0, ld = 0;
    DevBuf buf;
    const uint16_t* row(int64_t i) const { return buf.as<uint16_t>() + i * ld; }
};
struct Vec {  // float32
    int64_t n = 0;
    DevBuf buf;
    const float* p() const { return buf.as<float>(); }
};

// Where a tensor of the file goes.
struct Slot {
    Mat* mat = nullptr;
    Vec* vec = nullptr;
    int64_t row0 = 0, rows = 0, cols = 0;
    int64_t step = 1, col0 = 0;  // rows of the matrix from one of the tensor's to the next; its first column there
    float factor = 1.f;          // of a vector
    bool needed = true, set = false;
};

struct StackLayer {
    mi355x_stack_layer c{};
    std::vector<double> decay;
    Vec norm1, norm1b, norm2, norm2b, canon, dwa, mix_norm, dkv_norm, bias_i, bias_f, ls1, ls2, vmix;
    // in: every projection of the mixer's input, one after the other, and from row proj_n on those of a parallel feed-forward,
    // a row of gate and one of up in turn. o: the output projection, with the feed-forward's down beside it from column
    // down_at on. up: a gated feed-forward's rows in turn likewise.
    Mat in, o, ukv, up, down;
    int64_t proj_n = 0, down_at = 0;
    int64_t g_at = 0, gates_at = 0;    // rows of `in` where W_g and the two gates' begin
    DevBuf cos_t, sin_t, cache, values, S, n, m, conv_state, decay_f, decay_pow;
    DevBuf out_mid;                    // s1 / s2 of a parallel layer, unless two_products
    bool two_products = false;         // an s2 too small beside its s1
    bool mixes_first = false;          // the first layer of those with value_mix
    int64_t ldc = 0;
    int64_t mixed() const { return (int64_t)c.heads * c.vdim; }
    bool recurrent() const { return c.mixer == MI355X_MIXER_MLSTM || c.mixer == MI355X_MIXER_LIGHTNING; }
    bool by_heads() const { return c.mixer == MI355X_MIXER_ATTENTION; }
};

struct Stack : Decoder {
    mi355x_stack_config c{};
    std::vector<StackLayer> layers;
    Mat embed, pairs, head_w;
    Vec embed_norm, final_norm;
    std::map<std::string, Slot> slots;

    // activations of up to max_rows rows; *_f float32, *_b bfloat16
    DevBuf streams, x, h, y, in_f, in_b, proj_f, proj_b, gates, scanned, mix_f, mix_b, up_f, up_b, last_f, last_b, rows_dev, ws;
    DevBuf q_b, keys_b, values_b;  // attention of a prompt: turned queries; latent: all positions' keys, and their values transposed
    DevBuf first_values;           // of a pass: what layers with value_mix mix in
    DevBuf held;                   // the tokens of every position [batch, context], where the embedding takes pairs

    mi355x_status set_tensor(const char* tensor, int dtype, const void* host, int64_t n_elems) override;
    mi355x_status finalize(int64_t max_tokens) override;
    mi355x_status forward(int64_t s) override;
    mi355x_status head(const int64_t* rows, int64_t n) override;
    mi355x_status step() override;
    mi355x_status reset() override;
    bool runs_in_portions() const override { return true; }

    bool half() const { return c.dtype == MI355X_BF16; }
    bool has(int flag) const { return (c.flags & flag) != 0; }
    bool parallel() const { return has(MI355X_STACK_PARALLEL); }
    const Mat& output() const { return has(MI355X_STACK_OUTPUT_MATRIX) ? head_w : embed; }
    int64_t width() const { return c.width; }
    void name_tensors();
    Latent latent(const StackLayer& l, int64_t s, const int32_t* pos) const;
    HeadAttention attention(const StackLayer& l, int64_t s, const int32_t* pos) const;
    Recurrence recurrence(const StackLayer& l, int64_t s, bool tiles) const;
    mi355x_status pass(const int32_t* tokens, int64_t s, const int32_t* pos);
    mi355x_status mix(StackLayer& l, int64_t s, bool tiles, const int32_t* pos);
    mi355x_status layer_output(StackLayer& l, bool tiles, int64_t rows);
    mi355x_status rotation(StackLayer& l);
    mi355x_status layer_scales(StackLayer& l);
    mi355x_status prompt_attention(const Latent& a, const Mat& o);
    // out = act(x . W[row0, row0 + n)^T) by the kernel for this many rows and x's form (bfloat16 if b, else float32); of W's
    // columns and of x's [k0, k1) (k1 0: to the end)
    mi355x_status product(const Mat& w, int64_t row0, int64_t n, const DevBuf& f, const DevBuf& b, bool tiles, int64_t rows, const ProductOut& out,
                          int64_t k0 = 0, int64_t k1 = 0);
};

mi355x_status Stack::product(const Mat& w, int64_t row0, int64_t n, const DevBuf& f, const DevBuf& b, bool tiles, int64_t rows, const ProductOut& out, int64_t k0,
                             int64_t k1) {
    const int64_t k = (k1 ? k1 : w.k) - k0;
    const uint16_t* m = w.row(row0) + k0;
    if (tiles) STACK_HIP(gemm_bf16(m, w.ld, b.as<uint16_t>() + k0, w.ld, rows, n, k, out, stream), "product");
    else if (half() && rows > 1 && rows <= kGemvRows) STACK_HIP(gemv_bf16_rows(m, w.ld, f.as<float>() + k0, w.ld, rows, n, k, out, stream), "product");
    else if (rows <= kGemvRows) STACK_HIP(gemv_bf16(m, w.ld, f.as<float>() + k0, w.ld, rows, n, k, out, stream), "product");
    else STACK_HIP(gemm_f32(m, w.ld, f.as<float>() + k0, w.ld, rows, n, k, out, stream), "product");
    return MI355X_OK;
}

Latent Stack::latent(const StackLayer& l, int64_t s, const int32_t* pos) const {
    Latent a;
    a.heads = l.c.heads; a.dim = l.c.dim; a.rot_dim = l.c.rot_dim; a.vdim = l.c.vdim; a.rank = l.c.kv_rank;
    a.scale = (float)l.c.scale; a.eps = (float)c.eps;
    a.cos_t = l.cos_t.as<float>(); a.sin_t = l.sin_t.as<float>();
    a.norm_w = l.dkv_norm.p();
    a.w_uk = l.ukv.row(0); a.w_uv = l.ukv.row((int64_t)l.c.heads * l.c.dim); a.ldw = l.ukv.ld;
    a.cache = l.cache.p; a.cache_bf16 = half(); a.ldc = l.ldc; a.context = pad64(context);
    a.batch = batch; a.s = s;
    a.past = pos ? 0 : cache_len; a.past_dev = pos;
    return a;
}

HeadAttention Stack::attention(const StackLayer& l, int64_t s, const int32_t* pos) const {
    HeadAttention a;
    a.heads = l.c.heads; a.kv_heads = l.c.kv_heads; a.dim = l.c.dim; a.vdim = l.c.vdim;
    a.scale = (float)l.c.scale; a.softcap = (float)l.c.softcap;
    a.unit = l.c.unit_qk != 0; a.eps = (float)c.eps;
    a.rot_dim = l.c.rot_dim; a.cos_t = l.cos_t.as<float>(); a.sin_t = l.sin_t.as<float>();
    a.proj = proj_f.as<float>(); a.ldp = l.proj_n;
    a.gated = l.c.head_gate != 0;
    if (l.c.value_mix && l.mixes_first) a.first_out = first_values.as<float>();
    else if (l.c.value_mix) { a.first = first_values.as<float>(); a.mix = l.vmix.p(); }
    a.keys = l.cache.p; a.values = l.values.p; a.cache_bf16 = half(); a.ldk = l.ldc; a.context = pad64(context);
    a.batch = batch; a.s = s;
    a.past = pos ? 0 : cache_len; a.past_dev = pos;
    return a;
}

Recurrence Stack::recurrence(const StackLayer& l, int64_t s, bool tiles) const {
    Recurrence r;
    const int64_t qk = (int64_t)l.c.heads * l.c.dim;
    r.bf16 = tiles;
    if (tiles) {
        r.ld = pad64(l.gates_at);
        r.q = proj_b.as<uint16_t>(); r.k = proj_b.as<uint16_t>() + qk; r.v = proj_b.as<uint16_t>() + 2 * qk;
    } else {
        r.ld = l.in.n;
        r.q = proj_f.as<float>(); r.k = proj_f.as<float>() + qk; r.v = proj_f.as<float>() + 2 * qk;
    }
    if (l.c.mixer == MI355X_MIXER_MLSTM) {
        r.gates = tiles ? gates.as<float>() : proj_f.as<float>() + l.gates_at; r.ldg = tiles ? 2 * l.c.heads : l.in.n;
        r.bias_i = l.bias_i.p(); r.bias_f = l.bias_f.p();
        r.cap = (float)l.c.gate_cap;
        r.q_scale = (float)(1.0 / std::sqrt((double)l.c.dim));
        r.n = l.n.as<float>(); r.m = l.m.as<float>();
    } else {
        r.decay = l.decay_f.as<float>(); r.decay_pow = l.decay_pow.as<float>();
    }
    r.S = l.S.as<float>();
    r.out = scanned.as<float>(); r.ldo = l.mixed();
    r.batch = batch; r.heads = l.c.heads; r.dim = l.c.dim; r.vdim = l.c.vdim; r.s = s;
    r.ws = ws.as<float>();
    return r;
}

// A prompt's latent attention: keys and transposed values of all positions from the cached latents, then the attention on
// them. The sequences' caches lie one behind the other: one product for all of them where most of the capacity is held
// (what lies behind a sequence's positions is finite and is not looked at), else one a sequence.
mi355x_status Stack::prompt_attention(const Latent& a, const Mat& o) {
    const int64_t n = a.past + a.s, kn = (int64_t)a.heads * a.dim, vn = (int64_t)a.heads * a.vdim, ldv = batch * a.context, qn = (int64_t)a.heads * (a.dim + a.rot_dim);
    const bool at_once = batch > 1 && 2 * n > a.context;
    for (int b = 0; b < (at_once ? 1 : batch); b++) {
        const uint16_t* latents = (const uint16_t*)a.cache + b * a.context * a.ldc;
        const int64_t rows = at_once ? batch * a.context : n;
        ProductOut k;
        k.bf16 = keys_b.as<uint16_t>() + b * a.context * kn; k.ld = kn;
        STACK_HIP(gemm_bf16(a.w_uk, a.ldw, latents, a.ldc, rows, kn, a.rank, k, stream), "keys");
        ProductOut v;
        v.bf16 = values_b.as<uint16_t>() + b * a.context; v.ld = ldv;
        STACK_HIP(gemm_bf16(latents, a.ldc, a.w_uv, a.ldw, vn, rows, a.rank, v, stream), "values");
    }
    STACK_HIP(latent_prompt(a, q_b.as<uint16_t>(), qn, keys_b.as<uint16_t>(), kn, values_b.as<uint16_t>(), ldv, mix_b.as<uint16_t>(), o.ld, stream),
              "latent attention");
    return MI355X_OK;
}

// The mixer and behind it layer_output, for s positions a sequence.
mi355x_status Stack::mix(StackLayer& l, int64_t s, bool tiles, const int32_t* pos) {
    const int64_t rows = (int64_t)batch * s, mixed = l.mixed();
    if (l.by_heads()) {
        ProductOut p;  // float32: norms, the rotation and the mixing of values see what the product summed
        p.f32 = proj_f.as<float>(); p.ld = l.proj_n;
        if (l.in.n > l.proj_n) {
            p.pair_from = l.proj_n; p.pair_ld = l.o.ld;
            if (tiles) p.pair_bf16 = mix_b.as<uint16_t>() + l.down_at;
            else p.pair_f32 = mix_f.as<float>() + l.down_at;
        }
        if (mi355x_status st = product(l.in, 0, l.in.n, in_f, in_b, tiles, rows, p)) return st;
        const HeadAttention a = attention(l, s, pos);
        if (tiles && s >= kManyRows && heads_prompt_ok(a)) STACK_HIP(heads_prompt(a, q_b.as<uint16_t>(), mix_b.as<uint16_t>(), l.o.ld, stream), "attention");
        else STACK_HIP(heads_attend(a, ws.as<float>(), tiles ? nullptr : mix_f.as<float>(), tiles ? mix_b.as<uint16_t>() : nullptr, l.o.ld, stream), "attention");
    } else if (!l.recurrent()) {
        ProductOut p;  // float32: the latent's norm and the rotation see what the product summed
        p.f32 = proj_f.as<float>(); p.ld = l.in.n;
        if (mi355x_status st = product(l.in, 0, l.in.n, in_f, in_b, tiles, rows, p)) return st;
        const Latent a = latent(l, s, pos);
        const bool formed = tiles && s >= kManyRows && latent_prompt_ok(a);
        if (formed) {
            STACK_HIP(latent_prepare(a, proj_f.as<float>(), l.in.n, q_b.as<uint16_t>(), (int64_t)l.c.heads * (l.c.dim + l.c.rot_dim), stream),
                      "latents and rotation");
            if (mi355x_status st = prompt_attention(a, l.o)) return st;
        } else {
            STACK_HIP(latent_absorbed(a, proj_f.as<float>(), l.in.n, ws.as<float>(), tiles ? nullptr : mix_f.as<float>(),
                                      tiles ? mix_b.as<uint16_t>() : nullptr, l.o.ld, stream), "latent attention");
        }
    } else {
        ProductOut p;
        p.silu_n = l.c.mixer == MI355X_MIXER_LIGHTNING ? l.g_at : 0;
        if (tiles) {
            p.bf16 = proj_b.as<uint16_t>(); p.ld = pad64(l.gates_at);
            if (mi355x_status st = product(l.in, 0, l.gates_at, in_f, in_b, true, rows, p)) return st;
            if (l.in.n > l.gates_at) {  // the recurrence's gates are not rounded
                ProductOut g;
                g.f32 = gates.as<float>(); g.ld = l.in.n - l.gates_at;
                if (mi355x_status st = product(l.in, l.gates_at, g.ld, in_f, in_b, false, rows, g)) return st;
            }
        } else {
            p.f32 = proj_f.as<float>(); p.ld = l.in.n;
            if (mi355x_status st = product(l.in, 0, l.in.n, in_f, in_b, false, rows, p)) return st;
        }
        const Recurrence r = recurrence(l, s, tiles);
        if (tiles && s >= kChunked && recurrence_chunks_ok(r)) STACK_HIP(recurrence_chunks(r, stream), "recurrence in chunks");
        else STACK_HIP(recurrence_scan(r, stream), "recurrence");
        const void* g = tiles ? (const void*)(proj_b.as<uint16_t>() + l.g_at) : (const void*)(proj_f.as<float>() + l.g_at);
        STACK_HIP(gated_norm(scanned.as<float>(), g, tiles, tiles ? p.ld : l.in.n, l.mix_norm.p(), rows, (int)mixed,
                             l.c.mixer == MI355X_MIXER_MLSTM ? l.c.heads : 1, (float)c.eps, tiles ? nullptr : mix_f.as<float>(),
                             tiles ? mix_b.as<uint16_t>() : nullptr, l.o.ld, stream), "gated norm");
    }
    return layer_output(l, tiles, rows);
}

// The mixer's result, times its scale, into y; of a parallel layer, with the feed-forward's, added to x.
mi355x_status Stack::layer_output(StackLayer& l, bool tiles, int64_t rows) {
    ProductOut p;
    p.ld = width();
    if (has(MI355X_STACK_LAYER_SCALE)) p.scale = l.ls1.p();
    if (!parallel()) {
        p.f32 = y.as<float>();
        return product(l.o, 0, l.o.n, mix_f, mix_b, tiles, rows, p);
    }
    p.f32 = x.as<float>(); p.add = true;
    if (l.c.ff == 0) return product(l.o, 0, l.o.n, mix_f, mix_b, tiles, rows, p);
    if (l.two_products) {
        if (mi355x_status st = product(l.o, 0, l.o.n, mix_f, mix_b, tiles, rows, p, 0, l.down_at)) return st;
        p.scale = l.ls2.p();
        return product(l.o, 0, l.o.n, mix_f, mix_b, tiles, rows, p, l.down_at);
    }
    if (has(MI355X_STACK_LAYER_SCALE)) {
        p.scale = l.ls2.p(); p.mid = l.out_mid.as<float>(); p.split = l.down_at;
    }
    return product(l.o, 0, l.o.n, mix_f, mix_b, tiles, rows, p);
}

// s positions a sequence through all layers. pos: a decoding step, whose position is read from the device (s is 1) and
// which leaves the final norm of its rows in last_f; otherwise the residual is left in x.
mi355x_status Stack::pass(const int32_t* tokens, int64_t s, const int32_t* pos) {
    const int64_t rows = (int64_t)batch * s, W = width(), ldw = pad64(W);
    const bool tiles = half() && rows > kGemvRows;
    NormChain base;
    base.width = c.width; base.groups = c.norm_groups; base.eps = (float)c.eps; base.taps = c.taps;
    const bool convolves = c.taps > 0, averages = has(MI355X_STACK_DEPTH_AVERAGE), posts = has(MI355X_STACK_POST_NORMS);
    // whether a layer's products read float32 rows; the gates of a recurrence always do
    auto in_float = [&](const StackLayer& l) { return !tiles || l.c.mixer == MI355X_MIXER_MLSTM; };
    auto into_layer = [&](NormChain& a, size_t i) {  // the end of a chain: layer i's norm, or the final one
        if (i == layers.size()) {
            if (!pos) return;
            a.w_next = final_norm.p(); a.h_f32 = last_f.as<float>(); a.ldh = ldw;
            return;
        }
        a.w_next = layers[i].norm1.p();
        if (pos || !convolves) {
            if (convolves) { a.conv_w = layers[i].canon.p(); a.conv_state = layers[i].conv_state.as<float>(); }
            a.ldh = ldw;
            if (tiles) a.h_bf16 = in_b.as<uint16_t>();
            if (in_float(layers[i])) a.h_f32 = in_f.as<float>();
        } else {
            a.h_f32 = h.as<float>(); a.ldh = W;
        }
    };
    {
        NormChain a = base;
        a.tokens = tokens; a.table = embed.row(0); a.table_ld = embed.ld;
        if (has(MI355X_STACK_EMBED_NORM)) a.w_post = embed_norm.p();
        if (c.pair_buckets > 0) {
            a.pairs.table = pairs.row(0); a.pairs.ld = pairs.ld;
            a.pairs.buckets = c.pair_buckets; a.pairs.mul_prev = c.pair_mul_prev; a.pairs.mul_cur = c.pair_mul_cur;
            a.pairs.held = held.as<int32_t>(); a.pairs.held_ld = context; a.pairs.s = s;
            a.pairs.past = pos ? 0 : cache_len; a.pairs.past_dev = pos;
        }
        if (averages) a.stream_out = streams.as<float>();
        a.x_out = x.as<float>();
        into_layer(a, 0);
        STACK_HIP(norm_chain(a, rows, stream), "embedding");
    }
    for (size_t i = 0; i < layers.size(); i++) {
        StackLayer& l = layers[i];
        if (!pos && convolves) {
            STACK_HIP(causal_conv(h.as<float>(), l.canon.p(), l.conv_state.as<float>(), c.taps, batch, s, c.width, in_float(l) ? in_f.as<float>() : nullptr,
                                  tiles ? in_b.as<uint16_t>() : nullptr, ldw, stream), "convolution");
        }
        if (mi355x_status st = mix(l, s, tiles, pos)) return st;
        NormChain a = base;
        a.x = x.as<float>();
        if (parallel()) {  // the product has added to x
            into_layer(a, i + 1);
            if (a.w_next) STACK_HIP(norm_chain(a, rows, stream), "norm");
            continue;
        }
        a.y = y.as<float>(); a.ldy = W; a.w_post = posts ? l.norm1b.p() : nullptr; a.x_out = x.as<float>();
        if (l.c.ff > 0) {
            a.w_next = l.norm2.p(); a.ldh = ldw;
            if (tiles) a.h_bf16 = in_b.as<uint16_t>();
            else a.h_f32 = in_f.as<float>();
            STACK_HIP(norm_chain(a, rows, stream), "norms");
            ProductOut p;
            p.relu2 = true; p.ld = l.down.ld;
            if (tiles) p.bf16 = up_b.as<uint16_t>();
            else p.f32 = up_f.as<float>();
            if (l.c.mlp == MI355X_MLP_SWIGLU) { p.pair_from = 0; p.pair_f32 = p.f32; p.pair_bf16 = p.bf16; p.pair_ld = p.ld; }
            if (mi355x_status st = product(l.up, 0, l.up.n, in_f, in_b, tiles, rows, p)) return st;
            ProductOut d;
            d.f32 = y.as<float>(); d.ld = W;
            if (has(MI355X_STACK_LAYER_SCALE)) d.scale = l.ls2.p();
            if (mi355x_status st = product(l.down, 0, l.down.n, up_f, up_b, tiles, rows, d)) return st;
            a = base;
            a.x = x.as<float>(); a.y = y.as<float>(); a.ldy = W; a.w_post = posts ? l.norm2b.p() : nullptr; a.x_out = x.as<float>();
        }
        if (averages) {
            a.stream_out = i + 1 < layers.size() ? streams.as<float>() + (i + 1) * max_rows * W : nullptr;
            a.streams = streams.as<float>(); a.stream_stride = max_rows * W; a.n_streams = (int)i + 1; a.dwa = l.dwa.p();
        }
        into_layer(a, i + 1);
        STACK_HIP(norm_chain(a, rows, stream), "norms and depth average");
    }
    return MI355X_OK;
}

mi355x_status Stack::forward(int64_t s) {
    if (mi355x_status st = pass(tokens_dev.as<int32_t>(), s, nullptr)) return st;
    cache_len += s;
    return MI355X_OK;
}

mi355x_status Stack::head(const int64_t* rows, int64_t n) {
    if (n <= 0) return MI355X_OK;
    const bool tiles = half() && n > kGemvRows;
    STACK_HIP(hipMemcpyAsync(rows_dev.p, rows, (size_t)n * 8, hipMemcpyHostToDevice, stream), "upload rows");
    STACK_HIP(norm_rows(x.as<float>(), rows_dev.as<int64_t>(), n, final_norm.p(), c.width, c.norm_groups, (float)c.eps, tiles ? nullptr : last_f.as<float>(),
                        tiles ? last_b.as<uint16_t>() : nullptr, embed.ld, stream), "final norm");
    ProductOut p;
    p.f32 = logits.as<float>(); p.ld = vocab;
    return product(output(), 0, vocab, last_f, last_b, tiles, n, p);
}

mi355x_status Stack::step() {
    if (mi355x_status st = pass(next_tok.as<int32_t>(), 1, state.as<int32_t>())) return st;
    ProductOut p;
    p.f32 = logits.as<float>(); p.ld = vocab;
    return product(output(), 0, vocab, last_f, last_b, false, batch, p);  // float32 rows, however many
}

mi355x_status Stack::reset() {
    cache_len = 0;
    if (!ready) return MI355X_OK;
    for (StackLayer& l : layers)  // a cache's rows are written before they are read; the rest is read as it is
        for (DevBuf* b : {&l.conv_state, &l.S, &l.n, &l.m})
            if (b->p) STACK_HIP(hipMemsetAsync(b->p, 0, b->bytes, stream), "clear states");
    return MI355X_OK;
}

// The tensors' names and where each goes. Sizes are known from the configuration.
void Stack::name_tensors() {
    const int64_t W = width();
    auto mat = [&](const std::string& s, Mat& m, int64_t row0, int64_t rows, int64_t cols, int64_t step = 1, int64_t col0 = 0) {
        Slot v;
        v.mat = &m; v.row0 = row0; v.rows = rows; v.cols = cols; v.step = step; v.col0 = col0;
        slots[s] = v;
        m.n = std::max(m.n, row0 + (rows - 1) * step + 1);
        m.k = std::max(m.k, col0 + cols);
        m.ld = pad64(m.k);
    };
    auto vec = [&](const std::string& s, Vec& d, int64_t n, bool needed = true, float factor = 1.f) {
        Slot v;
        v.vec = &d; v.rows = 1; v.cols = n; v.needed = needed; v.factor = factor;
        slots[s] = v;
        d.n = n;
    };
    mat("embed", embed, 0, vocab, W);
    if (c.pair_buckets > 0) mat("bigram", pairs, 0, c.pair_buckets + 1, W);
    if (has(MI355X_STACK_EMBED_NORM)) vec("embed.norm", embed_norm, W);
    vec("final.norm", final_norm, W, true, (float)c.logit_scale);
    if (has(MI355X_STACK_OUTPUT_MATRIX)) mat("head", head_w, 0, vocab, W);
    for (size_t i = 0; i < layers.size(); i++) {
        StackLayer& l = layers[i];
        const std::string p = "l" + std::to_string(i) + ".", mp = p + "mix.";
        const int64_t H = l.c.heads, qk = H * l.c.dim, mixed = l.mixed();
        vec(p + "norm1", l.norm1, W);
        if (has(MI355X_STACK_POST_NORMS)) vec(p + "norm1b", l.norm1b, W);
        if (c.taps > 0) vec(p + "canon1", l.canon, W * c.taps);
        if (has(MI355X_STACK_DEPTH_AVERAGE)) vec(p + "dwa", l.dwa, (int64_t)i + 2);
        if (has(MI355X_STACK_LAYER_SCALE)) {
            vec(p + "ls1", l.ls1, W);
            vec(p + "ls2", l.ls2, W, l.c.ff > 0);
        }
        mat(mp + "o", l.o, 0, W, mixed);
        if (l.by_heads()) {
            const int64_t kn = (int64_t)l.c.kv_heads * l.c.dim, vn = (int64_t)l.c.kv_heads * l.c.vdim, gates = l.c.head_gate ? H : 0;
            mat(mp + "q", l.in, 0, qk, W);
            mat(mp + "k", l.in, qk, kn, W);
            mat(mp + "v", l.in, qk + kn, vn, W);
            vec(mp + "vmix", l.vmix, 1, l.c.value_mix && !l.mixes_first);
            if (gates) mat(mp + "g", l.in, qk + kn + vn, gates, W);
            l.in.n = l.proj_n = (qk + kn + vn + gates + 3) / 4 * 4;
        }
        if (l.c.ff > 0) {
            Mat& first = parallel() ? l.in : l.up;
            if (l.c.mlp == MI355X_MLP_SWIGLU) {
                mat(p + "mlp.gate", first, l.proj_n * parallel(), l.c.ff, W, 2);
                mat(p + "mlp.up", first, l.proj_n * parallel() + 1, l.c.ff, W, 2);
            } else {
                mat(p + "mlp.up", first, 0, l.c.ff, W);
            }
            if (parallel()) {
                l.down_at = pad64(mixed);
                mat(p + "mlp.down", l.o, 0, W, l.c.ff, 1, l.down_at);
            } else {
                if (has(MI355X_STACK_POST_NORMS)) vec(p + "norm2b", l.norm2b, W);
                vec(p + "norm2", l.norm2, W);
                mat(p + "mlp.down", l.down, 0, W, l.c.ff);
            }
        }
        if (l.by_heads()) continue;
        if (!l.recurrent()) {
            const int64_t qn = H * (l.c.dim + l.c.rot_dim);
            mat(mp + "q", l.in, 0, qn, W);
            mat(mp + "dkv", l.in, qn, l.c.kv_rank + l.c.rot_dim, W);
            vec(mp + "dkv.norm", l.dkv_norm, l.c.kv_rank);
            mat(mp + "uk", l.ukv, 0, qk, l.c.kv_rank);
            mat(mp + "uv", l.ukv, qk, mixed, l.c.kv_rank);
            continue;
        }
        mat(mp + "q", l.in, 0, qk, W);
        mat(mp + "k", l.in, qk, qk, W);
        mat(mp + "v", l.in, 2 * qk, mixed, W);
        l.g_at = 2 * qk + mixed;
        mat(mp + "g", l.in, l.g_at, mixed, W);
        l.gates_at = l.g_at + mixed;
        vec(mp + "norm", l.mix_norm, mixed);
        if (l.c.mixer == MI355X_MIXER_MLSTM) {
            mat(mp + "i", l.in, l.gates_at, H, W);
            mat(mp + "f", l.in, l.gates_at + H, H, W);
            vec(mp + "i.b", l.bias_i, H);
            vec(mp + "f.b", l.bias_f, H);
        }
    }
}

mi355x_status Stack::set_tensor(const char* tensor, int dtype, const void* host, int64_t n_elems) {
    auto it = slots.find(tensor);
    if (it == slots.end()) return capi_fail(MI355X_ERR_SHAPE, "mi355x: stack: unknown tensor %s", tensor);
    Slot& v = it->second;
    if (v.rows * v.cols != n_elems)
        return capi_fail(MI355X_ERR_SHAPE, "mi355x: stack: %s of %lld elements, want [%lld, %lld]", tensor, (long long)n_elems, (long long)v.rows, (long long)v.cols);
    if (dtype != kBF16 && !(v.vec && dtype == kF32)) return capi_fail(MI355X_ERR_DTYPE, "mi355x: stack: %s of dtype %d, want bfloat16", tensor, dtype);
    if (v.vec) {
        std::vector<float> f((size_t)n_elems);
        if (dtype == kF32) {
            memcpy(f.data(), host, f.size() * 4);
        } else {
            for (int64_t i = 0; i < n_elems; i++) {
                const uint32_t bits = (uint32_t)((const uint16_t*)host)[i] << 16;
                memcpy(&f[(size_t)i], &bits, 4);
            }
        }
        for (float& x : f) x *= v.factor;
        if (!v.vec->buf.p) STACK_HIP(v.vec->buf.alloc(f.size() * 4), "hipMalloc(weight)");
        STACK_HIP(hipMemcpy(v.vec->buf.p, f.data(), f.size() * 4, hipMemcpyHostToDevice), "hipMemcpy(weight)");
    } else {
        Mat& m = *v.mat;
        if (!m.buf.p) {
            STACK_HIP(m.buf.alloc((size_t)m.n * m.ld * 2), "hipMalloc(weight)");
            STACK_HIP(hipMemset(m.buf.p, 0, (size_t)m.n * m.ld * 2), "hipMemset(weight)");
        }
        STACK_HIP(hipMemcpy2D(m.buf.as<uint16_t>() + v.row0 * m.ld + v.col0, (size_t)(v.step * m.ld) * 2, host, (size_t)v.cols * 2, (size_t)v.cols * 2, (size_t)v.rows,
                              hipMemcpyHostToDevice), "hipMemcpy(weight)");
    }
    v.set = true;
    ready = false;
    return MI355X_OK;
}

// The cosines and sines of all positions' angles. Frequencies base^(-2 i / rot_dim), with Llama 3.1's scaling where it is asked for:
// wavelengths beyond original / low positions are stretched by the factor, those below original / high are not, and
// between the two the share of each goes with original / wavelength.
mi355x_status Stack::rotation(StackLayer& l) {
    if (l.c.rot_dim == 0) return MI355X_OK;
    const int half_n = l.c.rot_dim / 2;
    std::vector<float> cs((size_t)context * half_n), sn((size_t)context * half_n);
    for (int i = 0; i < half_n; i++) {
        double f = std::pow(l.c.rot_base, -2.0 * i / (double)l.c.rot_dim);
        if (l.c.rot_factor > 0) {
            const double turns = l.c.rot_original * f / (2 * M_PI);  // original / wavelength
            if (turns < l.c.rot_low) f /= l.c.rot_factor;
            else if (turns <= l.c.rot_high && l.c.rot_high > l.c.rot_low) {
                const double share = (turns - l.c.rot_low) / (l.c.rot_high - l.c.rot_low);
                f = (1 - share) * f / l.c.rot_factor + share * f;
            }
        }
        for (int64_t p = 0; p < context; p++) {
            cs[p * half_n + i] = (float)std::cos((double)p * f);
            sn[p * half_n + i] = (float)std::sin((double)p * f);
        }
    }
    STACK_HIP(l.cos_t.alloc(cs.size() * 4), "hipMalloc");
    STACK_HIP(l.sin_t.alloc(sn.size() * 4), "hipMalloc");
    STACK_HIP(hipMemcpy(l.cos_t.p, cs.data(), cs.size() * 4, hipMemcpyHostToDevice), "hipMemcpy(angles)");
    STACK_HIP(hipMemcpy(l.sin_t.p, sn.data(), sn.size() * 4, hipMemcpyHostToDevice), "hipMemcpy(angles)");
    return MI355X_OK;
}

// s1 / s2 for the one product of a parallel layer's two results; two products where a quotient would drown the other part.
mi355x_status Stack::layer_scales(StackLayer& l) {
    l.two_products = false;
    if (!parallel() || !has(MI355X_STACK_LAYER_SCALE) || l.c.ff == 0) return MI355X_OK;
    const int64_t W = width();
    std::vector<float> s1(W), s2(W);
    STACK_HIP(hipMemcpy(s1.data(), l.ls1.buf.p, W * 4, hipMemcpyDeviceToHost), "hipMemcpy(scales)");
    STACK_HIP(hipMemcpy(s2.data(), l.ls2.buf.p, W * 4, hipMemcpyDeviceToHost), "hipMemcpy(scales)");
    for (int64_t i = 0; i < W; i++) {
        if (!(std::fabs(s2[i]) > 1e-12f * std::fabs(s1[i]))) l.two_products = true;
        s1[i] /= s2[i];
    }
    if (l.two_products) return MI355X_OK;
    STACK_HIP(l.out_mid.alloc(W * 4), "hipMalloc");
    STACK_HIP(hipMemcpy(l.out_mid.p, s1.data(), W * 4, hipMemcpyHostToDevice), "hipMemcpy(scales)");
    return MI355X_OK;
}

mi355x_status Stack::finalize(int64_t max_tokens) {
    for (const auto& kv : slots)
        if (kv.second.needed && !kv.second.set) return capi_fail(MI355X_ERR_SHAPE, "mi355x: stack: tensor %s missing", kv.first.c_str());
    const int64_t W = width();
    int64_t per = 8192 / batch;  // rows of a pass: longer calls go in portions
    per = per < 1 ? 1 : per;
    if (max_tokens > context) max_tokens = context;
    const int64_t R = batch * (max_tokens < per ? max_tokens : per);
    const int64_t logit_n = R < 256 ? R : 256 > batch ? 256 : batch;
    if (mi355x_status st = alloc_common(R, logit_n < batch ? batch : logit_n)) return st;
    auto zeroed = [&](DevBuf& b, size_t bytes) -> mi355x_status {
        STACK_HIP(b.alloc(bytes), "hipMalloc");
        STACK_HIP(hipMemset(b.p, 0, b.bytes), "hipMemset");
        return MI355X_OK;
    };
#define STACK_BUF(buf, n)                                              \
    do {                                                               \
        if (mi355x_status st_ = zeroed(buf, (size_t)(n))) return st_;  \
    } while (0)
    int64_t in_n = 0, mixed = 0, mix_ld = 0, ff = 0, gate_n = 0, q_n = 0, keys_n = 0, values_n = 0, first_n = 0;
    size_t ws_floats = 0;
    bool recurrent = false;
    for (StackLayer& l : layers) {
        recurrent = recurrent || l.recurrent();
        in_n = std::max(in_n, l.by_heads() ? l.proj_n : l.in.n);
        mix_ld = std::max(mix_ld, l.o.ld);
        mixed = l.mixed() > mixed ? l.mixed() : mixed;
        ff = std::max(ff, parallel() ? (int64_t)0 : (int64_t)l.c.ff);
        const int64_t H = l.c.heads;
        if (c.taps > 1) STACK_BUF(l.conv_state, (size_t)batch * (c.taps - 1) * W * 4);
        if (mi355x_status st = layer_scales(l)) return st;
        if (l.by_heads()) {
            l.ldc = (l.c.dim + 7) / 8 * 8;
            const size_t positions = (size_t)batch * l.c.kv_heads * pad64(context) * (half() ? 2 : 4);
            STACK_BUF(l.cache, positions * l.ldc);
            STACK_BUF(l.values, positions * l.c.vdim);
            if (mi355x_status st = rotation(l)) return st;
            const HeadAttention a = attention(l, 1, nullptr);
            const size_t need = heads_attend_ws_floats(a, heads_prompt_ok(a) ? std::min(R, (int64_t)batch * kManyRows) : R);
            ws_floats = need > ws_floats ? need : ws_floats;
            q_n = std::max(q_n, H * l.ldc);
            if (l.c.value_mix) first_n = std::max(first_n, (int64_t)l.c.kv_heads * l.c.vdim);
            continue;
        }
        if (!l.recurrent()) {
            l.ldc = (l.c.kv_rank + l.c.rot_dim + 7) / 8 * 8;
            // rows are read to a multiple of 64 elements of the latent: more than the last row has
            STACK_BUF(l.cache, ((size_t)batch * pad64(context) * l.ldc + pad64(l.ldc) + 64) * (half() ? 2 : 4));
            if (mi355x_status st = rotation(l)) return st;
            const size_t need = latent_absorbed_ws_floats(latent(l, 1, nullptr), R);
            ws_floats = need > ws_floats ? need : ws_floats;
            q_n = H * (l.c.dim + l.c.rot_dim) > q_n ? H * (l.c.dim + l.c.rot_dim) : q_n;
            keys_n = H * l.c.dim > keys_n ? H * l.c.dim : keys_n;
            values_n = l.mixed() > values_n ? l.mixed() : values_n;
            continue;
        }
        STACK_BUF(l.S, (size_t)batch * H * l.c.dim * l.c.vdim * 4);
        if (half()) {
            const size_t need = recurrence_chunk_ws_floats(batch, l.c.heads, l.c.dim, l.c.vdim, R / batch);
            ws_floats = need > ws_floats ? need : ws_floats;
        }
        if (l.c.mixer == MI355X_MIXER_MLSTM) {
            gate_n = 2 * H > gate_n ? 2 * H : gate_n;
            STACK_BUF(l.n, (size_t)batch * H * recurrence_slices(l.c.vdim) * l.c.dim * 4);
            STACK_BUF(l.m, (size_t)batch * H * recurrence_slices(l.c.vdim) * 4);
        } else {
            std::vector<float> d(H), pw((size_t)H * (kRecurrenceChunk + 1));
            for (int64_t i = 0; i < H; i++) {
                d[i] = (float)l.decay[i];
                for (int j = 0; j <= kRecurrenceChunk; j++) pw[i * (kRecurrenceChunk + 1) + j] = (float)std::pow((double)d[i], j);
            }
            STACK_BUF(l.decay_f, d.size() * 4);
            STACK_BUF(l.decay_pow, pw.size() * 4);
            STACK_HIP(hipMemcpy(l.decay_f.p, d.data(), d.size() * 4, hipMemcpyHostToDevice), "hipMemcpy(decays)");
            STACK_HIP(hipMemcpy(l.decay_pow.p, pw.data(), pw.size() * 4, hipMemcpyHostToDevice), "hipMemcpy(decays)");
        }
    }
    // rows are padded to a multiple of 64 elements that a product may read; the layers' sizes share the buffers
    if (has(MI355X_STACK_DEPTH_AVERAGE)) STACK_BUF(streams, (size_t)layers.size() * R * W * 4);
    STACK_BUF(x, (size_t)R * W * 4);
    if (c.taps > 0) STACK_BUF(h, (size_t)R * W * 4);
    if (!parallel()) STACK_BUF(y, (size_t)R * W * 4);
    if (c.pair_buckets > 0) STACK_BUF(held, (size_t)batch * context * 4);
    STACK_BUF(first_values, (size_t)R * first_n * 4);
    STACK_BUF(in_f, (size_t)R * pad64(W) * 4);
    STACK_BUF(proj_f, (size_t)R * in_n * 4);
    if (recurrent) STACK_BUF(scanned, (size_t)R * mixed * 4);
    STACK_BUF(mix_f, (size_t)R * mix_ld * 4);
    STACK_BUF(up_f, (size_t)R * pad64(ff) * 4);
    STACK_BUF(last_f, (size_t)logit_rows * pad64(W) * 4);
    STACK_BUF(rows_dev, (size_t)logit_rows * 8);
    STACK_BUF(ws, ws_floats * 4);
    if (half() && R > kGemvRows) {
        STACK_BUF(in_b, (size_t)R * pad64(W) * 2);
        STACK_BUF(mix_b, (size_t)R * mix_ld * 2);
        STACK_BUF(up_b, (size_t)R * pad64(ff) * 2);
        if (recurrent) STACK_BUF(proj_b, (size_t)R * pad64(in_n) * 2);
        STACK_BUF(gates, (size_t)R * gate_n * 4);
        STACK_BUF(last_b, (size_t)logit_rows * pad64(W) * 2);
        STACK_BUF(q_b, (size_t)R * q_n * 2);
        if (keys_n > 0) {
            STACK_BUF(keys_b, (size_t)batch * pad64(context) * keys_n * 2);
            STACK_BUF(values_b, (size_t)values_n * batch * pad64(context) * 2);  // read in whole tiles of 64 keys
        }
    }
#undef STACK_BUF
    cache_len = 0;
    ready = true;
    return MI355X_OK;
}

}  // namespace

}  // namespace mimir

extern "C" {

mi355x_status mi355x_stack_create(const mi355x_stack_config* cfg, const mi355x_stack_layer* layers, void** out) {
    using namespace mimir;
    if (!cfg || !layers || !out) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: stack_create: null pointer");
    const auto& c = *cfg;
    const bool parallel = c.flags & MI355X_STACK_PARALLEL;
    if (c.width <= 0 || c.width > 15360 || c.vocab <= 0 || c.layers <= 0 || c.layers > 1024 || c.context <= 0 || c.batch <= 0 || c.batch > 8192 || c.taps < 0 ||
        c.pair_buckets < 0 || c.pair_buckets >= INT32_MAX || (c.pair_buckets > 0 && (c.pair_mul_prev < 0 || c.pair_mul_cur < 0 || c.pair_mul_prev > INT32_MAX || c.pair_mul_cur > INT32_MAX)) ||
        (parallel && (c.taps > 0 || (c.flags & (MI355X_STACK_POST_NORMS | MI355X_STACK_DEPTH_AVERAGE)))) || c.norm_groups <= 0 || c.norm_groups > 512 || c.width % c.norm_groups != 0 || !(c.eps > 0))
        return capi_fail(MI355X_ERR_SHAPE, "mi355x: stack: hyperparameters: width %d in %d groups, %d layers, %d taps, vocabulary %d, context %d, batch %d",
                         c.width, c.norm_groups, c.layers, c.taps, c.vocab, c.context, c.batch);
    if (c.dtype != MI355X_F32 && c.dtype != MI355X_BF16) return capi_fail(MI355X_ERR_DTYPE, "mi355x: stack: compute dtype %d", c.dtype);
    auto m = std::make_unique<Stack>();
    m->c = c;
    m->name = "stack"; m->vocab = c.vocab; m->context = c.context; m->batch = c.batch;
    m->layers.resize(c.layers);
    int first_mixed = -1;
    for (int i = 0; i < c.layers; i++) {
        const auto& l = layers[i];
        bool ok = l.heads > 0 && l.heads <= 4096 && l.dim > 0 && l.vdim > 0 && l.ff >= 0 && (int64_t)l.heads * l.vdim <= 15360;
        if (l.mixer == MI355X_MIXER_ATTENTION)
            ok = ok && l.kv_heads > 0 && l.heads % l.kv_heads == 0 && l.dim <= kHeadAttentionMax && l.vdim <= kHeadAttentionMax && l.rot_dim >= 0 && l.rot_dim % 2 == 0 &&
                 l.rot_dim <= l.dim && (l.rot_dim == 0 || l.rot_base > 0) && l.softcap >= 0;
        else if (parallel) ok = false;
        else if (l.mixer == MI355X_MIXER_LATENT) ok = ok && l.rot_dim > 0 && l.rot_dim % 2 == 0 && l.kv_rank > 0 && l.kv_rank <= 1024 && l.rot_dim <= 1024 && l.rot_base > 0;
        else if (l.mixer == MI355X_MIXER_MLSTM) ok = ok && l.dim <= kRecurrenceMaxDim && l.gate_cap > 0;
        else if (l.mixer == MI355X_MIXER_LIGHTNING) ok = ok && l.dim <= kRecurrenceMaxDim && l.decay;
        else ok = false;
        ok = ok && (l.mlp == MI355X_MLP_RELU2 || l.mlp == MI355X_MLP_SWIGLU) && !(parallel && l.ff > 0 && l.mlp != MI355X_MLP_SWIGLU);
        if (l.mixer == MI355X_MIXER_ATTENTION && l.value_mix) {  // all of them mix the first one's values
            if (first_mixed < 0) first_mixed = i;
            const auto& f = layers[first_mixed];
            ok = ok && l.kv_heads == f.kv_heads && l.vdim == f.vdim;
            m->layers[i].mixes_first = first_mixed == i;
        }
        if (!ok)
            return capi_fail(MI355X_ERR_SHAPE, "mi355x: stack: layer %d: mixer %d with %d heads (%d) of %d and %d features, %d rotated, latent of %d, feed-forward %d", i,
                             l.mixer, l.heads, l.kv_heads, l.dim, l.vdim, l.rot_dim, l.kv_rank, l.mlp);
        m->layers[i].c = l;
        if (l.mixer == MI355X_MIXER_LIGHTNING) m->layers[i].decay.assign(l.decay, l.decay + l.heads);
        m->layers[i].c.decay = nullptr;
    }
    m->name_tensors();
    *out = (Decoder*)m.release();
    return MI355X_OK;
}

mi355x_status mi355x_stack_tensor(void* model, int64_t i, char* name, size_t size, int64_t* rows, int64_t* cols) {
    using namespace mimir;
    if (!model || !name || size == 0 || !rows || !cols) return capi_fail(MI355X_ERR_INTERNAL, "mi355x: stack_tensor: null pointer");
    const auto& slots = ((Stack*)(Decoder*)model)->slots;
    if (i < 0 || i >= (int64_t)slots.size()) return capi_fail(MI355X_ERR_INDEX, "mi355x: stack_tensor: tensor %lld of %zu", (long long)i, slots.size());
    auto it = slots.begin();
    std::advance(it, i);
    snprintf(name, size, "%s", it->first.c_str());
    *rows = it->second.rows;
    *cols = it->second.cols;
    return MI355X_OK;
}

}  // extern "C"
