// The Ruvenex decoder: a session over a model folder.  A layer reads one norm with all of its sublayers and adds
//
//   x += sig(G1 h + b1) * (ls * W_o attn(h) + rs * W_o' hgrn2(h)) + sig(G2 h + b2) * W_down gelu(W_up h),  h = norm(x)
//
// so everything that reads h is one stacked product with the activations in its epilogue, everything that ends in x
// one product over the concatenated mixer outputs with the gates and scales in its epilogue, and between the two
// stand the mixers: three launches a layer and token, the norm included.  Several tokens (prompt passes, portions)
// take the matrix-core products and the mixers' several-token kernels.
#include <cmath>
#include <map>
#include <string>
#include <utility>
#include <vector>

#include "device_dense.h"
#include "device_sample.h"
#include "model_folder.h"
#include "seq_mixers.h"
#include "session.h"

namespace {

constexpr uint32_t kPassMax = 2048;   // most positions of a pass
constexpr uint32_t kLogitRows = 64;   // most positions whose logits are computed together

struct RuvenexLayer {
    float *norm = nullptr;
    RmiDense w_in, w_out;  // all that reads h, row segments below; all that ends in x, columns attn | hgrn2 | ff
    RmiRowSegs in;
    RmiColSegs out;
    RmiAttnShape attn{};
    RmiRecurShape recur{};
    float *conv = nullptr, *cos_t = nullptr, *sin_t = nullptr, *recur_norm = nullptr;
    void *k_cache = nullptr, *v_cache = nullptr;
    float *hist[2] = {nullptr, nullptr};
    float *state[2] = {nullptr, nullptr};
    uint32_t k_attn = 0, k_recur = 0;  // where the recurrence's and the feed-forward's columns begin
};

// the embedding of the next token, the argmax kernel's last act
template <typename T>
struct EmbedDense {
    const T *table;
    uint32_t ld, vocab;
    float scale;
    float *x;
    uint32_t n;
    __device__ __forceinline__ void operator()(uint32_t token) const {
        if (token >= vocab) token = vocab - 1;
        for (uint32_t i = threadIdx.x; i < n; i += 256) x[i] = to_f32(table[size_t(token) * ld + i]) * scale;
    }
};

}  // namespace

struct rmi_hip_ruvenex : RmiSession {
    uint32_t elem = 2;  // bytes of a weight / activation element
    uint32_t width = 0, n_layer = 0, k_in = 0, cap_pad = 0, pass_rows = 0, logit_rows = 0;
    float eps = 0, embed_scale = 1;
    std::vector<RuvenexLayer> layers;
    RmiDense embed, head;
    float *final_norm = nullptr;
    // activations of a pass, token-major
    float *x = nullptr, *u = nullptr, *gate = nullptr, *rq = nullptr, *rf = nullptr, *rv = nullptr, *rg1 = nullptr, *rg2 = nullptr;
    void *h = nullptr, *act = nullptr, *q = nullptr;
    float *logits = nullptr;
    void *attn_scratch = nullptr;
    float *recur_scratch = nullptr;
    uint32_t *want_rows = nullptr;
    uint32_t position = 0;         // tokens of the current sequence so far
    int now = 0;              // which of a layer's two history and state buffers the last pass left
    uint32_t embedded = ~0u;       // the position whose embedding the last sampling launch left in x

    void begin_sequence() override {
        position = 0;
        embedded = ~0u;
    }
    int enqueue_layers(uint32_t step0, uint32_t n, hipStream_t st, float *host_layers = nullptr);
    int enqueue_logits(const uint32_t *rows, uint32_t n_rows, hipStream_t st);
    int enqueue_sample(uint32_t step0, const uint32_t *rows, uint32_t n_rows, hipStream_t st);
    int embed_tokens(uint32_t step0, uint32_t n, hipStream_t st) {
        return rmi_dense_embed(elem, embed, tok + step0, vocab, embed_scale, x, n, width, st);
    }
    int set_rows(const uint32_t *want, uint32_t n_want, hipStream_t st);

    int enqueue_step(uint32_t step, hipStream_t st) override;
    const float *step_logits() const override { return logits; }
    bool pass_possible(uint32_t step0, uint32_t n) const override { return n <= pass_rows && step0 + n <= capacity; }
    int enqueue_pass(uint32_t step0, uint32_t n, const uint32_t *want, uint32_t n_want, bool sample, hipStream_t st) override;
    uint32_t max_pass_want() const override { return logit_rows; }
    const float *pass_logits(uint32_t, uint32_t i) const override { return logits + size_t(i) * vocab; }
    int feed(const uint32_t *tokens, uint32_t n, const uint32_t *want, uint32_t n_want, float *out, float *host_layers);
    bool load(const RmiModelFolder &f, uint32_t elem_bytes, uint32_t cap);
};

// The layers over positions step0 .. step0 + n - 1, whose embeddings are in x.  host_layers: the residual stream
// behind every layer, [layer][n][width] (synchronises; for comparisons).
int rmi_hip_ruvenex::enqueue_layers(uint32_t step0, uint32_t n, hipStream_t st, float *host_layers) {
    int rc = RMI_HIP_OK;
    for (uint32_t l = 0; l < n_layer && rc == RMI_HIP_OK; l++) {
        const RuvenexLayer &y = layers[l];
        RmiAttnArgs a{};
        a.u = u;
        a.hist_in = y.hist[now];
        a.hist_out = y.hist[now ^ 1];
        a.conv = y.conv;
        a.cos_t = y.cos_t;
        a.sin_t = y.sin_t;
        a.q = q;
        a.k_cache = y.k_cache;
        a.v_cache = y.v_cache;
        a.gate = gate;
        a.out = act;
        a.out_ld = y.w_out.ld;
        a.pos0 = step0;
        a.n_tokens = n;
        a.scratch = attn_scratch;
        RmiRecurArgs r{};
        r.q = rq;
        r.f = rf;
        r.v = rv;
        r.state_in = y.state[now];
        r.state_out = y.state[now ^ 1];
        r.norm = y.recur_norm;
        r.out = static_cast<uint8_t *>(act) + size_t(y.k_attn) * elem;
        r.out_ld = y.w_out.ld;
        r.pos0 = step0;
        r.n_tokens = n;
        r.scratch = recur_scratch;
        if (n == 1 && rmi_dense_gemv_fits(elem, k_in)) {
            rc = rmi_dense_norm_gemv(elem, y.w_in, x, y.norm, eps, width, y.in, st);
            if (rc == RMI_HIP_OK) rc = rmi_mixers_step(elem, &y.attn, &a, &y.recur, &r, st);
            if (rc == RMI_HIP_OK) rc = rmi_dense_gemv_residual(elem, y.w_out, act, y.out, x, width, st);
        } else {
            rc = rmi_dense_norm(elem, x, nullptr, y.norm, eps, h, n, width, k_in, st);
            if (rc == RMI_HIP_OK) rc = rmi_dense_gemm(elem, y.w_in, h, y.in, n, st);
            if (rc == RMI_HIP_OK) rc = rmi_attn_pass(elem, y.attn, a, st);
            if (rc == RMI_HIP_OK) rc = rmi_recur_pass(elem, y.recur, r, st);
            if (rc == RMI_HIP_OK) rc = rmi_dense_gemm_residual(elem, y.w_out, act, y.out, x, width, n, st);
        }
        if (host_layers && rc == RMI_HIP_OK) {
            RMI_HIP_CHECK(hipStreamSynchronize(st));
            RMI_HIP_CHECK(hipMemcpy(host_layers + size_t(l) * n * width, x, size_t(n) * width * 4, hipMemcpyDeviceToHost));
        }
    }
    now ^= 1;
    position = step0 + n;
    return rc;
}

// logits[i] = head . norm(x[rows[i]]); rows in HBM, nullptr: 0 .. n_rows - 1
int rmi_hip_ruvenex::enqueue_logits(const uint32_t *rows, uint32_t n_rows, hipStream_t st) {
    RmiRowSegs s{};
    s.n_segs = 1;
    s.n_rows = head.n_rows;
    s.s[0] = RmiRowSeg{logits, nullptr, nullptr, 0, vocab, vocab, uint16_t(kActNone), 0};
    rmi_row_segs_done(&s);
    if (n_rows == 1 && !rows && rmi_dense_gemv_fits(elem, k_in)) return rmi_dense_norm_gemv(elem, head, x, final_norm, eps, width, s, st);
    const int rc = rmi_dense_norm(elem, x, rows, final_norm, eps, h, n_rows, width, k_in, st);
    return rc == RMI_HIP_OK ? rmi_dense_gemm(elem, head, h, s, n_rows, st) : rc;
}

int rmi_hip_ruvenex::enqueue_sample(uint32_t step0, const uint32_t *rows, uint32_t n_rows, hipStream_t st) {
    hipLaunchKernelGGL(argmax_partial_kernel, dim3(kArgmaxGroups, n_rows), dim3(256), 0, st, logits, vocab, static_cast<Top *>(partial));
    auto finish = [&](auto embed_next) {
        hipLaunchKernelGGL((argmax_final_batch_kernel<decltype(embed_next)>), dim3(n_rows), dim3(256), 0, st,
                           static_cast<const Top *>(partial), kArgmaxGroups, static_cast<StepParams *>(params), step0, rows, tok, step_argmax,
                           step_top2, nonfinite, embed_next);
    };
    if (elem == 2)
        finish(EmbedDense<rmi_bf16>{static_cast<const rmi_bf16 *>(embed.data), embed.ld, vocab, embed_scale, x, width});
    else
        finish(EmbedDense<float>{static_cast<const float *>(embed.data), embed.ld, vocab, embed_scale, x, width});
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int rmi_hip_ruvenex::set_rows(const uint32_t *want, uint32_t n_want, hipStream_t st) {
    RMI_HIP_CHECK(hipMemcpyAsync(want_rows, want, size_t(n_want) * 4, hipMemcpyHostToDevice, st));
    RMI_HIP_CHECK(hipStreamSynchronize(st));  // the host array is the caller's
    return RMI_HIP_OK;
}

int rmi_hip_ruvenex::enqueue_step(uint32_t step, hipStream_t st) {
    int rc = embedded == step ? RMI_HIP_OK : embed_tokens(step, 1, st);
    if (rc == RMI_HIP_OK) rc = enqueue_layers(step, 1, st);
    if (rc == RMI_HIP_OK) rc = enqueue_logits(nullptr, 1, st);
    if (rc == RMI_HIP_OK) rc = enqueue_sample(step, nullptr, 1, st);
    embedded = step + 1;
    return rc;
}

int rmi_hip_ruvenex::enqueue_pass(uint32_t step0, uint32_t n, const uint32_t *want, uint32_t n_want, bool sample, hipStream_t st) {
    int rc = embed_tokens(step0, n, st);
    if (rc == RMI_HIP_OK) rc = enqueue_layers(step0, n, st);
    std::vector<uint32_t> rows(want, want + n_want);
    if (sample && (rows.empty() || rows.back() != n - 1)) rows.push_back(n - 1);
    embedded = ~0u;
    if (rc != RMI_HIP_OK || rows.empty()) return rc;
    if (rows.size() > logit_rows) return rmi_fail(RMI_HIP_E_INVALID, "logits of more than %u positions of a pass", logit_rows);
    rc = set_rows(rows.data(), uint32_t(rows.size()), st);
    if (rc == RMI_HIP_OK) rc = enqueue_logits(want_rows, uint32_t(rows.size()), st);
    if (rc == RMI_HIP_OK) rc = enqueue_sample(step0, want_rows, uint32_t(rows.size()), st);
    if (rows.back() == n - 1) embedded = step0 + n;
    return rc;
}

// The next n tokens of the sequence, with no sampling: logits of the places in `want`, in that order.
int rmi_hip_ruvenex::feed(const uint32_t *tokens, uint32_t n, const uint32_t *want, uint32_t n_want, float *out, float *host_layers) {
    if (n && !tokens) return rmi_fail(RMI_HIP_E_INVALID, "null tokens");
    if (n_want && (!want || !out)) return rmi_fail(RMI_HIP_E_INVALID, "null want or logits");
    if (uint64_t(position) + n > capacity)
        return rmi_fail(RMI_HIP_E_INVALID, "%u + %u tokens exceed the capacity %u", position, n, capacity);
    for (uint32_t i = 0; i < n; i++)
        if (tokens[i] >= vocab) return rmi_fail(RMI_HIP_E_INVALID, "token id %u outside the vocabulary", tokens[i]);
    for (uint32_t i = 0; i < n_want; i++)
        if (want[i] >= n) return rmi_fail(RMI_HIP_E_INVALID, "place %u of a step of %u tokens", want[i], n);
    if (host_layers && n > pass_rows) return rmi_fail(RMI_HIP_E_INVALID, "the residual stream of at most %u tokens", pass_rows);
    RmiThreadCtx *ctx = rmi_thread_ctx();
    if (!ctx) return RMI_HIP_E_RUNTIME;
    hipStream_t st = ctx->stream;
    const uint32_t step0 = position;
    if (n) RMI_HIP_CHECK(hipMemcpyAsync(tok + step0, tokens, size_t(n) * 4, hipMemcpyHostToDevice, st));
    RMI_HIP_CHECK(hipStreamSynchronize(st));
    embedded = ~0u;
    const uint32_t most = prompt_pass ? (prompt_pass < pass_rows ? prompt_pass : pass_rows) : 1;
    for (uint32_t at = 0; at < n;) {
        const uint32_t m = n - at < most ? n - at : most;
        int rc = embed_tokens(step0 + at, m, st);
        if (rc == RMI_HIP_OK) rc = enqueue_layers(step0 + at, m, st, host_layers);
        if (rc != RMI_HIP_OK) return rc;
        std::vector<uint32_t> rows, slots;  // this pass's rows, and where their logits go
        for (uint32_t i = 0; i < n_want; i++)
            if (want[i] >= at && want[i] < at + m) {
                rows.push_back(want[i] - at);
                slots.push_back(i);
            }
        for (size_t i = 0; i < rows.size(); i += logit_rows) {
            const uint32_t k = uint32_t(rows.size() - i < logit_rows ? rows.size() - i : logit_rows);
            if (m > 1) rc = set_rows(rows.data() + i, k, st);
            if (rc == RMI_HIP_OK) rc = m > 1 ? enqueue_logits(want_rows, k, st) : enqueue_logits(nullptr, 1, st);
            if (rc != RMI_HIP_OK) return rc;
            RMI_HIP_CHECK(hipStreamSynchronize(st));
            for (uint32_t j = 0; j < k; j++)
                RMI_HIP_CHECK(hipMemcpy(out + size_t(slots[i + j]) * vocab, logits + size_t(m > 1 ? j : 0) * vocab, size_t(vocab) * 4,
                                        hipMemcpyDeviceToHost));
        }
        at += m;
    }
    RMI_HIP_CHECK(hipStreamSynchronize(st));
    return RMI_HIP_OK;
}

// ------------------------------------------------------------------ loading

namespace {

// What a constructor reads from the folder: the first thing missing or out of place ends it with a message.
struct Reader {
    const RmiModelFolder &f;
    bool ok = true;

    void fail(const std::string &what) {
        if (ok) rmi_set_error("%s", what.c_str());
        ok = false;
    }
    const RmiJson *object(const RmiJson *o, const char *key) {
        const RmiJson *v = o ? o->get(key) : nullptr;
        if (!v || v->type != RmiJson::kObject) {
            fail(std::string("config.json: no object '") + key + "'");
            return nullptr;
        }
        return v;
    }
    double number(const RmiJson *o, const char *key) {
        const RmiJson *v = o ? o->get(key) : nullptr;
        if (!v || v->type != RmiJson::kNumber) {
            fail(std::string("config.json: no number '") + key + "'");
            return 0;
        }
        return v->number;
    }
    uint32_t size(const RmiJson *o, const char *key, bool zero_ok = false) {
        const double v = number(o, key);
        if (ok && (v != std::floor(v) || v < (zero_ok ? 0 : 1) || v > 0x7fffffff)) fail(std::string("config.json: '") + key + "' is not a size");
        return ok ? uint32_t(v) : 1;
    }
    const RmiTensor *tensor(const std::string &name, std::vector<uint64_t> shape) {
        const RmiTensor *t = f.tensors.find(name);
        if (!t) {
            fail("Missing tensor: " + name);
            return nullptr;
        }
        if (t->shape != shape || t->dtype > RmiTensor::kF32) {
            fail("Invalid tensor " + name + ": shape or type");
            return nullptr;
        }
        return t;
    }
};

void f32_to_bf16_host(const RmiTensor &t, uint64_t at, uint64_t n, uint16_t *dst) {
    if (t.dtype == RmiTensor::kBf16) {
        memcpy(dst, t.data + 2 * at, 2 * n);
        return;
    }
    for (uint64_t i = 0; i < n; i++) {
        const float v = rmi_tensor_f32(t, at + i);
        uint32_t b;
        memcpy(&b, &v, 4);
        dst[i] = uint16_t((b + 0x7fff + ((b >> 16) & 1)) >> 16);
    }
}

// A dense weight put together on the host from blocks of tensors, then uploaded.
struct DenseBuilder {
    uint32_t elem, n_rows, k_pad, ld;
    std::vector<uint8_t> bytes;
    DenseBuilder(uint32_t e, uint32_t rows, uint32_t k)
        : elem(e), n_rows(rows), k_pad(k), ld(rmi_dense_ld(k, e)), bytes(size_t(rows) * ld * e, 0) {}
    void put(const RmiTensor *t, uint32_t row0, uint32_t col0) {
        if (!t) return;
        const uint64_t rows = t->shape[0], cols = t->shape[1];
        for (uint64_t r = 0; r < rows; r++) {
            uint8_t *dst = bytes.data() + (size_t(row0 + r) * ld + col0) * elem;
            if (elem == 2)
                f32_to_bf16_host(*t, r * cols, cols, reinterpret_cast<uint16_t *>(dst));
            else
                for (uint64_t i = 0; i < cols; i++) {
                    const float v = rmi_tensor_f32(*t, r * cols + i);
                    memcpy(dst + 4 * i, &v, 4);
                }
        }
    }
    bool upload(RmiSession *s, RmiDense *out) const {
        out->data = s->alloc_bytes(bytes.size(), false);
        out->n_rows = n_rows;
        out->k_pad = k_pad;
        out->ld = ld;
        if (!out->data) return false;
        if (hipMemcpy(out->data, bytes.data(), bytes.size(), hipMemcpyHostToDevice) != hipSuccess) {
            rmi_set_error("weight upload failed");
            return false;
        }
        return true;
    }
};

float *upload_vector(RmiSession *s, const RmiTensor *t) {
    if (!t) return nullptr;
    std::vector<float> v(t->count);
    for (uint64_t i = 0; i < t->count; i++) v[i] = rmi_tensor_f32(*t, i);
    return s->upload(v.data(), v.size());
}

}  // namespace

bool rmi_hip_ruvenex::load(const RmiModelFolder &folder, uint32_t elem_bytes, uint32_t cap) {
    Reader rd{folder};
    const RmiJson &c = folder.config;
    const RmiJson *arch = c.get("architecture");
    if (!arch || arch->text != "Ruvenex") {
        rmi_set_error("config.json: architecture '%s' is not Ruvenex", arch ? arch->text.c_str() : "");
        return false;
    }
    elem = elem_bytes;
    width = rd.size(&c, "width");
    vocab = rd.size(&c, "vocab");
    capacity = cap;
    cap_pad = rmi_dense_pad(cap, kKeyBlock);
    eps = float(rd.number(rd.object(&c, "norm"), "eps"));
    embed_scale = float(rd.number(rd.object(&c, "embedding"), "scale"));
    const RmiJson *ls = c.get("layers");
    if (!ls || ls->type != RmiJson::kArray) rd.fail("config.json: no list 'layers'");
    if (!rd.ok) return false;
    n_layer = uint32_t(ls->items.size());
    k_in = rmi_dense_pad(width, kDenseKAlign);
    pass_rows = cap < kPassMax ? cap : kPassMax;
    prompt_pass = pass_rows;
    if (uint64_t(vocab) * k_in > (uint64_t(1) << 40) || width > (1u << 20) || cap_pad > 0x7fffffffu / kMaxHeadDim) {
        rmi_set_error("unsupported model shape: a width or the cache overflows");
        return false;
    }

    // the embedding and the output
    for (int i = 0; i < 2; i++) {
        DenseBuilder b(elem, rmi_dense_pad(vocab, kDenseRowAlign), k_in);
        b.put(rd.tensor(i ? "head" : "embed", {vocab, width}), 0, 0);
        if (!rd.ok || !b.upload(this, i ? &head : &embed)) return false;
    }
    if (!(final_norm = upload_vector(this, rd.tensor("final.norm", {width})))) return false;

    // sizes first: the activation buffers are shared by the layers
    struct Sizes {
        uint32_t channels, n_recur, n_recur_v, ff;
        double rot_base;
    };
    std::vector<Sizes> sizes(n_layer);
    layers.resize(n_layer);
    uint32_t max_channels = 1, max_heads = 1, max_rq = 1, max_rv = 1, max_ld = kDenseKAlign;
    size_t max_q = 1, max_attn_scratch = 0, max_recur_scratch = 1;
    for (uint32_t l = 0; l < n_layer; l++) {
        const RmiJson *e = &ls->items[l], *type = e->get("type");
        if (!type || type->text != "parallel") rd.fail("config.json: layer " + std::to_string(l) + " has a type other than 'parallel'");
        const RmiJson *mix = rd.object(e, "mixer"), *left = rd.object(mix, "left"), *right = rd.object(mix, "right"), *rot = rd.object(left, "rot");
        RuvenexLayer &y = layers[l];
        Sizes &z = sizes[l];
        RmiAttnShape &a = y.attn;
        a.heads = rd.size(left, "heads");
        a.kv_heads = rd.size(left, "kv_heads");
        a.dim = rd.size(left, "dim");
        a.vdim = rd.size(left, "vdim");
        a.taps = rd.size(left, "conv");
        a.scale = float(rd.number(left, "scale"));
        a.rot_dims = rd.size(rot, "dims", true);
        z.rot_base = rd.number(rot, "base");
        a.eps = eps;
        a.capacity = cap_pad;
        RmiRecurShape &r = y.recur;
        r.heads = rd.size(right, "heads");
        r.dim = rd.size(right, "dim");
        r.vdim = rd.size(right, "vdim");
        r.eps = eps;
        const double left_scale = rd.number(mix, "left_scale"), right_scale = rd.number(mix, "right_scale");
        z.ff = 0;
        const RmiJson *mlp = e->get("mlp");
        if (mlp && !mlp->is_null()) {
            const RmiJson *kind = mlp->get("kind");
            if (!kind || kind->text != "dense") rd.fail("config.json: layer " + std::to_string(l) + " has a feed-forward that is not 'dense'");
            z.ff = rd.size(mlp, "ff");
        }
        if (!rd.ok) return false;
        if (a.heads % a.kv_heads || a.dim > kMaxHeadDim || a.vdim > kMaxHeadDim || r.dim > kMaxHeadDim || r.vdim > kMaxHeadDim ||
            a.taps > kMaxTaps || a.rot_dims > a.dim || a.rot_dims % 2 || a.heads > (1u << 16) || r.heads > (1u << 16) || z.ff > (1u << 24)) {
            rmi_set_error("unsupported model shape in layer %u (head sizes up to %u, up to %u taps)", l, kMaxHeadDim, kMaxTaps);
            return false;
        }
        a.dk_pad = rmi_dense_pad(a.dim, 32);
        a.dv_pad = rmi_dense_pad(a.vdim, 16);
        r.d_pad = rmi_dense_pad(r.dim, 16);
        r.v_pad = rmi_dense_pad(r.vdim, 16);
        z.channels = (a.heads + a.kv_heads) * a.dim + a.kv_heads * a.vdim;
        z.n_recur = r.heads * r.dim;
        z.n_recur_v = r.heads * r.vdim;
        y.k_attn = rmi_dense_pad(a.heads * a.vdim, kDenseKAlign);
        y.k_recur = y.k_attn + rmi_dense_pad(z.n_recur_v, kDenseKAlign);
        y.w_out.k_pad = y.k_recur + (z.ff ? rmi_dense_pad(z.ff, kDenseKAlign) : 0);
        const RmiColSeg sa{nullptr, float(left_scale), y.k_attn}, sr{nullptr, float(right_scale), y.k_recur}, sf{nullptr, 1.0f, y.w_out.k_pad};
        y.out.s[0] = sa;
        y.out.s[1] = sr;
        y.out.s[2] = sf;
        y.out.n_segs = z.ff ? 3 : 2;
        auto grow = [](auto &m, auto v) {
            if (v > m) m = v;
        };
        grow(max_channels, z.channels);
        grow(max_heads, a.heads);
        grow(max_rq, z.n_recur);
        grow(max_rv, z.n_recur_v);
        grow(max_ld, rmi_dense_ld(y.w_out.k_pad, elem));
        grow(max_q, size_t(pass_rows) * a.heads * a.dk_pad * elem);
        grow(max_attn_scratch, rmi_attn_scratch_bytes(a));
        grow(max_recur_scratch, rmi_recur_scratch_floats(r, pass_rows));
    }
    const size_t rows = pass_rows;
    logit_rows = pass_rows < kLogitRows ? pass_rows : kLogitRows;
    if (!alloc_sampling() || !(x = alloc<float>(rows * width, true)) || !(u = alloc<float>(rows * max_channels, true)) ||
        !(gate = alloc<float>(rows * max_heads, true)) || !(rq = alloc<float>(rows * max_rq, true)) || !(rf = alloc<float>(rows * max_rq, true)) ||
        !(rv = alloc<float>(rows * max_rv, true)) || !(rg1 = alloc<float>(rows * width, true)) || !(rg2 = alloc<float>(rows * width, true)) ||
        !(h = alloc_bytes(rows * rmi_dense_ld(k_in, elem) * elem, true)) || !(act = alloc_bytes(rows * max_ld * elem, true)) || !(q = alloc_bytes(max_q, true)) ||
        !(logits = alloc<float>(size_t(logit_rows) * vocab, true)) || !(attn_scratch = alloc_bytes(max_attn_scratch + 16, true)) ||
        !(recur_scratch = alloc<float>(max_recur_scratch, true)) || !(want_rows = alloc<uint32_t>(kLogitRows, true)) ||
        !(partial = alloc_bytes(size_t(logit_rows) * kArgmaxGroups * kTopBytes, false)))
        return false;

    std::map<std::pair<uint32_t, double>, std::pair<float *, float *>> rotations;
    for (uint32_t l = 0; l < n_layer; l++) {
        RuvenexLayer &y = layers[l];
        const Sizes &z = sizes[l];
        const RmiAttnShape &a = y.attn;
        const RmiRecurShape &r = y.recur;
        const std::string p = "l" + std::to_string(l) + ".", L = p + "mix.left.", R = p + "mix.right.";
        const uint32_t n_q = a.heads * a.dim, n_k = a.kv_heads * a.dim, n_v = a.kv_heads * a.vdim;
        float *f_bias = upload_vector(this, rd.tensor(R + "f.b", {z.n_recur})), *lower = upload_vector(this, rd.tensor(R + "lower", {z.n_recur}));
        float *b1 = upload_vector(this, rd.tensor(p + "rg1.b", {width})), *b2 = nullptr;
        if (z.ff) b2 = upload_vector(this, rd.tensor(p + "rg2.b", {width}));
        if (!f_bias || !lower || !b1 || (z.ff && !b2)) return false;

        // everything that reads h
        struct Part {
            std::string name;
            uint32_t n, ld;
            void *dst;
            uint16_t act, out_elem;
            const float *bias, *lower;
        };
        std::vector<Part> parts = {
            {L + "q", n_q, z.channels, u, kActNone, 0, nullptr, nullptr},
            {L + "k", n_k, z.channels, u + n_q, kActNone, 0, nullptr, nullptr},
            {L + "v", n_v, z.channels, u + n_q + n_k, kActNone, 0, nullptr, nullptr},
            {L + "g", a.heads, a.heads, gate, kActSigmoid, 0, nullptr, nullptr},
            {R + "q", z.n_recur, z.n_recur, rq, kActSilu, 0, nullptr, nullptr},
            {R + "f", z.n_recur, z.n_recur, rf, kActForgetGate, 0, f_bias, lower},
            {R + "v", z.n_recur_v, z.n_recur_v, rv, kActNone, 0, nullptr, nullptr},
            {p + "rg1", width, width, rg1, kActSigmoid, 0, b1, nullptr},
        };
        if (z.ff) {
            parts.push_back({p + "rg2", width, width, rg2, kActSigmoid, 0, b2, nullptr});
            parts.push_back({p + "mlp.up", z.ff, rmi_dense_ld(y.w_out.k_pad, elem), static_cast<uint8_t *>(act) + size_t(y.k_recur) * elem, kActGeluTanh, 1, nullptr, nullptr});
        }
        uint32_t n_rows = 0;
        for (const Part &q1 : parts) {
            RmiRowSeg &s = y.in.s[y.in.n_segs++];
            s.y = q1.dst;
            s.bias = q1.bias;
            s.lower = q1.lower;
            s.row0 = n_rows;
            s.n = q1.n;
            s.ld = q1.ld;
            s.act = q1.act;
            s.out_elem = q1.out_elem;
            n_rows += rmi_dense_pad(q1.n, kDenseRowAlign);
        }
        y.in.n_rows = n_rows;
        rmi_row_segs_done(&y.in);
        {
            DenseBuilder b(elem, n_rows, k_in);
            for (size_t i = 0; i < parts.size() && rd.ok; i++) b.put(rd.tensor(parts[i].name, {parts[i].n, width}), y.in.s[i].row0, 0);
            if (!rd.ok || !b.upload(this, &y.w_in)) return false;
        }
        // everything that ends in x
        y.out.s[0].gate = y.out.s[1].gate = rg1;
        if (z.ff) y.out.s[2].gate = rg2;
        {
            DenseBuilder b(elem, rmi_dense_pad(width, kDenseRowAlign), y.w_out.k_pad);
            b.put(rd.tensor(L + "o", {width, uint64_t(a.heads) * a.vdim}), 0, 0);
            b.put(rd.tensor(R + "o", {width, z.n_recur_v}), 0, y.k_attn);
            if (z.ff) b.put(rd.tensor(p + "mlp.down", {width, z.ff}), 0, y.k_recur);
            if (!rd.ok || !b.upload(this, &y.w_out)) return false;
        }
        if (!(y.norm = upload_vector(this, rd.tensor(p + "norm1", {width}))) || !(y.recur_norm = upload_vector(this, rd.tensor(R + "norm", {r.vdim}))))
            return false;
        // the three convolutions, one below the other
        std::vector<float> taps;
        const std::pair<const char *, uint32_t> convs[] = {{"q.conv", n_q}, {"k.conv", n_k}, {"v.conv", n_v}};
        for (const auto &cv : convs) {
            const RmiTensor *t = rd.tensor(L + cv.first, {cv.second, a.taps});
            if (!t) return false;
            for (uint64_t i = 0; i < t->count; i++) taps.push_back(rmi_tensor_f32(*t, i));
        }
        auto &rot = rotations[{a.rot_dims, z.rot_base}];
        if (!rot.first) {
            const uint32_t half = a.rot_dims / 2;
            std::vector<float> ct(size_t(cap_pad) * half), sn(ct.size());
            for (uint32_t i = 0; i < half; i++) {
                const double f = std::pow(z.rot_base, -2.0 * i / a.rot_dims);
                for (uint32_t t = 0; t < cap_pad; t++) {
                    ct[size_t(t) * half + i] = float(std::cos(t * f));
                    sn[size_t(t) * half + i] = float(std::sin(t * f));
                }
            }
            rot = {upload(ct.data(), ct.size()), upload(sn.data(), sn.size())};
        }
        y.cos_t = rot.first;
        y.sin_t = rot.second;
        const size_t hist = size_t(a.taps - 1) * z.channels;
        if (!y.cos_t || !y.sin_t || !(y.conv = upload(taps.data(), taps.size())) || !(y.hist[0] = alloc<float>(hist, true)) ||
            !(y.hist[1] = alloc<float>(hist, true)) || !(y.k_cache = alloc_bytes(size_t(a.kv_heads) * cap_pad * a.dk_pad * elem, true)) ||
            !(y.v_cache = alloc_bytes(size_t(a.kv_heads) * cap_pad * a.dv_pad * elem, true)) ||
            !(y.state[0] = alloc<float>(size_t(r.heads) * r.d_pad * r.v_pad, true)) ||
            !(y.state[1] = alloc<float>(size_t(r.heads) * r.d_pad * r.v_pad, true)))
            return false;
    }
    if (hipDeviceSynchronize() != hipSuccess) {
        rmi_set_error("weight upload failed");
        return false;
    }
    return rd.ok;
}

extern "C" {

rmi_hip_ruvenex *rmi_hip_ruvenex_open(const char *dir, int dtype, uint32_t capacity) {
    if (!rmi_ready()) {
        rmi_set_error("rmi_hip_init has not succeeded");
        return nullptr;
    }
    if (!dir || capacity == 0 || (dtype != RMI_HIP_DTYPE_BF16 && dtype != RMI_HIP_DTYPE_F32)) {
        rmi_set_error("null folder, no capacity, or an element type other than bf16 and f32");
        return nullptr;
    }
    if (!rmi_thread_ctx()) return nullptr;
    RmiModelFolder f;
    if (!f.open(dir)) return nullptr;
    rmi_hip_ruvenex *s = new rmi_hip_ruvenex();
    if (!s->load(f, dtype == RMI_HIP_DTYPE_F32 ? 4 : 2, capacity)) {
        delete s;
        return nullptr;
    }
    return s;
}

void rmi_hip_ruvenex_destroy(rmi_hip_ruvenex *s) { delete s; }

int rmi_hip_ruvenex_sizes(const rmi_hip_ruvenex *s, uint32_t *vocab, uint32_t *width, uint32_t *n_layer, uint32_t *capacity) {
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    if (vocab) *vocab = s->vocab;
    if (width) *width = s->width;
    if (n_layer) *n_layer = s->n_layer;
    if (capacity) *capacity = s->capacity;
    return RMI_HIP_OK;
}

uint32_t rmi_hip_ruvenex_position(const rmi_hip_ruvenex *s) { return s ? s->position : 0; }

int rmi_hip_ruvenex_reset(rmi_hip_ruvenex *s) {
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    s->begin_sequence();
    return RMI_HIP_OK;
}

int rmi_hip_ruvenex_step(rmi_hip_ruvenex *s, const uint32_t *tokens, uint32_t n_tokens, const uint32_t *want, uint32_t n_want, float *logits,
                         float *layers) {
    RMI_REQUIRE_INIT();
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    return s->feed(tokens, n_tokens, want, n_want, logits, layers);
}

int rmi_hip_ruvenex_generate(rmi_hip_ruvenex *s, const uint32_t *prompt, uint32_t n_prompt, uint32_t max_new, uint32_t *generated,
                             uint32_t *step_argmax, float *step_top2, const uint32_t *dump_steps, uint32_t n_dump, float *dump_logits,
                             double *seconds) {
    return rmi_session_generate(s, prompt, n_prompt, max_new, generated, step_argmax, step_top2, dump_steps, n_dump, dump_logits, seconds);
}

int rmi_hip_ruvenex_set_prompt_passes(rmi_hip_ruvenex *s, int enabled) {
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    s->prompt_pass = enabled <= 0 ? 0u : enabled == 1 || uint32_t(enabled) > s->pass_rows ? s->pass_rows : uint32_t(enabled);
    return RMI_HIP_OK;
}

int rmi_hip_ruvenex_set_stop_ids(rmi_hip_ruvenex *s, const uint32_t *ids, uint32_t n_ids) { return rmi_session_set_stop_ids(s, ids, n_ids); }

}  // extern "C"
