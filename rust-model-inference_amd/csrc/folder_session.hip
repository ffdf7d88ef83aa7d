// The sessions over model folders (folder_session.h): what they share, the registry and the C ABI.
#include "folder_session.h"

#include "device_dense.h"
#include "device_sample.h"

namespace {

// the embedding of the next token, the argmax kernel's last act
template <typename T>
struct EmbedNext {
    RmiEmbed e;
    uint32_t pos;
    __device__ __forceinline__ void operator()(uint32_t token) const { embed_row<T>(e, token, pos, 0); }
};

struct Architecture {
    const char *name;
    rmi_hip_folder_session *(*create)();
};
constexpr Architecture kArchitectures[] = {{"Ruvenex", rmi_new_ruvenex}, {"Vogizen", rmi_new_vogizen}};

}  // namespace

RmiEmbed rmi_hip_folder_session::embed_to() const {
    RmiEmbed e = embedding;
    e.table = embed.data;
    e.ld = embed.ld;
    e.vocab = vocab;
    e.n = width;
    e.x = x;
    e.x_also = x_embedded;
    return e;
}

int rmi_hip_folder_session::embed_tokens(uint32_t step0, uint32_t n, hipStream_t st) {
    return rmi_dense_embed(elem, embed_to(), tok + step0, step0, n, st);
}

// logits[i] = head . the input of x[rows[i]]; rows in HBM, nullptr: 0 .. n_rows - 1
int rmi_hip_folder_session::enqueue_logits(const uint32_t *rows, uint32_t n_rows, hipStream_t st) {
    RmiRowSegs s{};
    s.n_segs = 1;
    s.n_rows = head.n_rows;
    s.s[0].y = logits;
    s.s[0].n = s.s[0].ld = vocab;
    s.s[0].act = kActNone;
    rmi_row_segs_done(&s);
    const RmiInput in = head_input();
    if (n_rows == 1 && !rows && rmi_dense_gemv_fits(elem, k_in)) return rmi_dense_gemv(elem, head, in, s, st);
    const int rc = rmi_dense_input(elem, in, rows, h, n_rows, k_in, st);
    return rc == RMI_HIP_OK ? rmi_dense_gemm(elem, head, h, s, n_rows, st) : rc;
}

// last: the place of the pass's last sampled position, whose token's embedding is left for the next step
int rmi_hip_folder_session::enqueue_sample(uint32_t step0, const uint32_t *rows, uint32_t n_rows, uint32_t last, hipStream_t st) {
    hipLaunchKernelGGL(argmax_partial_kernel, dim3(kArgmaxGroups, n_rows), dim3(256), 0, st, logits, vocab, static_cast<Top *>(partial));
    auto finish = [&](auto embed_next) {
        hipLaunchKernelGGL((argmax_final_batch_kernel<decltype(embed_next)>), dim3(n_rows), dim3(256), 0, st,
                           static_cast<const Top *>(partial), kArgmaxGroups, static_cast<StepParams *>(params), step0, rows, tok, step_argmax,
                           step_top2, nonfinite, embed_next);
    };
    if (elem == 2)
        finish(EmbedNext<rmi_bf16>{embed_to(), step0 + last + 1});
    else
        finish(EmbedNext<float>{embed_to(), step0 + last + 1});
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

int rmi_hip_folder_session::set_rows(const uint32_t *want, uint32_t n_want, hipStream_t st) {
    RMI_HIP_CHECK(hipMemcpyAsync(want_rows, want, size_t(n_want) * 4, hipMemcpyHostToDevice, st));
    RMI_HIP_CHECK(hipStreamSynchronize(st));  // the host array is the caller's
    return RMI_HIP_OK;
}

int rmi_hip_folder_session::enqueue_step(uint32_t step, hipStream_t st) {
    int rc = embedded == step ? RMI_HIP_OK : embed_tokens(step, 1, st);
    if (rc == RMI_HIP_OK) rc = enqueue_layers(step, 1, st, nullptr);
    if (rc == RMI_HIP_OK) rc = enqueue_logits(nullptr, 1, st);
    if (rc == RMI_HIP_OK) rc = enqueue_sample(step, nullptr, 1, 0, st);
    embedded = step + 1;
    return rc;
}

int rmi_hip_folder_session::enqueue_pass(uint32_t step0, uint32_t n, const uint32_t *want, uint32_t n_want, bool sample, hipStream_t st) {
    int rc = embed_tokens(step0, n, st);
    if (rc == RMI_HIP_OK) rc = enqueue_layers(step0, n, st, nullptr);
    std::vector<uint32_t> rows(want, want + n_want);
    if (sample && (rows.empty() || rows.back() != n - 1)) rows.push_back(n - 1);
    embedded = ~0u;
    if (rc != RMI_HIP_OK || rows.empty()) return rc;
    if (rows.size() > logit_rows) return rmi_fail(RMI_HIP_E_INVALID, "logits of more than %u positions of a pass", logit_rows);
    rc = set_rows(rows.data(), uint32_t(rows.size()), st);
    if (rc == RMI_HIP_OK) rc = enqueue_logits(want_rows, uint32_t(rows.size()), st);
    if (rc == RMI_HIP_OK) rc = enqueue_sample(step0, want_rows, uint32_t(rows.size()), rows.back(), st);
    if (rows.back() == n - 1) embedded = step0 + n;
    return rc;
}

// The next n tokens of the sequence, with no sampling: logits of the places in `want`, in that order.
int rmi_hip_folder_session::feed(const uint32_t *tokens, uint32_t n, const uint32_t *want, uint32_t n_want, float *out, float *host_layers) {
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

int rmi_hip_folder_session::copy_layer(float *host_layers, uint32_t run, uint32_t n, hipStream_t st) {
    RMI_HIP_CHECK(hipStreamSynchronize(st));
    RMI_HIP_CHECK(hipMemcpy(host_layers + size_t(run) * n * width, x, size_t(n) * width * 4, hipMemcpyDeviceToHost));
    return RMI_HIP_OK;
}

float *rmi_hip_folder_session::upload_vector(const RmiTensor *t) {
    if (!t) return nullptr;
    std::vector<float> v(t->count);
    for (uint64_t i = 0; i < t->count; i++) v[i] = rmi_tensor_f32(*t, i);
    return upload(v.data(), v.size());
}

bool rmi_hip_folder_session::load_common(RmiFolderReader &rd) {
    const RmiJson &c = rd.f.config;
    width = rd.size(&c, "width");
    vocab = rd.size(&c, "vocab");
    eps = float(rd.number(rd.object(&c, "norm"), "eps"));
    embedding.scale = float(rd.number(rd.object(&c, "embedding"), "scale"));
    const RmiJson *ls = c.get("layers");
    if (!ls || ls->type != RmiJson::kArray) rd.fail("config.json: no list 'layers'");
    if (!rd.ok) return false;
    k_in = rmi_dense_pad(width, kDenseKAlign);
    pass_rows = capacity < kPassMax ? capacity : kPassMax;
    prompt_pass = pass_rows;
    logit_rows = pass_rows < kLogitRows ? pass_rows : kLogitRows;
    if (width > kInputMax || uint64_t(vocab) * k_in > (uint64_t(1) << 40)) {
        rmi_set_error("unsupported model shape: a width of up to %u", kInputMax);
        return false;
    }
    RmiDenseBuilder b(elem, rmi_dense_pad(vocab, kDenseRowAlign), k_in);
    b.put(rd.tensor("embed", {vocab, width}), 0, 0);
    return rd.ok && b.upload(this, &embed);
}

bool rmi_hip_folder_session::alloc_common(uint32_t max_k) {
    if (max_k < k_in) max_k = k_in;
    return alloc_sampling() && (x = alloc<float>(size_t(pass_rows) * width, true)) &&
           (h = alloc_bytes(size_t(pass_rows) * (max_k + 128) * elem, true)) && (logits = alloc<float>(size_t(logit_rows) * vocab, true)) &&
           (want_rows = alloc<uint32_t>(kLogitRows, true)) && (partial = alloc_bytes(size_t(logit_rows) * kArgmaxGroups * kTopBytes, false));
}

extern "C" {

rmi_hip_folder_session *rmi_hip_folder_open(const char *dir, const char *architecture, int dtype, uint32_t capacity) {
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
    const RmiJson *arch = f.config.get("architecture");
    const std::string name = arch ? arch->text : "";
    if (architecture && name != architecture) {
        rmi_set_error("config.json: architecture '%s' is not %s", name.c_str(), architecture);
        return nullptr;
    }
    for (const Architecture &a : kArchitectures) {
        if (name != a.name) continue;
        rmi_hip_folder_session *s = a.create();
        s->elem = dtype == RMI_HIP_DTYPE_F32 ? 4 : 2;
        s->capacity = capacity;
        bool ok = s->load(f);
        if (ok && hipDeviceSynchronize() != hipSuccess) {
            rmi_set_error("weight upload failed");
            ok = false;
        }
        if (ok) return s;
        delete s;
        return nullptr;
    }
    rmi_set_error("config.json: no session for architecture '%s'", name.c_str());
    return nullptr;
}

void rmi_hip_folder_destroy(rmi_hip_folder_session *s) { delete s; }

int rmi_hip_folder_sizes(const rmi_hip_folder_session *s, uint32_t *vocab, uint32_t *width, uint32_t *n_layer, uint32_t *capacity) {
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    if (vocab) *vocab = s->vocab;
    if (width) *width = s->width;
    if (n_layer) *n_layer = s->n_runs;
    if (capacity) *capacity = s->capacity;
    return RMI_HIP_OK;
}

uint32_t rmi_hip_folder_position(const rmi_hip_folder_session *s) { return s ? s->position : 0; }

int rmi_hip_folder_reset(rmi_hip_folder_session *s) {
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    s->begin_sequence();
    return RMI_HIP_OK;
}

int rmi_hip_folder_step(rmi_hip_folder_session *s, const uint32_t *tokens, uint32_t n_tokens, const uint32_t *want, uint32_t n_want,
                        float *logits, float *layers) {
    RMI_REQUIRE_INIT();
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    return s->feed(tokens, n_tokens, want, n_want, logits, layers);
}

int rmi_hip_folder_generate(rmi_hip_folder_session *s, const uint32_t *prompt, uint32_t n_prompt, uint32_t max_new, uint32_t *generated,
                            uint32_t *step_argmax, float *step_top2, const uint32_t *dump_steps, uint32_t n_dump, float *dump_logits,
                            double *seconds) {
    return rmi_session_generate(s, prompt, n_prompt, max_new, generated, step_argmax, step_top2, dump_steps, n_dump, dump_logits, seconds);
}

int rmi_hip_folder_set_prompt_passes(rmi_hip_folder_session *s, int enabled) {
    if (!s) return rmi_fail(RMI_HIP_E_INVALID, "null session");
    s->prompt_pass = enabled <= 0 ? 0u : enabled == 1 || uint32_t(enabled) > s->pass_rows ? s->pass_rows : uint32_t(enabled);
    return RMI_HIP_OK;
}

int rmi_hip_folder_set_stop_ids(rmi_hip_folder_session *s, const uint32_t *ids, uint32_t n_ids) { return rmi_session_set_stop_ids(s, ids, n_ids); }

// the names from when Ruvenex was the only design
rmi_hip_ruvenex *rmi_hip_ruvenex_open(const char *dir, int dtype, uint32_t capacity) { return rmi_hip_folder_open(dir, "Ruvenex", dtype, capacity); }
void rmi_hip_ruvenex_destroy(rmi_hip_ruvenex *s) { rmi_hip_folder_destroy(s); }
int rmi_hip_ruvenex_sizes(const rmi_hip_ruvenex *s, uint32_t *vocab, uint32_t *width, uint32_t *n_layer, uint32_t *capacity) {
    return rmi_hip_folder_sizes(s, vocab, width, n_layer, capacity);
}
uint32_t rmi_hip_ruvenex_position(const rmi_hip_ruvenex *s) { return rmi_hip_folder_position(s); }
int rmi_hip_ruvenex_reset(rmi_hip_ruvenex *s) { return rmi_hip_folder_reset(s); }
int rmi_hip_ruvenex_step(rmi_hip_ruvenex *s, const uint32_t *tokens, uint32_t n_tokens, const uint32_t *want, uint32_t n_want, float *logits,
                         float *layers) {
    return rmi_hip_folder_step(s, tokens, n_tokens, want, n_want, logits, layers);
}
int rmi_hip_ruvenex_generate(rmi_hip_ruvenex *s, const uint32_t *prompt, uint32_t n_prompt, uint32_t max_new, uint32_t *generated,
                             uint32_t *step_argmax, float *step_top2, const uint32_t *dump_steps, uint32_t n_dump, float *dump_logits,
                             double *seconds) {
    return rmi_hip_folder_generate(s, prompt, n_prompt, max_new, generated, step_argmax, step_top2, dump_steps, n_dump, dump_logits, seconds);
}
int rmi_hip_ruvenex_set_prompt_passes(rmi_hip_ruvenex *s, int enabled) { return rmi_hip_folder_set_prompt_passes(s, enabled); }
int rmi_hip_ruvenex_set_stop_ids(rmi_hip_ruvenex *s, const uint32_t *ids, uint32_t n_ids) { return rmi_hip_folder_set_stop_ids(s, ids, n_ids); }

}  // extern "C"
