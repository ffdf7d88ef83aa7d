// What the sessions over model folders have in common (session.h beneath it): the sequence they hold, the embedding,
// the logits and sampling, feeding recorded tokens, and the reading of sizes and tensors.  A design adds its layers.
#pragma once

#include <cmath>
#include <string>
#include <vector>

#include "dense.h"
#include "model_folder.h"
#include "session.h"

constexpr uint32_t kPassMax = 2048;  // most positions of a pass
constexpr uint32_t kLogitRows = 64;  // most positions whose logits are computed together

struct rmi_hip_folder_session : RmiSession {
    uint32_t elem = 2;  // bytes of a weight / activation element
    uint32_t width = 0, n_runs = 0, k_in = 0, pass_rows = 0, logit_rows = 0;  // n_runs: layers, each as often as it runs
    float eps = 0;
    RmiDense embed, head;  // (a design that ties the two sets both to the same weight)
    RmiEmbed embedding{};  // but for the buffers
    float *x = nullptr;    // the residual stream of a pass, [token][width]; a design may exchange it for another buffer
    float *x_embedded = nullptr;  // a copy of the embedding output, for designs that read it again
    void *h = nullptr;            // the operand of the product under way
    float *logits = nullptr;
    uint32_t *want_rows = nullptr;
    uint32_t position = 0;    // tokens of the current sequence so far
    uint32_t embedded = ~0u;  // the position whose embedding the last sampling launch left in x

    // Sizes, weights and buffers; false + error text.
    virtual bool load(const RmiModelFolder &f) = 0;
    // The layers over positions step0 .. step0 + n - 1, whose embeddings are in x.  host_layers: the residual stream
    // behind every layer run, [run][n][width] (synchronises; for comparisons).
    virtual int enqueue_layers(uint32_t step0, uint32_t n, hipStream_t st, float *host_layers) = 0;
    // What the head reads of the stream behind the last layer (x_out is not used).
    virtual RmiInput head_input() const = 0;

    void begin_sequence() override {
        position = 0;
        embedded = ~0u;
    }
    int enqueue_step(uint32_t step, hipStream_t st) override;
    const float *step_logits() const override { return logits; }
    bool pass_possible(uint32_t step0, uint32_t n) const override { return n <= pass_rows && step0 + n <= capacity; }
    int enqueue_pass(uint32_t step0, uint32_t n, const uint32_t *want, uint32_t n_want, bool sample, hipStream_t st) override;
    uint32_t max_pass_want() const override { return logit_rows; }
    const float *pass_logits(uint32_t, uint32_t i) const override { return logits + size_t(i) * vocab; }
    int feed(const uint32_t *tokens, uint32_t n, const uint32_t *want, uint32_t n_want, float *out, float *host_layers);

  protected:
    // width, vocab, eps and the rest of what every design has; then, with operands of up to max_k columns, the buffers
    bool load_common(struct RmiFolderReader &rd);
    bool alloc_common(uint32_t max_k);
    float *upload_vector(const RmiTensor *t);
    int copy_layer(float *host_layers, uint32_t run, uint32_t n, hipStream_t st);

  private:
    RmiEmbed embed_to() const;
    int embed_tokens(uint32_t step0, uint32_t n, hipStream_t st);
    int enqueue_logits(const uint32_t *rows, uint32_t n_rows, hipStream_t st);
    int enqueue_sample(uint32_t step0, const uint32_t *rows, uint32_t n_rows, uint32_t last, hipStream_t st);
    int set_rows(const uint32_t *want, uint32_t n_want, hipStream_t st);
};

// the sessions that config.json's architecture chooses between
rmi_hip_folder_session *rmi_new_ruvenex();
rmi_hip_folder_session *rmi_new_vogizen();

// What a constructor reads from the folder: the first thing missing or out of place ends it with a message.
struct RmiFolderReader {
    const RmiModelFolder &f;
    bool ok = true;
    explicit RmiFolderReader(const RmiModelFolder &folder) : f(folder) {}

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

// A dense weight put together on the host from blocks of tensors, then uploaded.
struct RmiDenseBuilder {
    uint32_t elem, n_rows, k_pad, ld;
    std::vector<uint8_t> bytes;
    RmiDenseBuilder(uint32_t e, uint32_t rows, uint32_t k)
        : elem(e), n_rows(rows), k_pad(k), ld(rmi_dense_ld(k, e)), bytes(size_t(rows) * ld * e, 0) {}
    // columns [src_col, src_col + cols) of t (cols 0: all) from (row0, col0) on, its rows row_step apart
    void put(const RmiTensor *t, uint32_t row0, uint32_t col0, uint32_t row_step = 1, uint64_t src_col = 0, uint64_t cols = 0) {
        if (!t) return;
        const uint64_t rows = t->shape[0], all = t->shape[1];
        if (!cols) cols = all;
        for (uint64_t r = 0; r < rows; r++) {
            uint8_t *dst = bytes.data() + (size_t(row0 + r * row_step) * ld + col0) * elem;
            if (elem == 2)
                rmi_tensor_bf16(*t, r * all + src_col, cols, reinterpret_cast<uint16_t *>(dst));
            else
                for (uint64_t i = 0; i < cols; i++) {
                    const float v = rmi_tensor_f32(*t, r * all + src_col + i);
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
