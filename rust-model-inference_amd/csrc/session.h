// What every decoder session has: its device allocations, the token and sampling arrays, stop ids, and the
// generation loop that schedules prompt passes and single steps (Qwen3Session::generate_inner,
// src/models/qwen3.rs:581-1158, is the loop's model).
#pragma once

#include <vector>

#include "rmi_internal.h"

constexpr uint32_t kArgmaxGroups = 256;
constexpr size_t kTopBytes = 16;  // one Top of device_sample.h

struct RmiSession {
    uint32_t vocab = 0, capacity = 0;
    uint32_t *tok = nullptr, *step_argmax = nullptr, *nonfinite = nullptr;
    float *step_top2 = nullptr;
    void *partial = nullptr;
    void *params = nullptr;          // StepParams in HBM
    std::vector<void *> owned;       // every device allocation but the weights', freed with the session
    std::vector<uint32_t> stop_ids;  // generation ends before the first of these (EOS, im_end)
    uint32_t prompt_pass = 0;        // prompt positions per pass, 0 = every position its own step

    RmiSession() = default;
    RmiSession(const RmiSession &) = delete;
    RmiSession &operator=(const RmiSession &) = delete;
    virtual ~RmiSession();

    // a device allocation that lives as long as the session; nullptr and the error text on failure
    void *alloc_bytes(size_t nbytes, bool zero);
    template <typename T>
    T *alloc(size_t count, bool zero = false) {
        return static_cast<T *>(alloc_bytes(count * sizeof(T), zero));
    }
    float *upload(const float *host, size_t n);
    bool alloc_sampling();  // the arrays above, for `capacity` positions

    // A new sequence begins at position 0.
    virtual void begin_sequence() {}
    // One position: its logits in step_logits(), its argmax, top two logits and the next token on the device.
    virtual int enqueue_step(uint32_t step, hipStream_t st) = 0;
    virtual const float *step_logits() const = 0;
    // Whether the prompt positions step0 .. step0 + n - 1 can go through one pass.
    virtual bool pass_possible(uint32_t step0, uint32_t n) const = 0;
    // Such a pass, after which the session stands where a single step would have left it.  want (ascending, below n):
    // the positions whose logits the caller reads; a session may compute more.  sample: the pass ends the prompt.
    virtual int enqueue_pass(uint32_t step0, uint32_t n, const uint32_t *want, uint32_t n_want, bool sample, hipStream_t st) = 0;
    virtual uint32_t max_pass_want() const { return 0xffffffffu; }
    // the logits of want[i] = offset
    virtual const float *pass_logits(uint32_t offset, uint32_t i) const = 0;
};

// rmi_hip_<model>_generate: see rmi_hip_qwen3_generate in the header
int rmi_session_generate(RmiSession *s, const uint32_t *prompt, uint32_t n_prompt, uint32_t max_new, uint32_t *generated,
                         uint32_t *step_argmax, float *step_top2, const uint32_t *dump_steps, uint32_t n_dump,
                         float *dump_logits, double *seconds);
int rmi_session_set_stop_ids(RmiSession *s, const uint32_t *ids, uint32_t n_ids);
