// The generation loop of the decoder sessions (session.h).  Host code only.
#include "session.h"

#include <algorithm>
#include <chrono>

RmiSession::~RmiSession() {
    for (void *p : owned) (void)hipFree(p);
}

void *RmiSession::alloc_bytes(size_t nbytes, bool zero) {
    void *p = nullptr;
    const size_t n = nbytes ? nbytes : 16;
    if (hipMalloc(&p, n) != hipSuccess) {
        rmi_set_error("hipMalloc of %zu bytes failed", nbytes);
        return nullptr;
    }
    owned.push_back(p);
    if (zero && hipMemset(p, 0, n) != hipSuccess) {
        rmi_set_error("hipMemset of %zu bytes failed", nbytes);
        return nullptr;
    }
    return p;
}

float *RmiSession::upload(const float *host, size_t n) {
    float *d = alloc<float>(n);
    if (d && n && hipMemcpy(d, host, n * 4, hipMemcpyHostToDevice) != hipSuccess) {
        rmi_set_error("hipMemcpy of a session's constants failed");
        return nullptr;
    }
    return d;
}

bool RmiSession::alloc_sampling() {
    return (tok = alloc<uint32_t>(size_t(capacity) + 1, true)) && (step_argmax = alloc<uint32_t>(capacity, true)) &&
           (step_top2 = alloc<float>(size_t(2) * capacity, true)) && (nonfinite = alloc<uint32_t>(1, true)) &&
           (partial = alloc_bytes(kArgmaxGroups * kTopBytes, false)) && (params = alloc_bytes(8, true));
}

int rmi_session_set_stop_ids(RmiSession *s, const uint32_t *ids, uint32_t n_ids) {
    if (!s || (n_ids && !ids)) return rmi_fail(RMI_HIP_E_INVALID, "null session or ids");
    if (n_ids > 16) return rmi_fail(RMI_HIP_E_INVALID, "at most 16 stop ids");
    s->stop_ids.assign(ids, ids + n_ids);
    return RMI_HIP_OK;
}

int rmi_session_generate(RmiSession *s, const uint32_t *prompt, uint32_t n_prompt, uint32_t max_new, uint32_t *generated,
                         uint32_t *step_argmax, float *step_top2, const uint32_t *dump_steps, uint32_t n_dump,
                         float *dump_logits, double *seconds) {
    RMI_REQUIRE_INIT();
    if (!s || !prompt || n_prompt == 0 || (max_new && !generated))
        return rmi_fail(RMI_HIP_E_INVALID, "null session, prompt or output");
    const uint32_t vocab = s->vocab;
    if (size_t(n_prompt) + max_new > s->capacity)
        return rmi_fail(RMI_HIP_E_INVALID, "%u prompt + %u new tokens exceed the capacity %u", n_prompt, max_new, s->capacity);
    for (uint32_t i = 0; i < n_prompt; i++)
        if (prompt[i] >= vocab) return rmi_fail(RMI_HIP_E_INVALID, "token id %u outside the vocabulary", prompt[i]);
    RmiThreadCtx *ctx = rmi_thread_ctx();
    if (!ctx) return RMI_HIP_E_RUNTIME;
    hipStream_t st = ctx->stream;
    const uint32_t steps = n_prompt + max_new - 1;
    float *d_dump = nullptr;
    if (n_dump) {
        if (!dump_steps || !dump_logits) return rmi_fail(RMI_HIP_E_INVALID, "null dump arrays");
        RMI_HIP_CHECK(hipMalloc(reinterpret_cast<void **>(&d_dump), size_t(n_dump) * vocab * 4));
    }
    std::vector<uint32_t> dumps(dump_steps, dump_steps + n_dump);  // ascending, each once: what passes are asked for
    std::sort(dumps.begin(), dumps.end());
    dumps.erase(std::unique(dumps.begin(), dumps.end()), dumps.end());
    int rc = RMI_HIP_OK;
    const uint32_t start[2] = {0u, n_prompt};  // StepParams: position, prompt length
    hipError_t e = hipMemcpyAsync(s->tok, prompt, size_t(n_prompt) * 4, hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipMemcpyAsync(s->params, start, sizeof start, hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipMemsetAsync(s->nonfinite, 0, 4, st);
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    s->begin_sequence();
    const auto t0 = std::chrono::steady_clock::now();
    // Without stop ids every step is enqueued at once.  With them the host looks at the tokens every
    // kStopCheck generated steps (one small copy) and ends the run at the first stop id, which is not part of
    // the result (src/models/qwen3.rs:1123-1130: the loop breaks before the token is pushed).
    constexpr uint32_t kStopCheck = 32;
    const bool stops = !s->stop_ids.empty() && max_new > 0;
    uint32_t n_valid = max_new, steps_done = 0, checked = 0;
    std::vector<uint32_t> seen(stops ? max_new : 0), want;
    auto dump = [&](uint32_t step, const float *logits) {
        for (uint32_t d = 0; d < n_dump && e == hipSuccess; d++)
            if (dump_steps[d] == step)
                e = hipMemcpyAsync(d_dump + size_t(d) * vocab, logits, size_t(vocab) * 4, hipMemcpyDeviceToDevice, st);
    };
    while (e == hipSuccess && rc == RMI_HIP_OK && steps_done < steps) {
        uint32_t until = steps;
        if (stops) {
            const uint32_t base = steps_done < n_prompt - 1 ? n_prompt - 1 : steps_done;
            until = steps - base > kStopCheck ? base + kStopCheck : steps;
        }
        for (uint32_t step = steps_done; e == hipSuccess && rc == RMI_HIP_OK && step < until;) {
            // prompt positions go several to a pass while they can (their tokens are known); the rest step by step
            uint32_t n = step < n_prompt ? n_prompt - step : 0;
            if (n > s->prompt_pass) n = s->prompt_pass;
            if (n > until - step) n = until - step;
            if (n > 1 && s->pass_possible(step, n)) {
                const auto first = std::lower_bound(dumps.begin(), dumps.end(), step);
                want.assign(first, std::lower_bound(first, dumps.end(), step + n));
                // a pass that could not hold every position asked for (the sampled one may come on top) ends before
                if (want.size() >= s->max_pass_want()) {
                    want.resize(s->max_pass_want() - 1);
                    n = want.back() + 1 - step;
                }
                for (uint32_t &w : want) w -= step;
                rc = s->enqueue_pass(step, n, want.data(), uint32_t(want.size()), step + n == n_prompt, st);
                for (uint32_t i = 0; rc == RMI_HIP_OK && i < want.size(); i++) dump(step + want[i], s->pass_logits(want[i], i));
                step += n;
                continue;
            }
            rc = s->enqueue_step(step, st);
            if (rc == RMI_HIP_OK) dump(step, s->step_logits());
            step++;
        }
        steps_done = until;
        if (!stops || e != hipSuccess || rc != RMI_HIP_OK) continue;
        const uint32_t have = steps_done - (n_prompt - 1);  // tokens sampled so far
        e = hipStreamSynchronize(st);
        if (e == hipSuccess && have > checked)
            e = hipMemcpy(seen.data() + checked, s->tok + n_prompt + checked, size_t(have - checked) * 4, hipMemcpyDeviceToHost);
        bool hit = false;
        for (; e == hipSuccess && checked < have && !hit; checked++)
            for (uint32_t id : s->stop_ids)
                if (seen[checked] == id) {
                    n_valid = checked;
                    hit = true;
                    break;
                }
        if (hit) break;
    }
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    if (seconds) *seconds = std::chrono::duration<double>(std::chrono::steady_clock::now() - t0).count();
    uint32_t nonfinite = 0;
    if (e == hipSuccess && rc == RMI_HIP_OK) {
        if (n_valid) e = hipMemcpy(generated, s->tok + n_prompt, size_t(n_valid) * 4, hipMemcpyDeviceToHost);
        if (e == hipSuccess && step_argmax) e = hipMemcpy(step_argmax, s->step_argmax, size_t(steps_done) * 4, hipMemcpyDeviceToHost);
        if (e == hipSuccess && step_top2) e = hipMemcpy(step_top2, s->step_top2, size_t(steps_done) * 8, hipMemcpyDeviceToHost);
        if (e == hipSuccess && n_dump) e = hipMemcpy(dump_logits, d_dump, size_t(n_dump) * vocab * 4, hipMemcpyDeviceToHost);
        if (e == hipSuccess) e = hipMemcpy(&nonfinite, s->nonfinite, 4, hipMemcpyDeviceToHost);
    }
    if (d_dump) (void)hipFree(d_dump);
    if (rc != RMI_HIP_OK) return rc;
    if (e != hipSuccess) return rmi_fail(RMI_HIP_E_RUNTIME, "decode failed: %s", hipGetErrorString(e));
    if (nonfinite) return rmi_fail(RMI_HIP_E_RUNTIME, "non-finite logits in %u steps", nonfinite);
    return int(n_valid);
}
