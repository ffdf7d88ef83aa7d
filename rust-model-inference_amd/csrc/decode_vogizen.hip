// The Vogizen decoder: a session over a model folder.  A layer, with n1 and n2 its layer norms, m its mixer
// (sliding-window latent attention, or the gated delta rule), s1 and s2 its scales and E its part of a table by token,
//
//   x += s1 * m(n1(x));   x += s2 * W_down (relu(W_gate n2(x)) * W_up n2(x))   (where it has a feed-forward);
//   x += rms(P (gelu(G x) * E[token])) * w
//
// with a run of layers looped: each pass of it has its own cache and state and begins with x <- W [x ; embedding].
//
// What ends a layer needs the whole of its result before x is known (the rms), so it stays a pending sum that the next
// reader of x forms in its prologue: the norm in front of the next layer, the loop's product, or the head.  In a
// product of one token that prologue runs in every workgroup and the first one stores the new x into a second buffer.
// Launches of a layer and token: norm + all that reads it; the mixer (the delta rule one launch, latent attention two:
// norms + up-projections, attention); output + scale + residual; G; P; a feed-forward adds two.
#include <cmath>
#include <string>
#include <vector>

#include "folder_session.h"
#include "seq_mixers.h"

namespace {

struct VogizenLayer {
    bool delta = false, ffn = false;
    float *norm1 = nullptr, *norm2 = nullptr, *side_norm = nullptr;
    RmiDense w_in, w_out, w_uq, w_ukv, w_ff, w_down, w_gate, w_proj;  // w_ff: (gate, up) rows in turn
    RmiRowSegs in, uq, ukv, ff, gate, proj;
    RmiColSegs out, down;
    // latent attention
    RmiAttnShape attn{};
    uint32_t q_rank = 0, kv_rank = 0;
    float *dq_norm = nullptr, *dkv_norm = nullptr, *ones = nullptr;
    // the delta rule
    RmiDeltaShape rule{};
    float *conv = nullptr, *head_norm = nullptr, *rate = nullptr, *bias = nullptr;
};

// A layer as often as a token runs through it, each time with a cache or state of its own.
struct VogizenRun {
    uint32_t layer = 0;
    bool loop_begins = false;
    void *k_cache = nullptr, *v_cache = nullptr;
    float *hist[2] = {nullptr, nullptr}, *state[2] = {nullptr, nullptr};
};

// the columns of a product that adds to the stream: one segment, scaled by a vector
RmiColSegs scaled_columns(const float *scale, uint32_t k_pad) {
    RmiColSegs c{};
    c.n_segs = 1;
    c.s[0] = RmiColSeg{scale, 0, 1.0f, k_pad};
    return c;
}

struct VogizenSession : rmi_hip_folder_session {
    std::vector<VogizenLayer> layers;
    std::vector<VogizenRun> runs;
    bool looped = false;
    RmiDense w_loop, side_table;
    float *final_norm = nullptr;
    // activations of a pass, token-major
    float *x_next = nullptr;  // the other buffer of the stream
    float *u = nullptr, *beta = nullptr, *decay = nullptr, *gate = nullptr, *cq = nullptr, *ckv = nullptr, *y = nullptr, *side_f32 = nullptr;
    void *act = nullptr, *q = nullptr, *side = nullptr;
    void *attn_scratch = nullptr;
    float *delta_scratch = nullptr;
    const float *pending = nullptr;  // the weight of the result in y that x still lacks
    int now = 0;                     // which of a run's two history and state buffers the last pass left

    void begin_sequence() override {
        rmi_hip_folder_session::begin_sequence();
        pending = nullptr;
    }
    bool load(const RmiModelFolder &f) override;
    int enqueue_layers(uint32_t step0, uint32_t n, hipStream_t st, float *host_layers) override;
    RmiInput head_input() const override { return stream(kNormLayer, final_norm); }

  private:
    // the stream, with what it still lacks, as a product's input
    RmiInput stream(RmiNorm norm, const float *weight) const {
        RmiInput in;
        in.x = x;
        in.n = width;
        in.norm = norm;
        in.weight = weight;
        in.eps = in.y_eps = eps;
        if (pending) {
            in.y = y;
            in.y_weight = pending;
        }
        return in;
    }
    // a latent under its RMS norm
    RmiInput latent(const float *c, uint32_t n, const float *weight) const {
        RmiInput in;
        in.x = c;
        in.n = n;
        in.norm = kNormRms;
        in.weight = weight;
        in.eps = eps;
        return in;
    }
    // x = what x is to be, now
    int settle(uint32_t n, hipStream_t st) {
        if (!pending) return RMI_HIP_OK;
        RmiInput in = stream(kNormNone, nullptr);
        in.x_out = x;
        pending = nullptr;
        return rmi_dense_input(elem, in, nullptr, nullptr, n, k_in, st);
    }
    int read(const RmiDense &w, RmiInput in, const RmiRowSegs &segs, uint32_t n, bool one, hipStream_t st);
    int loop_in(uint32_t n, bool one, hipStream_t st);
    int mixer(const VogizenLayer &l, const VogizenRun &r, uint32_t step0, uint32_t n, bool one, hipStream_t st);
    int add(const RmiDense &w, const RmiColSegs &segs, uint32_t n, bool one, hipStream_t st) {
        return one ? rmi_dense_gemv_residual(elem, w, act, segs, x, width, st) : rmi_dense_gemm_residual(elem, w, act, segs, x, width, n, st);
    }
    bool fits(uint32_t k) const { return rmi_dense_gemv_fits(elem, rmi_dense_pad(k, kDenseKAlign)); }
    bool load_latent(RmiFolderReader &rd, VogizenLayer &l, const std::string &p);
    bool load_delta(RmiFolderReader &rd, VogizenLayer &l, const std::string &p);
    bool load_ffn(RmiFolderReader &rd, VogizenLayer &l, const std::string &p, uint32_t ff);
    bool stack(RmiFolderReader &rd, RmiDense *w, RmiRowSegs *segs, const std::vector<std::pair<std::string, RmiRowSeg>> &parts, uint32_t k);
    bool output(RmiFolderReader &rd, RmiDense *w, RmiColSegs *segs, const std::string &name, const std::string &scale, uint32_t k);
    bool one_token_gemv = true;  // every input fits the products of one token
    // the largest of what the shared buffers hold
    uint32_t max_u = 1, max_heads = 1, max_values = 1, max_q_rank = 1, max_kv_rank = 1, max_ld = kDenseKAlign, max_k = kDenseKAlign;
    size_t max_q = 1, max_attn_scratch = 0, max_delta_scratch = 1;
};

// segs = w . the stream (and, once x holds it, what was pending is no longer)
int VogizenSession::read(const RmiDense &w, RmiInput in, const RmiRowSegs &segs, uint32_t n, bool one, hipStream_t st) {
    if (one) {
        if (in.y) in.x_out = x_next;
        const int rc = rmi_dense_gemv(elem, w, in, segs, st);
        if (in.y) std::swap(x, x_next);
        pending = nullptr;
        return rc;
    }
    if (in.y) in.x_out = x;
    pending = nullptr;
    const int rc = rmi_dense_input(elem, in, nullptr, h, n, w.k_pad, st);
    return rc == RMI_HIP_OK ? rmi_dense_gemm(elem, w, h, segs, n, st) : rc;
}

int VogizenSession::loop_in(uint32_t n, bool one, hipStream_t st) {
    RmiInput in = stream(kNormNone, nullptr);
    in.x2 = x_embedded;
    in.n2 = width;
    in.k2 = k_in;
    RmiRowSegs s{};
    s.n_segs = 1;
    s.n_rows = w_loop.n_rows;
    s.s[0].y = one ? x_next : x;  // (of several tokens x has become the operand before it is written)
    s.s[0].n = s.s[0].ld = width;
    s.s[0].act = kActNone;
    rmi_row_segs_done(&s);
    pending = nullptr;
    if (one) {
        const int rc = rmi_dense_gemv(elem, w_loop, in, s, st);
        std::swap(x, x_next);
        return rc;
    }
    const int rc = rmi_dense_input(elem, in, nullptr, h, n, w_loop.k_pad, st);
    return rc == RMI_HIP_OK ? rmi_dense_gemm(elem, w_loop, h, s, n, st) : rc;
}

// the mixer's result in act, from what the product in front of it left
int VogizenSession::mixer(const VogizenLayer &l, const VogizenRun &r, uint32_t step0, uint32_t n, bool one, hipStream_t st) {
    if (l.delta) {
        RmiDeltaArgs a{};
        a.u = u;
        a.hist_in = r.hist[now];
        a.hist_out = r.hist[now ^ 1];
        a.conv = l.conv;
        a.b = beta;
        a.a = decay;
        a.rate = l.rate;
        a.bias = l.bias;
        a.gate = gate;
        a.norm = l.head_norm;
        a.state_in = r.state[now];
        a.state_out = r.state[now ^ 1];
        a.out = act;
        a.out_ld = l.w_out.ld;
        a.pos0 = step0;
        a.n_tokens = n;
        a.scratch = delta_scratch;
        return n == 1 ? rmi_delta_step(elem, l.rule, a, st) : rmi_delta_pass(elem, l.rule, a, st);
    }
    const RmiInput in_q = latent(cq, l.q_rank, l.dq_norm), in_kv = latent(ckv, l.kv_rank, l.dkv_norm);
    int rc;
    if (one) {
        rc = rmi_dense_gemv_pair(elem, l.w_uq, in_q, l.uq, l.w_ukv, in_kv, l.ukv, st);
    } else {
        rc = rmi_dense_input(elem, in_q, nullptr, h, n, l.w_uq.k_pad, st);
        if (rc == RMI_HIP_OK) rc = rmi_dense_gemm(elem, l.w_uq, h, l.uq, n, st);
        if (rc == RMI_HIP_OK) rc = rmi_dense_input(elem, in_kv, nullptr, h, n, l.w_ukv.k_pad, st);
        if (rc == RMI_HIP_OK) rc = rmi_dense_gemm(elem, l.w_ukv, h, l.ukv, n, st);
    }
    if (rc != RMI_HIP_OK) return rc;
    RmiAttnArgs a{};
    a.u = u;
    a.conv = l.ones;
    a.q = q;
    a.k_cache = r.k_cache;
    a.v_cache = r.v_cache;
    a.out = act;
    a.out_ld = l.w_out.ld;
    a.pos0 = step0;
    a.n_tokens = n;
    a.scratch = attn_scratch;
    return n == 1 ? rmi_mixers_step(elem, &l.attn, &a, nullptr, nullptr, st) : rmi_attn_pass(elem, l.attn, a, st);
}

int VogizenSession::enqueue_layers(uint32_t step0, uint32_t n, hipStream_t st, float *host_layers) {
    const bool one = n == 1 && one_token_gemv, in_prologue = !one || width <= kGemvAddMax;
    int rc = RMI_HIP_OK;
    pending = nullptr;
    for (uint32_t i = 0; i < runs.size() && rc == RMI_HIP_OK; i++) {
        const VogizenRun &r = runs[i];
        const VogizenLayer &l = layers[r.layer];
        if (r.loop_begins) rc = loop_in(n, one, st);
        if (rc == RMI_HIP_OK) rc = read(l.w_in, stream(kNormLayer, l.norm1), l.in, n, one, st);
        if (rc == RMI_HIP_OK) rc = mixer(l, r, step0, n, one, st);
        if (rc == RMI_HIP_OK) rc = add(l.w_out, l.out, n, one, st);
        if (l.ffn) {
            if (rc == RMI_HIP_OK) rc = read(l.w_ff, stream(kNormLayer, l.norm2), l.ff, n, one, st);
            if (rc == RMI_HIP_OK) rc = add(l.w_down, l.down, n, one, st);
        }
        RmiRowSegs g = l.gate;
        g.s[0].mul_tok = tok + step0;
        if (one) g.s[0].y = side_f32;
        g.s[0].out_elem = one ? 0 : 1;
        if (rc == RMI_HIP_OK) rc = read(l.w_gate, stream(kNormNone, nullptr), g, n, one, st);
        if (rc != RMI_HIP_OK) return rc;
        if (one) {
            RmiInput in;
            in.x = side_f32;
            in.n = g.s[0].n;
            rc = rmi_dense_gemv(elem, l.w_proj, in, l.proj, st);
        } else {
            rc = rmi_dense_gemm(elem, l.w_proj, side, l.proj, n, st);
        }
        pending = l.side_norm;
        if (rc == RMI_HIP_OK && (host_layers || !in_prologue)) rc = settle(n, st);
        if (rc == RMI_HIP_OK && host_layers) rc = copy_layer(host_layers, i, n, st);
    }
    now ^= 1;
    position = step0 + n;
    return rc;
}

// ------------------------------------------------------------------ loading

RmiRowSeg segment(void *y, uint32_t n, uint32_t ld, RmiAct act) {
    RmiRowSeg s{};
    s.y = y;
    s.n = n;
    s.ld = ld;
    s.act = uint16_t(act);
    return s;
}

// Tensors [n, k] one below the other, each with its segment (whose row0 is set here).
bool VogizenSession::stack(RmiFolderReader &rd, RmiDense *w, RmiRowSegs *segs, const std::vector<std::pair<std::string, RmiRowSeg>> &parts, uint32_t k) {
    uint32_t rows = 0;
    for (const auto &p : parts) {
        RmiRowSeg &s = segs->s[segs->n_segs++] = p.second;
        s.row0 = rows;
        rows += rmi_dense_pad(s.n, kDenseRowAlign);
    }
    segs->n_rows = rows;
    rmi_row_segs_done(segs);
    RmiDenseBuilder b(elem, rows, rmi_dense_pad(k, kDenseKAlign));
    for (size_t i = 0; i < parts.size() && rd.ok; i++) b.put(rd.tensor(parts[i].first, {parts[i].second.n, k}), segs->s[i].row0, 0);
    return rd.ok && b.upload(this, w);
}

// A tensor [width, k] whose result joins the stream under a scale.
bool VogizenSession::output(RmiFolderReader &rd, RmiDense *w, RmiColSegs *segs, const std::string &name, const std::string &scale, uint32_t k) {
    float *s = upload_vector(rd.tensor(scale, {width}));
    RmiDenseBuilder b(elem, rmi_dense_pad(width, kDenseRowAlign), rmi_dense_pad(k, kDenseKAlign));
    b.put(rd.tensor(name, {width, k}), 0, 0);
    *segs = scaled_columns(s, b.k_pad);
    return rd.ok && s && b.upload(this, w);
}

bool VogizenSession::load_latent(RmiFolderReader &rd, VogizenLayer &l, const std::string &p) {
    const std::string m = p + "mix.";
    const RmiAttnShape &a = l.attn;
    const uint32_t nk = a.heads * a.dim, nv = a.heads * a.vdim, ld = 2 * nk + nv;
    if (!stack(rd, &l.w_in, &l.in, {{m + "dq", segment(cq, l.q_rank, l.q_rank, kActNone)}, {m + "dkv", segment(ckv, l.kv_rank, l.kv_rank, kActNone)}}, width) ||
        !stack(rd, &l.w_uq, &l.uq, {{m + "uq", segment(u, nk, ld, kActNone)}}, l.q_rank) ||
        !stack(rd, &l.w_ukv, &l.ukv, {{m + "uk", segment(u + nk, nk, ld, kActNone)}, {m + "uv", segment(u + 2 * nk, nv, ld, kActNone)}}, l.kv_rank) ||
        !output(rd, &l.w_out, &l.out, m + "o", p + "ls1", nv))
        return false;
    const std::vector<float> ones(ld, 1.0f);  // queries, keys and values pass through as they are
    return (l.dq_norm = upload_vector(rd.tensor(m + "dq.norm", {l.q_rank}))) && (l.dkv_norm = upload_vector(rd.tensor(m + "dkv.norm", {l.kv_rank}))) &&
           (l.ones = upload(ones.data(), ones.size()));
}

bool VogizenSession::load_delta(RmiFolderReader &rd, VogizenLayer &l, const std::string &p) {
    const std::string m = p + "mix.";
    const RmiDeltaShape &s = l.rule;
    const uint32_t nk = s.kv_heads * s.dim, nv = s.heads * s.vdim, ld = 2 * nk + nv;
    const RmiTensor *a_log = rd.tensor(m + "A_log", {s.heads});
    if (!a_log) return false;
    std::vector<float> rate(s.heads);
    for (uint32_t i = 0; i < s.heads; i++) rate[i] = float(std::exp(double(rmi_tensor_f32(*a_log, i))));
    if (!(l.rate = upload(rate.data(), rate.size())) || !(l.bias = upload_vector(rd.tensor(m + "dt_bias", {s.heads})))) return false;
    if (!stack(rd, &l.w_in, &l.in,
               {{m + "q", segment(u, nk, ld, kActNone)},
                {m + "k", segment(u + nk, nk, ld, kActNone)},
                {m + "v", segment(u + 2 * nk, nv, ld, kActNone)},
                {m + "b", segment(beta, s.heads, s.heads, kActNone)},
                {m + "a", segment(decay, s.heads, s.heads, kActNone)},
                {m + "g", segment(gate, nv, nv, kActSilu)}},
               width) ||
        !output(rd, &l.w_out, &l.out, m + "o", p + "ls1", nv))
        return false;
    std::vector<float> taps;  // the three convolutions, one below the other
    const std::pair<const char *, uint32_t> convs[] = {{"q.conv", nk}, {"k.conv", nk}, {"v.conv", nv}};
    for (const auto &c : convs) {
        const RmiTensor *t = rd.tensor(m + c.first, {c.second, s.taps});
        if (!t) return false;
        for (uint64_t i = 0; i < t->count; i++) taps.push_back(rmi_tensor_f32(*t, i));
    }
    return (l.conv = upload(taps.data(), taps.size())) && (l.head_norm = upload_vector(rd.tensor(m + "norm", {s.vdim})));
}

bool VogizenSession::load_ffn(RmiFolderReader &rd, VogizenLayer &l, const std::string &p, uint32_t ff) {
    RmiRowSeg &s = l.ff.s[0];
    s = segment(act, 2 * ff, rmi_dense_ld(rmi_dense_pad(ff, kDenseKAlign), elem), kActReluGlu);
    s.out_elem = 1;
    l.ff.n_segs = 1;
    l.ff.n_rows = rmi_dense_pad(2 * ff, kDenseRowAlign);
    rmi_row_segs_done(&l.ff);
    RmiDenseBuilder b(elem, l.ff.n_rows, k_in);
    b.put(rd.tensor(p + "mlp.gate", {ff, width}), 0, 0, 2);
    b.put(rd.tensor(p + "mlp.up", {ff, width}), 1, 0, 2);
    return rd.ok && b.upload(this, &l.w_ff) && output(rd, &l.w_down, &l.down, p + "mlp.down", p + "ls2", ff) &&
           (l.norm2 = upload_vector(rd.tensor(p + "norm2", {width})));
}

bool VogizenSession::load(const RmiModelFolder &folder) {
    RmiFolderReader rd(folder);
    if (!load_common(rd)) return false;
    head = embed;
    const RmiJson &c = folder.config;
    const std::vector<RmiJson> &ls = c.get("layers")->items;
    const uint32_t n_layer = uint32_t(ls.size()), side_dim = rd.size(rd.object(&c, "token_side"), "dim");
    uint32_t start = 0, stop = 0, times = 1;
    const RmiJson *loop = c.get("loop");
    if ((looped = loop && !loop->is_null())) {
        loop = rd.object(&c, "loop");
        start = rd.size(loop, "start", true);
        stop = rd.size(loop, "stop");
        times = rd.size(loop, "times");
        if (rd.ok && (start >= stop || stop > n_layer || times > 1024)) rd.fail("config.json: 'loop' names layers that do not exist");
    }
    if (!rd.ok) return false;

    // sizes first: the activation buffers are shared by the layers
    auto grow = [](auto &m, auto v) {
        if (v > m) m = v;
    };
    auto grow_k = [&](uint32_t k) { grow(max_k, rmi_dense_pad(k, kDenseKAlign)); };
    layers.resize(n_layer);
    std::vector<uint32_t> ff(n_layer, 0);
    for (uint32_t i = 0; i < n_layer; i++) {
        const std::string where = "config.json: layer " + std::to_string(i);
        const RmiJson *type = ls[i].get("type"), *mix = rd.object(&ls[i], "mixer"), *mlp = ls[i].get("mlp");
        VogizenLayer &l = layers[i];
        uint64_t n_k, n_v;
        if (type && type->text == "delta") {
            l.delta = true;
            RmiDeltaShape &s = l.rule;
            s.heads = rd.size(mix, "heads");
            s.kv_heads = rd.size(mix, "kv_heads");
            s.dim = rd.size(mix, "dim");
            s.vdim = rd.size(mix, "vdim");
            s.taps = rd.size(mix, "conv");
            s.eps = eps;
            s.d_pad = rmi_dense_pad(s.dim, 16);
            s.v_pad = rmi_dense_pad(s.vdim, 16);
            if (rd.ok && (s.heads % s.kv_heads || s.d_pad > kMaxHeadDim || s.v_pad > kMaxHeadDim || s.taps > kMaxTaps))
                rd.fail(where + ": unsupported shape (head sizes up to " + std::to_string(kMaxHeadDim) + ", up to " + std::to_string(kMaxTaps) + " taps)");
            n_k = uint64_t(s.kv_heads) * s.dim;
            n_v = uint64_t(s.heads) * s.vdim;
            grow(max_heads, s.heads);
            if (rd.ok) grow(max_values, uint32_t(n_v));
            if (rd.ok) grow(max_delta_scratch, rmi_delta_scratch_floats(s, pass_rows));
        } else if (type && type->text == "latent_attention") {
            RmiAttnShape &a = l.attn;
            a.heads = a.kv_heads = rd.size(mix, "heads");
            a.dim = rd.size(mix, "dim");
            a.vdim = rd.size(mix, "vdim");
            a.scale = float(rd.number(mix, "scale"));
            a.window = rd.size(rd.object(mix, "mask"), "size");
            l.q_rank = rd.size(mix, "q_rank");
            l.kv_rank = rd.size(mix, "kv_rank");
            a.taps = 1;
            a.eps = eps;
            a.dk_pad = rmi_dense_pad(a.dim, 32);
            a.dv_pad = rmi_dense_pad(a.vdim, 16);
            if (a.window > capacity) a.window = capacity;  // (it never shows)
            a.capacity = rmi_attn_rows(a.window, pass_rows, capacity);
            if (rd.ok && (a.dk_pad > kMaxHeadDim || a.dv_pad > kMaxHeadDim || l.q_rank > kInputMax || l.kv_rank > kInputMax))
                rd.fail(where + ": unsupported shape (head sizes up to " + std::to_string(kMaxHeadDim) + ")");
            n_k = uint64_t(a.heads) * a.dim;
            n_v = uint64_t(a.heads) * a.vdim;
            grow(max_q_rank, l.q_rank);
            grow(max_kv_rank, l.kv_rank);
            grow_k(l.q_rank);
            grow_k(l.kv_rank);
            one_token_gemv = one_token_gemv && fits(l.q_rank) && fits(l.kv_rank);
            if (rd.ok) grow(max_q, size_t(pass_rows) * a.heads * a.dk_pad * elem);
            if (rd.ok) grow(max_attn_scratch, rmi_attn_scratch_bytes(a));
        } else {
            rd.fail(where + " has a type other than 'delta' and 'latent_attention'");
            return false;
        }
        if (rd.ok && 2 * n_k + n_v > (1u << 24)) rd.fail(where + ": unsupported shape");
        if (mlp && !mlp->is_null()) {
            const RmiJson *kind = mlp->get("kind");
            if (!kind || kind->text != "dense") rd.fail(where + " has a feed-forward that is not 'dense'");
            ff[i] = rd.size(mlp, "ff");
            if (ff[i] > (1u << 24)) rd.fail(where + ": unsupported shape");
            l.ffn = true;
        }
        if (!rd.ok) return false;
        grow(max_u, uint32_t(2 * n_k + n_v));
        grow(max_ld, rmi_dense_ld(rmi_dense_pad(uint32_t(n_v), kDenseKAlign), elem));
        grow(max_ld, rmi_dense_ld(rmi_dense_pad(ff[i], kDenseKAlign), elem));
    }
    if (looped) grow_k(2 * k_in);
    one_token_gemv = one_token_gemv && rmi_dense_gemv_fits(elem, k_in) && (!looped || rmi_dense_gemv_fits(elem, 2 * k_in)) && fits(side_dim) && side_dim <= kInputMax;
    if (uint64_t(side_dim) * n_layer > (1u << 24)) rd.fail("config.json: unsupported 'token_side'");
    if (!rd.ok) return false;

    const size_t rows = pass_rows;
    const uint32_t side_ld = rmi_dense_ld(rmi_dense_pad(side_dim, kDenseKAlign), elem);
    if (!alloc_common(max_k) || !(x_next = alloc<float>(rows * width, true)) || !(u = alloc<float>(rows * max_u, true)) ||
        !(beta = alloc<float>(rows * max_heads, true)) || !(decay = alloc<float>(rows * max_heads, true)) ||
        !(gate = alloc<float>(rows * max_values, true)) || !(cq = alloc<float>(rows * max_q_rank, true)) ||
        !(ckv = alloc<float>(rows * max_kv_rank, true)) || !(y = alloc<float>(rows * width, true)) || !(side_f32 = alloc<float>(side_dim, true)) ||
        !(act = alloc_bytes(rows * max_ld * elem, true)) || !(q = alloc_bytes(max_q, true)) || !(side = alloc_bytes(rows * side_ld * elem, true)) ||
        !(attn_scratch = alloc_bytes(max_attn_scratch + 16, true)) || !(delta_scratch = alloc<float>(max_delta_scratch, true)))
        return false;
    if (looped && !(x_embedded = alloc<float>(rows * width, true))) return false;

    std::vector<double> turns((width + 1) / 2);  // of the sinusoidal position vector
    for (size_t i = 0; i < turns.size(); i++) turns[i] = std::pow(10000.0, -2.0 * double(i) / width) / 6.283185307179586476925286766559;
    double *d_turns = alloc<double>(turns.size());
    if (!d_turns || hipMemcpy(d_turns, turns.data(), turns.size() * 8, hipMemcpyHostToDevice) != hipSuccess) return false;
    embedding.turns = d_turns;

    if (!(final_norm = upload_vector(rd.tensor("final.norm", {width})))) return false;
    if (looped) {
        RmiDenseBuilder b(elem, rmi_dense_pad(width, kDenseRowAlign), 2 * k_in);
        const RmiTensor *t = rd.tensor("loop.in", {width, 2 * uint64_t(width)});
        b.put(t, 0, 0, 1, 0, width);
        b.put(t, 0, k_in, 1, width, width);
        if (!rd.ok || !b.upload(this, &w_loop)) return false;
    }
    {
        RmiDenseBuilder b(elem, vocab, rmi_dense_pad(side_dim * n_layer, kDenseKAlign));
        b.put(rd.tensor("side.embed", {vocab, uint64_t(side_dim) * n_layer}), 0, 0);
        if (!rd.ok || !b.upload(this, &side_table)) return false;
    }
    for (uint32_t i = 0; i < n_layer; i++) {
        VogizenLayer &l = layers[i];
        const std::string p = "l" + std::to_string(i) + ".";
        if (!(l.norm1 = upload_vector(rd.tensor(p + "norm1", {width}))) || !(l.side_norm = upload_vector(rd.tensor(p + "side.norm", {width})))) return false;
        if (!(l.delta ? load_delta(rd, l, p) : load_latent(rd, l, p)) || (l.ffn && !load_ffn(rd, l, p, ff[i]))) return false;
        RmiRowSeg g = segment(side, side_dim, side_ld, kActGeluTanh);
        g.mul = static_cast<const uint8_t *>(side_table.data) + size_t(i) * side_dim * elem;
        g.mul_ld = side_table.ld;
        g.mul_rows = vocab;
        if (!stack(rd, &l.w_gate, &l.gate, {{p + "side.gate", g}}, width) ||
            !stack(rd, &l.w_proj, &l.proj, {{p + "side.proj", segment(y, width, width, kActNone)}}, side_dim))
            return false;
    }

    auto add_run = [&](uint32_t i, bool begins) {
        VogizenRun r;
        r.layer = i;
        r.loop_begins = begins;
        const VogizenLayer &l = layers[i];
        bool ok = true;
        if (l.delta) {
            const RmiDeltaShape &s = l.rule;
            const size_t hist = size_t(s.taps - 1) * (2 * s.kv_heads * s.dim + s.heads * s.vdim), state = size_t(s.heads) * s.d_pad * s.v_pad;
            for (int j = 0; j < 2; j++) ok = ok && (r.hist[j] = alloc<float>(hist, true)) && (r.state[j] = alloc<float>(state, true));
        } else {
            const RmiAttnShape &a = l.attn;
            ok = (r.k_cache = alloc_bytes(size_t(a.heads) * a.capacity * a.dk_pad * elem, true)) &&
                 (r.v_cache = alloc_bytes(size_t(a.heads) * a.capacity * a.dv_pad * elem, true));
        }
        runs.push_back(r);
        return ok;
    };
    bool ok = true;
    for (uint32_t i = 0; i < start; i++) ok = ok && add_run(i, false);
    for (uint32_t t = 0; t < times; t++)
        for (uint32_t i = start; i < stop; i++) ok = ok && add_run(i, i == start);
    for (uint32_t i = stop; i < n_layer; i++) ok = ok && add_run(i, false);
    n_runs = uint32_t(runs.size());
    return ok && rd.ok;
}

}  // namespace

rmi_hip_folder_session *rmi_new_vogizen() { return new VogizenSession(); }
