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

#include "folder_session.h"
#include "seq_mixers.h"

namespace {

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

struct RuvenexSession : rmi_hip_folder_session {
    uint32_t cap_pad = 0;
    std::vector<RuvenexLayer> layers;
    float *final_norm = nullptr;
    // activations of a pass, token-major
    float *u = nullptr, *gate = nullptr, *rq = nullptr, *rf = nullptr, *rv = nullptr, *rg1 = nullptr, *rg2 = nullptr;
    void *act = nullptr, *q = nullptr;
    void *attn_scratch = nullptr;
    float *recur_scratch = nullptr;
    int now = 0;  // which of a layer's two history and state buffers the last pass left

    bool load(const RmiModelFolder &f) override;
    int enqueue_layers(uint32_t step0, uint32_t n, hipStream_t st, float *host_layers) override;
    RmiInput normed(const float *weight) const {
        RmiInput in;
        in.x = x;
        in.n = width;
        in.norm = kNormRms;
        in.weight = weight;
        in.eps = eps;
        return in;
    }
    RmiInput head_input() const override { return normed(final_norm); }
};

int RuvenexSession::enqueue_layers(uint32_t step0, uint32_t n, hipStream_t st, float *host_layers) {
    int rc = RMI_HIP_OK;
    for (uint32_t l = 0; l < n_runs && rc == RMI_HIP_OK; l++) {
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
            rc = rmi_dense_gemv(elem, y.w_in, normed(y.norm), y.in, st);
            if (rc == RMI_HIP_OK) rc = rmi_mixers_step(elem, &y.attn, &a, &y.recur, &r, st);
            if (rc == RMI_HIP_OK) rc = rmi_dense_gemv_residual(elem, y.w_out, act, y.out, x, width, st);
        } else {
            rc = rmi_dense_input(elem, normed(y.norm), nullptr, h, n, k_in, st);
            if (rc == RMI_HIP_OK) rc = rmi_dense_gemm(elem, y.w_in, h, y.in, n, st);
            if (rc == RMI_HIP_OK) rc = rmi_attn_pass(elem, y.attn, a, st);
            if (rc == RMI_HIP_OK) rc = rmi_recur_pass(elem, y.recur, r, st);
            if (rc == RMI_HIP_OK) rc = rmi_dense_gemm_residual(elem, y.w_out, act, y.out, x, width, n, st);
        }
        if (host_layers && rc == RMI_HIP_OK) rc = copy_layer(host_layers, l, n, st);
    }
    now ^= 1;
    position = step0 + n;
    return rc;
}

bool RuvenexSession::load(const RmiModelFolder &folder) {
    RmiFolderReader rd(folder);
    if (!load_common(rd)) return false;
    const std::vector<RmiJson> &ls = folder.config.get("layers")->items;
    const uint32_t n_layer = n_runs = uint32_t(ls.size());
    cap_pad = rmi_dense_pad(capacity, kKeyBlock);
    if (cap_pad > 0x7fffffffu / kMaxHeadDim) {
        rmi_set_error("unsupported model shape: the cache overflows");
        return false;
    }
    {
        RmiDenseBuilder b(elem, rmi_dense_pad(vocab, kDenseRowAlign), k_in);
        b.put(rd.tensor("head", {vocab, width}), 0, 0);
        if (!rd.ok || !b.upload(this, &head)) return false;
    }
    if (!(final_norm = upload_vector(rd.tensor("final.norm", {width})))) return false;

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
        const RmiJson *e = &ls[l], *type = e->get("type");
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
        a.v_norm = true;
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
        const RmiColSeg sa{nullptr, width, float(left_scale), y.k_attn}, sr{nullptr, width, float(right_scale), y.k_recur},
            sf{nullptr, width, 1.0f, y.w_out.k_pad};
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
    if (!alloc_common(0) || !(u = alloc<float>(rows * max_channels, true)) || !(gate = alloc<float>(rows * max_heads, true)) ||
        !(rq = alloc<float>(rows * max_rq, true)) || !(rf = alloc<float>(rows * max_rq, true)) || !(rv = alloc<float>(rows * max_rv, true)) ||
        !(rg1 = alloc<float>(rows * width, true)) || !(rg2 = alloc<float>(rows * width, true)) ||
        !(act = alloc_bytes(rows * max_ld * elem, true)) || !(q = alloc_bytes(max_q, true)) ||
        !(attn_scratch = alloc_bytes(max_attn_scratch + 16, true)) || !(recur_scratch = alloc<float>(max_recur_scratch, true)))
        return false;

    std::map<std::pair<uint32_t, double>, std::pair<float *, float *>> rotations;
    for (uint32_t l = 0; l < n_layer; l++) {
        RuvenexLayer &y = layers[l];
        const Sizes &z = sizes[l];
        const RmiAttnShape &a = y.attn;
        const RmiRecurShape &r = y.recur;
        const std::string p = "l" + std::to_string(l) + ".", L = p + "mix.left.", R = p + "mix.right.";
        const uint32_t n_q = a.heads * a.dim, n_k = a.kv_heads * a.dim, n_v = a.kv_heads * a.vdim;
        float *f_bias = upload_vector(rd.tensor(R + "f.b", {z.n_recur})), *lower = upload_vector(rd.tensor(R + "lower", {z.n_recur}));
        float *b1 = upload_vector(rd.tensor(p + "rg1.b", {width})), *b2 = nullptr;
        if (z.ff) b2 = upload_vector(rd.tensor(p + "rg2.b", {width}));
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
            RmiDenseBuilder b(elem, n_rows, k_in);
            for (size_t i = 0; i < parts.size() && rd.ok; i++) b.put(rd.tensor(parts[i].name, {parts[i].n, width}), y.in.s[i].row0, 0);
            if (!rd.ok || !b.upload(this, &y.w_in)) return false;
        }
        // everything that ends in x
        y.out.s[0].gate = y.out.s[1].gate = rg1;
        if (z.ff) y.out.s[2].gate = rg2;
        {
            RmiDenseBuilder b(elem, rmi_dense_pad(width, kDenseRowAlign), y.w_out.k_pad);
            b.put(rd.tensor(L + "o", {width, uint64_t(a.heads) * a.vdim}), 0, 0);
            b.put(rd.tensor(R + "o", {width, z.n_recur_v}), 0, y.k_attn);
            if (z.ff) b.put(rd.tensor(p + "mlp.down", {width, z.ff}), 0, y.k_recur);
            if (!rd.ok || !b.upload(this, &y.w_out)) return false;
        }
        if (!(y.norm = upload_vector(rd.tensor(p + "norm1", {width}))) || !(y.recur_norm = upload_vector(rd.tensor(R + "norm", {r.vdim}))))
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
    return rd.ok;
}

}  // namespace

rmi_hip_folder_session *rmi_new_ruvenex() { return new RuvenexSession(); }
