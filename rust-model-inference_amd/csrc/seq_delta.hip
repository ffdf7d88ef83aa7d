// The gated delta rule (seq_mixers.h): kernels for single tokens and for passes of several.
#include "device_conv.h"
#include "device_dense.h"
#include "seq_mixers.h"

namespace {

constexpr uint32_t kRunTaps = 4;  // up to here the taps and a window of rows sit in registers

__host__ __device__ inline uint32_t delta_channels(const RmiDeltaShape &s) { return 2 * s.kv_heads * s.dim + s.heads * s.vdim; }
// where the channels of key head g's queries and keys, and of head h's values, begin
__device__ __forceinline__ uint32_t q_channel(const RmiDeltaShape &s, uint32_t g) { return g * s.dim; }
__device__ __forceinline__ uint32_t k_channel(const RmiDeltaShape &s, uint32_t g) { return (s.kv_heads + g) * s.dim; }
__device__ __forceinline__ uint32_t v_channel(const RmiDeltaShape &s, uint32_t h) { return 2 * s.kv_heads * s.dim + h * s.vdim; }

__device__ __forceinline__ float delta_beta(const RmiDeltaShape &s, const RmiDeltaArgs &a, uint32_t t, uint32_t h) {
    return sigmoid_t<float>(a.b[size_t(t) * s.heads + h]);
}
__device__ __forceinline__ float delta_decay(const RmiDeltaShape &s, const RmiDeltaArgs &a, uint32_t t, uint32_t h) {
    return expf(-a.rate[h] * softplus_f32(a.a[size_t(t) * s.heads + h] + a.bias[h]));
}

// the history that head h passes on: its values' channels, and as the first of its group the queries' and keys'
__device__ __forceinline__ void delta_carry(const RmiDeltaShape &s, const RmiDeltaArgs &a, const ConvCtx &x, uint32_t h, uint32_t threads) {
    const uint32_t group = s.heads / s.kv_heads, g = h / group;
    for (uint32_t d = threadIdx.x; d < s.vdim; d += threads) conv_carry(x, a.hist_out, a.n_tokens, v_channel(s, h) + d);
    if (h % group) return;
    for (uint32_t d = threadIdx.x; d < s.dim; d += threads) {
        conv_carry(x, a.hist_out, a.n_tokens, q_channel(s, g) + d);
        conv_carry(x, a.hist_out, a.n_tokens, k_channel(s, g) + d);
    }
}

// ---- one token: a workgroup a head.  A thread keeps a quad of columns of every slices-th state row; one walk over the
// state gives both S^T k and S^T q, and with them
//   u = beta (v - g S^T k),   o = g S^T q + (k . q) u,   S' = g S + k u^T
constexpr uint32_t kStepThreads = 512;
template <typename T, int NR>
__global__ __launch_bounds__(kStepThreads) void delta_step_kernel(RmiDeltaShape s, RmiDeltaArgs a) {
    __shared__ __attribute__((aligned(16))) float ks[kMaxHeadDim], qs[kMaxHeadDim], vs[kMaxHeadDim], us[kMaxHeadDim], red[8];
    __shared__ __attribute__((aligned(16))) float part[2][4 * kStepThreads];  // [S^T k, S^T q][slice][column]
    const uint32_t tid = threadIdx.x, lane = tid & 63, h = blockIdx.x, group = s.heads / s.kv_heads, g = h / group;
    const ConvCtx x{a.u, a.hist_in, a.conv, delta_channels(s), s.taps};
    const uint32_t n_ch = 2 * s.dim + s.vdim;  // this head's channels: queries, keys, values
    auto channel = [&](uint32_t e) { return e < s.dim ? q_channel(s, g) + e : e < 2 * s.dim ? k_channel(s, g) + e - s.dim : v_channel(s, h) + e - 2 * s.dim; };
    auto put = [&](uint32_t e, float z) {
        z *= sigmoid_t<T>(z);
        if (e < s.dim) qs[e] = z;
        else if (e < 2 * s.dim) ks[e - s.dim] = z;
        else vs[e - 2 * s.dim] = z;
    };
    // the convolution's operands first, the state's behind them: everything waits for the former
    float row[2][kRunTaps], tap[2][kRunTaps];
    uint32_t ch[2];
    const bool run = s.taps <= kRunTaps;
    if (run) {
#pragma unroll
        for (uint32_t i = 0; i < 2; i++) {
            const uint32_t e = tid + i * kStepThreads;
            ch[i] = channel(e < n_ch ? e : 0);
#pragma unroll
            for (uint32_t back = 0; back < kRunTaps; back++) {  // (every load is issued; what does not count is cleared below)
                const uint32_t b = back < s.taps ? back : s.taps - 1;
                const float *src = back == 0 || b == 0 ? a.u : a.hist_in + size_t(s.taps - 1 - b) * x.channels;
                row[i][back] = src[ch[i]];
                tap[i][back] = a.conv[ch[i] * s.taps + s.taps - 1 - b];
            }
        }
    }
    const float decay = delta_decay(s, a, 0, h), beta = delta_beta(s, a, 0, h);
    const uint32_t quads = s.v_pad / 4, slices = kStepThreads / quads, col = tid % quads, sl = tid / quads;
    const size_t at = size_t(h) * s.d_pad * s.v_pad + col * 4;
    f32x4 r[NR];
#pragma unroll
    for (uint32_t j = 0; j < NR; j++) {
        const uint32_t d = sl + j * slices;
        r[j] = *reinterpret_cast<const f32x4 *>(a.state_in + at + size_t(d < s.d_pad ? d : 0) * s.v_pad);
    }
    const float gate = tid < s.vdim ? a.gate[size_t(h) * s.vdim + tid] : 0.0f, weight = tid < s.vdim ? a.norm[tid] : 0.0f;
    if (run) {
#pragma unroll
        for (uint32_t i = 0; i < 2; i++) {
            const uint32_t e = tid + i * kStepThreads;
            float z = 0.0f;
#pragma unroll
            for (uint32_t back = kRunTaps; back-- > 0;) z = __builtin_fmaf(tap[i][back], back < s.taps && a.pos0 >= back ? row[i][back] : 0.0f, z);
            if (e < n_ch) put(e, z);
            if (e < n_ch && (e >= 2 * s.dim || h % group == 0)) {  // the rows that the next token looks back on
#pragma unroll
                for (uint32_t back = 0; back + 1 < kRunTaps; back++)
                    if (back + 1 < s.taps) a.hist_out[size_t(s.taps - 2 - back) * x.channels + ch[i]] = row[i][back];
            }
        }
    } else {
        for (uint32_t e = tid; e < n_ch; e += kStepThreads) put(e, conv_at(x, 0, a.pos0, channel(e)));
        delta_carry(s, a, x, h, kStepThreads);
    }
    for (uint32_t d = s.dim + tid; d < s.d_pad; d += kStepThreads) qs[d] = ks[d] = 0.0f;
    for (uint32_t d = s.vdim + tid; d < s.v_pad; d += kStepThreads) vs[d] = 0.0f;
    __syncthreads();
    float qq = 0.0f, kk = 0.0f, kq = 0.0f;  // every wave for itself
    for (uint32_t d = lane; d < s.d_pad; d += 64) {
        const float q = qs[d], k = ks[d];
        qq = __builtin_fmaf(q, q, qq);
        kk = __builtin_fmaf(k, k, kk);
        kq = __builtin_fmaf(k, q, kq);
    }
    const float rk = 1.0f / sqrtf(wave_sum_f32(kk) + 1e-6f), rq = 1.0f / sqrtf(wave_sum_f32(qq) + 1e-6f) / sqrtf(float(s.dim));
    kq = wave_sum_f32(kq) * rk * rq;
    if (sl < slices) {
        f32x4 pk = {0.f, 0.f, 0.f, 0.f}, pq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (uint32_t j = 0; j < NR; j++) {
            const uint32_t d = sl + j * slices;
            const bool live = d < s.d_pad && a.pos0;
            const float k = ks[live ? d : 0], q = qs[live ? d : 0];
            if (!live) r[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int e = 0; e < 4; e++) {
                pk[e] = __builtin_fmaf(r[j][e], k, pk[e]);
                pq[e] = __builtin_fmaf(r[j][e], q, pq[e]);
            }
        }
        *reinterpret_cast<f32x4 *>(&part[0][sl * s.v_pad + col * 4]) = pk;
        *reinterpret_cast<f32x4 *>(&part[1][sl * s.v_pad + col * 4]) = pq;
    }
    __syncthreads();
    float o = 0.0f;
    if (tid < s.v_pad) {
        float sk = 0.0f, sq = 0.0f;
        for (uint32_t i = 0; i < slices; i++) {
            sk += part[0][i * s.v_pad + tid];
            sq += part[1][i * s.v_pad + tid];
        }
        const float u = beta * (vs[tid] - decay * (rk * sk));
        us[tid] = u;
        o = __builtin_fmaf(kq, u, decay * (rq * sq));
    }
    const float sq = wave_sum_f32(o * o);
    if (lane == 0) red[tid >> 6] = sq;
    __syncthreads();
    if (sl < slices) {
        const f32x4 u = *reinterpret_cast<const f32x4 *>(us + col * 4);
#pragma unroll
        for (uint32_t j = 0; j < NR; j++) {
            const uint32_t d = sl + j * slices;
            if (d >= s.d_pad) continue;
            const float k = rk * ks[d];
            f32x4 n;
#pragma unroll
            for (int e = 0; e < 4; e++) n[e] = __builtin_fmaf(k, u[e], decay * r[j][e]);
            *reinterpret_cast<f32x4 *>(a.state_out + at + size_t(d) * s.v_pad) = n;
        }
    }
    float total = 0.0f;
#pragma unroll
    for (uint32_t i = 0; i < kStepThreads / 64; i++) total += red[i];
    const float norm = 1.0f / sqrtf(total / float(s.vdim) + s.eps);
    if (tid < s.vdim) static_cast<T *>(a.out)[size_t(h) * s.vdim + tid] = from_f32<T>(o * norm * weight * gate);
}

// ---- several tokens, in chunks of sixteen.  With G_t the product of g over the chunk's tokens up to t and
// D_ts = g_{s+1} .. g_t (running products: nothing is divided by a decay):
//   u_t = beta_t (v_t - G_t S0^T k_t - sum_{s < t} D_ts (k_s . k_t) u_s), a unit lower triangular system (1 + A) u = b
//   o_t = G_t S0^T q_t + sum_{s <= t} D_ts (q_t . k_s) u_s
//   S'  = G_15 S0 + sum_s D_15,s k_s u_s^T
// With T = (1 + A)^-1 diag(beta), by forward substitution, and M = D (q k^T), everything that meets the state does so as
//   u = T v - W S0,   W = T G k;      o = M T v + Q S0,   Q = G q - M W
// so the first kernel makes W, Q, T v and M T v for all chunks at once, and the second, which walks the chunks with the
// state in the matrix cores' accumulators, has two products a chunk between one state and the next.
constexpr uint32_t kChunk = 16;
struct DeltaScratch {
    float *w, *q, *kt, *v, *o, *dk;
};
__host__ __device__ inline size_t delta_scratch_at(float *p, const RmiDeltaShape &s, uint32_t n_chunks, DeltaScratch *w) {
    const size_t hc = size_t(s.heads) * n_chunks, rows_k = hc * kChunk * s.d_pad, rows_v = hc * kChunk * s.v_pad;
    size_t at = 0;
    auto take = [&](size_t n) {
        const size_t was = at;
        at += n;
        return was;
    };
    const size_t wk = take(rows_k), q = take(rows_k), v = take(rows_v), o = take(rows_v);
    const size_t kt = take(size_t(s.kv_heads) * n_chunks * kChunk * s.d_pad), dk = take(hc * 2 * kChunk);
    if (w) {
        w->w = p + wk;   // [head][chunk][16][d_pad]
        w->q = p + q;    // [head][chunk][16][d_pad]
        w->v = p + v;    // [head][chunk][v_pad][16]: T v
        w->o = p + o;    // [head][chunk][16][v_pad]: M T v, then o
        w->kt = p + kt;  // [kv_head][chunk][d_pad][16]
        w->dk = p + dk;  // [head][chunk][D_15 of 16, G_15]
    }
    return at;
}

// channel c convolved over the sixteen tokens of a chunk (t0 a multiple of 16; tokens past the end: zero)
template <typename T>
__device__ __forceinline__ void conv_chunk(const ConvCtx &x, const RmiDeltaArgs &a, uint32_t t0, uint32_t c, float (&y)[kChunk]) {
    if (x.taps <= kRunTaps) {
        float row[kChunk + kRunTaps - 1], w[kRunTaps];
#pragma unroll
        for (uint32_t i = 0; i < kRunTaps; i++) w[i] = i < x.taps ? x.conv[c * x.taps + x.taps - 1 - i] : 0.0f;  // i tokens back
#pragma unroll
        for (uint32_t i = 0; i < kRunTaps - 1; i++) {  // the rows before the chunk's first
            const uint32_t back = kRunTaps - 1 - i;
            row[i] = 0.0f;
            if (t0 >= back) row[i] = x.u[size_t(t0 - back < a.n_tokens ? t0 - back : a.n_tokens - 1) * x.channels + c];
            else if (back < x.taps && a.pos0 >= back) row[i] = x.hist[size_t(x.taps - 1 - back) * x.channels + c];  // (t0 = 0)
        }
#pragma unroll
        for (uint32_t i = 0; i < kChunk; i++) row[kRunTaps - 1 + i] = x.u[size_t(t0 + i < a.n_tokens ? t0 + i : a.n_tokens - 1) * x.channels + c];
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) {
            y[t] = 0.0f;
#pragma unroll
            for (uint32_t i = kRunTaps; i-- > 0;) y[t] = __builtin_fmaf(w[i], row[t + kRunTaps - 1 - i], y[t]);
        }
    } else {
        for (uint32_t t = 0; t < kChunk; t++) y[t] = t0 + t < a.n_tokens ? conv_at(x, t0 + t, a.pos0, c) : 0.0f;
    }
#pragma unroll
    for (uint32_t t = 0; t < kChunk; t++) y[t] = t0 + t < a.n_tokens ? y[t] * sigmoid_t<T>(y[t]) : 0.0f;
}

// one chunk of one head; the first head of a group also stores the group's k
constexpr uint32_t kTl = kChunk + 4;  // rows of sixteen tokens in LDS
__host__ __device__ inline uint32_t factors_lds_floats(const RmiDeltaShape &s) { return 2 * kChunk * (s.d_pad + 4) + (s.d_pad + s.v_pad) * kTl; }
constexpr uint32_t kFactorThreads = 512;
template <typename T>
__global__ __launch_bounds__(kFactorThreads) void delta_factors_kernel(RmiDeltaShape s, RmiDeltaArgs a, uint32_t n_pad) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    const uint32_t ld = s.d_pad + 4;
    float *ql = reinterpret_cast<float *>(lds_raw), *kl = ql + kChunk * ld;  // [16][d_pad + 4]
    float *kt = kl + kChunk * ld, *vt = kt + s.d_pad * kTl;                  // [d_pad][20], [v_pad][20]
    __shared__ __attribute__((aligned(16))) float dm[kChunk][kChunk], am[kChunk][kTl], mm[kChunk][kTl], tm[kChunk][kTl], beta[kChunk], decay[kChunk], gl[kChunk];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6))), chunk = blockIdx.x, h = blockIdx.y,
                   t0 = chunk * kChunk;
    const uint32_t group = s.heads / s.kv_heads, g = h / group;
    const ConvCtx x{a.u, a.hist_in, a.conv, delta_channels(s), s.taps};
    DeltaScratch ws;
    delta_scratch_at(a.scratch, s, n_pad, &ws);
    const size_t hc = size_t(h) * n_pad + chunk;
    for (uint32_t e = tid; e < 2 * s.d_pad + s.v_pad; e += kFactorThreads) {
        const bool is_v = e >= 2 * s.d_pad, is_k = !is_v && e >= s.d_pad;
        const uint32_t d = is_v ? e - 2 * s.d_pad : is_k ? e - s.d_pad : e;
        float y[kChunk];
        if (d < (is_v ? s.vdim : s.dim)) {
            conv_chunk<T>(x, a, t0, (is_v ? v_channel(s, h) : is_k ? k_channel(s, g) : q_channel(s, g)) + d, y);
        } else {
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) y[t] = 0.0f;
        }
        if (is_v) {
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t += 4) *reinterpret_cast<f32x4 *>(vt + d * kTl + t) = f32x4{y[t], y[t + 1], y[t + 2], y[t + 3]};
        } else {
            float *dst = (is_k ? kl : ql) + d;
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) dst[t * ld] = y[t];
        }
    }
    if (tid >= 128 && tid < 128 + kChunk) {
        const uint32_t t = tid - 128;
        const bool live = t0 + t < a.n_tokens;  // a token past the end changes nothing
        decay[t] = live ? delta_decay(s, a, t0 + t, h) : 1.0f;
        beta[t] = live ? delta_beta(s, a, t0 + t, h) : 0.0f;
    }
    __syncthreads();
    if (tid < kChunk) {  // column s of D
        float w = 1.0f;
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) {
            if (t > tid) w *= decay[t];
            dm[t][tid] = t < tid ? 0.0f : w;
        }
        ws.dk[hc * 2 * kChunk + tid] = w;
    } else if (tid == 64) {
        float w = 1.0f;
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) {
            w *= decay[t];
            gl[t] = w;
        }
        ws.dk[hc * 2 * kChunk + kChunk] = w;
    }
    // unit length
    for (uint32_t t = wave; t < kChunk; t += kFactorThreads / 64) {
        float qq = 0.0f, kk = 0.0f;
        for (uint32_t d = lane; d < s.d_pad; d += 64) {
            qq = __builtin_fmaf(ql[t * ld + d], ql[t * ld + d], qq);
            kk = __builtin_fmaf(kl[t * ld + d], kl[t * ld + d], kk);
        }
        const float rq = 1.0f / sqrtf(wave_sum_f32(qq) + 1e-6f) / sqrtf(float(s.dim)), rk = 1.0f / sqrtf(wave_sum_f32(kk) + 1e-6f);
        for (uint32_t d = lane; d < s.d_pad; d += 64) {
            ql[t * ld + d] *= rq;
            kt[d * kTl + t] = kl[t * ld + d] *= rk;
        }
    }
    __syncthreads();
    const uint32_t fr = lane & 15, q4 = lane >> 4;
    auto quad = [](const float *p) { return *reinterpret_cast<const f32x4 *>(p); };
    if (wave < 2) {  // wave 0: k k^T and the triangular system; wave 1: q k^T
        const float *lhs = wave == 0 ? kl : ql;
        f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
        for (uint32_t d = 0; d < s.d_pad; d += 32) {
            acc[0] = mma16_f32(quad(lhs + fr * ld + d + q4 * 4), quad(kl + fr * ld + d + q4 * 4), acc[0]);
            if (d + 16 < s.d_pad) acc[1] = mma16_f32(quad(lhs + fr * ld + d + 16 + q4 * 4), quad(kl + fr * ld + d + 16 + q4 * 4), acc[1]);
        }
        const f32x4 dot = acc[0] + acc[1];  // row t = 4 q4 + r, column s = fr
#pragma unroll
        for (uint32_t r = 0; r < 4; r++) {
            const uint32_t t = q4 * 4 + r;
            (wave == 0 ? am : mm)[t][fr] = dot[r] * dm[t][fr] * (wave == 0 ? beta[t] : 1.0f);
        }
        if (wave == 0) {
            rmi_wave_lds_fence();
            // lane j < 16 solves for column j; the entries on and above the diagonal are never read
            float c[kChunk];
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) {
                float v = t == fr ? 1.0f : 0.0f;
#pragma unroll
                for (uint32_t e = 0; e < t; e++) v = __builtin_fmaf(-am[t][e], c[e], v);
                c[t] = v;
            }
            if (lane < 16) {
                const float b = beta[fr];
#pragma unroll
                for (uint32_t t = 0; t < kChunk; t++) tm[t][fr] = c[t] * b;
            }
        }
    } else if (h % group == 0) {
        float *dst = ws.kt + (size_t(g) * n_pad + chunk) * kChunk * s.d_pad;
        for (uint32_t e = tid - 128; e < s.d_pad * (kChunk / 4); e += kFactorThreads - 128) *reinterpret_cast<f32x4 *>(dst + e * 4) = quad(kt + (e >> 2) * kTl + (e & 3) * 4);
    }
    __syncthreads();
    // A result (row 4g + r, column fr) is the next product's right operand as it lies, and its transpose's left one.  What
    // goes to memory by token is computed transposed, four channels of token fr in a lane, for one store.
    const f32x4 tr = quad(&tm[fr][q4 * 4]), mr = quad(&mm[fr][q4 * 4]), gt = quad(gl + q4 * 4), zero = {0.f, 0.f, 0.f, 0.f};
    const uint32_t k_tiles = s.d_pad / 16, tiles = k_tiles + s.v_pad / 16;
    for (uint32_t i = wave; i < tiles; i += kFactorThreads / 64) {
        if (i < k_tiles) {
            const f32x4 gk = quad(kt + (i * 16 + fr) * kTl + q4 * 4) * gt;
            const f32x4 w = mma16_f32(tr, gk, zero), wt = mma16_f32(gk, tr, zero), mw = mma16_f32(w, mr, zero);
            const uint32_t c = i * 16 + q4 * 4;
            const size_t to = (hc * kChunk + fr) * s.d_pad + c;
            *reinterpret_cast<f32x4 *>(ws.w + to) = wt;
            *reinterpret_cast<f32x4 *>(ws.q + to) = quad(ql + fr * ld + c) * gl[fr] - mw;
        } else {
            const uint32_t c0 = (i - k_tiles) * 16;
            const f32x4 v = mma16_f32(tr, quad(vt + (c0 + fr) * kTl + q4 * 4), zero), o = mma16_f32(v, mr, zero);
            *reinterpret_cast<f32x4 *>(ws.v + (hc * s.v_pad + c0 + fr) * kChunk + q4 * 4) = v;
            *reinterpret_cast<f32x4 *>(ws.o + (hc * kChunk + fr) * s.v_pad + c0 + q4 * 4) = o;
        }
    }
}

// One workgroup: sixteen value channels of one head, over all chunks of the pass; wave w holds the state's row tiles
// w, w + 4, ..  A tile in accumulator form (row 4g + r in register r) is the right operand of the next product as it lies.
// The waves' parts of W S meet in LDS at the chunk's barrier; those of Q S, which nothing waits for, once in four chunks,
// when each wave finishes o of one of the four.  All of it is one straight line, for a whole number of fours (a chunk
// without tokens leaves the state alone): a branch around a load or a store would make the waits behind it waits for
// all.  Workgroups of one head share an XCD: they read the same W, Q and k.
// FULL: the state has 4 TPW row tiles; otherwise the missing ones stay zero.
constexpr uint32_t kScanGroup = 4;
inline uint32_t scan_chunks(uint32_t n_tokens) { return (n_tokens + kChunk * kScanGroup - 1) / (kChunk * kScanGroup) * kScanGroup; }
__device__ __forceinline__ f32x4 quad_at(const float *base, uint32_t byte) { return *reinterpret_cast<const f32x4 *>(reinterpret_cast<const char *>(base) + byte); }

template <int TPW, bool FULL>
__global__ __launch_bounds__(256) void delta_scan_kernel(RmiDeltaShape s, RmiDeltaArgs a, uint32_t n_pad) {
    __shared__ f32x4 part_w[2][4][64], part_q[kScanGroup][4][64];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6))), fr = lane & 15, g4 = lane >> 4;
    const uint32_t v_tiles = s.v_pad / 16, n_tiles = s.d_pad / 16;
    uint32_t v_tile, h;
    rmi_gemm_tile_of(blockIdx.x, v_tiles, s.heads, 0u, 0u, v_tile, h);
    const uint32_t v0 = v_tile * 16, g = h / (s.heads / s.kv_heads);
    DeltaScratch ws;
    delta_scratch_at(a.scratch, s, n_pad, &ws);
    // this head's first chunk, and from there bytes: of a lane's pieces, and from chunk to chunk
    const float *pw = ws.w + size_t(h) * n_pad * kChunk * s.d_pad, *pq = ws.q + size_t(h) * n_pad * kChunk * s.d_pad;
    const float *pk = ws.kt + size_t(g) * n_pad * kChunk * s.d_pad, *pv = ws.v + size_t(h) * n_pad * kChunk * s.v_pad;
    const float *pd = ws.dk + size_t(h) * n_pad * 2 * kChunk;
    float *po = ws.o + size_t(h) * n_pad * kChunk * s.v_pad;
    const size_t step_k = size_t(kChunk) * s.d_pad, step_v = size_t(kChunk) * s.v_pad;  // floats
    uint32_t off_w[TPW], off_k[TPW];
    bool has[TPW];
    f32x4 st[TPW];
    const size_t at = size_t(h) * s.d_pad * s.v_pad + v0 + fr;
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        has[i] = FULL || wave + 4 * i < n_tiles;
        const uint32_t tile = has[i] ? wave + 4 * i : n_tiles - 1;
        off_w[i] = (fr * s.d_pad + tile * 16 + g4 * 4) * 4;
        off_k[i] = ((tile * 16 + fr) * kChunk + g4 * 4) * 4;
        st[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (a.pos0 == 0 || !has[i]) continue;
#pragma unroll
        for (int r = 0; r < 4; r++) st[i][r] = a.state_in[at + size_t(tile * 16 + g4 * 4 + r) * s.v_pad];
    }
    const uint32_t off_v = ((v0 + fr) * kChunk + g4 * 4) * 4, off_d = g4 * 16;
    struct Operands {
        f32x4 w[TPW], q[TPW], kt[TPW];
        f32x4 v, d;
        float keep;
    };
    auto load = [&](uint32_t chunk) {
        Operands x;
        const uint32_t c = chunk < n_pad ? chunk : n_pad - 1;
#pragma unroll
        for (int i = 0; i < TPW; i++) x.w[i] = quad_at(pw + c * step_k, off_w[i]);
        x.v = quad_at(pv + c * step_v, off_v);
        x.d = quad_at(pd + size_t(c) * 2 * kChunk, off_d);
        x.keep = pd[size_t(c) * 2 * kChunk + kChunk];
#pragma unroll
        for (int i = 0; i < TPW; i++) x.q[i] = quad_at(pq + c * step_k, off_w[i]);
#pragma unroll
        for (int i = 0; i < TPW; i++) x.kt[i] = quad_at(pk + c * step_k, off_k[i]);
        return x;
    };
    const uint32_t off_o = g4 * 4 * s.v_pad + v0 + fr;
    auto load_o = [&](uint32_t chunk) {
        const float *p = po + (chunk < n_pad ? chunk : n_pad - 1) * step_v;
        return f32x4{p[off_o], p[off_o + s.v_pad], p[off_o + 2 * s.v_pad], p[off_o + 3 * s.v_pad]};
    };
    constexpr uint32_t kAhead = TPW <= 2 ? 4 : 2;  // chunks whose operands are on their way
    static_assert(kScanGroup % kAhead == 0, "ring slots by compile-time index");
    Operands ring[kAhead];
#pragma unroll
    for (uint32_t j = 0; j < kAhead; j++) {
        ring[j] = load(j);
        asm volatile("" ::: "memory");  // in this order, and here: the waits in the loop count on it
    }
    f32x4 left = load_o(wave);
    asm volatile("" ::: "memory");
    for (uint32_t chunk0 = 0; chunk0 < n_pad; chunk0 += kScanGroup) {
#pragma unroll
        for (uint32_t j = 0; j < kScanGroup; j++) {
            const uint32_t chunk = chunk0 + j;
            const Operands &x = ring[j % kAhead];
            f32x4 w = {0.f, 0.f, 0.f, 0.f}, q = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < TPW; i++) w = mma16_f32(x.w[i], st[i], w);
            part_w[j & 1][wave][lane] = w;
            __builtin_amdgcn_sched_barrier(0);  // Q S stays behind the barrier, under the wait for the others' parts
            __syncthreads();  // (two buffers: the next chunk's writes cannot meet this one's reads)
            const f32x4 p0 = part_w[j & 1][0][lane], p1 = part_w[j & 1][1][lane], p2 = part_w[j & 1][2][lane], p3 = part_w[j & 1][3][lane];
#pragma unroll
            for (int i = 0; i < TPW; i++) q = mma16_f32(x.q[i], st[i], q);
            const f32x4 du = x.d * (x.v - ((p0 + p1) + (p2 + p3)));
#pragma unroll
            for (int i = 0; i < TPW; i++) {
                f32x4 k = x.kt[i];
                if (!FULL)
#pragma unroll
                    for (int r = 0; r < 4; r++) k[r] = has[i] ? k[r] : 0.0f;
                st[i] = mma16_f32(k, du, st[i] * x.keep);
            }
            part_q[j][wave][lane] = q;
            ring[j % kAhead] = load(chunk + kAhead);
            asm volatile("" ::: "memory");
        }
        __syncthreads();
        const f32x4 q = (part_q[wave][0][lane] + part_q[wave][1][lane]) + (part_q[wave][2][lane] + part_q[wave][3][lane]);
        float *dst = po + (chunk0 + wave) * step_v + off_o;
#pragma unroll
        for (uint32_t r = 0; r < 4; r++) dst[size_t(r) * s.v_pad] = left[r] + q[r];
        left = load_o(chunk0 + kScanGroup + wave);
        asm volatile("" ::: "memory");
    }
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        if (!has[i]) continue;
#pragma unroll
        for (int r = 0; r < 4; r++) a.state_out[at + size_t((wave + 4 * i) * 16 + g4 * 4 + r) * s.v_pad] = st[i][r];
    }
}

// a wave: one (token, head): o over its root mean square, times the weight and the gate; workgroup 0 of a head also
// carries the convolution's history on
template <typename T>
__global__ __launch_bounds__(256) void delta_norm_kernel(RmiDeltaShape s, RmiDeltaArgs a, uint32_t n_pad) {
    const uint32_t lane = threadIdx.x & 63, t = blockIdx.x * 4 + (threadIdx.x >> 6), h = blockIdx.y;
    if (blockIdx.x == 0) delta_carry(s, a, ConvCtx{a.u, a.hist_in, a.conv, delta_channels(s), s.taps}, h, 256);
    if (t >= a.n_tokens) return;
    DeltaScratch ws;
    delta_scratch_at(a.scratch, s, n_pad, &ws);
    const float *o = ws.o + (size_t(h) * n_pad * kChunk + t) * s.v_pad, *gate = a.gate + (size_t(t) * s.heads + h) * s.vdim;
    float v[kMaxHeadDim / 64], sq = 0.0f;
#pragma unroll
    for (uint32_t j = 0; j < kMaxHeadDim / 64; j++) {
        v[j] = lane + j * 64 < s.vdim ? o[lane + j * 64] : 0.0f;
        sq = __builtin_fmaf(v[j], v[j], sq);
    }
    const float r = 1.0f / sqrtf(wave_sum_f32(sq) / float(s.vdim) + s.eps);
#pragma unroll
    for (uint32_t j = 0; j < kMaxHeadDim / 64; j++) {
        const uint32_t d = lane + j * 64;
        if (d < s.vdim) static_cast<T *>(a.out)[size_t(t) * a.out_ld + size_t(h) * s.vdim + d] = from_f32<T>(v[j] * r * a.norm[d] * gate[d]);
    }
}

int check_delta(const RmiDeltaShape &s) {
    if (s.heads == 0 || s.kv_heads == 0 || s.heads % s.kv_heads || s.dim == 0 || s.vdim == 0 || s.d_pad % 16 || s.v_pad % 16 || s.d_pad < s.dim ||
        s.v_pad < s.vdim || s.d_pad > kMaxHeadDim || s.v_pad > kMaxHeadDim || s.taps == 0 || s.taps > kMaxTaps)
        return rmi_fail(RMI_HIP_E_INVALID, "bad delta rule shape");
    return RMI_HIP_OK;
}

template <typename T>
int delta_pass(const RmiDeltaShape &s, const RmiDeltaArgs &a, hipStream_t st) {
    const uint32_t n_pad = scan_chunks(a.n_tokens);
    const size_t lds = size_t(factors_lds_floats(s)) * 4;
    const int rc = rmi_allow_lds(delta_factors_kernel<T>, lds);
    if (rc != RMI_HIP_OK) return rc;
    hipLaunchKernelGGL(delta_factors_kernel<T>, dim3(n_pad, s.heads), dim3(kFactorThreads), lds, st, s, a, n_pad);
    auto scan = [&](auto kernel) { hipLaunchKernelGGL(kernel, dim3(s.v_pad / 16 * s.heads), dim3(256), 0, st, s, a, n_pad); };
    if (s.d_pad <= 64)
        s.d_pad == 64 ? scan(delta_scan_kernel<1, true>) : scan(delta_scan_kernel<1, false>);
    else if (s.d_pad <= 128)
        s.d_pad == 128 ? scan(delta_scan_kernel<2, true>) : scan(delta_scan_kernel<2, false>);
    else
        s.d_pad == 256 ? scan(delta_scan_kernel<4, true>) : scan(delta_scan_kernel<4, false>);
    hipLaunchKernelGGL(delta_norm_kernel<T>, dim3((a.n_tokens + 3) / 4, s.heads), dim3(256), 0, st, s, a, n_pad);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

template <typename T>
int delta_step(const RmiDeltaShape &s, const RmiDeltaArgs &a, hipStream_t st) {
    const uint32_t slices = kStepThreads / (s.v_pad / 4), rows = (s.d_pad + slices - 1) / slices;  // at most 32
    auto go = [&](auto kernel) { hipLaunchKernelGGL(kernel, dim3(s.heads), dim3(kStepThreads), 0, st, s, a); };
    if (rows <= 8)
        go(delta_step_kernel<T, 8>);
    else
        go(delta_step_kernel<T, 32>);
    RMI_HIP_CHECK(hipGetLastError());
    return RMI_HIP_OK;
}

}  // namespace

size_t rmi_delta_scratch_floats(const RmiDeltaShape &s, uint32_t max_tokens) {
    return delta_scratch_at(nullptr, s, scan_chunks(max_tokens), nullptr);
}

int rmi_delta_pass(uint32_t elem_bytes, const RmiDeltaShape &s, const RmiDeltaArgs &a, hipStream_t st) {
    if (a.n_tokens == 0) return RMI_HIP_OK;
    const int rc = check_delta(s);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? delta_pass<rmi_bf16>(s, a, st) : delta_pass<float>(s, a, st);
}

int rmi_delta_step(uint32_t elem_bytes, const RmiDeltaShape &s, const RmiDeltaArgs &a, hipStream_t st) {
    if (a.n_tokens != 1) return rmi_fail(RMI_HIP_E_INVALID, "a step takes one token");
    const int rc = check_delta(s);
    if (rc != RMI_HIP_OK) return rc;
    return elem_bytes == 2 ? delta_step<rmi_bf16>(s, a, st) : delta_step<float>(s, a, st);
}
