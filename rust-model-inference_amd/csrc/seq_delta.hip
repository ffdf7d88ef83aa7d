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
    __shared__ float ks[kMaxHeadDim], qs[kMaxHeadDim], vs[kMaxHeadDim], us[kMaxHeadDim], red[8];
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
// The first kernel makes what does not need the state, for all chunks at once: q, k, v, M = D (q k^T), the inverse
// T = (1 + A)^-1 diag(beta) by forward substitution, G and D_15.  The second walks the chunks with the state in the
// matrix cores' accumulators.
constexpr uint32_t kChunk = 16;
struct DeltaScratch {
    float *q, *k, *kt, *v, *o, *m, *t, *gd;
};
__host__ __device__ inline size_t delta_scratch_at(float *p, const RmiDeltaShape &s, uint32_t n_chunks, DeltaScratch *w) {
    const size_t kc = size_t(s.kv_heads) * n_chunks * kChunk * s.d_pad, hc = size_t(s.heads) * n_chunks;
    size_t at = 0;
    auto take = [&](size_t n) {
        const size_t was = at;
        at += n;
        return was;
    };
    const size_t q = take(kc), k = take(kc), kt = take(kc);
    const size_t v = take(hc * kChunk * s.v_pad), o = take(hc * kChunk * s.v_pad);
    const size_t m = take(hc * kChunk * kChunk), t = take(hc * kChunk * kChunk), gd = take(hc * 2 * kChunk);
    if (w) {
        w->q = p + q;    // [kv_head][chunk][16][d_pad], unit, over sqrt(dim)
        w->k = p + k;    // [kv_head][chunk][16][d_pad], unit
        w->kt = p + kt;  // [kv_head][chunk][d_pad][16]
        w->v = p + v;    // [head][chunk][16][v_pad]
        w->o = p + o;    // [head][chunk][16][v_pad]
        w->m = p + m;    // [head][chunk][16 t][16 s]
        w->t = p + t;    // [head][chunk][16 t][16 s]
        w->gd = p + gd;  // [head][chunk][G of 16, D_15 of 16]
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
            if (t0 >= back) row[i] = x.u[size_t(t0 - back) * x.channels + c];
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

// one chunk of one head; the first head of a group also stores the group's q and k
template <typename T>
__global__ __launch_bounds__(256) void delta_factors_kernel(RmiDeltaShape s, RmiDeltaArgs a, uint32_t n_chunks) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    const uint32_t ld = s.d_pad + 4;
    float *ql = reinterpret_cast<float *>(lds_raw), *kl = ql + kChunk * ld;  // [16][d_pad + 4]
    __shared__ float dm[kChunk][kChunk], am[kChunk][kChunk + 1], beta[kChunk], decay[kChunk];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, chunk = blockIdx.x, h = blockIdx.y, t0 = chunk * kChunk;
    const uint32_t group = s.heads / s.kv_heads, g = h / group;
    const bool first = h % group == 0;
    const ConvCtx x{a.u, a.hist_in, a.conv, delta_channels(s), s.taps};
    DeltaScratch ws;
    delta_scratch_at(a.scratch, s, n_chunks, &ws);
    const size_t hc = size_t(h) * n_chunks + chunk, kc = (size_t(g) * n_chunks + chunk) * kChunk * s.d_pad;
    float y[kChunk];
    for (uint32_t e = tid; e < 2 * s.d_pad + s.v_pad; e += 256) {
        const bool is_v = e >= 2 * s.d_pad, is_k = !is_v && e >= s.d_pad;
        const uint32_t d = is_v ? e - 2 * s.d_pad : is_k ? e - s.d_pad : e;
        const bool live = d < (is_v ? s.vdim : s.dim);
        if (live) {
            conv_chunk<T>(x, a, t0, (is_v ? v_channel(s, h) : is_k ? k_channel(s, g) : q_channel(s, g)) + d, y);
        } else {
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) y[t] = 0.0f;
        }
        if (is_v) {
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) ws.v[(hc * kChunk + t) * s.v_pad + d] = y[t];
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
        ws.gd[hc * 2 * kChunk + kChunk + tid] = w;
    } else if (tid == 64) {
        float w = 1.0f;
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) {
            w *= decay[t];
            ws.gd[hc * 2 * kChunk + t] = w;
        }
    }
    // unit length: four tokens a wave
    for (uint32_t t = wave; t < kChunk; t += 4) {
        float qq = 0.0f, kk = 0.0f;
        for (uint32_t d = lane; d < s.d_pad; d += 64) {
            qq = __builtin_fmaf(ql[t * ld + d], ql[t * ld + d], qq);
            kk = __builtin_fmaf(kl[t * ld + d], kl[t * ld + d], kk);
        }
        const float rq = 1.0f / sqrtf(wave_sum_f32(qq) + 1e-6f) / sqrtf(float(s.dim)), rk = 1.0f / sqrtf(wave_sum_f32(kk) + 1e-6f);
        for (uint32_t d = lane; d < s.d_pad; d += 64) {
            const float q = ql[t * ld + d] * rq, k = kl[t * ld + d] * rk;
            ql[t * ld + d] = q;
            kl[t * ld + d] = k;
            if (first) {
                ws.q[kc + t * s.d_pad + d] = q;
                ws.k[kc + t * s.d_pad + d] = k;
            }
        }
    }
    __syncthreads();
    if (first && wave >= 2) {
        for (uint32_t e = tid - 128; e < s.d_pad * (kChunk / 4); e += 128) {
            const uint32_t d = e >> 2, t = (e & 3) * 4;
            *reinterpret_cast<f32x4 *>(ws.kt + kc + d * kChunk + t) = f32x4{kl[t * ld + d], kl[(t + 1) * ld + d], kl[(t + 2) * ld + d], kl[(t + 3) * ld + d]};
        }
    }
    if (wave >= 2) return;
    // wave 0: k k^T and the triangular system; wave 1: q k^T
    const uint32_t fr = lane & 15, q4 = lane >> 4;
    const float *lhs = wave == 0 ? kl : ql;
    f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    for (uint32_t d = 0; d < s.d_pad; d += 32) {
        acc[0] = mma16_f32(*reinterpret_cast<const f32x4 *>(lhs + fr * ld + d + q4 * 4), *reinterpret_cast<const f32x4 *>(kl + fr * ld + d + q4 * 4), acc[0]);
        if (d + 16 < s.d_pad)
            acc[1] = mma16_f32(*reinterpret_cast<const f32x4 *>(lhs + fr * ld + d + 16 + q4 * 4), *reinterpret_cast<const f32x4 *>(kl + fr * ld + d + 16 + q4 * 4), acc[1]);
    }
    const f32x4 dot = acc[0] + acc[1];  // row t = 4 q4 + r, column s = fr
    if (wave == 1) {
#pragma unroll
        for (uint32_t r = 0; r < 4; r++) ws.m[hc * kChunk * kChunk + (q4 * 4 + r) * kChunk + fr] = dot[r] * dm[q4 * 4 + r][fr];
        return;
    }
#pragma unroll
    for (uint32_t r = 0; r < 4; r++) am[q4 * 4 + r][fr] = dot[r] * dm[q4 * 4 + r][fr] * beta[q4 * 4 + r];
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
        for (uint32_t t = 0; t < kChunk; t++) ws.t[hc * kChunk * kChunk + t * kChunk + fr] = c[t] * b;
    }
}

// One workgroup: sixteen value channels of one head, over all chunks of the pass; wave w holds the state's row tiles
// w, w + 4, ..  A tile in accumulator form (row 4g + r in register r) is the right operand of the next product as it
// lies, and so are v - G (k S) and u.
template <int TPW>
__global__ __launch_bounds__(256) void delta_scan_kernel(RmiDeltaShape s, RmiDeltaArgs a, uint32_t n_chunks) {
    __shared__ f32x4 part[2][2][4][64];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = uint32_t(__builtin_amdgcn_readfirstlane(int(tid >> 6))), fr = lane & 15, g4 = lane >> 4;
    const uint32_t h = blockIdx.y, v0 = blockIdx.x * 16, n_tiles = s.d_pad / 16, g = h / (s.heads / s.kv_heads);
    DeltaScratch ws;
    delta_scratch_at(a.scratch, s, n_chunks, &ws);
    f32x4 st[TPW];
    const size_t at = size_t(h) * s.d_pad * s.v_pad + v0 + fr;
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        const uint32_t tile = wave + 4 * i;
        st[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (a.pos0 == 0 || tile >= n_tiles) continue;
#pragma unroll
        for (int r = 0; r < 4; r++) st[i][r] = a.state_in[at + size_t(tile * 16 + g4 * 4 + r) * s.v_pad];
    }
    struct Operands {
        f32x4 q[TPW], k[TPW], kt[TPW];
        f32x4 v, m, t, gt, dt;
        float keep;
    };
    auto load = [&](uint32_t chunk) {
        Operands x;
        const size_t hc = size_t(h) * n_chunks + chunk, kc = (size_t(g) * n_chunks + chunk) * kChunk * s.d_pad;
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            const uint32_t tile = wave + 4 * i < n_tiles ? wave + 4 * i : n_tiles - 1;
            x.k[i] = *reinterpret_cast<const f32x4 *>(ws.k + kc + fr * s.d_pad + tile * 16 + g4 * 4);
            x.q[i] = *reinterpret_cast<const f32x4 *>(ws.q + kc + fr * s.d_pad + tile * 16 + g4 * 4);
            x.kt[i] = *reinterpret_cast<const f32x4 *>(ws.kt + kc + (tile * 16 + fr) * kChunk + g4 * 4);
        }
        x.m = *reinterpret_cast<const f32x4 *>(ws.m + hc * kChunk * kChunk + fr * kChunk + g4 * 4);
        x.t = *reinterpret_cast<const f32x4 *>(ws.t + hc * kChunk * kChunk + fr * kChunk + g4 * 4);
        x.gt = *reinterpret_cast<const f32x4 *>(ws.gd + hc * 2 * kChunk + g4 * 4);
        x.dt = *reinterpret_cast<const f32x4 *>(ws.gd + hc * 2 * kChunk + kChunk + g4 * 4);
        x.keep = ws.gd[hc * 2 * kChunk + kChunk - 1];
#pragma unroll
        for (int r = 0; r < 4; r++) x.v[r] = ws.v[(hc * kChunk + g4 * 4 + r) * s.v_pad + v0 + fr];
        return x;
    };
    constexpr uint32_t kAhead = TPW <= 2 ? 4 : 2;  // chunks whose operands are on their way
    Operands ring[kAhead];
#pragma unroll
    for (uint32_t j = 0; j < kAhead; j++) ring[j] = load(j < n_chunks ? j : n_chunks - 1);
    for (uint32_t chunk0 = 0; chunk0 < n_chunks; chunk0 += kAhead) {
#pragma unroll
        for (uint32_t j = 0; j < kAhead; j++) {
            const uint32_t chunk = chunk0 + j;
            if (chunk >= n_chunks) break;
            const Operands &x = ring[j];
            f32x4 ks = {0.f, 0.f, 0.f, 0.f}, qs = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < TPW; i++) {
                if (wave + 4 * i >= n_tiles) continue;
                ks = mma16_f32(x.k[i], st[i], ks);
                qs = mma16_f32(x.q[i], st[i], qs);
            }
            part[chunk & 1][0][wave][lane] = ks;
            part[chunk & 1][1][wave][lane] = qs;
            __syncthreads();  // (two buffers: the next chunk's writes cannot meet this one's reads)
            const f32x4 p = (part[chunk & 1][0][0][lane] + part[chunk & 1][0][1][lane]) + (part[chunk & 1][0][2][lane] + part[chunk & 1][0][3][lane]);
            const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
            const f32x4 u = mma16_f32(x.t, x.v - x.gt * p, zero);
            const f32x4 du = x.dt * u;
#pragma unroll
            for (int i = 0; i < TPW; i++) {
                if (wave + 4 * i >= n_tiles) continue;
                st[i] = mma16_f32(x.kt[i], du, st[i] * x.keep);
            }
            if (wave == (chunk & 3)) {
                const f32x4 q = (part[chunk & 1][1][0][lane] + part[chunk & 1][1][1][lane]) + (part[chunk & 1][1][2][lane] + part[chunk & 1][1][3][lane]);
                const f32x4 o = mma16_f32(x.m, u, x.gt * q);
                float *dst = ws.o + ((size_t(h) * n_chunks + chunk) * kChunk + g4 * 4) * s.v_pad + v0 + fr;
#pragma unroll
                for (int r = 0; r < 4; r++) dst[size_t(r) * s.v_pad] = o[r];
            }
            ring[j] = load(chunk + kAhead < n_chunks ? chunk + kAhead : n_chunks - 1);
        }
    }
#pragma unroll
    for (int i = 0; i < TPW; i++) {
        const uint32_t tile = wave + 4 * i;
        if (tile >= n_tiles) continue;
#pragma unroll
        for (int r = 0; r < 4; r++) a.state_out[at + size_t(tile * 16 + g4 * 4 + r) * s.v_pad] = st[i][r];
    }
}

// a wave: one (token, head): o over its root mean square, times the weight and the gate; workgroup 0 of a head also
// carries the convolution's history on
template <typename T>
__global__ __launch_bounds__(256) void delta_norm_kernel(RmiDeltaShape s, RmiDeltaArgs a, uint32_t n_chunks) {
    const uint32_t lane = threadIdx.x & 63, t = blockIdx.x * 4 + (threadIdx.x >> 6), h = blockIdx.y;
    if (blockIdx.x == 0) delta_carry(s, a, ConvCtx{a.u, a.hist_in, a.conv, delta_channels(s), s.taps}, h, 256);
    if (t >= a.n_tokens) return;
    DeltaScratch ws;
    delta_scratch_at(a.scratch, s, n_chunks, &ws);
    const float *o = ws.o + (size_t(h) * n_chunks * kChunk + t) * s.v_pad, *gate = a.gate + (size_t(t) * s.heads + h) * s.vdim;
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
    const uint32_t n_chunks = (a.n_tokens + kChunk - 1) / kChunk;
    const size_t lds = 2 * size_t(kChunk) * (s.d_pad + 4) * 4;
    hipLaunchKernelGGL(delta_factors_kernel<T>, dim3(n_chunks, s.heads), dim3(256), lds, st, s, a, n_chunks);
    auto scan = [&](auto kernel) { hipLaunchKernelGGL(kernel, dim3(s.v_pad / 16, s.heads), dim3(256), 0, st, s, a, n_chunks); };
    if (s.d_pad <= 64)
        scan(delta_scan_kernel<1>);
    else if (s.d_pad <= 128)
        scan(delta_scan_kernel<2>);
    else
        scan(delta_scan_kernel<4>);
    hipLaunchKernelGGL(delta_norm_kernel<T>, dim3((a.n_tokens + 3) / 4, s.heads), dim3(256), 0, st, s, a, n_chunks);
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
    return delta_scratch_at(nullptr, s, (max_tokens + kChunk - 1) / kChunk, nullptr);
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
