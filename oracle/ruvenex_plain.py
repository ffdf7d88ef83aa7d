"""Plain, slow numpy statement of the Ruvenex decoder, one function per mechanism, written from the equations.

Test infrastructure only: it shares no code with the product path, and nothing in the product imports it.  Every
function takes whole sequences ([tokens, channels], position 0 first) and computes in the dtype of its inputs
(float64 in the tests).  Notation: h is what a sublayer reads, t a position, p the same as a number.
"""
import json
import struct

import numpy as np


def rms_unit(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + x.dtype.type(eps))


def rms_norm(x, weight, eps):
    return rms_unit(x, eps) * weight


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z**3)))


def causal_conv(u, taps):
    """y[t, c] = sum_j taps[c, j] u[t - (n - 1) + j, c], rows before the first being zero."""
    n = taps.shape[1]
    y = np.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                y[t] += taps[:, j] * u[s]
    return y


def rotate_interleaved(x, dims, base, first_pos=0):
    """x [tokens, heads, dim]: the pairs (2i, 2i+1), i < dims/2, turned by p * base^(-2i/dims)."""
    y = x.copy()
    p = np.arange(first_pos, first_pos + x.shape[0], dtype=np.float64)
    for i in range(dims // 2):
        a = p * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(a).astype(x.dtype)[:, None], np.sin(a).astype(x.dtype)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        y[:, :, 2 * i] = u * c - v * s
        y[:, :, 2 * i + 1] = v * c + u * s
    return y


def causal_attention(q, k, v, scale):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; query head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]), q.dtype)
    for h in range(H):
        g = h // group
        for t in range(T):
            s = (k[: t + 1, g] @ q[t, h]) * scale
            w = np.exp(s - s.max())
            out[t, h] = (w / w.sum()) @ v[: t + 1, g]
    return out


def gated_linear_recurrence(q, f, v, state=None):
    """Per head S <- diag(f) S + (1 - f) v^T, then o = S^T q.  q, f [T, H, d], v [T, H, e] -> [T, H, e], S."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), q.dtype) if state is None else state.copy()
    out = np.zeros((T, H, v.shape[2]), q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = f[t, h][:, None] * S[h] + np.outer(1.0 - f[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def forget_gate(z, bias, lower):
    return lower + (1.0 - lower) * sigmoid(z + bias)


def attention_mixer(h, w, p, c, eps):
    """The attention half of a parallel mixer; p = the tensors' prefix, c = its sizes."""
    T, H, G = h.shape[0], c["heads"], c["kv_heads"]
    q, k, v = (causal_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    q = rotate_interleaved(q.reshape(T, H, c["dim"]), c["rot"]["dims"], c["rot"]["base"])
    k = rotate_interleaved(k.reshape(T, G, c["dim"]), c["rot"]["dims"], c["rot"]["base"])
    v = rms_unit(v.reshape(T, G, c["vdim"]), eps)
    o = causal_attention(q, k, v, h.dtype.type(c["scale"]))
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[p + "o"].T


def hgrn2_mixer(h, w, p, c, eps):
    """The recurrent half of a parallel mixer."""
    T, H, d, e = h.shape[0], c["heads"], c["dim"], c["vdim"]
    q = silu(h @ w[p + "q"].T).reshape(T, H, d)
    f = forget_gate(h @ w[p + "f"].T, w[p + "f.b"], w[p + "lower"]).reshape(T, H, d)
    v = (h @ w[p + "v"].T).reshape(T, H, e)
    o, _ = gated_linear_recurrence(q, f, v)
    return rms_norm(o, w[p + "norm"], eps).reshape(T, -1) @ w[p + "o"].T


def parallel_mixer(h, w, p, c, eps):
    d = h.dtype.type
    return d(c["left_scale"]) * attention_mixer(h, w, p + "left.", c["left"], eps) + \
        d(c["right_scale"]) * hgrn2_mixer(h, w, p + "right.", c["right"], eps)


def feed_forward(h, w, p):
    return gelu_tanh(h @ w[p + "up"].T) @ w[p + "down"].T


def residual_gate(h, w, name):
    return sigmoid(h @ w[name].T + w[name + ".b"])


def layer(x, w, i, c, eps):
    p = f"l{i}."
    h = rms_norm(x, w[p + "norm1"], eps)
    y = residual_gate(h, w, p + "rg1") * parallel_mixer(h, w, p + "mix.", c["mixer"], eps)
    if c.get("mlp") is not None:
        y = y + residual_gate(h, w, p + "rg2") * feed_forward(h, w, p + "mlp.")
    return x + y


def forward(config, w, tokens, dtype=np.float64, layers_out=None):
    """Logits [tokens, vocab] of one whole sequence; w maps tensor names to arrays of any float type."""
    w = {n: (a.astype(dtype) if a.dtype.kind == "f" else a) for n, a in w.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)] * dtype(config["embedding"]["scale"])
    for i, c in enumerate(config["layers"]):
        x = layer(x, w, i, c, eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def read_safetensors(path):
    """name -> array (bfloat16 widened to float32)."""
    with open(path, "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        head = json.loads(f.read(n))
        data = f.read()
    out = {}
    for name, t in head.items():
        if name == "__metadata__":
            continue
        raw = data[t["data_offsets"][0]: t["data_offsets"][1]]
        if t["dtype"] == "BF16":
            a = (np.frombuffer(raw, np.uint16).astype(np.uint32) << 16).view(np.float32)
        else:
            a = np.frombuffer(raw, {"F32": np.float32, "I32": np.int32, "F16": np.float16}[t["dtype"]])
        out[name] = a.reshape(t["shape"])
    return out
