"""Plain, slow numpy statement of the Vogizen decoder, one function per mechanism, written from the equations.

Test infrastructure only: it shares no code with the product path, and nothing in the product imports it.  Every
function takes whole sequences ([tokens, channels], position 0 first) and computes in the dtype of its inputs
(float64 in the tests).  Notation: h is what a sublayer reads, t a position, p the same as a number.
"""
import numpy as np
from ruvenex_plain import causal_conv, gelu_tanh, read_safetensors, rms_norm, rms_unit, sigmoid, silu  # noqa: F401


def layer_norm(x, weight, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + x.dtype.type(eps)) * weight


def position_vector(p, width):
    """sin and cos of p * 10000^(-2i / width) in turn."""
    a = np.asarray(p, np.float64)[:, None] * 10000.0 ** (-2.0 * (np.arange(width) // 2) / width)
    return np.where(np.arange(width) % 2 == 0, np.sin(a), np.cos(a))


def window_attention(q, k, v, scale, window):
    """q, k [T, H, d], v [T, H, e] -> [T, H, e]; position t sees t - window + 1 .. t."""
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[2]), q.dtype)
    for t in range(T):
        lo = max(0, t - window + 1)
        for h in range(H):
            s = (k[lo: t + 1, h] @ q[t, h]) * scale
            w = np.exp(s - s.max())
            out[t, h] = (w / w.sum()) @ v[lo: t + 1, h]
    return out


def latent_attention_mixer(h, w, p, c, eps):
    T, H = h.shape[0], c["heads"]
    q = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T
    latent = rms_norm(h @ w[p + "dkv"].T, w[p + "dkv.norm"], eps)
    k, v = latent @ w[p + "uk"].T, latent @ w[p + "uv"].T
    o = window_attention(q.reshape(T, H, c["dim"]), k.reshape(T, H, c["dim"]), v.reshape(T, H, c["vdim"]), h.dtype.type(c["scale"]),
                         c["mask"]["size"])
    return o.reshape(T, -1) @ w[p + "o"].T


def unit(x):
    """x over its length along the last axis."""
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + x.dtype.type(1e-6))


def softplus(z):
    return np.maximum(z, 0) + np.log1p(np.exp(-np.abs(z)))


def decay(z, bias, a_log):
    return np.exp(-np.exp(a_log) * softplus(z + bias))


def gated_delta_rule(q, k, v, g, beta, state=None):
    """q, k [T, H, d], v [T, H, e], g, beta [T, H] -> o [T, H, e] and the state [H, d, e] behind the last token."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), q.dtype) if state is None else state.copy()
    out = np.zeros_like(v)
    for t in range(T):
        for h in range(H):
            S[h] = g[t, h] * S[h]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] = S[h] + np.outer(k[t, h], u)
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def delta_mixer(h, w, p, c, eps):
    T, H, G, d, e = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = unit(q.reshape(T, G, d)) * h.dtype.type(d**-0.5)
    k = unit(k.reshape(T, G, d))
    share = np.arange(H) // (H // G)
    beta = sigmoid(h @ w[p + "b"].T)
    g = decay(h @ w[p + "a"].T, w[p + "dt_bias"], w[p + "A_log"])
    o, _ = gated_delta_rule(q[:, share], k[:, share], v.reshape(T, H, e), g, beta)
    o = rms_norm(o, w[p + "norm"], eps) * silu(h @ w[p + "g"].T).reshape(T, H, e)
    return o.reshape(T, -1) @ w[p + "o"].T


MIXERS = {"latent_attention": latent_attention_mixer, "delta": delta_mixer}


def feed_forward(h, w, p):
    return (np.maximum(h @ w[p + "gate"].T, 0) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def token_side(x, e, w, p, eps):
    y = (gelu_tanh(x @ w[p + "gate"].T) * e) @ w[p + "proj"].T
    return rms_norm(y, w[p + "norm"], eps)


def layer(x, w, i, config, tokens):
    c, p, eps = config["layers"][i], f"l{i}.", config["norm"]["eps"]
    x = x + w[p + "ls1"] * MIXERS[c["type"]](layer_norm(x, w[p + "norm1"], eps), w, p + "mix.", c["mixer"], eps)
    if c.get("mlp") is not None:
        x = x + w[p + "ls2"] * feed_forward(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
    n = config["token_side"]["dim"]
    return x + token_side(x, w["side.embed"][tokens][:, i * n: (i + 1) * n], w, p + "side.", eps)


def layer_runs(config):
    """(layer, whether a pass of the loop begins with it), in the order of execution."""
    n, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, False) for i in range(a)] + [(i, i == a) for _ in range(loop["times"]) for i in range(a, b)] + [(i, False) for i in range(b, n)]


def embedding(config, w, tokens, dtype=np.float64):
    x = w["embed"][tokens] * dtype(config["embedding"]["scale"])
    return x + position_vector(np.arange(len(tokens)), config["width"]).astype(dtype)


def forward(config, w, tokens, dtype=np.float64, layers_out=None):
    """Logits [tokens, vocab] of one whole sequence; w maps tensor names to arrays of any float type."""
    w = {n: a.astype(dtype) for n, a in w.items()}
    tokens = np.asarray(tokens)
    x = x0 = embedding(config, w, tokens, dtype)
    for i, begins in layer_runs(config):
        if begins:
            x = np.concatenate([x, x0], 1) @ w["loop.in"].T
        x = layer(x, w, i, config, tokens)
        if layers_out is not None:
            layers_out.append(x.copy())
    return layer_norm(x, w["final.norm"], config["norm"]["eps"]) @ w["embed"].T
