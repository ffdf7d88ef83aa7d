"""Writes model folders (config.json and model.safetensors): the synthetic models of the benchmark."""
import json
import os
import struct

import numpy as np


def bf16_bits(a):
    """f32 -> bf16 bits, to nearest even."""
    b = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((b + 0x7FFF + ((b >> 16) & 1)) >> 16).astype(np.uint16)


def write_safetensors(path, tensors):
    """tensors: (name, uint16 bf16 bits) pairs."""
    head, at = {}, 0
    for name, a in tensors:
        head[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + a.nbytes]}
        at += a.nbytes
    text = json.dumps(head).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for _, a in tensors:
            f.write(a.tobytes())


def _write(path, cfg, tensors):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(path, "model.safetensors"), tensors)
    return cfg


def synthetic_ruvenex_config(n_layer, width, ff, heads, kv_heads, dim, rheads, rdim, vocab):
    layer = {"type": "parallel", "mlp": {"kind": "dense", "ff": ff},
             "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "conv": 4,
                                "rot": {"dims": dim // 2, "base": 1e6}, "scale": dim**-0.5},
                       "right": {"heads": rheads, "dim": rdim, "vdim": rdim}, "left_scale": 1.0, "right_scale": 0.8}}
    return {"architecture": "Ruvenex", "embedding": {"scale": 1.0}, "layers": [layer] * n_layer, "norm": {"eps": 1e-6},
            "vocab": vocab, "width": width}


def write_synthetic_ruvenex(path, seed, **sizes):
    """A random model of those sizes.  One layer's weights are drawn and stored once for every layer (each layer's
    copy has its own place in the file and in HBM)."""
    cfg = synthetic_ruvenex_config(**sizes)
    rng = np.random.default_rng(seed)
    W, V, c = cfg["width"], cfg["vocab"], cfg["layers"][0]
    a, r, ff = c["mixer"]["left"], c["mixer"]["right"], c["mlp"]["ff"]

    def mat(out, inp):
        return bf16_bits(rng.standard_normal((out, inp), dtype=np.float32) / np.sqrt(inp))

    def vec(n, mean, spread):
        return bf16_bits(mean + spread * rng.standard_normal(n))

    nq, nk, nv, nr = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"], r["heads"] * r["dim"]
    nrv = r["heads"] * r["vdim"]
    layer = {"norm1": vec(W, 1, 0.1), "mix.left.g": mat(a["heads"], W), "mix.left.o": mat(W, a["heads"] * a["vdim"]),
             "mix.right.q": mat(nr, W), "mix.right.f": mat(nr, W), "mix.right.f.b": vec(nr, 2, 1),
             "mix.right.lower": bf16_bits(rng.uniform(0, 0.9, nr)), "mix.right.v": mat(nrv, W), "mix.right.norm": vec(r["vdim"], 1, 0.1),
             "mix.right.o": mat(W, nrv), "mlp.up": mat(ff, W), "mlp.down": mat(W, ff), "rg1": mat(W, W), "rg1.b": vec(W, 0, 0.5),
             "rg2": mat(W, W), "rg2.b": vec(W, 0, 0.5)}
    for n, size in (("q", nq), ("k", nk), ("v", nv)):
        layer[f"mix.left.{n}"] = mat(size, W)
        layer[f"mix.left.{n}.conv"] = bf16_bits(0.3 * rng.standard_normal((size, a["conv"])) + (np.arange(a["conv"]) == a["conv"] - 1))
    tensors = [("embed", mat(V, W)), ("final.norm", vec(W, 1, 0.1)), ("head", mat(V, W))]
    for i in range(len(cfg["layers"])):
        tensors += [(f"l{i}.{n}", t) for n, t in layer.items()]
    return _write(path, cfg, tensors)


def synthetic_vogizen_config(layers, width, ff, heads, dim, q_rank, kv_rank, window, rheads, rkv_heads, rdim, side, vocab, loop):
    """layers: "d" (delta rule) or "a" (latent attention) each; loop: (start, stop, times)."""
    kinds = {"d": ("delta", {"heads": rheads, "kv_heads": rkv_heads, "dim": rdim, "vdim": rdim, "conv": 4}),
             "a": ("latent_attention", {"heads": heads, "dim": dim, "vdim": dim, "q_rank": q_rank, "kv_rank": kv_rank,
                                        "scale": dim**-0.5, "mask": {"size": window}})}
    entries = [{"type": kinds[k][0], "mixer": kinds[k][1], "mlp": {"kind": "dense", "ff": ff}} for k in layers]
    return {"architecture": "Vogizen", "embedding": {"scale": 1.0}, "layers": entries, "loop": dict(zip(("start", "stop", "times"), loop)),
            "norm": {"eps": 1e-6}, "token_side": {"dim": side}, "vocab": vocab, "width": width}


def write_synthetic_vogizen(path, seed, **sizes):
    """A random model of those sizes.  One layer's weights of either kind are drawn and stored once for every such layer
    (each layer's copy has its own place in the file and in HBM)."""
    cfg = synthetic_vogizen_config(**sizes)
    rng = np.random.default_rng(seed)
    W, V, side = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"]

    def mat(out, inp):
        return bf16_bits(rng.standard_normal((out, inp), dtype=np.float32) / np.sqrt(inp))

    def vec(n, mean, spread):
        return bf16_bits(mean + spread * rng.standard_normal(n))

    def layer(entry):
        m, ff = entry["mixer"], entry["mlp"]["ff"]
        t = {"norm1": vec(W, 1, 0.1), "norm2": vec(W, 1, 0.1), "ls1": vec(W, 0.5, 0.1), "ls2": vec(W, 0.5, 0.1), "mlp.gate": mat(ff, W),
             "mlp.up": mat(ff, W), "mlp.down": mat(W, ff), "side.gate": mat(side, W), "side.proj": mat(W, side), "side.norm": vec(W, 0.3, 0.1),
             "mix.o": mat(W, m["heads"] * m["vdim"])}
        if entry["type"] == "delta":
            nk, nv = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, size in (("q", nk), ("k", nk), ("v", nv)):
                t[f"mix.{n}"] = mat(size, W)
                t[f"mix.{n}.conv"] = bf16_bits(0.3 * rng.standard_normal((size, m["conv"])) + (np.arange(m["conv"]) == m["conv"] - 1))
            t.update({"mix.b": mat(m["heads"], W), "mix.a": mat(m["heads"], W), "mix.A_log": vec(m["heads"], 0, 0.5),
                      "mix.dt_bias": vec(m["heads"], -2, 1), "mix.g": mat(nv, W), "mix.norm": vec(m["vdim"], 1, 0.1)})
        else:
            nk, nv, rq, rk = m["heads"] * m["dim"], m["heads"] * m["vdim"], m["q_rank"], m["kv_rank"]
            t.update({"mix.dq": mat(rq, W), "mix.dq.norm": vec(rq, 1, 0.1), "mix.uq": mat(nk, rq), "mix.dkv": mat(rk, W),
                      "mix.dkv.norm": vec(rk, 1, 0.1), "mix.uk": mat(nk, rk), "mix.uv": mat(nv, rk)})
        return t

    kinds = {}
    for entry in cfg["layers"]:
        if entry["type"] not in kinds:
            kinds[entry["type"]] = layer(entry)
    tensors = [("embed", mat(V, W)), ("final.norm", vec(W, 1, 0.1)), ("loop.in", mat(W, 2 * W)),
               ("side.embed", np.tile(mat(V, side), (1, len(cfg["layers"]))))]
    for i, entry in enumerate(cfg["layers"]):
        tensors += [(f"l{i}.{n}", t) for n, t in kinds[entry["type"]].items()]
    return _write(path, cfg, tensors)
