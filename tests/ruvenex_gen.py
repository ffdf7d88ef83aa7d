"""Small random Ruvenex models for the tests: a configuration, weights rounded to bf16, and the model folder."""
import json
import os
import struct

import numpy as np


def bf16_round(a):
    b = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((b + 0x7FFF + ((b >> 16) & 1)) & np.uint32(0xFFFF0000)).view(np.float32)


def layer_config(heads=4, kv_heads=2, dim=16, vdim=16, taps=3, rot_dims=8, base=10000.0, scale=None, rheads=2, rdim=16, rvdim=16,
                 left_scale=0.9, right_scale=0.7, ff=48):
    return {"type": "parallel",
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps,
                               "rot": {"dims": rot_dims, "base": base}, "scale": dim**-0.5 if scale is None else scale},
                      "right": {"heads": rheads, "dim": rdim, "vdim": rvdim}, "left_scale": left_scale, "right_scale": right_scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, width=40, vocab=60, eps=1e-5, embed_scale=3.0):
    return {"architecture": "Ruvenex", "embedding": {"scale": embed_scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


def weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = bf16_round(rng.standard_normal((out, inp)) * gain / np.sqrt(inp))

    def vec(name, n, mean, spread):
        w[name] = bf16_round(mean + spread * rng.standard_normal(n))

    mat("embed", V, W, np.sqrt(W) / cfg["embedding"]["scale"])
    for i, c in enumerate(cfg["layers"]):
        p, a, r = f"l{i}.", c["mixer"]["left"], c["mixer"]["right"]
        L, R = p + "mix.left.", p + "mix.right."
        vec(p + "norm1", W, 1.0, 0.2)
        for n, size in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
            mat(L + n, size, W, 1.5)
            w[L + n + ".conv"] = bf16_round(rng.standard_normal((size, a["conv"])) * 0.4 + (np.arange(a["conv"]) == a["conv"] - 1))
        mat(L + "g", a["heads"], W)
        mat(L + "o", W, a["heads"] * a["vdim"])
        mat(R + "q", r["heads"] * r["dim"], W)
        mat(R + "f", r["heads"] * r["dim"], W)
        vec(R + "f.b", r["heads"] * r["dim"], 1.0, 2.0)
        w[R + "lower"] = bf16_round(rng.uniform(0.0, 0.9, r["heads"] * r["dim"]))
        mat(R + "v", r["heads"] * r["vdim"], W)
        vec(R + "norm", r["vdim"], 1.0, 0.2)
        mat(R + "o", W, r["heads"] * r["vdim"])
        mat(p + "rg1", W, W)
        vec(p + "rg1.b", W, 0.5, 0.5)
        if c["mlp"] is not None:
            mat(p + "mlp.up", c["mlp"]["ff"], W, 1.5)
            mat(p + "mlp.down", W, c["mlp"]["ff"])
            mat(p + "rg2", W, W)
            vec(p + "rg2.b", W, 0.5, 0.5)
    vec("final.norm", W, 1.0, 0.2)
    mat("head", V, W)
    return w


def write_folder(path, cfg, w):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, data, at = {}, [], 0
    for name, a in w.items():
        b = (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype(np.uint16).tobytes()
        head[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(b)]}
        data.append(b)
        at += len(b)
    text = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text + b"".join(data))
    return str(path)


def tokens(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()
