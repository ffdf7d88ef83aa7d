"""Small random Vogizen models for the tests: a configuration and weights rounded to bf16 (folders as ruvenex_gen
writes them)."""
import numpy as np
from ruvenex_gen import bf16_round, tokens, write_folder  # noqa: F401


def delta(heads=4, kv_heads=2, dim=16, vdim=24, taps=3, ff=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def latent(heads=3, dim=16, vdim=20, q_rank=24, kv_rank=18, window=11, scale=None, ff=40):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": dim**-0.5 if scale is None else scale, "mask": {"size": window}},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, width=40, vocab=60, eps=1e-5, embed_scale=3.0, side=8, loop=(0, 1, 1)):
    c = {"architecture": "Vogizen", "embedding": {"scale": embed_scale}, "layers": layers, "norm": {"eps": eps}, "token_side": {"dim": side},
         "vocab": vocab, "width": width}
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    W, V, side = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"]
    w = {}

    def mat(name, out, inp, gain=1.0):
        w[name] = bf16_round(rng.standard_normal((out, inp)) * gain / np.sqrt(inp))

    def vec(name, n, mean, spread):
        w[name] = bf16_round(mean + spread * rng.standard_normal(n))

    mat("embed", V, W, np.sqrt(W) / cfg["embedding"]["scale"])
    mat("side.embed", V, side * len(cfg["layers"]), np.sqrt(side * len(cfg["layers"])))
    if "loop" in cfg:
        mat("loop.in", W, 2 * W)
    for i, c in enumerate(cfg["layers"]):
        p, m = f"l{i}.", c["mixer"]
        M = p + "mix."
        vec(p + "norm1", W, 1.0, 0.2)
        vec(p + "ls1", W, 0.6, 0.2)
        nv = m["heads"] * m["vdim"]
        if c["type"] == "delta":
            nk = m["kv_heads"] * m["dim"]
            for n, size in (("q", nk), ("k", nk), ("v", nv)):
                mat(M + n, size, W, 1.5)
                w[M + n + ".conv"] = bf16_round(rng.standard_normal((size, m["conv"])) * 0.4 + (np.arange(m["conv"]) == m["conv"] - 1))
            mat(M + "b", m["heads"], W)
            mat(M + "a", m["heads"], W)
            vec(M + "A_log", m["heads"], -0.5, 1.0)
            vec(M + "dt_bias", m["heads"], -2.0, 1.0)
            vec(M + "norm", m["vdim"], 1.0, 0.2)
            mat(M + "g", nv, W)
        else:
            nk = m["heads"] * m["dim"]
            mat(M + "dq", m["q_rank"], W)
            vec(M + "dq.norm", m["q_rank"], 1.0, 0.2)
            mat(M + "uq", nk, m["q_rank"], 1.5)
            mat(M + "dkv", m["kv_rank"], W)
            vec(M + "dkv.norm", m["kv_rank"], 1.0, 0.2)
            mat(M + "uk", nk, m["kv_rank"], 1.5)
            mat(M + "uv", nv, m["kv_rank"])
        mat(M + "o", W, nv)
        if c["mlp"] is not None:
            ff = c["mlp"]["ff"]
            vec(p + "norm2", W, 1.0, 0.2)
            vec(p + "ls2", W, 0.6, 0.2)
            mat(p + "mlp.gate", ff, W)
            mat(p + "mlp.up", ff, W)
            mat(p + "mlp.down", W, ff)
        mat(p + "side.gate", side, W, 0.7)
        mat(p + "side.proj", W, side)
        vec(p + "side.norm", W, 0.4, 0.1)
    vec("final.norm", W, 1.0, 0.2)
    return w
