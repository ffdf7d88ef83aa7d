"""What the GPU tests of the model-folder sessions share."""
import numpy as np

F32, BF16 = "float32", "bfloat16"
TOL = {F32: 3e-5, BF16: 4e-2}


def rel(got, want):
    """Largest row error: root mean square over the row's, against the typical row's size."""
    d = np.asarray(got, np.float64) - want
    return float(np.sqrt((d * d).mean(-1)).max() / np.sqrt((want * want).mean()))


def portions(n, sizes):
    """Slices that cut n tokens into portions of the given sizes (the last one repeats)."""
    out, at = [], 0
    while at < n:
        k = min(sizes[min(len(out), len(sizes) - 1)], n - at)
        out.append(slice(at, at + k))
        at += k
    return out


def feed(s, tokens, sizes):
    """Logits of every position, the tokens cut into portions."""
    return np.concatenate([s.step(tokens[p], range(p.stop - p.start)) for p in portions(len(tokens), sizes)])


def feed_layers(s, tokens, sizes):
    """The residual stream behind every layer run, the tokens cut into portions."""
    return np.concatenate([s.step(tokens[p], (), layers=True)[1] for p in portions(len(tokens), sizes)], 1)


class Opener:
    """Writes a model's folder and opens its session; close() ends them all."""

    def __init__(self, hip, tmp_path, gen):
        self.hip, self.tmp_path, self.gen, self.opened = hip, tmp_path, gen, []

    def __call__(self, cfg, w=None, dtype=F32, capacity=256):
        w = self.gen.weights(cfg) if w is None else w
        s = self.hip.models.open_session(self.gen.write_folder(self.tmp_path / f"m{len(self.opened)}", cfg, w), capacity, dtype)
        self.opened.append(s)
        return s, w

    def close(self):
        for s in self.opened:
            s.close()
