"""The plain statement of the Ruvenex decoder against hand-worked values and properties of each mechanism, and the
parts of the product that need no GPU: model folders, the registry, the trace replay."""
import json

import numpy as np
import pytest
import ruvenex_gen as G
import ruvenex_plain as P


def test_conv_is_causal_and_ordered():
    u = np.array([[1.0], [10.0], [100.0]])
    y = P.causal_conv(u, np.array([[3.0, 2.0, 1.0]]))
    assert y[:, 0].tolist() == [1.0, 12.0, 123.0]


def test_rotation_is_interleaved_partial_and_relative():
    x = np.zeros((4, 1, 6))
    x[:, 0, 0] = 1.0
    x[:, 0, 5] = 7.0
    y = P.rotate_interleaved(x, 4, 100.0)
    assert np.allclose(y[:, 0, 0], np.cos(np.arange(4))) and np.allclose(y[:, 0, 1], np.sin(np.arange(4)))
    assert (y[:, 0, 5] == 7.0).all()
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((2, 1, 1, 8))
    dots = [(P.rotate_interleaved(q, 8, 50.0, p + 3) * P.rotate_interleaved(k, 8, 50.0, p)).sum() for p in (0, 5, 90)]
    assert np.allclose(dots, dots[0])


def test_attention_sees_its_past_and_its_group():
    v = np.arange(8.0).reshape(4, 2, 1)
    q = np.zeros((4, 4, 2))
    out = P.causal_attention(q, np.ones((4, 2, 2)), v, 1.0)  # equal weights: running means
    assert np.allclose(out[:, 0, 0], [0, 1, 2, 3]) and np.allclose(out[:, 1], out[:, 0]) and np.allclose(out[:, 2], out[:, 0] + 1)


def test_recurrence_extremes_and_split():
    rng = np.random.default_rng(1)
    q, f, v = rng.standard_normal((5, 1, 3)), rng.uniform(0, 1, (5, 1, 3)), rng.standard_normal((5, 1, 2))
    o, _ = P.gated_linear_recurrence(q, np.zeros_like(f), v)  # forgets at once: only the token itself
    assert np.allclose(o[:, 0], q[:, 0].sum(-1, keepdims=True) * v[:, 0])
    o, _ = P.gated_linear_recurrence(q, np.ones_like(f), v)  # never forgets and never writes
    assert (o == 0).all()
    whole, s = P.gated_linear_recurrence(q, f, v)
    a, sa = P.gated_linear_recurrence(q[:2], f[:2], v[:2])
    b, sb = P.gated_linear_recurrence(q[2:], f[2:], v[2:], sa)
    assert np.allclose(np.concatenate([a, b]), whole) and np.allclose(s, sb)


def test_scalar_functions():
    z = np.array([-30.0, -1.0, 0.0, 2.0, 30.0])
    assert np.allclose(P.sigmoid(z), 1 / (1 + np.exp(-z)))
    assert np.allclose(P.gelu_tanh(z), [0, -0.15880801, 0, 1.95459769, 30], atol=1e-7)
    assert np.allclose(P.forget_gate(z, -z, 0.25), 0.625)
    x = np.array([[3.0, 4.0]])
    assert np.allclose(P.rms_norm(x, np.array([1.0, 2.0]), 12.5), x / 5.0 * [1, 2])


def test_later_tokens_change_nothing():
    cfg = G.config([G.layer_config(), G.layer_config(ff=None)])
    w, t = G.weights(cfg), G.tokens(cfg, 9)
    assert np.allclose(P.forward(cfg, w, t)[:6], P.forward(cfg, w, t[:6]), rtol=1e-12, atol=1e-12)


def test_folder_architecture_and_registry(rmi, tmp_path):
    cfg = G.config([G.layer_config()])
    G.write_folder(tmp_path, cfg, G.weights(cfg))
    H = rmi.hip
    buf = H.C.create_string_buffer(32)
    assert H.lib.rmi_hip_model_folder_architecture(str(tmp_path).encode(), buf, 32) == 7 and buf.value == b"Ruvenex"
    assert rmi.models.folder_architecture(str(tmp_path)) == "Ruvenex"
    assert rmi.models.session_class("Ruvenex") is rmi.decode.RuvenexSession
    with pytest.raises(ValueError, match="no session for architecture 'Other'"):
        rmi.models.session_class("Other")


@pytest.mark.parametrize("text", ["", "{", '{"architecture": 3}', '{"a": [1,]}', '{"architecture": "X"} x', "[1]", '{"architecture": "\\u12"}'])
def test_bad_config_is_an_error(rmi, tmp_path, text):
    (tmp_path / "config.json").write_text(text)
    assert rmi.hip.lib.rmi_hip_model_folder_architecture(str(tmp_path).encode(), None, 0) == -1
    assert rmi.hip.last_error()


def test_config_reader_takes_any_json(rmi, tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"x": [True, None, -1.5e3, {"y": "é\n\"\\"}], "architecture": "Über"}))
    buf = rmi.hip.C.create_string_buffer(32)
    assert rmi.hip.lib.rmi_hip_model_folder_architecture(str(tmp_path).encode(), buf, 32) == 5
    assert buf.value.decode() == "Über"


class FakeSession:
    def __init__(self):
        self.log = []

    def reset(self):
        self.log.append("reset")

    def step(self, tokens, want):
        self.log.append((list(tokens), list(want)))
        return np.array([[tokens[i], 0.5] for i in want], np.float32).reshape(len(want), 2)


def test_replay_writes_what_is_wanted(rmi, tmp_path):
    s = FakeSession()
    r = rmi.replay.Replay(s, str(tmp_path))
    r.run({"step": 0, "entries": [{"id": "a", "tokens": [5, 6], "want": []}], "end": []})
    r.run({"step": 1, "entries": [{"id": "a", "tokens": [7, 8, 9], "want": [2, 0]}], "end": ["a"]})
    with pytest.raises(ValueError):
        r.run({"step": 2, "entries": [{"id": "b", "tokens": [1], "want": []}, {"id": "c", "tokens": [1], "want": []}], "end": []})
    assert s.log[:4] == ["reset", ([5, 6], []), ([7, 8, 9], [2, 0]), "reset"]
    assert not (tmp_path / "0.f32").exists()
    assert np.fromfile(tmp_path / "1.f32", "<f4").tolist() == [9, 0.5, 7, 0.5]
