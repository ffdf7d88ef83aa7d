"""The plain statement of the Vogizen decoder against hand-worked values and properties of each mechanism, and the parts
of the product that need no GPU."""
import numpy as np
import pytest
import vogizen_gen as G
import vogizen_plain as P


def test_layer_norm():
    x = np.array([[1.0, 3.0, 5.0, 7.0]])
    assert np.allclose(P.layer_norm(x, np.array([1.0, 1.0, 2.0, 1.0]), 4.0), [[-1.0, -1.0 / 3, 2.0 / 3, 1.0]])


def test_position_vector_is_interleaved():
    v = P.position_vector([0, 1, 7], 6)
    assert np.allclose(v[0], [0, 1, 0, 1, 0, 1])
    f = 10000.0 ** (-2 / 6)
    assert np.allclose(v[2, :4], [np.sin(7), np.cos(7), np.sin(7 * f), np.cos(7 * f)])
    assert P.position_vector([3], 5).shape == (1, 5)


def test_window_holds_itself_and_the_ones_before():
    v = np.arange(6.0).reshape(6, 1, 1)
    out = P.window_attention(np.zeros((6, 1, 2)), np.ones((6, 1, 2)), v, 1.0, 3)  # equal weights: means over the window
    assert np.allclose(out[:, 0, 0], [0, 0.5, 1, 2, 3, 4])
    assert np.allclose(P.window_attention(np.zeros((6, 1, 2)), np.ones((6, 1, 2)), v, 1.0, 1), v)


def test_delta_rule_replaces_what_a_key_holds():
    k = np.zeros((3, 1, 2))
    k[:, 0, 0] = 1.0  # the same unit key three times
    v = np.array([[[5.0]], [[7.0]], [[-2.0]]])
    o, s = P.gated_delta_rule(k, k, v, np.ones((3, 1)), np.ones((3, 1)))
    assert np.allclose(o, v) and np.allclose(s[0], [[-2.0], [0.0]])  # full step, no decay: the last value, not a sum
    o, _ = P.gated_delta_rule(k, k, v, np.ones((3, 1)), np.full((3, 1), 0.5))
    assert np.allclose(o[:, 0, 0], [2.5, 4.75, 1.375])
    o, _ = P.gated_delta_rule(k, np.zeros_like(k), v, np.full((3, 1), 0.5), np.ones((3, 1)))
    assert (o == 0).all()
    other = np.zeros((1, 1, 2))
    other[0, 0, 1] = 1.0
    o, s = P.gated_delta_rule(other, other, np.array([[[3.0]]]), np.full((1, 1), 0.25), np.ones((1, 1)), s)
    assert np.allclose(s[0], [[-0.5], [3.0]])  # the decay comes before the write


def test_delta_rule_in_two_parts():
    rng = np.random.default_rng(1)
    q, k, v = rng.standard_normal((5, 2, 3)), rng.standard_normal((5, 2, 3)), rng.standard_normal((5, 2, 4))
    g, b = rng.uniform(0, 1, (5, 2)), rng.uniform(0, 1, (5, 2))
    whole, s = P.gated_delta_rule(q, k, v, g, b)
    x, sx = P.gated_delta_rule(q[:2], k[:2], v[:2], g[:2], b[:2])
    y, sy = P.gated_delta_rule(q[2:], k[2:], v[2:], g[2:], b[2:], sx)
    assert np.allclose(np.concatenate([x, y]), whole) and np.allclose(s, sy)


def test_scalar_functions():
    z = np.array([-50.0, -1.0, 0.0, 2.0, 50.0])
    assert np.allclose(P.softplus(z), [0, 0.31326169, 0.69314718, 2.12692801, 50.0])
    assert np.allclose(P.decay(np.zeros(1), 0.0, 0.0), 0.5)
    assert np.allclose(P.unit(np.array([[3.0, 4.0]])), [[0.6, 0.8]])


def test_layers_of_a_loop_run_again():
    cfg = G.config([G.delta() for _ in range(4)], loop=(1, 3, 2))
    assert P.layer_runs(cfg) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert P.layer_runs(G.config([G.delta()] * 2, loop=None)) == [(0, False), (1, False)]


def test_later_tokens_change_nothing():
    cfg = G.config([G.delta(), G.latent(), G.delta(ff=20)], loop=(1, 3, 2))
    w, t = G.weights(cfg), G.tokens(cfg, 14)
    assert np.allclose(P.forward(cfg, w, t)[:9], P.forward(cfg, w, t[:9]), rtol=1e-11, atol=1e-11)


def test_folder_architecture_and_registry(rmi, tmp_path):
    cfg = G.config([G.delta()])
    G.write_folder(tmp_path, cfg, G.weights(cfg))
    H = rmi.hip
    buf = H.C.create_string_buffer(32)
    assert H.lib.rmi_hip_model_folder_architecture(str(tmp_path).encode(), buf, 32) == 7 and buf.value == b"Vogizen"
    assert rmi.models.session_class(rmi.models.folder_architecture(str(tmp_path))) is rmi.decode.VogizenSession


@pytest.mark.parametrize("layers", ["d", "da", "dad"])
def test_synthetic_models_have_every_tensor(rmi, tmp_path, layers):
    cfg = rmi.folder.write_synthetic_vogizen(tmp_path, 3, layers=layers, loop=(0, 1, 2), width=24, ff=20, heads=2, dim=6, q_rank=10, kv_rank=8,
                                             window=5, rheads=4, rkv_heads=2, rdim=8, side=4, vocab=30)
    out = P.forward(cfg, P.read_safetensors(tmp_path / "model.safetensors"), [3, 1, 2])
    assert out.shape == (3, 30) and np.isfinite(out).all()
