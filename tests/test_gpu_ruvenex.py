"""The Ruvenex session on the GPU against the plain statement of its equations (oracle/ruvenex_plain.py): every
mechanism alone, sizes that fit no tile, passes, portions and single tokens, borders of key blocks and recurrence
chunks, extreme forget gates, sequences one after the other, and greedy generation."""
import json
import subprocess
import sys

import numpy as np
import pytest
import ruvenex_gen as G
import ruvenex_plain as P
from conftest import ROOT
from folder_helpers import BF16, F32, TOL, Opener, feed, rel

pytestmark = pytest.mark.gpu


@pytest.fixture
def open_model(hip, tmp_path):
    o = Opener(hip, tmp_path, G)
    yield o
    o.close()


def only(w, keep):
    """Zero the output projections of every sublayer but `keep`, so that one mechanism is all there is."""
    for name in w:
        if name.endswith((".left.o", ".right.o", ".mlp.down")) and not name.endswith(keep):
            w[name] = np.zeros_like(w[name])
    return w


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("keep", [".left.o", ".right.o", ".mlp.down"])
def test_each_sublayer_alone(open_model, dtype, keep):
    cfg = G.config([G.layer_config()])
    s, w = open_model(cfg, only(G.weights(cfg, 3), keep), dtype)
    t, ref = G.tokens(cfg, 45), []
    P.forward(cfg, w, t, layers_out=ref)
    x0 = w["embed"][t] * cfg["embedding"]["scale"]
    _, whole = s.step(t, (), layers=True)
    s.reset()
    steps = np.concatenate([s.step([k], (), layers=True)[1] for k in t], 1)
    for got in (whole, steps):  # what the layer adds
        assert rel(got[0] - x0, ref[0] - x0) < TOL[dtype]


SHAPES = {
    "one of everything": dict(heads=1, kv_heads=1, dim=2, vdim=1, taps=1, rot_dims=2, rheads=1, rdim=1, rvdim=1, ff=1),
    "no rotation": dict(rot_dims=0),
    "whole head rotated": dict(dim=24, rot_dims=24, base=77.0),
    "wide values": dict(dim=8, vdim=40, rot_dims=4),
    "wide keys": dict(dim=72, vdim=12, rot_dims=20),
    "no sharing": dict(heads=3, kv_heads=3, taps=2),
    "five to a key head": dict(heads=10, kv_heads=2, taps=5),
    "more queries than a tile": dict(heads=20, kv_heads=1, taps=4),
    "heads of 128": dict(heads=2, kv_heads=1, dim=128, vdim=128, rot_dims=32, rdim=128, rvdim=128),
    "heads of 256": dict(heads=2, kv_heads=1, dim=256, vdim=250, rot_dims=64, rdim=256, rvdim=256),
    "odd recurrence": dict(rheads=3, rdim=37, rvdim=21),
    "recurrence narrow and deep": dict(rdim=130, rvdim=5),
    "recurrence shallow and wide": dict(rdim=5, rvdim=130),
    "large scores": dict(scale=4.0),
    "scales": dict(left_scale=-2.5, right_scale=0.0),
    "no feed-forward": dict(ff=None),
    "odd feed-forward": dict(ff=77),
}


@pytest.mark.parametrize("name", SHAPES)
def test_shapes(open_model, name):
    cfg = G.config([G.layer_config(**SHAPES[name])], width=36)
    s, w = open_model(cfg)
    t = G.tokens(cfg, 70)
    ref = P.forward(cfg, w, t)
    for sizes in ([70], [33, 1], [2, 3, 19, 5, 17]):
        s.reset()
        assert rel(feed(s, t, sizes), ref) < TOL[F32], sizes


@pytest.mark.parametrize("width,vocab,eps,scale", [(33, 7, 1e-5, 1.0), (64, 130, 0.3, 0.02), (130, 33, 1e-6, 50.0), (256, 64, 1e-5, 1.0)])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_widths_and_constants(open_model, width, vocab, eps, scale, dtype):
    cfg = G.config([G.layer_config(), G.layer_config(heads=2, kv_heads=1)], width, vocab, eps, scale)
    s, w = open_model(cfg, None, dtype)
    t = G.tokens(cfg, 40)
    ref = P.forward(cfg, w, t)
    assert rel(feed(s, t, [29, 1, 1, 9]), ref) < TOL[dtype]


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_layers_of_different_shapes(open_model, dtype):
    cfg = G.config([G.layer_config(), G.layer_config(heads=6, kv_heads=3, dim=40, vdim=8, taps=6, rot_dims=2, base=5.0, ff=None),
                    G.layer_config(heads=1, kv_heads=1, dim=64, vdim=64, taps=1, rot_dims=64, rheads=5, rdim=20, rvdim=50, ff=200),
                    G.layer_config(rot_dims=8, base=500.0)], width=72)
    s, w = open_model(cfg, None, dtype)
    t = G.tokens(cfg, 90)
    ref = P.forward(cfg, w, t)
    for sizes in ([90], [2, 31, 1, 40, 3], [60, 1]):
        s.reset()
        assert rel(feed(s, t, sizes), ref) < TOL[dtype], sizes


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("sizes", [[1], [2], [3], [15, 2], [16], [17], [31, 2, 1], [32], [33], [64, 65], [100, 1], [127, 2], [129]])
def test_portions(open_model, dtype, sizes):
    cfg = G.config([G.layer_config(heads=6, kv_heads=2, taps=4), G.layer_config(dim=32, vdim=24, ff=None)])
    s, w = open_model(cfg, None, dtype)
    t = G.tokens(cfg, 200)
    got = feed(s, t, sizes)
    s.reset()
    whole = feed(s, t, [200])
    assert rel(got, whole) < TOL[dtype] / 2
    assert rel(got, P.forward(cfg, w, t)) < TOL[dtype]


def standing_out(dim=32, taps=2):
    """A model in which a query of one token meets its own earlier key with a score far above the rest: keys and
    queries share their projection, and the values' convolution tells apart where that earlier token stood."""
    cfg = G.config([G.layer_config(heads=2, kv_heads=1, dim=dim, vdim=16, taps=taps, rot_dims=2, base=1e9, scale=1.0)], width=64, vocab=200)
    w = only(G.weights(cfg, 5), ".left.o")
    k = w["l0.mix.left.k"]
    k[:2] = 0  # the rotated pair stays out of the scores
    w["l0.mix.left.q"] = np.concatenate([k, k])
    for n in ("q", "k"):
        c = np.zeros_like(w[f"l0.mix.left.{n}.conv"])
        c[:, -1] = 1.0
        w[f"l0.mix.left.{n}.conv"] = c
    w["l0.mix.left.v.conv"][:] = 0.7
    return cfg, w


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_one_key_among_many_at_every_border(open_model, dtype):
    cfg, w = standing_out()
    s, _ = open_model(cfg, w, dtype, 1400)
    rng = np.random.default_rng(2)
    n, special = 1300, 199
    base = rng.integers(0, 199, n)
    tol = {F32: 1e-4, BF16: 6e-2}[dtype]
    for p in (0, 1, 2, 15, 16, 31, 32, 33, 63, 64, 127, 128, 129, 255, 256, 511, 512, 1023, 1024, 1279, 1280, n - 3, n - 2):
        t = base.copy()
        t[[p, n - 1]] = special
        h = P.rms_norm(w["embed"][t].astype(np.float64) * cfg["embedding"]["scale"], w["l0.norm1"], 1e-5)
        x = w["embed"][t[-1]] * cfg["embedding"]["scale"]
        want = P.attention_mixer(h, {k: v.astype(np.float64) for k, v in w.items()}, "l0.mix.left.", cfg["layers"][0]["mixer"]["left"], 1e-5) \
            if p == 0 else None
        # only the last position is needed: its weights over all keys
        k = P.rotate_interleaved((h @ w["l0.mix.left.k"].T).reshape(n, 1, -1), 2, 1e9)[:, 0]
        v = P.rms_unit(P.causal_conv(h @ w["l0.mix.left.v"].T, w["l0.mix.left.v.conv"].astype(np.float64)), 1e-5)
        sc = k @ k[-1]
        a = np.exp(sc - sc.max())
        a /= a.sum()
        assert 0.3 < a[p] < 0.7, (p, a[p])  # the far key and the query's own share the weight
        o = np.concatenate([(a @ v) * P.sigmoid(h[-1] @ g) for g in w["l0.mix.left.g"]]) @ w["l0.mix.left.o"].T
        if want is not None:
            assert np.allclose(o, want[-1])
        y = P.residual_gate(h[-1], w, "l0.rg1") * cfg["layers"][0]["mixer"]["left_scale"] * o
        for last in (1, 2, 20):  # decoded, a short portion, a longer one
            s.reset()
            s.step(t[: n - last])
            _, lay = s.step(t[n - last:], (), layers=True)
            assert rel(lay[0, -1] - x, y) < tol, (p, last)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_forget_gates_from_none_to_all(open_model, dtype):
    """Channels that forget at once, never, and anything between, side by side in one head, over many chunks."""
    cfg = G.config([G.layer_config(rheads=2, rdim=24, rvdim=16)])
    w = only(G.weights(cfg, 7), ".right.o")
    w["l0.mix.right.lower"][:] = 0
    w["l0.mix.right.lower"][::3] = 0.99609375
    w["l0.mix.right.f.b"][:] = G.bf16_round(np.linspace(-25, 25, 48))
    w["l0.mix.right.norm"][:] = 1
    s, _ = open_model(cfg, w, dtype, 512)
    t = G.tokens(cfg, 400)
    ref = P.forward(cfg, w, t)
    for sizes in ([400], [7, 300, 1], [390, 1]):
        s.reset()
        # (the head norm magnifies a state that all but vanished)
        assert rel(feed(s, t, sizes), ref) < {F32: 2e-4, BF16: TOL[BF16]}[dtype], sizes


def test_first_token_stays_in_the_state(open_model):
    """A channel that hardly forgets: the sequence's first token shows hundreds of tokens later."""
    cfg = G.config([G.layer_config(rheads=1, rdim=4, rvdim=8, right_scale=3.0)], eps=1e-9)
    w = only(G.weights(cfg, 9), ".right.o")
    w["l0.mix.right.lower"][:] = 0.99609375
    w["l0.mix.right.f.b"][:] = -4.0
    s, _ = open_model(cfg, w, F32, 512)
    t = [0] + [1] * 399
    u = [2] + t[1:]
    ra, rb = P.forward(cfg, w, t), P.forward(cfg, w, u)
    assert rel(rb[-1:], ra[-1:]) > 1e-3  # it does show, far above the tolerance
    for tok, ref in ((t, ra), (u, rb)):
        for sizes in ([400], [1, 2, 370, 1]):
            s.reset()
            assert rel(feed(s, tok, sizes)[-3:], ref[-3:]) < TOL[F32]


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_sequences_one_after_the_other(open_model, dtype):
    """What an ended sequence left in cache, history and state does not reach the next one."""
    cfg = G.config([G.layer_config(taps=5), G.layer_config()])
    s, w = open_model(cfg, None, dtype)
    seqs = [G.tokens(cfg, n, n) for n in (1, 200, 3, 70, 2, 129)]
    first = []
    for t in seqs:
        s.reset()
        first.append(feed(s, t, [max(len(t) - 3, 1), 1]))
        assert s.position == len(t)
    for t, a in list(zip(seqs, first))[::-1]:
        s.reset()
        assert np.array_equal(feed(s, t, [max(len(t) - 3, 1), 1]), a)  # the same cuts: the same bits
        assert rel(a, P.forward(cfg, w, t)) < TOL[dtype]


def test_long_decoding(open_model):
    cfg = G.config([G.layer_config(heads=4, kv_heads=1, taps=4), G.layer_config()])
    s, w = open_model(cfg, None, F32, 700)
    t = G.tokens(cfg, 700)
    assert rel(feed(s, t, [5, 1]), P.forward(cfg, w, t)) < TOL[F32]


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_prompts_longer_than_a_pass(open_model, dtype):
    cfg = G.config([G.layer_config(heads=2, kv_heads=1, dim=8, vdim=8, rot_dims=4, rheads=1)], width=32, vocab=20)
    s, w = open_model(cfg, None, dtype, 2600)
    t = G.tokens(cfg, 2550)
    ref = P.forward(cfg, w, t)
    places = [0, 1, 2046, 2047, 2048, 2049, 2050, 2300, 2549]
    assert rel(s.step(t, places), ref[places]) < TOL[dtype]
    s.set_prompt_passes(500)
    s.reset()
    assert rel(s.step(t, places[::-1]), ref[places[::-1]]) < TOL[dtype]
    assert rel(s.step([3], [0]), P.forward(cfg, w, t + [3])[-1:]) < TOL[dtype]


def test_large_products(open_model):
    """Enough rows and tokens for the largest tiles of the products, and the attention launch for many columns."""
    for dtype in (F32, BF16):
        cfg = G.config([G.layer_config(heads=16, kv_heads=2, dim=64, vdim=64, rot_dims=16, rheads=8, rdim=64, rvdim=64, ff=1300)], width=512,
                       vocab=300)
        s, w = open_model(cfg, None, dtype, 700)
        t = G.tokens(cfg, 650)
        ref = []
        P.forward(cfg, w, t, np.float32, ref)
        _, lay = s.step(t, (), layers=True)
        assert rel(lay[0], ref[0]) < TOL[dtype]


@pytest.mark.parametrize("passes", [True, False, 7])
def test_greedy_generation(open_model, passes):
    cfg = G.config([G.layer_config(taps=4), G.layer_config(ff=None)], vocab=150)
    s, w = open_model(cfg)
    s.set_prompt_passes(passes)
    prompt, new = G.tokens(cfg, 23), 12
    r = s.generate(prompt, new, dump_steps=[0, 5, 6, 22, 24, 33])
    seq = list(prompt)
    for _ in range(new):
        ref = P.forward(cfg, w, seq)
        top = np.sort(ref[-1])[::-1]
        assert top[0] - top[1] > 1e-3  # no tie that rounding could turn
        seq.append(int(ref[-1].argmax()))
    assert r["tokens"].tolist() == seq[23:]
    ref = P.forward(cfg, w, seq)
    assert rel(r["dump"], ref[[0, 5, 6, 22, 24, 33]]) < TOL[F32]
    assert r["argmax"][22:].tolist() == seq[23:]
    assert np.allclose(r["top2"][22:, 0], ref[22:-1].max(-1), rtol=1e-4)
    # generating again, then stopping before a token of the result
    assert s.generate(prompt, new)["tokens"].tolist() == seq[23:]
    stop = seq[30]
    s.set_stop_ids([stop])
    assert s.generate(prompt, new)["tokens"].tolist() == seq[23: 23 + seq[23:].index(stop)]


def test_generation_in_bf16_follows_its_own_logits(open_model):
    cfg = G.config([G.layer_config(), G.layer_config()], vocab=150)
    s, _ = open_model(cfg, None, BF16)
    prompt = G.tokens(cfg, 40)
    out = s.generate(prompt, 30)["tokens"].tolist()
    s.reset()
    logits = feed(s, prompt + out[:-1], [40, 1])[39:]
    assert logits.argmax(-1).tolist() == out


def test_generation_repeats_bit_for_bit(open_model):
    """Keys divided over workgroups that hand their parts to whichever arrives last: the order of arrival does not show."""
    cfg = G.config([G.layer_config(heads=4, kv_heads=2, dim=64, vdim=64, rot_dims=16)] * 3, vocab=150)
    s, _ = open_model(cfg, None, BF16, 1300)
    prompt = G.tokens(cfg, 900)
    runs = [s.generate(prompt, 300) for _ in range(4)]
    for r in runs[1:]:
        assert np.array_equal(r["tokens"], runs[0]["tokens"])
        assert np.array_equal(r["top2"][899:].view(np.uint32), runs[0]["top2"][899:].view(np.uint32))


def test_errors_are_reported(hip, open_model, tmp_path):
    cfg = G.config([G.layer_config()])
    s, w = open_model(cfg, None, F32, 8)
    for call in (lambda: s.step([60]), lambda: s.step(range(9)), lambda: s.step([1], [1]), lambda: s.generate([1] * 5, 4)):
        with pytest.raises(hip.hip.RmiHipError):
            call()
    assert s.position == 0 and s.step([1], [0]).shape == (1, 60)
    bad = dict(w)
    del bad["l0.rg2.b"]
    with pytest.raises(hip.hip.RmiHipError, match="Missing tensor: l0.rg2.b"):
        open_model(cfg, bad)
    bad = dict(w, head=w["head"][:, :-1])
    with pytest.raises(hip.hip.RmiHipError, match="Invalid tensor head"):
        open_model(cfg, bad)
    for change in (dict(kv_heads=3), dict(dim=300), dict(rot_dims=3), dict(heads=0)):
        other = G.config([G.layer_config(**change)])
        with pytest.raises(hip.hip.RmiHipError):
            open_model(other, w)
    other = json.loads(json.dumps(cfg))
    other["layers"][0]["mlp"]["kind"] = "sparse"
    with pytest.raises(hip.hip.RmiHipError, match="not 'dense'"):
        open_model(other, w)


def test_trace_run(open_model, tmp_path):
    cfg = G.config([G.layer_config()])
    w = G.weights(cfg)
    folder, out = G.write_folder(tmp_path / "model", cfg, w), tmp_path / "out"
    out.mkdir()
    t = G.tokens(cfg, 12)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:5], "want": [0, 4]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t[5:6], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": t[6:], "want": [5]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": t[:3], "want": [2]}], "end": ["b"]}]
    r = subprocess.run([sys.executable, f"{ROOT}/bin/trace_run", "--model", folder, "--dtype", F32, "--out", str(out), "--max-tokens", "12"],
                       input="".join(json.dumps(x) + "\n" for x in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    ref = P.forward(cfg, w, t)
    for step, rows in ((0, [0, 4]), (2, [11]), (3, [2])):
        assert rel(np.fromfile(out / f"{step}.f32", "<f4").reshape(-1, 60), ref[rows]) < TOL[F32]
    assert not (out / "1.f32").exists()


def test_command_line_generates(hip, tmp_path, capsys):
    """`python -m rust-model-inference_amd` on a model folder and on a GGUF file: the sessions' own tokens."""
    import importlib

    cli = importlib.import_module("rust-model-inference_amd.__main__")
    cfg = G.config([G.layer_config()])
    folder = G.write_folder(tmp_path / "m", cfg, G.weights(cfg))
    gguf = str(tmp_path / "q.gguf")
    hip.gguf.write_synthetic_qwen3(gguf, 3, n_layer=1, n_embd=64, n_head=2, n_head_kv=1, head_dim=32, n_ff=64, vocab=96)
    for path, args in ((folder, ["--dtype", F32]), (gguf, [])):
        s = hip.models.open_session(path, 32, F32)
        want = s.generate([5, 17, 3], 9)["tokens"].tolist()
        s.close()
        assert cli.main(["--model", path, "--tokens", "5,17,3", "--max-new", "9", *args]) == 0
        assert [int(t) for t in capsys.readouterr().out.strip().split(",")] == want
