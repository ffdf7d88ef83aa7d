"""The Vogizen session on the GPU against the plain statement of its equations (oracle/vogizen_plain.py): every
mechanism alone, sizes that fit no tile, loops, passes, portions and single tokens, keys on both sides of a window's
edge, the ring cache behind its end, extreme decays, sequences one after the other, and greedy generation."""
import copy
import json
import subprocess
import sys

import numpy as np
import pytest
import vogizen_gen as G
import vogizen_plain as P
from conftest import ROOT
from folder_helpers import BF16, F32, TOL, Opener, feed, feed_layers, rel

pytestmark = pytest.mark.gpu


@pytest.fixture
def open_model(hip, tmp_path):
    o = Opener(hip, tmp_path, G)
    yield o
    o.close()


def only(w, keep):
    """Silence every sublayer but `keep` (the end of its last tensor's name), so that one mechanism is all there is."""
    for name in w:
        if name.endswith((".ls1", ".ls2", ".side.norm")) and not name.endswith(keep):
            w[name] = np.zeros_like(w[name])
    return w


def reference_layers(cfg, w, t):
    ref = []
    P.forward(cfg, w, t, layers_out=ref)
    return ref


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("kind,keep", [("delta", ".ls1"), ("latent", ".ls1"), ("latent", ".ls2"), ("delta", ".side.norm")])
def test_each_sublayer_alone(open_model, dtype, kind, keep):
    cfg = G.config([G.delta() if kind == "delta" else G.latent()], loop=None)
    s, w = open_model(cfg, only(G.weights(cfg, 3), keep), dtype)
    t = G.tokens(cfg, 45)
    ref = reference_layers(cfg, w, t)
    x0 = P.embedding(cfg, w, np.asarray(t))
    for sizes in ([45], [1], [20, 2, 1]):
        s.reset()
        assert rel(feed_layers(s, t, sizes)[0] - x0, ref[0] - x0) < TOL[dtype], sizes  # what the layer adds


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_embedding_and_loop_product_alone(open_model, dtype):
    cfg = G.config([G.delta()], loop=(0, 1, 3), width=50)
    s, w = open_model(cfg, only(G.weights(cfg, 3), "nothing"), dtype, 3000)
    t = G.tokens(cfg, 2500)
    ref = reference_layers(cfg, w, t)
    got = [s.step(t[:2048], (), layers=True)[1], s.step(t[2048:2499], (), layers=True)[1], s.step(t[2499:], (), layers=True)[1]]
    for i in range(3):  # positions far along, in a pass and alone
        assert rel(np.concatenate(got, 1)[i], ref[i]) < {F32: 3e-6, BF16: 1e-2}[dtype]


SHAPES = {
    "delta, one of everything": G.delta(heads=1, kv_heads=1, dim=1, vdim=1, taps=1),
    "delta, no sharing": G.delta(heads=3, kv_heads=3, taps=2),
    "delta, five to a key head": G.delta(heads=10, kv_heads=2, taps=4),
    "delta, long convolution": G.delta(taps=7),
    "delta, odd sizes": G.delta(heads=3, kv_heads=1, dim=37, vdim=21, taps=4, ff=33),
    "delta, narrow and deep": G.delta(dim=130, vdim=5),
    "delta, shallow and wide": G.delta(dim=5, vdim=130),
    "delta, heads of 128": G.delta(heads=2, kv_heads=1, dim=128, vdim=128, taps=4),
    "delta, heads of 256": G.delta(heads=2, kv_heads=1, dim=256, vdim=250, taps=4),
    "delta, 240 wide": G.delta(heads=1, kv_heads=1, dim=48, vdim=240, taps=4, ff=70),
    "latent, one of everything": G.latent(heads=1, dim=1, vdim=1, q_rank=1, kv_rank=1, window=1, ff=1),
    "latent, window of two": G.latent(window=2),
    "latent, odd heads": G.latent(heads=5, dim=13, vdim=7, q_rank=31, kv_rank=9, window=30),
    "latent, wide values": G.latent(dim=8, vdim=40, window=33),
    "latent, wide keys": G.latent(dim=72, vdim=12, window=64, ff=None),
    "latent, wide latents": G.latent(q_rank=300, kv_rank=270, window=17),
    "latent, heads of 128": G.latent(heads=2, dim=128, vdim=128, window=40),
    "latent, heads of 256": G.latent(heads=2, dim=256, vdim=250, window=40),
    "latent, window never full": G.latent(window=1000),
    "latent, large scores": G.latent(scale=3.0, window=48),
    "latent, odd feed-forward": G.latent(ff=77),
}


@pytest.mark.parametrize("name", SHAPES)
def test_shapes(open_model, name):
    cfg = G.config([SHAPES[name]], width=36, loop=None)
    s, w = open_model(cfg)
    t = G.tokens(cfg, 70)
    ref = P.forward(cfg, w, t)
    for sizes in ([70], [33, 1], [2, 3, 19, 5, 17]):
        s.reset()
        assert rel(feed(s, t, sizes), ref) < TOL[F32], sizes


@pytest.mark.parametrize("width,vocab,eps,scale,side", [(33, 7, 1e-5, 1.0, 1), (64, 130, 0.3, 0.02, 24), (130, 33, 1e-6, 50.0, 40), (256, 64, 1e-3, 1.0, 260)])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_widths_and_constants(open_model, width, vocab, eps, scale, side, dtype):
    if dtype == BF16:
        side = max(side, 6)  # (one number over its own size is a sign, which rounding can turn)
    cfg = G.config([G.delta(), G.latent(), G.delta(heads=2, kv_heads=1, ff=50)], width, vocab, eps, scale, side, loop=(0, 2, 2))
    s, w = open_model(cfg, None, dtype)
    t = G.tokens(cfg, 40)
    ref = P.forward(cfg, w, t)
    assert rel(feed(s, t, [29, 1, 1, 9]), ref) < TOL[dtype]


@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 5, 2), (1, 3, 3), (2, 5, 2), (4, 5, 4), (0, 3, 1)])
def test_loops(open_model, loop):
    """Every pass of a loop has its own cache and state and begins with the loop's product, the first one too."""
    cfg = G.config([G.delta(), G.latent(window=6), G.delta(heads=2, kv_heads=2, taps=5, ff=30), G.latent(ff=None), G.delta(dim=9)], loop=loop)
    s, w = open_model(cfg)
    assert s.n_layer == len(P.layer_runs(cfg))
    t = G.tokens(cfg, 50)
    ref = reference_layers(cfg, w, t)
    for sizes in ([50], [1], [17, 2, 1, 30]):
        s.reset()
        got = feed_layers(s, t, sizes)
        for i, r in enumerate(ref):
            assert rel(got[i], r) < TOL[F32], (sizes, i)
    s.reset()
    assert rel(feed(s, t, [40, 1]), P.forward(cfg, w, t)) < TOL[F32]  # the same without layers read out between


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_layers_of_different_shapes(open_model, dtype):
    cfg = G.config([G.delta(), G.latent(heads=6, dim=40, vdim=8, window=25), G.delta(heads=5, kv_heads=5, dim=20, vdim=50, taps=6, ff=200),
                    G.latent(heads=1, dim=64, vdim=64, q_rank=70, kv_rank=33, window=3, ff=None)], width=72, side=20, loop=(1, 4, 2))
    s, w = open_model(cfg, None, dtype)
    t = G.tokens(cfg, 90)
    ref = P.forward(cfg, w, t)
    for sizes in ([90], [2, 31, 1, 40, 3], [60, 1]):
        s.reset()
        assert rel(feed(s, t, sizes), ref) < TOL[dtype], sizes


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("sizes", [[1], [2], [3], [15, 2], [16], [17], [31, 2, 1], [32], [33], [64, 65], [100, 1], [127, 2], [129]])
def test_portions(open_model, dtype, sizes):
    cfg = G.config([G.delta(taps=4), G.latent(window=45), G.delta(dim=32, taps=5, ff=40)], loop=(0, 2, 2))
    s, w = open_model(cfg, None, dtype)
    t = G.tokens(cfg, 200)
    got = feed(s, t, sizes)
    s.reset()
    whole = feed(s, t, [200])
    assert rel(got, whole) < TOL[dtype] / 2
    assert rel(got, P.forward(cfg, w, t)) < TOL[dtype]


def standing_out(window, heads=2, dim=32):
    """A model in which token 199 meets an earlier token 198 with a score far above the rest: queries and keys are the same
    function of one half of the embedding, which those two share; values come from the other half, in which they differ."""
    cfg = G.config([G.latent(heads=heads, dim=dim, vdim=24, q_rank=40, kv_rank=40, window=window, scale=0.3, ff=None)], width=64, vocab=200, loop=None)
    w = only(G.weights(cfg, 5), ".ls1")
    w["embed"] = w["embed"] * 16  # outweighs the position
    w["embed"][199, :32] = w["embed"][198, :32]
    w["l0.mix.dkv"][:20, 32:] = 0
    w["l0.mix.dkv"][20:, :32] = 0
    w["l0.mix.uk"][:, 20:] = 0
    w["l0.mix.uv"][:, :20] = 0
    w["l0.mix.dq"] = w["l0.mix.dkv"]
    w["l0.mix.dq.norm"] = w["l0.mix.dkv.norm"]
    w["l0.mix.uq"] = w["l0.mix.uk"]
    return cfg, w


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("window", [1, 2, 5, 31, 32, 33, 64, 65, 100, 128, 257, 300])
def test_keys_inside_and_outside_the_window(open_model, dtype, window):
    cfg, w = standing_out(window)
    s, _ = open_model(cfg, w, dtype, 400)
    rng = np.random.default_rng(window)
    wider, narrower = copy.deepcopy(cfg), copy.deepcopy(cfg)
    wider["layers"][0]["mixer"]["mask"]["size"] = window + 1
    narrower["layers"][0]["mixer"]["mask"]["size"] = max(window - 1, 1)
    for n in {window + 1, window + 2, window + 31, window + 40, 330}:
        for back in {window - 1, window}:  # the last key that is seen, the first that is not
            t = rng.integers(0, 198, n)
            t[n - 1 - back] = 198
            t[n - 1] = 199
            ref, x = reference_layers(cfg, w, t)[0], P.embedding(cfg, w, t)
            y = (ref - x)[-1:]
            if window > 1:  # a window one token off would show
                off = reference_layers(wider if back == window else narrower, w, t)[0]
                assert rel((off - x)[-1:], y) > 0.1
            for last in (1, 2, 20, n):  # decoded, a short portion, a longer one, the whole prompt
                s.reset()
                if last < n:
                    s.step(t[: n - last])
                _, lay = s.step(t[n - min(last, n):], (), layers=True)
                assert rel(lay[0, -1:] - x[-1:], y) < {F32: 1e-4, BF16: 0.06}[dtype], (n, back, last)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_ring_cache_behind_its_end(open_model, dtype):
    """More positions than the ring of a windowed cache has rows: prompts, portions and single tokens across its end."""
    window, n = 70, 2400
    cfg, w = standing_out(window, heads=1)
    s, _ = open_model(cfg, w, dtype, n)
    t = np.random.default_rng(8).integers(0, 198, n)
    for p in (2047, 2051, 2060, 2111, 2116, 2120, 2143, 2148, 2155, 2176, 2200, 2300, 2399):  # a key met again at the window's edge
        t[p - window + 1], t[p] = 198, 199
    ref, x = reference_layers(cfg, w, t)[0], P.embedding(cfg, w, t)
    for sizes in ([2048, 352], [2048, 40, 1], [1000, 1000, 37], [2048, 62, 2, 31, 1, 64]):
        s.reset()
        got = feed_layers(s, t, sizes)
        assert rel(got[0][-400:] - x[-400:], (ref - x)[-400:]) < {F32: 1e-4, BF16: 0.06}[dtype], sizes


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_decays_from_none_to_all(open_model, dtype):
    """Heads that forget at once, hardly ever, and anything between, and a step size from nothing to all, over many chunks."""
    cfg = G.config([G.delta(heads=12, kv_heads=2, dim=24, vdim=16, taps=4)], loop=None)
    w = only(G.weights(cfg, 7), ".ls1")
    w["l0.mix.A_log"][:] = G.bf16_round(np.linspace(-8, 5, 12))
    w["l0.mix.dt_bias"][:] = G.bf16_round(np.tile([-12, -3, 3, 25], 3))
    w["l0.mix.b"] *= 8
    s, _ = open_model(cfg, w, dtype, 512)
    t = G.tokens(cfg, 400)
    ref = P.forward(cfg, w, t)
    for sizes in ([400], [7, 300, 1], [390, 1]):
        s.reset()
        assert rel(feed(s, t, sizes), ref) < {F32: 2e-4, BF16: TOL[BF16]}[dtype], sizes


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_one_key_written_over_and_over(open_model, dtype):
    """Hardly any decay and the full step size at ever the same token: what the state holds is replaced each time, which a
    sum of powers of the chunk's matrix would get wrong."""
    cfg = G.config([G.delta(heads=2, kv_heads=1, dim=16, vdim=16, taps=2)], loop=None, vocab=5)
    w = only(G.weights(cfg, 11), ".ls1")
    w["embed"] *= 16
    w["l0.mix.A_log"][:] = -10
    w["l0.mix.b"][:] = np.sign(w["embed"][2]) * 0.5  # sigmoid near one for this token
    s, _ = open_model(cfg, w, dtype, 512)
    t = [2] * 150 + [3] + [2] * 120
    ref = P.forward(cfg, w, t)
    for sizes in ([271], [3, 140, 1], [100, 2, 1]):
        s.reset()
        assert rel(feed(s, t, sizes), ref) < {F32: 1e-4, BF16: TOL[BF16]}[dtype], sizes


def test_first_token_stays_in_the_state(open_model):
    """A head that hardly forgets: the sequence's first token shows hundreds of tokens later."""
    cfg = G.config([G.delta(heads=1, kv_heads=1, dim=16, vdim=8, taps=1)], eps=1e-9, loop=None)
    w = only(G.weights(cfg, 3), ".ls1")
    w["embed"] *= 16
    w["l0.mix.A_log"][:] = -12.0
    w["l0.mix.b"][:] = 0
    for n in "qkv":
        w[f"l0.mix.{n}.conv"][:] = 1
    w["l0.mix.q"] = w["l0.mix.k"]  # a token reads what its like wrote
    t = [0] + [1] * 398 + [0]
    u = [2] + t[1:]
    x = P.embedding(cfg, w, np.asarray(t))[-1:]
    ra, rb = reference_layers(cfg, w, t)[0][-1:] - x, reference_layers(cfg, w, u)[0][-1:] - x
    assert rel(rb, ra) > 0.1  # it does show, far above the tolerance
    s, _ = open_model(cfg, w, F32, 512)
    for tok, ref in ((t, ra), (u, rb)):
        for sizes in ([400], [1, 2, 370, 1]):
            s.reset()
            assert rel(feed_layers(s, tok, sizes)[0][-1:] - x, ref) < 1e-3  # (the stream is far larger than what is added)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_sequences_one_after_the_other(open_model, dtype):
    """What an ended sequence left in cache, history and state does not reach the next one."""
    cfg = G.config([G.delta(taps=5), G.latent(window=50), G.delta()], loop=(0, 2, 2))
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
    cfg = G.config([G.delta(taps=4), G.latent(window=90)], loop=(1, 2, 2))
    s, w = open_model(cfg, None, F32, 700)
    t = G.tokens(cfg, 700)
    assert rel(feed(s, t, [5, 1]), P.forward(cfg, w, t)) < 2 * TOL[F32]


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_prompts_longer_than_a_pass(open_model, dtype):
    cfg = G.config([G.delta(heads=2, kv_heads=1, dim=8, vdim=8), G.latent(heads=1, dim=8, vdim=8, window=300)], width=32, vocab=20, loop=(0, 2, 2))
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
        cfg = G.config([G.delta(heads=16, kv_heads=8, dim=64, vdim=64, taps=4, ff=1300), G.latent(heads=16, dim=64, vdim=64, q_rank=384, kv_rank=128,
                                                                                                  window=200, ff=1300)],
                       width=512, vocab=300, side=64, loop=(0, 2, 1))
        s, w = open_model(cfg, None, dtype, 700)
        t = G.tokens(cfg, 650)
        ref = []
        P.forward(cfg, w, t, np.float32, ref)
        _, lay = s.step(t, (), layers=True)
        for i in range(2):
            assert rel(lay[i], ref[i]) < TOL[dtype]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("width", [1030, 4100])
def test_wide_streams(open_model, dtype, width):
    """More channels than a workgroup holds in one quad a thread, and than a token's product adds to in its prologue."""
    cfg = G.config([G.delta(heads=2, kv_heads=1, ff=30), G.latent(ff=None)], width=width, vocab=9, loop=(0, 2, 2) if width < 2000 else None)
    s, w = open_model(cfg, None, dtype, 64)
    t = G.tokens(cfg, 30)
    assert rel(feed(s, t, [25, 1, 1, 3]), P.forward(cfg, w, t)) < TOL[dtype]


@pytest.mark.parametrize("passes", [True, False, 7])
def test_greedy_generation(open_model, passes):
    cfg = G.config([G.delta(taps=4), G.latent(window=9), G.delta(ff=30)], vocab=150, loop=(0, 2, 2))
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
    cfg = G.config([G.delta(), G.latent(), G.delta()], vocab=150, loop=(1, 3, 2))
    s, _ = open_model(cfg, None, BF16)
    prompt = G.tokens(cfg, 40)
    out = s.generate(prompt, 30)["tokens"].tolist()
    s.reset()
    logits = feed(s, prompt + out[:-1], [40, 1])[39:]
    assert logits.argmax(-1).tolist() == out


def test_generation_repeats_bit_for_bit(open_model):
    cfg = G.config([G.delta(heads=4, dim=64, vdim=64, taps=4), G.latent(heads=4, dim=64, vdim=64, window=700)] * 2, vocab=150, loop=(0, 2, 2))
    s, _ = open_model(cfg, None, BF16, 1300)
    prompt = G.tokens(cfg, 900)
    runs = [s.generate(prompt, 300) for _ in range(4)]
    for r in runs[1:]:
        assert np.array_equal(r["tokens"], runs[0]["tokens"])
        assert np.array_equal(r["top2"][899:].view(np.uint32), runs[0]["top2"][899:].view(np.uint32))


def test_errors_are_reported(hip, open_model):
    cfg = G.config([G.delta(), G.latent()], loop=(0, 2, 2))
    s, w = open_model(cfg, None, F32, 8)
    for call in (lambda: s.step([60]), lambda: s.step(range(9)), lambda: s.step([1], [1]), lambda: s.generate([1] * 5, 4)):
        with pytest.raises(hip.hip.RmiHipError):
            call()
    assert s.position == 0 and s.step([1], [0]).shape == (1, 60)
    for name in ("loop.in", "side.embed", "l1.norm2", "l0.mix.dt_bias", "l1.mix.uk", "l0.ls1"):
        bad = dict(w)
        del bad[name]
        with pytest.raises(hip.hip.RmiHipError, match=f"Missing tensor: {name}"):
            open_model(cfg, bad)
    with pytest.raises(hip.hip.RmiHipError, match="Invalid tensor embed"):
        open_model(cfg, dict(w, embed=w["embed"][:, :-1]))
    for change in (dict(layers=[G.delta(heads=4, kv_heads=3)]), dict(layers=[G.delta(dim=300)]), dict(layers=[G.latent(vdim=300)]),
                   dict(layers=[G.latent(window=0)]), dict(layers=[{"type": "other", "mixer": {}, "mlp": None}]),
                   dict(loop={"start": 1, "stop": 1, "times": 2}), dict(loop={"start": 0, "stop": 3, "times": 2}), dict(token_side={})):
        with pytest.raises(hip.hip.RmiHipError):
            open_model(dict(cfg, **change), w)
    other = copy.deepcopy(cfg)
    other["layers"][1]["mlp"]["kind"] = "sparse"
    with pytest.raises(hip.hip.RmiHipError, match="not 'dense'"):
        open_model(other, w)
    with pytest.raises(hip.hip.RmiHipError, match="architecture 'Vogizen' is not Ruvenex"):
        hip.decode.RuvenexSession(G.write_folder(open_model.tmp_path / "other", cfg, w), 8)


def test_trace_run(tmp_path):
    cfg = G.config([G.delta(), G.latent(window=4)], loop=(0, 2, 2))
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
    import importlib

    cli = importlib.import_module("rust-model-inference_amd.__main__")
    cfg = G.config([G.latent(), G.delta()], loop=(1, 2, 3))
    folder = G.write_folder(tmp_path / "m", cfg, G.weights(cfg))
    s = hip.models.open_session(folder, 32, F32)
    want = s.generate([5, 17, 3], 9)["tokens"].tolist()
    s.close()
    assert cli.main(["--model", folder, "--tokens", "5,17,3", "--max-new", "9", "--dtype", F32]) == 0
    assert [int(t) for t in capsys.readouterr().out.strip().split(",")] == want
