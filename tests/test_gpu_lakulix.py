"""Lakulix on the GPU against the plain numpy forward: every mechanism alone, prompts, decoding, portions, states that are
used again, distances and positions at every edge, and generation through the framework's own entry points."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from . import lakulix_common as lc
from .stack_common import close, feed, tokens_of
from oracle import lakulix as plain

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ("float32", "bfloat16")

MIXED = lc.config([lc.lightning(ff=56), lc.attention(ff=40), lc.wkv(), lc.attention(heads=2, kv_heads=1, dim=8, vdim=20), lc.wkv(heads=2, dim=36)],
                  loop={"start": 1, "stop": 4, "times": 2})

ONE_LAYER = {
    "lightning": (lc.config([lc.lightning()]), {}),
    "lightning wide values": (lc.config([lc.lightning(heads=2, dim=16, vdim=68)], width=64), {}),
    "lightning narrow values": (lc.config([lc.lightning(heads=5, dim=130, vdim=7)], width=96), {}),
    "lightning one head": (lc.config([lc.lightning(heads=1, dim=33, vdim=33)], width=40), {}),
    "lightning 128": (lc.config([lc.lightning(heads=2, dim=128, vdim=128)], width=128), {}),
    "lightning 256": (lc.config([lc.lightning(heads=1, dim=256, vdim=64)], width=64), {}),
    "lightning decay of one": (lc.config([lc.lightning(heads=3, decay=[1.0, 0.5, 1e-3])]), {}),
    "wkv": (lc.config([lc.wkv()]), {}),
    "wkv 64": (lc.config([lc.wkv(heads=2, dim=64)], width=96), dict(rank=16)),
    "wkv odd": (lc.config([lc.wkv(heads=5, dim=7)], width=50), dict(rank=1)),
    "wkv wide rank": (lc.config([lc.wkv(heads=1, dim=90)], width=64), dict(rank=70)),
    "wkv 128": (lc.config([lc.wkv(heads=1, dim=128)], width=64), {}),
    "wkv 192": (lc.config([lc.wkv(heads=1, dim=192)], width=64), {}),
    "attention": (lc.config([lc.attention()]), {}),
    "attention one head": (lc.config([lc.attention(heads=1, kv_heads=1, dim=17, vdim=9)], width=33), {}),
    "attention many per group": (lc.config([lc.attention(heads=12, kv_heads=1, dim=16, vdim=24)]), {}),
    "attention no sharing": (lc.config([lc.attention(heads=3, kv_heads=3, dim=64, vdim=64)]), dict(bias_rows=32)),
    "attention 128": (lc.config([lc.attention(heads=4, kv_heads=2, dim=128, vdim=100)], width=96), dict(bias_rows=20)),
    "attention 256": (lc.config([lc.attention(heads=2, kv_heads=1, dim=200, vdim=256)], width=64), {}),
    "attention wide values": (lc.config([lc.attention(heads=3, kv_heads=1, dim=40, vdim=150)]), {}),
    "attention wide keys": (lc.config([lc.attention(heads=3, kv_heads=1, dim=150, vdim=40)]), {}),
    "attention far buckets": (lc.config([lc.attention(bias_max=300)]), dict(bias_rows=8)),
    "feed-forward": (lc.config([lc.lightning(heads=1, dim=4, vdim=4, ff=200)]), {}),
    "feed-forward narrow": (lc.config([lc.wkv(heads=1, dim=8, ff=3)]), {}),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(ONE_LAYER))
def test_one_layer(ctx, name, dtype):
    cfg, kw = ONE_LAYER[name]
    t = lc.tensors(cfg, 11, **kw)
    tokens = tokens_of(cfg, 150)
    want, runs = lc.oracle(cfg, t).forward(tokens)
    m = lc.product(cfg, t, dtype, ctx)
    got, layers = m.forward_rows(tokens, range(len(tokens)), layers=True)
    assert np.abs(layers - runs).max() <= lc.LIMIT[dtype] * np.abs(runs).max()
    assert close(got, want, dtype)
    m.reset()
    assert close(feed(m, tokens[:90], [1] * 90), want[:90], dtype)
    m.close()


@pytest.fixture(scope="module")
def mixed():
    t = lc.tensors(MIXED, 3, pb=-5.0)
    tokens = tokens_of(MIXED, 330)
    want, runs = lc.oracle(MIXED, t).forward(tokens)
    return t, tokens, want, runs


@pytest.mark.parametrize("dtype", DTYPES)
def test_layers_of_a_looped_model(ctx, mixed, dtype):
    t, tokens, want, runs = mixed
    m = lc.product(MIXED, t, dtype, ctx)
    got, layers = m.forward_rows(tokens[:80], range(80), layers=True)
    assert layers.shape[0] == 8
    assert np.abs(layers - runs[:, :80]).max() <= 2 * lc.LIMIT[dtype] * np.abs(runs[:, :80]).max()
    assert close(got, want[:80], dtype, 2)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_and_reuse(ctx, mixed, dtype):
    """Every way of cutting gives the same logits; a state that another request has used gives them again."""
    t, tokens, want, _ = mixed
    m = lc.product(MIXED, t, dtype, ctx)
    n = len(tokens)
    for cuts in ([n], [2] * (n // 2), [3, 5, 7] * 22, [1, 63, 1, 64, 65, 2, 31, 32, 33, 38], [128, 1, 1, 1, 127, 2, 70], [17] * 19 + [7], [n - 40] + [1] * 40):
        m.reset()
        assert close(feed(m, tokens, cuts), want, dtype, 2), cuts[:6]
        other = tokens_of(MIXED, 70, seed=9)  # a shorter request over what the long one left
        m.reset()
        assert close(feed(m, other, [69, 1]), lc.oracle(MIXED, t).forward(other)[0], dtype, 2)
    m.close()


def test_prompt_chunks(ctx, mixed, monkeypatch):
    """A prompt longer than what goes through the layers at once: wanted places and layer outputs on both sides of every seam."""
    t, tokens, want, runs = mixed
    monkeypatch.setenv("AXQ_PROMPT_CHUNK", "50")
    m = lc.product(MIXED, t, "float32", ctx)
    places = [0, 48, 49, 50, 51, 99, 100, 149, 150, 151, 298, 300, 329]
    got, layers = m.forward_rows(tokens, places, layers=True)
    assert close(got, want[places], "float32", 2)
    assert np.abs(layers - runs).max() <= 2 * lc.LIMIT["float32"] * np.abs(runs).max()
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(ctx, mixed, dtype):
    t, tokens, want, _ = mixed
    m = lc.product(MIXED, t, dtype, ctx)
    assert close(feed(m, tokens, [1] * len(tokens)), want, dtype, 2)
    m.close()


def test_prompt_and_decoding_agree_to_rounding(ctx, mixed):
    t, tokens, _, _ = mixed
    m = lc.product(MIXED, t, "float32", ctx)
    a = feed(m, tokens, [len(tokens)])
    m.reset()
    b = feed(m, tokens, [1] * len(tokens))
    m.reset()
    assert lc.error(a, b).max() < 2 * lc.LIMIT["float32"]
    assert np.array_equal(feed(m, tokens, [len(tokens)]), a)  # the same cut again: the same bits
    m.close()


@pytest.mark.parametrize("loop,cut", [(None, 0), ({"start": 0, "stop": 3, "times": 3}, 0), ({"start": 2, "stop": 3, "times": 2}, 0), ({"start": 1, "stop": 2, "times": 1}, 0)])
def test_loops(ctx, loop, cut):
    cfg = lc.config([lc.wkv(), lc.attention(), lc.lightning()], loop=loop, softcap=None)
    t = lc.tensors(cfg, 21)
    tokens = tokens_of(cfg, 60)
    want = lc.oracle(cfg, t).forward(tokens)[0]
    m = lc.product(cfg, t, "float32", ctx)
    assert lc.error(feed(m, tokens, [25, 1, 1, 33]), want).max() < 2 * lc.LIMIT["float32"]
    m.close()


# ---- keys at chosen distances: one score stands out -----------------------------------------------------------------
def _pointing_model(dim, vdim, bias_rows, bias_max, max_positions=400):
    """One attention layer without feed-forward whose only strong score is between token 1 (asks) and token 2 (answers):
    every other weight is about sigmoid(-9), that one near one half, where its bias matters.  Token 2's value is large."""
    cfg = lc.config([lc.attention(heads=2, kv_heads=1, dim=dim, vdim=vdim, bias_max=bias_max, scale=1.0 / np.sqrt(dim), coef=0.0, every=5)],
                    width=64, vocab=40, max_positions=max_positions, softcap=None)
    t = lc.tensors(cfg, 31, bias_rows=bias_rows, pb=-9.0)
    t["pos"][:] = 0.0
    rng = np.random.default_rng(1)
    # input channel 0 is on for token 1 alone and channel 1 for token 2; queries, keys and values read them strongly
    t["embed"][:, :2] = 0.0
    t["embed"][1, 0] = t["embed"][2, 1] = 4.0
    t["l0.norm1.b"][:2] = 0.0
    a = rng.standard_normal(dim)
    t["l0.mix.q"][:, 0] = lc.bf16(np.tile(8.0 * a, 2))
    t["l0.mix.k"][:, 1] = lc.bf16(8.0 * a)
    t["l0.mix.v"][:, 1] = lc.bf16(8.0 * rng.standard_normal(vdim))
    t["l0.mix.q.norm"][:] = 1.0
    t["l0.mix.k.norm"][:] = lc.bf16(np.full(dim, 9.0 / np.sqrt(dim)))
    return cfg, t


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,vdim", [(32, 48), (128, 128)])
def test_far_keys_and_every_bucket_edge(ctx, dtype, dim, vdim):
    """A key at every distance that is special to the tables (bucket edges) or the kernels (chunks, tiles), asked for in a
    prompt and by a decoded token; with its bias one bucket off the answer would differ."""
    cfg, t = _pointing_model(dim, vdim, bias_rows=8, bias_max=64)
    t["l0.mix.rel"][:] = np.array([0.0, -3.0, 2.0, -2.0, 3.0, -1.5, 2.5, -2.5], np.float32)[:, None]
    edges = [n for n in range(1, 80) if plain.distance_bucket(n, 8, 64) != plain.distance_bucket(n - 1, 8, 64)]
    dist = sorted(set(d + o for d in edges + [31, 32, 63, 64, 127, 128, 191, 192, 255, 256, 300] for o in (-1, 0, 1) if d + o >= 1))
    m = lc.product(cfg, t, dtype, ctx)
    rng = np.random.default_rng(3)
    for d in dist:
        place = 5 if d % 2 else 63 if d < 250 else 2
        tokens = rng.integers(3, cfg["vocab"], place + d + 1)
        tokens[place], tokens[place + d] = 2, 1
        want = lc.oracle(cfg, t).forward(tokens)[0][-1:]
        without = tokens.copy()
        without[place] = 3
        far = lc.error(lc.oracle(cfg, t).forward(without)[0][-1:], want).max()
        assert far > 5 * lc.LIMIT["bfloat16"], "the key does not stand out"
        m.reset()
        assert close(m.forward_rows(tokens, [len(tokens) - 1]), want, dtype), d
        m.reset()
        m.forward_rows(tokens[:-1])
        assert close(m.feed(tokens[-1:], [0]), want, dtype), d
    m.close()


def test_distance_bias_alone(ctx):
    """Scores of zero (zero key norms): the weights are sigmoid(bias + number per head) and nothing else."""
    for bias_rows, bias_max in ((2, 5), (12, 13), (24, 96), (32, 400), (6, 3)):
        cfg = lc.config([lc.attention(bias_max=bias_max)], softcap=None)
        t = lc.tensors(cfg, 41, bias_rows=bias_rows, pb=-1.0)
        t["l0.mix.k.norm"][:] = 0.0
        t["l0.mix.rel"] = lc.bf16(2.0 * np.random.default_rng(2).standard_normal(t["l0.mix.rel"].shape))
        tokens = tokens_of(cfg, 200)
        if bias_max <= bias_rows // 2:  # no logarithmic part: everything beyond the exact rows is the last one
            half = bias_rows // 2
            real = plain.distance_bucket
            plain.distance_bucket = lambda n, rows, dmax: n if n < half else rows - 1
        want = lc.oracle(cfg, t).forward(tokens)[0]
        if bias_max <= bias_rows // 2:
            plain.distance_bucket = real
        m = lc.product(cfg, t, "float32", ctx)
        assert lc.error(feed(m, tokens, [120] + [1] * 80), want).max() < lc.LIMIT["float32"]
        m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_query_factor_steps(ctx, dtype):
    cfg = lc.config([lc.attention(coef=1.5, every=1), lc.attention(coef=-0.2, every=64)], softcap=None)
    t = lc.tensors(cfg, 51)
    tokens = tokens_of(cfg, 140)
    want = lc.oracle(cfg, t).forward(tokens)[0]
    m = lc.product(cfg, t, dtype, ctx)
    assert close(feed(m, tokens, [62, 1, 1, 1, 61, 1, 1, 1, 11]), want, dtype, 2)
    m.close()


def test_old_state_matters(ctx):
    """With slow decays the first tokens show hundreds of tokens later, in prompts and in decoding, across segments."""
    cfg = lc.config([lc.lightning(heads=2, dim=16, vdim=16, decay=[0.999, 1.0]), lc.wkv(heads=2, dim=16)], width=48, max_positions=900, softcap=None)
    t = lc.tensors(cfg, 61)
    t["l1.mix.w0"][:] = -8.0
    tokens = tokens_of(cfg, 800)
    changed = tokens.copy()
    changed[3] = (changed[3] + 1) % cfg["vocab"]
    want = lc.oracle(cfg, t).forward(tokens)[0]
    assert lc.error(lc.oracle(cfg, t).forward(changed)[0][-1:], want[-1:]).max() > 20 * lc.LIMIT["float32"]
    m = lc.product(cfg, t, "float32", ctx)
    for cuts in ([800], [1, 799], [401, 399], [770] + [1] * 30):
        m.reset()
        assert lc.error(feed(m, tokens, cuts), want).max() < 2 * lc.LIMIT["float32"], cuts[:3]
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_larger_sizes(ctx, dtype):
    """Sizes that take the big product tiles, several row tiles of attention and wide decode inputs."""
    cfg = lc.config([lc.attention(heads=8, kv_heads=2, dim=64, vdim=64, ff=6200), lc.lightning(heads=4, dim=64, vdim=64), lc.wkv(heads=8, dim=64)],
                    width=520, vocab=1000, max_positions=800)
    t = lc.tensors(cfg, 71, bias_rows=32, rank=24, pb=-6.0)
    tokens = tokens_of(cfg, 700)
    want = lc.oracle(cfg, t).forward(tokens)[0]
    m = lc.product(cfg, t, dtype, ctx)
    assert close(feed(m, tokens, [640, 57, 1, 1, 1]), want, dtype)
    m.close()


# ---- entry points ---------------------------------------------------------------------------------------------------
def _greedy(cfg, t, prompt, n):
    """Greedy continuation by the plain forward; also the smallest gap between the two best logits."""
    m, out, gap = lc.oracle(cfg, t), [], np.inf
    logits = m.forward(prompt)[0][-1]
    for _ in range(n):
        best = int(np.argmax(logits))
        two = np.sort(logits)[-2:]
        gap = min(gap, float(two[1] - two[0]))
        out.append(best)
        logits = m.forward([best])[0][-1]
    return out, gap


def test_greedy_generation(ctx, mixed):
    t, tokens, _, _ = mixed
    for n in (1, 2, 50):
        want, gap = _greedy(MIXED, t, tokens[:n], 40)
        assert gap > 1e-3
        m = lc.product(MIXED, t, "float32", ctx)
        out, _, _ = m.generate(tokens[:n], 40)
        assert out.tolist() == want
        assert m.seq_len() == n + 39
        m.reset()
        nxt, logits = m.forward_tokens(tokens[:n])
        assert nxt == want[0] and int(np.argmax(logits)) == nxt
        for k in range(5):
            assert m.forward(want[k])[0] == want[k + 1]
        out2, _, _ = m.generate_batch([tokens[:n]], 40)
        assert out2[0].tolist() == want
        m.close()


def test_sampling_is_repeatable_and_follows_the_logits(ctx, mixed):
    from axonml_amd.generation import GenerationConfig, TextGenerator

    t, tokens, _, _ = mixed
    m = lc.product(MIXED, t, "bfloat16", ctx)
    m.set_sampling(GenerationConfig(temperature=0.7, top_k=20, repetition_penalty=1.2), seed=3)
    a, _, _ = m.generate(tokens[:20], 30)
    m.reset()
    b, _, _ = m.generate(tokens[:20], 30)
    assert a.tolist() == b.tolist() and len(set(a.tolist())) > 3
    # greedy with a penalty: the sampler on the host's copy of the logits picks the same token
    cfg = GenerationConfig(do_sample=False, repetition_penalty=1.5)
    m.set_sampling(cfg)
    m.reset()
    nxt, logits = m.forward_tokens(tokens[:20])
    assert nxt == TextGenerator(cfg, ctx).get_next_token(logits, tokens[:20])
    m.close()


def test_beam_search(ctx):
    """One beam is greedy; with several, a state that cannot be rewound and one that can give the beams of the bookkeeping on
    the plain forward's logits."""
    from axonml_amd.generation import BeamSearch, beam_search_generate

    for layers in ([lc.wkv(), lc.attention()], [lc.attention(), lc.attention(ff=30)]):
        cfg = lc.config(layers)
        t = lc.tensors(cfg, 91)
        prompt = tokens_of(cfg, 7).tolist()
        bs = BeamSearch(3, 1.0, False, [])
        beams = bs.init_beams(prompt)
        for _ in range(5):
            beams = bs.expand_beams(beams, [lc.oracle(cfg, t).forward(b.tokens)[0][-1] for b in beams])
        m = lc.product(cfg, t, "float32", ctx)
        best, got = beam_search_generate(m, prompt, bs, 5)
        assert [b.tokens for b in got] == [b.tokens for b in beams] and best == bs.best_sequence(beams)
        m.reset()
        assert beam_search_generate(m, prompt, BeamSearch(1, 1.0, False, []), 6)[0][7:] == _greedy(cfg, t, prompt, 6)[0]
        m.close()


def test_cache_limit_and_refusals(ctx, mixed):
    from axonml_amd.quant import InvalidData, Overflow, QuantError, ShapeMismatch
    from axonml_amd.stack import StackModel
    from axonml_amd import lakulix

    t, tokens, want, _ = mixed
    m = lc.product(MIXED, t, "float32", ctx, cache_positions=70)
    assert lc.error(feed(m, tokens[:70], [60] + [1] * 10), want[:70]).max() < 2 * lc.LIMIT["float32"]
    with pytest.raises(Overflow):
        m.forward(int(tokens[70]))
    with pytest.raises(Overflow):
        m.forward_rows(tokens[:2])
    with pytest.raises((QuantError, RuntimeError)):
        m.truncate(10)  # a recurrent state cannot go back
    m.truncate(70)
    m.truncate(0)
    assert m.seq_len() == 0
    assert lc.error(feed(m, tokens[:30], [29, 1]), want[:30]).max() < 2 * lc.LIMIT["float32"]
    with pytest.raises(ShapeMismatch):
        m.set_batch(2)
    with pytest.raises((QuantError, RuntimeError)):
        m.forward_rows([0, MIXED["vocab"]])
    with pytest.raises((QuantError, RuntimeError)):
        m.forward_rows([1, 2, 3], [2, 1])
    with pytest.raises(InvalidData):  # true 32-bit takes bfloat16-exact weights only
        m.set_tensor(0, "mix.q", t["l0.mix.q"] * np.float32(1.0001))
    with pytest.raises(ShapeMismatch):
        m.set_tensor(0, "mix.q", t["l0.mix.q"][:, 1:])
    with pytest.raises((QuantError, RuntimeError)):
        m.set_tensor(0, "mix.nothing", t["l0.mix.q"])
    m.close()
    d = lakulix.describe(MIXED, lambda n: list(t[n].shape) if n in t else None)
    empty = StackModel(d, ctx=ctx)
    with pytest.raises(InvalidData):
        empty.forward(0)
    empty.close()


def test_weights_set_again_are_used(ctx):
    """The captured step must not go on reading a replaced weight or table."""
    cfg = lc.config([lc.attention(), lc.wkv()])
    t, other = lc.tensors(cfg, 81), lc.tensors(cfg, 82)
    tokens = tokens_of(cfg, 20)
    m = lc.product(cfg, t, "float32", ctx)
    feed(m, tokens, [10] + [1] * 10)
    for layer, name in ((0, "mix.q"), (0, "mix.rel"), (1, "mix.w2"), (1, "mix.u"), (-1, "head"), (0, "norm1")):
        full = name if layer < 0 else f"l{layer}.{name}"
        t[full] = other[full]
        m.set_tensor(layer, name, t[full])
    m.reset()
    assert lc.error(feed(m, tokens, [10] + [1] * 10), lc.oracle(cfg, t).forward(tokens)[0]).max() < 2 * lc.LIMIT["float32"]
    m.close()


def test_trace_program(tmp_path, mixed):
    """bin/trace_run on a checkpoint directory: portions, wanted places in any order, one request after the other."""
    t, tokens, want, _ = mixed
    lc.write_checkpoint(str(tmp_path), MIXED, t)
    out = tmp_path / "out"
    out.mkdir()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:50].tolist(), "want": [49, 0, 7]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[50:52].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [int(tokens[52])], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": tokens[:9].tolist(), "want": [8]}], "end": ["b"]}]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out), "--max-tokens", "60"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    read = lambda n: np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, MIXED["vocab"])  # noqa: E731
    assert lc.error(read(0), want[[49, 0, 7]]).max() < 2 * lc.LIMIT["float32"]
    assert not (out / "1.f32").exists()
    assert lc.error(read(2), want[52:53]).max() < 2 * lc.LIMIT["float32"]
    assert lc.error(read(3), want[8:9]).max() < 2 * lc.LIMIT["float32"]


def test_command_line_generates(tmp_path, mixed):
    t, tokens, _, _ = mixed
    lc.write_checkpoint(str(tmp_path), MIXED, t)
    want, gap = _greedy(MIXED, t, tokens[:6], 8)
    assert gap > 1e-3
    p = subprocess.run([sys.executable, "-m", "axonml_amd", "generate", "--model", str(tmp_path), "--dtype", "float32", "--tokens",
                        ",".join(str(x) for x in tokens[:6]), "--max-new-tokens", "8"], capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [int(x) for x in p.stdout.split()] == want


# ---- bfloat16 weights, on their own and under the LLaMA-shape model ---------------------------------------------------
def test_bf16_codec_and_products(ctx):
    from axonml_amd import quant as q

    rng = np.random.default_rng(4)
    x = rng.standard_normal(1003).astype(np.float32) * 10.0 ** rng.integers(-30, 30, 1003).astype(np.float32)
    qt = q.quantize_tensor(x, q.QuantType.BF16, ctx)
    assert np.array_equal(q.dequantize_tensor(qt, ctx), lc.bf16(x))
    for n, k in ((5, 3), (70, 72), (130, 512), (9, 1000), (300, 4160)):
        w = lc.bf16(rng.standard_normal((n, k)))
        dw = q.DeviceWeight.quantize(w, q.QuantType.BF16, ctx)
        assert np.array_equal(q.dequantize_tensor(dw.download(), ctx), w)
        b = rng.standard_normal(n).astype(np.float32)
        for batch in (1, 3, 50):
            v = rng.standard_normal((batch, k)).astype(np.float32)
            want = v.astype(np.float64) @ w.T.astype(np.float64) + b
            got = q.quantized_matmul(v, dw, b, ctx)
            assert np.abs(got - want).max() < 2e-5 * np.abs(want).max() + 1e-5 * np.sqrt(k)
        dw.free()


def test_llama_with_bf16_linears_and_rows(ctx):
    """forward_rows on the LLaMA-shape model agrees with its steps, with bfloat16 linears."""
    from axonml_amd.decode import QuantizedLlama
    from axonml_amd.quant import QuantType

    m = QuantizedLlama(ctx, vocab_size=320, hidden_size=256, intermediate_size=512, num_hidden_layers=2, num_attention_heads=4,
                       num_key_value_heads=2, head_dim=64, max_position_embeddings=120, rms_norm_eps=1e-5, rope_theta=10000.0)
    m.random_init(QuantType.BF16, 0.06, 1)
    tokens = np.random.default_rng(6).integers(0, 320, 80)
    steps = np.stack([m.forward(int(x))[1] for x in tokens])
    m.reset()
    rows = np.concatenate([m.forward_rows(tokens[:45], range(45)), m.forward_rows(tokens[45:50], range(5)), m.forward_rows(tokens[50:], range(30))])
    assert lc.error(rows, steps).max() < 1e-3
    m.close()
