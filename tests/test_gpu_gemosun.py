"""Gemosun on the GPU against the plain numpy forward: every mechanism alone, prompts, decoding, portions, caches that are
used again, keys on both sides of every window's and block's edge, and generation through the framework's own entry points."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from . import gemosun_common as gc
from .stack_common import close, feed, tokens_of, write_checkpoint
from oracle import gemosun as plain

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ("float32", "bfloat16")

MIXED = gc.config([gc.attention(mlp=gc.dense(56)), gc.attention(heads=6, kv_heads=3, dim=16, size=41, pool=7, mlp=gc.moe()), gc.attention(size=9, pool=3),
                   gc.attention(heads=2, kv_heads=1, dim=40, mlp=gc.moe(experts=8, top=3, groups=(2, 1), shared=0))])


def one(width=72, vocab=101, **kw):
    return gc.config([gc.attention(**kw)], width=width, vocab=vocab)


ONE_LAYER = {
    "attention": one(),
    "attention one head": one(heads=1, kv_heads=1, dim=18, width=33),
    "attention many per group": one(heads=12, kv_heads=1, dim=16),
    "attention no sharing": one(heads=3, kv_heads=3, dim=64, width=64),
    "attention 128": one(heads=4, kv_heads=2, dim=128, width=96, scale=0.1),
    "attention 200": one(heads=2, kv_heads=1, dim=200, width=64, scale=0.08),
    "attention 256": one(heads=2, kv_heads=2, dim=256, width=64, scale=0.06),
    "window of one": one(size=1, pool=2),
    "blocks of one": one(size=6, pool=1),
    "window of 64, blocks of 64": one(size=64, pool=64),
    "window of 65, blocks of 8": one(size=65, pool=8),
    "window past the end": one(size=500, pool=9),
    "no blocks": one(size=30, pool=None),
    "blocks wider than the window": one(size=4, pool=31),
    "no rotation": one(turn=None),
    "rotation as it is": one(turn=gc.rot(20, 500.0, None)),
    "rotation of two dimensions": one(turn=gc.rot(2, 100.0)),
    "rotation slowed throughout": one(turn=gc.rot(20, 100.0, {"factor": 8.0, "original": 9, "fast": 40.0, "slow": 9.0})),
    "rotation that ramps over its whole width": one(turn=gc.rot(20, 50.0, {"factor": 5.0, "original": 4000, "fast": 900.0, "slow": 0.2})),
    "dense": one(mlp=gc.dense(200)),
    "dense narrow": one(mlp=gc.dense(3)),
    "dense 32": one(mlp=gc.dense(32), width=64),
    "dense 97": one(mlp=gc.dense(97), width=65),
    "mixture": one(mlp=gc.moe()),
    "mixture without groups": one(mlp=gc.moe(groups=None, experts=5, top=3)),
    "mixture of all groups": one(mlp=gc.moe(groups=(3, 3), experts=9, top=4)),
    "mixture of one group of four": one(mlp=gc.moe(groups=(4, 1), experts=12, top=2)),
    "groups of one": one(mlp=gc.moe(groups=(6, 3), experts=6, top=3)),
    "mixture of one": one(mlp=gc.moe(groups=None, experts=1, top=1)),
    "one of many": one(mlp=gc.moe(groups=None, experts=7, top=1, shared=0)),
    "all of them": one(mlp=gc.moe(groups=None, experts=4, top=4)),
    "mixture of 64": one(mlp=gc.moe(groups=(8, 2), experts=64, top=5, ff=9)),
    "mixture of 96": one(mlp=gc.moe(groups=(8, 3), experts=96, top=6, ff=9)),
    "mixture of 130 without groups": one(mlp=gc.moe(groups=None, experts=130, top=9, ff=5)),
    "mixture, wide experts": one(mlp=gc.moe(ff=130, shared=70), width=130),
    "mixture, narrow experts": one(mlp=gc.moe(ff=1, shared=1), width=40),
    "layers of different rotations, with and without feed-forward": gc.config([gc.attention(turn=gc.rot(20, 500.0, None)), gc.attention(mlp=gc.dense(24)),
                                                                              gc.attention(turn=None), gc.attention(turn=gc.rot(8, 70.0))]),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(ONE_LAYER))
def test_one_layer(ctx, name, dtype):
    cfg = copy.deepcopy(ONE_LAYER[name])
    if name == "no blocks":  # the plain forward has no such case: a block that never ends
        cfg["layers"][0]["mixer"]["mask"]["pool"] = 100000
    t = gc.tensors(cfg, 11)
    tokens = tokens_of(cfg, 170)
    assert gc.margin(cfg, t, tokens) > 0.002
    want, runs = gc.oracle(cfg, t).forward(tokens)
    if name == "no blocks":
        del cfg["layers"][0]["mixer"]["mask"]["pool"]
    m = gc.product(cfg, t, dtype, ctx)
    got, layers = m.forward_rows(tokens, range(len(tokens)), layers=True)
    assert np.abs(layers - runs).max() <= gc.LIMIT[dtype] * np.abs(runs).max()
    assert close(got, want, dtype)
    m.reset()
    assert close(feed(m, tokens[:110], [1] * 110), want[:110], dtype)
    m.close()


@pytest.fixture(scope="module")
def mixed():
    t = gc.tensors(MIXED, 3)
    tokens = tokens_of(MIXED, 330)
    assert gc.margin(MIXED, t, tokens) > 0.002
    want, runs = gc.oracle(MIXED, t).forward(tokens)
    return t, tokens, want, runs


@pytest.mark.parametrize("dtype", DTYPES)
def test_layers(ctx, mixed, dtype):
    t, tokens, want, runs = mixed
    m = gc.product(MIXED, t, dtype, ctx)
    got, layers = m.forward_rows(tokens[:80], range(80), layers=True)
    assert layers.shape[0] == 4
    assert np.abs(layers - runs[:, :80]).max() <= 2 * gc.LIMIT[dtype] * np.abs(runs[:, :80]).max()
    assert close(got, want[:80], dtype, 2)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_and_reuse(ctx, mixed, dtype):
    """Every way of cutting gives the same logits; a cache that another request has used gives them again."""
    t, tokens, want, _ = mixed
    m = gc.product(MIXED, t, dtype, ctx)
    n = len(tokens)
    other = tokens_of(MIXED, 70, seed=9)
    other_want = gc.oracle(MIXED, t).forward(other)[0]
    for cuts in ([n], [2] * (n // 2), [3, 5, 7] * 22, [1, 63, 1, 64, 65, 2, 31, 32, 33, 38], [128, 1, 1, 1, 127, 2, 70], [17] * 19 + [7], [n - 40] + [1] * 40):
        m.reset()
        assert close(feed(m, tokens, cuts), want, dtype, 2), cuts[:6]
        m.reset()  # a shorter request over what the long one left
        assert close(feed(m, other, [69, 1]), other_want, dtype, 2)
    m.close()


def test_prompt_chunks(ctx, mixed, monkeypatch):
    """A prompt longer than what goes through the layers at once: wanted places and layer outputs on both sides of every seam."""
    t, tokens, want, runs = mixed
    monkeypatch.setenv("AXQ_PROMPT_CHUNK", "50")
    m = gc.product(MIXED, t, "float32", ctx)
    places = [0, 48, 49, 50, 51, 99, 100, 149, 150, 151, 298, 300, 329]
    got, layers = m.forward_rows(tokens, places, layers=True)
    assert close(got, want[places], "float32", 2)
    assert np.abs(layers - runs).max() <= 2 * gc.LIMIT["float32"] * np.abs(runs).max()
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(ctx, mixed, dtype):
    t, tokens, want, _ = mixed
    m = gc.product(MIXED, t, dtype, ctx)
    assert close(feed(m, tokens, [1] * len(tokens)), want, dtype, 2)
    m.close()


def test_prompt_and_decoding_agree_to_rounding(ctx, mixed):
    t, tokens, _, _ = mixed
    m = gc.product(MIXED, t, "float32", ctx)
    a = feed(m, tokens, [len(tokens)])
    m.reset()
    b = feed(m, tokens, [1] * len(tokens))
    m.reset()
    assert gc.error(a, b).max() < 2 * gc.LIMIT["float32"]
    assert np.array_equal(feed(m, tokens, [len(tokens)]), a)  # the same cut again: the same bits
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_going_back(ctx, mixed, dtype):
    """A sequence cut short inside a block and continued otherwise: the block's means are those of the new tokens."""
    t, tokens, want, _ = mixed
    m = gc.product(MIXED, t, dtype, ctx)
    for keep in (3, 62, 64, 101):
        wrong = (tokens[keep:keep + 60] + 1) % MIXED["vocab"]
        for cuts in ([40, 20], [1] * 60):
            m.reset()
            feed(m, tokens[:keep], [keep])
            feed(m, wrong, cuts)
            m.truncate(keep)
            rest = tokens[keep:keep + 110]
            assert close(feed(m, rest, [1] * 30 + [80] if keep % 2 else [90] + [1] * 20), want[keep:keep + 110], dtype, 2), (keep, cuts[:2])
    m.close()


def test_cache_of_any_length(ctx, mixed):
    """A cache whose last block has no room, and none at all for blocks."""
    t, tokens, want, _ = mixed
    for positions in (1, 2, 6, 64, 65, 83):
        m = gc.product(MIXED, t, "bfloat16", ctx, positions)
        assert close(feed(m, tokens[:positions], [positions]), want[:positions], "bfloat16", 2)
        m.reset()
        assert close(feed(m, tokens[:positions], [1] * positions), want[:positions], "bfloat16", 2)
        m.close()


# ---- keys at chosen distances: one score stands out -----------------------------------------------------------------
def _pointing_model(dim, size, pool):
    """One attention layer whose only strong score is between token 1 (asks) and token 2 (answers), strong enough that a block
    of `pool` tokens with token 2 among them stands out as well.  The signal is in the dimensions that are not rotated."""
    cfg = one(heads=2, kv_heads=1, dim=dim, size=size, pool=pool, scale=1.0 / np.sqrt(dim), turn=gc.rot(dim // 2), width=64, vocab=40)
    t = gc.tensors(cfg, 31)
    rng = np.random.default_rng(1)
    # input channel 0 is on for token 1 alone and channel 1 for token 2; queries and keys read them strongly
    t["embed"][:, :gc.CLASSES] = 0.0
    t["embed"][1, 0] = t["embed"][2, 1] = 4.0
    t["l0.mix.q"] *= 0.25
    t["l0.mix.k"][dim // 2:] *= 0.1
    a = np.zeros(dim)
    a[dim // 2:] = rng.choice([-1.0, 1.0], dim - dim // 2)
    strength = np.sqrt(11.0 * pool / (16.0 * np.sqrt(dim) / 2.0))
    t["l0.mix.q"][:, 0] = gc.bf16(np.tile(strength * a, 2))
    t["l0.mix.k"][:, 1] = gc.bf16(strength * a)
    t["l0.mix.g"][:] = 0.0
    return cfg, {k: gc.bf16(v) for k, v in t.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,size,pool", [(32, 24, 4), (64, 64, 3), (128, 70, 6), (64, 7, 9), (36, 128, 2)])
def test_window_and_block_edges(ctx, dtype, dim, size, pool):
    """Token 2 at every place relative to its block and every distance special to the window, to its block's turn to be seen, or to
    the kernels' tiles: in a prompt's last row and as a decoded token."""
    cfg, t = _pointing_model(dim, size, pool)
    mask = cfg["layers"][0]["mixer"]["mask"]
    m = gc.product(cfg, t, dtype, ctx, 800)
    rng = np.random.default_rng(3)
    far_limit, kinds = 3 * gc.LIMIT["bfloat16"], set()
    for place in (0, 1, pool - 1, pool, 62 + pool % 2, 64, 131):
        turn = (place // pool + 1) * pool - 1 + size - place  # the distance at which the block is seen
        for d in sorted({1, size - 2, size - 1, size, size + 1, turn - 1, turn, turn + 1, turn + 63, turn + 64 * pool} - {0, -1}):
            tokens = rng.integers(3, cfg["vocab"], place + d + 1)
            tokens[place], tokens[-1] = 2, 1
            want = gc.oracle(cfg, t).forward(tokens)[0][-1:]
            without = tokens.copy()
            without[place] = 3
            far = gc.error(gc.oracle(cfg, t).forward(without)[0][-1:], want).max()
            tok, blk = plain.visible(place + d, mask)
            seen = place in tok or place // pool in blk
            kinds.add((place in tok, place // pool in blk))
            assert far > far_limit if seen else far == 0.0, "the key does not stand out"
            m.reset()
            assert close(m.forward_rows(tokens, [len(tokens) - 1]), want, dtype), (place, d)
            m.reset()
            m.forward_rows(tokens[:-1])
            assert close(m.feed(tokens[-1:], [0]), want, dtype), (place, d)
    assert kinds == {(True, False), (False, True), (False, False)}
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_blocks_made_while_decoding(ctx, dtype):
    """Token 2 is decoded, so is everything up to the token that asks for its block; and the same cut into twos."""
    cfg, t = _pointing_model(32, 11, 4)
    m = gc.product(cfg, t, dtype, ctx)
    rng = np.random.default_rng(4)
    for place in (0, 5, 63, 70):
        tokens = rng.integers(3, cfg["vocab"], place + 40)
        tokens[place] = 2
        tokens[place + 1:place + 40:3] = 1
        want = gc.oracle(cfg, t).forward(tokens)[0]
        for cuts in ([1] * len(tokens), [2] * (len(tokens) // 2) + [1] * (len(tokens) % 2)):
            m.reset()
            assert close(feed(m, tokens, cuts), want, dtype), (place, cuts[0])
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_blocks(ctx, dtype):
    """More blocks than one tile of them, the first tokens far outside the window, and a far key through its block."""
    cfg, t = _pointing_model(64, 33, 2)
    m = gc.product(cfg, t, dtype, ctx, 1200)
    tokens = np.random.default_rng(5).integers(3, cfg["vocab"], 900)
    tokens[7], tokens[400], tokens[410], tokens[899] = 2, 1, 2, 1
    want = gc.oracle(cfg, t).forward(tokens)[0]
    for cuts in ([900], [450, 450], [870] + [1] * 30):
        m.reset()
        assert close(feed(m, tokens, cuts), want, dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_far_out(ctx, dtype):
    """Positions beyond the original length, with a score that only the rotation makes."""
    cfg = one(heads=1, kv_heads=1, dim=16, size=300, pool=5, scale=2.0, turn=gc.rot(16, 40.0, {"factor": 4.0, "original": 50, "fast": 6.0, "slow": 0.7}))
    t = gc.tensors(cfg, 41)
    tokens = tokens_of(cfg, 260)
    want = gc.oracle(cfg, t).forward(tokens)[0]
    m = gc.product(cfg, t, dtype, ctx)
    assert close(feed(m, tokens, [200] + [1] * 60), want, dtype, 2)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_larger_sizes(ctx, dtype):
    """Sizes that take the big product tiles, the big tiles of grouped products, several row tiles and wide decode inputs."""
    cfg = gc.config([gc.attention(heads=8, kv_heads=2, dim=64, size=200, pool=16, scale=0.125, turn=gc.rot(32), mlp=gc.dense(4300)),
                     gc.attention(heads=8, kv_heads=2, dim=64, size=100, pool=32, scale=0.125, turn=gc.rot(64),
                                  mlp=gc.moe(experts=8, top=4, ff=700, groups=(4, 3), shared=600))], width=520, vocab=1000)
    t = gc.tensors(cfg, 61)
    tokens = tokens_of(cfg, 500)
    assert gc.margin(cfg, t, tokens) > 0.002
    want = gc.oracle(cfg, t).forward(tokens)[0]
    m = gc.product(cfg, t, dtype, ctx, 600)
    assert close(feed(m, tokens, [440, 57, 1, 1, 1]), want, dtype, 2)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_experts_alone(ctx, dtype):
    """Every expert's turn: with all other parts silent a token's logits are those of its experts."""
    cfg = one(mlp=gc.moe(experts=12, top=1, groups=(4, 2), shared=0))
    t = gc.tensors(cfg, 64)
    t["l0.mix.o"][:] = 0.0
    chosen, real = set(), plain.choose
    tokens = np.arange(cfg["vocab"])

    def watched(s, router):
        c = real(s, router)
        chosen.update(c)
        return c

    plain.choose = watched
    try:
        want = gc.oracle(cfg, t).forward(tokens)[0]
    finally:
        plain.choose = real
    assert len(chosen) >= 5 and gc.margin(cfg, t, tokens) > 0.002
    m = gc.product(cfg, t, dtype, ctx)
    assert close(feed(m, tokens, [60] + [1] * 41), want, dtype)
    m.close()


def test_graph_replays_follow_the_router(ctx, mixed):
    """The captured decode step takes the experts of every token anew, between other work."""
    t, tokens, want, _ = mixed
    m, other = gc.product(MIXED, t, "float32", ctx), gc.product(MIXED, t, "float32", ctx)
    for i in range(60):
        assert close(m.feed(tokens[i:i + 1], [0]), want[i:i + 1], "float32", 4), i
        if i % 7 == 0:
            other.reset()
            other.forward_rows(tokens[:20 + i])
    m.close()
    other.close()


# ---- entry points ---------------------------------------------------------------------------------------------------
def _greedy(cfg, t, prompt, n):
    """Greedy continuation by the plain forward; also the smallest gap between the two best logits."""
    m, out, gap = gc.oracle(cfg, t), [], np.inf
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
        m = gc.product(MIXED, t, "float32", ctx)
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
    m = gc.product(MIXED, t, "bfloat16", ctx)
    m.set_sampling(GenerationConfig(temperature=0.7, top_k=20, repetition_penalty=1.2), seed=3)
    a, _, _ = m.generate(tokens[:20], 30)
    m.reset()
    b, _, _ = m.generate(tokens[:20], 30)
    assert a.tolist() == b.tolist() and len(set(a.tolist())) > 3
    cfg = GenerationConfig(do_sample=False, repetition_penalty=1.5)
    m.set_sampling(cfg)
    m.reset()
    nxt, logits = m.forward_tokens(tokens[:20])
    assert nxt == TextGenerator(cfg, ctx).get_next_token(logits, tokens[:20])
    m.close()


def test_beam_search(ctx):
    """One beam is greedy; several, on a cache that is rewound between them, are those of the bookkeeping on the plain forward."""
    from axonml_amd.generation import BeamSearch, beam_search_generate

    cfg = gc.config([gc.attention(size=6, pool=2, mlp=gc.moe()), gc.attention(size=4, pool=3)])
    t = gc.tensors(cfg, 91)
    prompt = tokens_of(cfg, 11).tolist()
    bs = BeamSearch(3, 1.0, False, [])
    beams = bs.init_beams(prompt)
    for _ in range(6):
        beams = bs.expand_beams(beams, [gc.oracle(cfg, t).forward(b.tokens)[0][-1] for b in beams])
    m = gc.product(cfg, t, "float32", ctx)
    best, got = beam_search_generate(m, prompt, bs, 6)
    assert [b.tokens for b in got] == [b.tokens for b in beams] and best == bs.best_sequence(beams)
    m.reset()
    assert beam_search_generate(m, prompt, BeamSearch(1, 1.0, False, []), 6)[0][11:] == _greedy(cfg, t, prompt, 6)[0]
    m.close()


def test_cache_limit_and_refusals(ctx, mixed):
    from axonml_amd import gemosun
    from axonml_amd.quant import InvalidData, Overflow, QuantError, ShapeMismatch
    from axonml_amd.stack import StackModel

    t, tokens, want, _ = mixed
    m = gc.product(MIXED, t, "float32", ctx, 70)
    assert gc.error(feed(m, tokens[:70], [60] + [1] * 10), want[:70]).max() < 2 * gc.LIMIT["float32"]
    with pytest.raises(Overflow):
        m.forward(int(tokens[70]))
    with pytest.raises(Overflow):
        m.forward_rows(tokens[:2])
    m.truncate(0)
    with pytest.raises(ShapeMismatch):
        m.set_batch(2)
    with pytest.raises((QuantError, RuntimeError)):
        m.forward_rows([0, MIXED["vocab"]])
    with pytest.raises(InvalidData):  # true 32-bit takes bfloat16-exact weights only
        m.set_tensor(1, "mlp.e2.up", t["l1.mlp.e2.up"] * np.float32(1.0001))
    with pytest.raises(ShapeMismatch):
        m.set_tensor(0, "dwa", t["l1.dwa"])
    with pytest.raises((QuantError, RuntimeError)):
        m.set_tensor(1, "mlp.e6.up", t["l1.mlp.e2.up"])  # of experts 0 .. 5
    m.close()
    empty = StackModel(gemosun.describe(MIXED, 30), ctx=ctx)
    with pytest.raises(InvalidData):
        empty.forward(0)
    empty.close()
    for change in (dict(heads=5, kv_heads=2), dict(dim=300), dict(scale=0.0), dict(turn=gc.rot(26)), dict(mlp=gc.moe(experts=7)), dict(mlp=gc.moe(top=5)),
                   dict(mlp=gc.moe(groups=(3, 4)))):
        with pytest.raises(ShapeMismatch):
            StackModel(gemosun.describe(one(**change), 30), ctx=ctx)


def test_weights_set_again_are_used(ctx):
    """The captured step must not go on reading a replaced weight."""
    cfg = gc.config([gc.attention(mlp=gc.moe()), gc.attention(mlp=gc.dense())])
    t, other = gc.tensors(cfg, 81), gc.tensors(cfg, 82)
    tokens = tokens_of(cfg, 20)
    m = gc.product(cfg, t, "float32", ctx)
    feed(m, tokens, [10] + [1] * 10)
    for layer, name in ((0, "mix.q"), (0, "mlp.e3.down"), (0, "mlp.shared.up"), (0, "dwa"), (1, "mlp.gate"), (1, "mlp.up"), (-1, "head"), (0, "norm1")):
        full = name if layer < 0 else f"l{layer}.{name}"
        t[full] = other[full]
        m.set_tensor(layer, name, t[full])
    m.reset()
    assert gc.error(feed(m, tokens, [10] + [1] * 10), gc.oracle(cfg, t).forward(tokens)[0]).max() < 2 * gc.LIMIT["float32"]
    m.close()


def test_trace_program(tmp_path, mixed):
    """bin/trace_run on a checkpoint directory: portions, wanted places in any order, one request after the other."""
    t, tokens, want, _ = mixed
    write_checkpoint(str(tmp_path), MIXED, t)
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
    assert gc.error(read(0), want[[49, 0, 7]]).max() < 2 * gc.LIMIT["float32"]
    assert not (out / "1.f32").exists()
    assert gc.error(read(2), want[52:53]).max() < 2 * gc.LIMIT["float32"]
    assert gc.error(read(3), want[8:9]).max() < 2 * gc.LIMIT["float32"]


def test_command_line_generates(tmp_path, mixed):
    t, tokens, _, _ = mixed
    write_checkpoint(str(tmp_path), MIXED, t)
    want, gap = _greedy(MIXED, t, tokens[:6], 8)
    assert gap > 1e-3
    p = subprocess.run([sys.executable, "-m", "axonml_amd", "generate", "--model", str(tmp_path), "--dtype", "float32", "--tokens",
                        ",".join(str(x) for x in tokens[:6]), "--max-new-tokens", "8"], capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [int(x) for x in p.stdout.split()] == want
