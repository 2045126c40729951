"""The plain Lakulix forward, on the CPU: it does not depend on how its tokens are cut, and every mechanism of the design
shows in the logits of the test models (a mistake planted in the plain forward is far beyond the tolerances the product is
held to)."""
import json

import numpy as np
import pytest

from . import lakulix_common as lc
from oracle import lakulix as plain

CFG = lc.config([lc.lightning(ff=56), lc.attention(ff=40), lc.wkv(), lc.attention(heads=2, kv_heads=1, dim=8, vdim=20)],
                loop={"start": 1, "stop": 3, "times": 2})


@pytest.fixture(scope="module")
def case():
    t = lc.tensors(CFG, 1)
    tokens = np.random.default_rng(2).integers(0, CFG["vocab"], 90)
    return t, tokens, lc.oracle(CFG, t).forward(tokens)[0]


@pytest.mark.parametrize("cuts", [[1] * 90, [2] * 45, [30, 1, 1, 58], [89, 1]])
def test_plain_forward_does_not_depend_on_the_cuts(case, cuts):
    t, tokens, whole = case
    m, at, out = lc.oracle(CFG, t), 0, []
    for n in cuts:
        out.append(m.forward(tokens[at:at + n])[0])
        at += n
    assert lc.error(np.concatenate(out), whole).max() < 1e-12


def _bucket_off_by_one(n, rows, dmax, real=plain.distance_bucket):
    return real(max(0, n - 1), rows, dmax)


MISTAKES = {
    "bucket": lambda mp: mp.setattr(plain, "distance_bucket", _bucket_off_by_one),
    "query factor": lambda mp: mp.setattr(plain, "query_temperature", lambda p, coef, every: 1.0),
    "query factor one step late": lambda mp: mp.setattr(plain, "query_temperature", lambda p, c, e: 1.0 + c * np.log(p // e + 1.0)),
    "poly norm constant": lambda mp: mp.setattr(plain, "poly_norm", lambda z, c, eps, real=plain.poly_norm: real(z, c, eps) - float(c[3])),
    "tanh norm": lambda mp: mp.setattr(plain, "dynamic_tanh", lambda x, a, w, b: np.tanh(a * x) * w),
}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_a_mistake_in_a_mechanism_shows(case, monkeypatch, name):
    t, tokens, whole = case
    MISTAKES[name](monkeypatch)
    e = lc.error(lc.oracle(CFG, t).forward(tokens)[0], whole)
    # (a late step of the query factor touches only the positions where it steps and what follows them)
    assert np.sort(e)[len(e) // 2] > 10 * lc.LIMIT["float32"] and e.max() > lc.LIMIT["bfloat16"] / 3


@pytest.mark.parametrize("tensor,change", [("l2.mix.u", 0.0), ("l2.mix.mu.w", 0.0), ("l2.mix.mu.r", 0.0), ("l2.mix.norm", 1.0), ("l0.mix.norm", 1.0),
                                           ("l1.mix.pb", -3.0), ("pos", 0.0), ("l1.mix.q.norm", 1.0), ("l1.mix.k.norm", 1.0), ("l0.mlp.act", 0.5)])
def test_every_small_tensor_shows(case, tensor, change):
    t, tokens, whole = case
    other = dict(t)
    other[tensor] = np.full_like(t[tensor], change)
    assert lc.error(lc.oracle(CFG, other).forward(tokens)[0], whole).max() > 50 * lc.LIMIT["float32"]


def test_passes_of_a_loop_keep_states_of_their_own(case):
    t, tokens, whole = case
    m = lc.oracle(CFG, t)
    m.forward(tokens[:40])
    m.state[3] = m.state[1]  # the second pass reads the first one's cache
    m.state[4] = m.state[2]
    assert lc.error(m.forward(tokens[40:])[0], whole[40:]).max() > 50 * lc.LIMIT["float32"]


def test_distance_buckets():
    # exact up to half the rows, every row used, the last one from 12 * 8^(11/12) = 80.7 on
    b = [plain.distance_bucket(n, 24, 96) for n in range(200)]
    assert b[:12] == list(range(12)) and b == sorted(b) and set(b) == set(range(24))
    assert b[80] == 22 and b[81] == 23 and b[199] == 23
    assert plain.distance_bucket(24, 24, 96) == 16 and plain.distance_bucket(23, 24, 96) == 15  # 12 * 8^(4/12) = 24: an edge


def test_description_follows_config_and_shapes():
    from axonml_amd import lakulix
    from axonml_amd.stack import ATTENTION, LIGHTNING, WKV

    t = lc.tensors(CFG, 1, bias_rows=10, rank=7)
    d = lakulix.describe(json.loads(json.dumps(CFG)), lambda n: list(t[n].shape) if n in t else None)
    assert [l.mixer for l in d.layers] == [LIGHTNING, ATTENTION, WKV, ATTENTION]
    assert (d.vocab_size, d.width, d.max_positions, d.loop) == (101, 72, 400, (1, 3, 2))
    assert d.layers[1].bias_rows == 10 and d.layers[1].bias_max == 40 and d.layers[2].decay_rank == 7
    assert [l.ff for l in d.layers] == [56, 40, 0, 0]
    assert {n for _, _, n in lakulix.tensor_names(d)} | {"embed"} == set(t)
    plain_cfg = dict(CFG, loop=None, logit_softcap=None)
    d = lakulix.describe(plain_cfg, lambda n: list(t[n].shape) if n in t else None)
    assert d.loop is None and d.logit_softcap == 0.0


def test_registry_names_and_refusals(tmp_path):
    from axonml_amd import registry
    from axonml_amd.hf_loader import UnsupportedFormat

    assert {"Lakulix", "LlamaForCausalLM", "MistralForCausalLM"} <= set(registry.architectures())
    assert registry.architecture_of({"architectures": ["LlamaForCausalLM"]}) == "LlamaForCausalLM"
    assert registry.architecture_of({"model_type": "mistral"}) == "MistralForCausalLM"
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Unheard"}))
    with pytest.raises(UnsupportedFormat):
        registry.load_model(str(tmp_path))


def test_replay_feeds_and_ends_requests(tmp_path):
    from axonml_amd import trace

    class Fake:
        vocab_size = 3
        log = []

        def reset(self):
            self.log.append("reset")

        def feed(self, tokens, want):
            self.log.append((tuple(tokens), tuple(want)))
            return np.array([[t, t + 1, t + 2] for t in (tokens[w] for w in want)], np.float32).reshape(-1, 3)

    lines = ['{"step": 0, "entries": [{"id": "a", "tokens": [5, 7, 3], "want": [2, 0]}], "end": []}',
             '{"step": 1, "entries": [{"id": "a", "tokens": [9], "want": []}], "end": ["a"]}', "",
             '{"step": 2, "entries": [{"id": "b", "tokens": [4], "want": [0]}], "end": ["b"]}']
    said = []
    trace.run(Fake(), lines, str(tmp_path), said.append)
    assert said == ["done 0", "done 1", "done 2"]
    assert np.array_equal(np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, 3), [[3, 4, 5], [5, 6, 7]])
    assert not (tmp_path / "1.f32").exists()
    assert np.array_equal(np.fromfile(tmp_path / "2.f32", "<f4"), [4, 5, 6])
    assert Fake.log == ["reset", ((5, 7, 3), (0, 2)), ((9,), ()), "reset", "reset", ((4,), (0,)), "reset"]
    with pytest.raises(ValueError):
        trace.run(Fake(), [lines[0], lines[3]], str(tmp_path), said.append)
