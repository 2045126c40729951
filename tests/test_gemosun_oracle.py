"""The plain Gemosun forward, on the CPU: it does not depend on how its tokens are cut, and every mechanism of the design
shows in the logits of the test models (a mistake planted in the plain forward is far beyond the tolerances the product is
held to); and how the product reads config.json."""
import copy

import numpy as np
import pytest

from . import gemosun_common as gc
from oracle import gemosun as plain

CFG = gc.config([gc.attention(mlp=gc.dense()), gc.attention(heads=6, kv_heads=3, size=17, pool=4, mlp=gc.moe()), gc.attention(),
                 gc.attention(heads=2, kv_heads=1, mlp=gc.moe(experts=8, top=3, groups=(2, 1)))])


@pytest.fixture(scope="module")
def case():
    t = gc.tensors(CFG, 1)
    tokens = np.random.default_rng(2).integers(0, CFG["vocab"], 90)
    return t, tokens, gc.oracle(CFG, t).forward(tokens)[0]


@pytest.mark.parametrize("cuts", [[1] * 90, [2] * 45, [30, 1, 1, 58], [89, 1]])
def test_plain_forward_does_not_depend_on_the_cuts(case, cuts):
    t, tokens, whole = case
    m, at, out = gc.oracle(CFG, t), 0, []
    for n in cuts:
        out.append(m.forward(tokens[at:at + n])[0])
        at += n
    assert gc.error(np.concatenate(out), whole).max() < 1e-11


def test_test_models_keep_away_from_close_choices(case):
    t, tokens, _ = case
    assert gc.margin(CFG, t, tokens) > 0.004


def _choose_without_groups(s, router, real=plain.choose):
    return real(s, {"top": router["top"]})


def _wide_window(i, mask, real=plain.visible):
    return real(i, {"size": mask["size"] + 1, "pool": mask["pool"]})[0], real(i, mask)[1]


def _early_blocks(i, mask, real=plain.visible):
    return real(i, mask)[0], real(i + 1, mask)[1]


def _late_blocks(i, mask, real=plain.visible):
    return real(i, mask)[0], real(i - 1, mask)[1] if i else []


MISTAKES = {
    "window": lambda mp: mp.setattr(plain, "visible", _wide_window),
    "blocks one token early": lambda mp: mp.setattr(plain, "visible", _early_blocks),
    "blocks one token late": lambda mp: mp.setattr(plain, "visible", _late_blocks),
    "no blocks": lambda mp: mp.setattr(plain, "visible", lambda i, mask, real=plain.visible: (real(i, mask)[0], [])),
    "blocks summed": lambda mp: mp.setattr(plain, "pooled", lambda x, b, pool: x[b * pool:(b + 1) * pool].sum(axis=0)),
    "groups": lambda mp: mp.setattr(plain, "choose", _choose_without_groups),
    "size of the rotation": lambda mp: mp.setattr(plain, "rotation", lambda r, real=plain.rotation: (real(r)[0], 1.0)),
    "frequencies as they are": lambda mp: mp.setattr(plain, "rotation", lambda r, real=plain.rotation: (real({**r, "scaling": None})[0], real(r)[1])),
    "gelu": lambda mp: mp.setattr(plain, "gelu_tanh", lambda z: z * plain.sigmoid(1.702 * z)),
    "relu": lambda mp: mp.setattr(plain, "relu_squared", lambda z: np.maximum(z, 0.0)),
    "mean in the norm": lambda mp: mp.setattr(plain, "layer_norm", lambda x, w, eps: x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w),
    "mean over the layers": lambda mp: mp.setattr(plain, "depth_average", lambda results, w: results[-1]),
}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_a_mistake_in_a_mechanism_shows(case, monkeypatch, name):
    t, tokens, whole = case
    MISTAKES[name](monkeypatch)
    e = gc.error(gc.oracle(CFG, t).forward(tokens)[0], whole)
    # (gelu's two approximations are near each other everywhere; a block early or late touches one position in `pool`)
    far = 20 * gc.LIMIT["float32"] if name == "gelu" else gc.LIMIT["bfloat16"] / 3
    assert np.median(e) > 10 * gc.LIMIT["float32"] and e.max() > far


@pytest.mark.parametrize("tensor,change", [("l0.mix.g", 0.0), ("l1.mlp.shared.sg", 0.0), ("l0.dwa", 0.5), ("l3.dwa", 0.5), ("l0.norm1", 1.0), ("l0.norm2", 1.0),
                                           ("l2.norm1", 1.0), ("final.norm", 1.0), ("l3.mlp.router", 0.1), ("l1.mlp.shared.down", 0.0)])
def test_every_small_tensor_shows(case, tensor, change):
    t, tokens, whole = case
    other = dict(t)
    other[tensor] = np.full_like(t[tensor], change)
    assert np.median(gc.error(gc.oracle(CFG, other).forward(tokens)[0], whole)) > gc.LIMIT["bfloat16"]


def test_description_and_names():
    from axonml_amd import gemosun

    d = gemosun.describe(CFG)
    t = gc.tensors(CFG, 1)
    assert {full for _, _, full in gemosun.tensor_names(d)} | {"embed"} == set(t)
    assert d.max_positions == 240 and gemosun.describe(CFG, 77).max_positions == 77
    assert [l.window for l in d.layers] == [23, 17, 23, 23] and [l.pool for l in d.layers] == [5, 4, 5, 5]
    assert [l.ff for l in d.layers] == [40, 20, 0, 20] and [l.shared_ff for l in d.layers] == [0, 28, 0, 28]
    plain_layers = gc.config([gc.attention(turn=None, mlp=gc.moe(groups=None, shared=0))])
    d = gemosun.describe(plain_layers)
    l = d.layers[0]
    assert (l.rot_dims, l.groups, l.groups_keep, l.shared_ff) == (0, 1, 1, 0) and d.max_positions == gemosun.DEFAULT_POSITIONS
    assert {full for _, _, full in gemosun.tensor_names(d)} | {"embed"} == set(gc.tensors(plain_layers, 1))


def test_what_the_design_does_not_have_is_refused():
    from axonml_amd import gemosun
    from axonml_amd.hf_loader import UnsupportedFormat
    from axonml_amd.quant import ShapeMismatch

    for path, value, error in ((("type",), "lightning", UnsupportedFormat), (("mlp", "kind"), "poly", UnsupportedFormat), (("mixer", "vdim"), 8, ShapeMismatch)):
        cfg = copy.deepcopy(CFG)
        at = cfg["layers"][0]
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        with pytest.raises(error):
            gemosun.describe(cfg)


def test_registry_knows_the_design():
    from axonml_amd import registry

    assert "Gemosun" in registry.architectures() and registry.architecture_of(CFG) == "Gemosun"
