"""Gemosun: a decoder of parallel layers (attention and feed-forward read two layer norms of the same stream) with softmax
attention over a sliding window of tokens and the means of the blocks before it, values that are the unrotated keys, partial
rotary positions (plain or YaRN), gated heads, dense GLU feed-forwards or grouped mixtures of experts, and a weighted mean
over all layers' results after every layer.

config.json: `vocab`, `width`, `layers` (each `type`, `mixer` sizes and constants, `mlp` or null), `norm.eps`.
"""
import numpy as np

from .hf_loader import HFLoader, UnsupportedFormat, set_embedding
from .quant import ShapeMismatch
from .stack import FF_GLU, FF_MOE, NORM_LAYER, SOFTMAX, LayerDescription, StackDescription, StackModel, bench_beside, bench_rates

DEFAULT_POSITIONS = 4096  # of a model that states no original length of its rotation


def _rotation(i, rot):
    if not rot:
        return {}
    out = dict(rot_dims=int(rot["dims"]), rot_base=float(rot["base"]))
    scaling = rot.get("scaling")
    if scaling:
        out.update(rot_original=int(scaling["original"]), rot_factor=float(scaling["factor"]), rot_fast=float(scaling["fast"]),
                   rot_slow=float(scaling["slow"]))
    return out


def _feed_forward(i, mlp):
    if mlp is None:
        return {}
    kind = mlp.get("kind", "dense")
    if kind == "dense":
        return dict(ff=int(mlp["ff"]), ff_kind=FF_GLU)
    if kind != "moe":
        raise UnsupportedFormat(f"layer {i}: feed-forward of kind {kind!r}")
    router = mlp["router"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    shared = mlp.get("shared")
    return dict(ff=int(mlp["expert"]["ff"]), ff_kind=FF_MOE, experts=int(router["experts"]), top=int(router["top"]), groups=int(groups["count"]),
                groups_keep=int(groups["keep"]), shared_ff=int(shared["ff"]) if shared else 0)


def _describe_layer(i, layer):
    if layer["type"] != "attention":
        raise UnsupportedFormat(f"layer {i}: mixer {layer['type']!r}")
    mix = layer["mixer"]
    heads, dim = int(mix["heads"]), int(mix["dim"])
    vdim = int(mix.get("vdim", dim))
    if vdim != dim:
        raise ShapeMismatch(f"Shape mismatch: layer {i}: values of {vdim} that are keys of {dim}")
    mask = mix.get("mask") or {}
    return LayerDescription(SOFTMAX, heads, dim, vdim, kv_heads=int(mix.get("kv_heads", heads)), scale=float(mix["scale"]),
                            window=int(mask.get("size") or 0), pool=int(mask.get("pool") or 0), keys_as_values=1, head_gate=1,
                            **_rotation(i, mix.get("rot")), **_feed_forward(i, layer.get("mlp")))


def default_positions(layers):
    """The longest sequence the rotations are made for."""
    reach = [int(l.rot_original * l.rot_factor) for l in layers if l.rot_original]
    return max(reach) if reach else DEFAULT_POSITIONS


def describe(cfg, positions=None):
    """config.json's contents -> StackDescription for sequences of up to `positions` tokens."""
    layers = [_describe_layer(i, l) for i, l in enumerate(cfg["layers"])]
    return StackDescription(vocab_size=int(cfg["vocab"]), width=int(cfg["width"]), max_positions=int(positions or default_positions(layers)),
                            layers=layers, norm_eps=float(cfg["norm"]["eps"]), norm=NORM_LAYER, position_table=False, parallel=True,
                            depth_average=True)


def tensor_names(description):
    """(layer, name in the layer, checkpoint name) of every tensor but the embedding."""
    out = [(-1, "final.norm", "final.norm"), (-1, "head", "head")]
    for i, l in enumerate(description.layers):
        names = ["norm1", "mix.q", "mix.k", "mix.g", "mix.o", "dwa"]
        if l.ff:
            names.append("norm2")
            if l.ff_kind == FF_MOE:
                names += [f"mlp.e{e}.{w}" for e in range(l.experts) for w in ("up", "down")] + ["mlp.router"]
                if l.shared_ff:
                    names += ["mlp.shared.up", "mlp.shared.down", "mlp.shared.sg"]
            else:
                names += ["mlp.gate", "mlp.up", "mlp.down"]
        out += [(i, n, f"l{i}.{n}") for n in names]
    return out


def build(cfg, get, dtype="bfloat16", positions=None, ctx=None):
    """A model from config.json's contents and get(name) -> f32 array."""
    d = describe(cfg, positions)
    model = StackModel(d, dtype, None, ctx)
    set_embedding(model, get("embed"))
    for layer, name, full in tensor_names(d):
        model.set_tensor(layer, name, get(full))
    return model


def load(path, dtype="bfloat16", positions=None, ctx=None):
    loader = HFLoader.from_local(path)
    cfg = loader.load_config()
    loader.load_tensors()
    return build(cfg, loader.get_tensor, dtype, positions, ctx)


# ---------------------------------------------------------------------------------------------------------------------
# Benchmark: random weights at sizes that resemble a real model's layers, beside the LLaMA-shape model of equal size.
# ---------------------------------------------------------------------------------------------------------------------
def bench_description(width, n_layers, positions, vocab=32000):
    """One dense layer, then mixtures of 16 experts in 4 groups, 4 per token, and a shared one, at LLaMA-like proportions."""
    heads = width // 128
    mix = dict(kv_heads=max(1, heads // 4), scale=128 ** -0.5, window=1024, pool=64, keys_as_values=1, head_gate=1, rot_dims=64, rot_base=10000.0,
               rot_original=1024, rot_factor=4.0, rot_fast=32.0, rot_slow=1.0)
    dense = LayerDescription(SOFTMAX, heads, 128, 128, ff=width * 7 // 2, ff_kind=FF_GLU, **mix)
    moe = LayerDescription(SOFTMAX, heads, 128, 128, ff=width, ff_kind=FF_MOE, experts=16, top=4, groups=4, groups_keep=2, shared_ff=width, **mix)
    return StackDescription(vocab_size=vocab, width=width, max_positions=positions, layers=[dense] + [moe] * (n_layers - 1), norm_eps=1e-5,
                            norm=NORM_LAYER, position_table=False, parallel=True, depth_average=True)


def linear_weights(d):
    """Elements of all linears a token passes, the head included."""
    total = d.vocab_size * d.width
    for l in d.layers:
        n = 2 * l.heads * l.dim + l.kv_heads * l.dim + l.heads
        if l.ff_kind == FF_MOE:
            n += l.experts + 2 * (l.top * l.ff + l.shared_ff)
        else:
            n += 3 * l.ff
        total += d.width * n
    return total


def bench(ctx, log=print, widths=(1024, 2048, 4096), n_layers=6, prompt_len=2048, new_tokens=128, beside=True):
    out = []
    for width in widths:
        d = bench_description(width, n_layers, prompt_len + new_tokens)
        weights = linear_weights(d)
        prompt = np.random.default_rng(0).integers(0, d.vocab_size, size=prompt_len, dtype=np.int32)
        m = StackModel(d, ctx=ctx)
        m.random_init(0.02, 1)
        r = {"width": width, "layers": len(d.layers), "linear_weights": weights, "prompt_tokens": prompt_len, "generated_tokens": new_tokens,
             "gemosun_bf16": bench_rates(m, weights, 2.0, prompt, new_tokens)}
        m.close()
        if beside:
            r.update(bench_beside(ctx, width, weights, d.vocab_size, prompt, new_tokens))
        for name, v in r.items():
            if isinstance(v, dict):
                log(f"  width {width} {name}: prefill {v['prefill_tokens_per_s']:.0f} tok/s ({v['prefill_tflops']:.0f} TFLOP/s), decode "
                    f"{v['decode_tokens_per_s']:.0f} tok/s ({v['decode_ms_per_token']:.3f} ms, {v['decode_weight_gbps']:.0f} GB/s of weights)")
        out.append(r)
    return out
