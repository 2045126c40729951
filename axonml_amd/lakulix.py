"""Lakulix: a decoder whose layers are lightning attention, sigmoid-weighted attention with a distance bias, or
RWKV-style time mixing, in the order config.json lists them, a range of layers possibly looped.

config.json: `vocab`, `width`, `max_positions`, `layers` (each `type`, `mixer` sizes and constants, `mlp` or null), `loop`
(`start`, `stop`, `times`, or absent), `norm.eps`, `logit_softcap`.  Sizes that the file does not state come from the
tensors: the rows of the distance table, the rank of the decay.
"""
import numpy as np

from .hf_loader import HFLoader, UnsupportedFormat, WeightNotFound, set_embedding
from .quant import ShapeMismatch
from .stack import ATTENTION, LIGHTNING, WKV, LayerDescription, StackDescription, StackModel, bench_beside, bench_rates

_NORM = ("", ".b", ".alpha")
_MIXER_TENSORS = {
    ATTENTION: ("q", "k", "v", "q.norm", "k.norm", "pb", "o"),
    LIGHTNING: ("q", "k", "v", "g", "norm", "o"),
    WKV: ("mu.r", "mu.k", "mu.v", "mu.g", "mu.w", "r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o"),
}


def _describe_layer(i, layer, shape_of):
    kind, mix, mlp = layer["type"], layer["mixer"], layer.get("mlp")
    ff = 0
    if mlp is not None:
        if mlp.get("kind", "dense") != "dense":
            raise UnsupportedFormat(f"layer {i}: feed-forward of kind {mlp['kind']!r}")
        ff = int(mlp["ff"])
    heads, dim = int(mix["heads"]), int(mix["dim"])
    if kind == "attention":
        temp = mix.get("q_temp") or {"coef": 0.0, "every": 0}
        rel = shape_of(f"l{i}.mix.rel")
        return LayerDescription(ATTENTION, heads, dim, int(mix.get("vdim", dim)), kv_heads=int(mix.get("kv_heads", heads)), ff=ff,
                                bias_rows=int(rel[0]) if rel else 0, bias_max=int(mix.get("bias_max", 0)), scale=float(mix["scale"]),
                                q_temp_every=int(temp["every"]), q_temp_coef=float(temp["coef"]))
    if kind == "lightning":
        if len(mix["decay"]) != heads:
            raise ShapeMismatch(f"Shape mismatch: layer {i}: {len(mix['decay'])} decays for {heads} heads")
        return LayerDescription(LIGHTNING, heads, dim, int(mix.get("vdim", dim)), ff=ff)
    if kind == "wkv":
        w1 = shape_of(f"l{i}.mix.w1")
        if not w1:
            raise WeightNotFound(f"l{i}.mix.w1")
        return LayerDescription(WKV, heads, dim, dim, ff=ff, decay_rank=int(w1[0]))
    raise UnsupportedFormat(f"layer {i}: mixer {kind!r}")


def describe(cfg, shape_of):
    """config.json's contents -> StackDescription; shape_of(name): a tensor's shape, or None."""
    loop = cfg.get("loop")
    return StackDescription(vocab_size=int(cfg["vocab"]), width=int(cfg["width"]), max_positions=int(cfg["max_positions"]),
                            layers=[_describe_layer(i, l, shape_of) for i, l in enumerate(cfg["layers"])], norm_eps=float(cfg["norm"]["eps"]),
                            logit_softcap=float(cfg.get("logit_softcap") or 0.0),
                            loop=(int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else None)


def tensor_names(description):
    """(layer, name in the layer, checkpoint name) of every tensor but the embedding."""
    out = [(-1, "pos", "pos"), (-1, "head", "head")] + [(-1, "final.norm" + s, "final.norm" + s) for s in _NORM]
    for i, l in enumerate(description.layers):
        names = ["norm1" + s for s in _NORM] + ["mix." + n for n in _MIXER_TENSORS[l.mixer]]
        if l.mixer == ATTENTION and l.bias_rows:
            names.append("mix.rel")
        if l.ff:
            names += ["norm2" + s for s in _NORM] + ["mlp.up", "mlp.down", "mlp.act"]
        out += [(i, n, f"l{i}.{n}") for n in names]
    return out


def build(cfg, get, shape_of, dtype="bfloat16", cache_positions=None, ctx=None):
    """A model from config.json's contents and get(name) -> f32 array."""
    d = describe(cfg, shape_of)
    model = StackModel(d, dtype, cache_positions, ctx)
    set_embedding(model, get("embed"))
    for layer, name, full in tensor_names(d):
        model.set_tensor(layer, name, get(full))
    for i, l in enumerate(cfg["layers"]):
        if l["type"] == "lightning":
            model.set_tensor(i, "mix.decay", np.asarray(l["mixer"]["decay"], dtype=np.float32))
    return model


def load(path, dtype="bfloat16", cache_positions=None, ctx=None):
    loader = HFLoader.from_local(path)
    cfg = loader.load_config()
    loader.load_tensors()
    return build(cfg, loader.get_tensor, loader.shape, dtype, cache_positions, ctx)


# ---------------------------------------------------------------------------------------------------------------------
# Benchmark: random weights at sizes that resemble a real model's layers, beside the LLaMA-shape model of equal size.
# ---------------------------------------------------------------------------------------------------------------------
def bench_description(width, n_blocks, positions, vocab=32000):
    """Blocks of lightning, attention + feed-forward, time mixing, attention + feed-forward, at LLaMA-like proportions."""
    ff, heads = width * 7 // 2, width // 128
    att = LayerDescription(ATTENTION, heads, 128, 128, kv_heads=max(1, heads // 4), ff=ff, bias_rows=32, bias_max=128, scale=128 ** -0.5,
                           q_temp_every=1024, q_temp_coef=0.1)
    block = [LayerDescription(LIGHTNING, heads, 128, 128), att, LayerDescription(WKV, width // 64, 64, 64, decay_rank=64), att]
    return StackDescription(vocab_size=vocab, width=width, max_positions=positions, layers=block * n_blocks, norm_eps=1e-5, logit_softcap=30.0)


def linear_weights(d):
    """Elements of all linears a token passes, the head included."""
    total = d.vocab_size * d.width
    for l in d.layers:
        out = l.heads * l.vdim
        if l.mixer == ATTENTION:
            n = l.heads * l.dim + l.kv_heads * (l.dim + l.vdim)
        elif l.mixer == LIGHTNING:
            n = 2 * l.heads * l.dim + 2 * out
        else:
            n = 4 * l.heads * l.dim + l.decay_rank * (1 + l.heads * l.dim // d.width)
        total += d.width * (n + out + 2 * l.ff)
    return total


def bench(ctx, log=print, widths=(1024, 2048, 4096), blocks=2, prompt_len=2048, new_tokens=128, beside=True):
    out = []
    for width in widths:
        d = bench_description(width, blocks, prompt_len + new_tokens)
        weights = linear_weights(d)
        prompt = np.random.default_rng(0).integers(0, d.vocab_size, size=prompt_len, dtype=np.int32)
        m = StackModel(d, ctx=ctx)
        m.random_init(0.02, 1)
        r = {"width": width, "layers": len(d.layers), "linear_weights": weights, "prompt_tokens": prompt_len, "generated_tokens": new_tokens,
             "lakulix_bf16": bench_rates(m, weights, 2.0, prompt, new_tokens)}
        m.close()
        if beside:
            r.update(bench_beside(ctx, width, weights, d.vocab_size, prompt, new_tokens))
        for name, v in r.items():
            if isinstance(v, dict):
                log(f"  width {width} {name}: prefill {v['prefill_tokens_per_s']:.0f} tok/s ({v['prefill_tflops']:.0f} TFLOP/s), decode "
                    f"{v['decode_tokens_per_s']:.0f} tok/s ({v['decode_ms_per_token']:.3f} ms, {v['decode_weight_gbps']:.0f} GB/s of weights)")
        out.append(r)
    return out
