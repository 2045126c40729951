"""Which class serves a checkpoint directory: config.json's architecture -> loader.

`load_model(path, ...)` reads the name from `architecture` or the first of `architectures` and calls the loader registered
for it: loader(path, dtype, max_positions, quant_type, ctx) -> DecoderModel.
"""
from .hf_loader import HFLoader, UnsupportedFormat, load_llama
from .quant import QuantType

_LOADERS = {}


def register(*architectures):
    def add(fn):
        for a in architectures:
            _LOADERS[a] = fn
        return fn
    return add


def architectures():
    return sorted(_LOADERS)


def architecture_of(cfg):
    name = cfg.get("architecture") or (cfg.get("architectures") or [None])[0]
    if name is None and cfg.get("model_type") in ("llama", "mistral"):
        name = cfg["model_type"].capitalize() + "ForCausalLM"
    return name


def load_model(path, dtype="bfloat16", max_positions=None, quant_type=None, ctx=None):
    """dtype: what a model kept in its checkpoint's format computes in; quant_type: the block type of models that are
    quantised as they are read; max_positions: the longest sequence to make room for (default: the model's own limit)."""
    name = architecture_of(HFLoader.from_local(path).load_config())
    if name not in _LOADERS:
        raise UnsupportedFormat(f"no model for architecture {name!r}: one of {architectures()}")
    return _LOADERS[name](path, dtype=dtype, max_positions=max_positions, quant_type=quant_type, ctx=ctx)


@register("LlamaForCausalLM", "MistralForCausalLM")
def _llama(path, dtype, max_positions, quant_type, ctx):
    if quant_type is None:
        quant_type = QuantType.F32 if dtype == "float32" else QuantType.Q4_K
    return load_llama(path, quant_type, ctx, max_positions)


@register("Lakulix")
def _lakulix(path, dtype, max_positions, quant_type, ctx):
    from .lakulix import load

    if quant_type not in (None, QuantType.BF16):
        raise UnsupportedFormat(f"Lakulix linears are kept in BF16, not {QuantType(quant_type)}")
    return load(path, dtype, max_positions, ctx)


@register("Gemosun")
def _gemosun(path, dtype, max_positions, quant_type, ctx):
    from .gemosun import load

    if quant_type not in (None, QuantType.BF16):
        raise UnsupportedFormat(f"Gemosun linears are kept in BF16, not {QuantType(quant_type)}")
    return load(path, dtype, max_positions, ctx)
