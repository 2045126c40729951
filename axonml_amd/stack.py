"""Models of described layers (`axq_model_create_stack`): a `DecoderModel` whose layers are a list of descriptions, each
with a mixer of its own kind, its sizes and an optional feed-forward, some of them possibly run several times.

A design is a function from its configuration to `StackDescription` (see `axonml_amd/lakulix.py`, `axonml_amd/gemosun.py`); the stepping, the
sampling and the generation are those of every decode model.
"""
import ctypes as C
import dataclasses
from typing import List, Optional

import numpy as np

from . import _lib
from .decode import DecoderModel
from .quant import default_context

ATTENTION, LIGHTNING, WKV, SOFTMAX = 0, 1, 2, 3
FF_POLY, FF_GLU, FF_MOE = 0, 1, 2
NORM_TANH, NORM_LAYER = 0, 1
COMPUTE = {"bfloat16": 0, "float32": 1}


@dataclasses.dataclass
class LayerDescription:
    mixer: int
    heads: int
    dim: int
    vdim: int
    kv_heads: int = 1            # attentions
    ff: int = 0                  # width of the feed-forward or of one expert; 0: no feed-forward
    bias_rows: int = 0           # attention: buckets of the distance bias, 0 for none
    bias_max: int = 0
    scale: float = 1.0           # attentions
    q_temp_every: int = 0        # attention: 0 for no query factor
    q_temp_coef: float = 0.0
    decay_rank: int = 0          # wkv

    window: int = 0              # softmax attention: tokens seen, 0 for all
    pool: int = 0                # softmax attention: tokens of a block seen as one before the window, 0 for none
    keys_as_values: int = 0      # softmax attention
    head_gate: int = 0           # softmax attention
    rot_dims: int = 0            # softmax attention: rotated dimensions
    rot_base: float = 10000.0
    rot_original: int = 0        # 0: frequencies as they are, else YaRN with the three below
    rot_factor: float = 1.0
    rot_fast: float = 0.0
    rot_slow: float = 0.0
    ff_kind: int = FF_POLY
    experts: int = 0             # mixture of experts
    top: int = 0
    groups: int = 0
    groups_keep: int = 0
    shared_ff: int = 0

    def to_c(self):
        return _lib.LayerConfig(**dataclasses.asdict(self))


@dataclasses.dataclass
class StackDescription:
    vocab_size: int
    width: int
    max_positions: int
    layers: List[LayerDescription]
    norm_eps: float
    logit_softcap: float = 0.0
    loop: Optional[tuple] = None  # (start, stop, times)
    norm: int = NORM_TANH
    position_table: bool = True
    parallel: bool = False
    depth_average: bool = False


class StackModel(DecoderModel):
    max_sequences = 1

    def __init__(self, description, dtype="bfloat16", cache_positions=None, ctx=None):
        ctx = ctx or default_context()
        self.description, self.dtype = description, dtype
        d = description
        layers = (_lib.LayerConfig * max(1, len(d.layers)))(*[l.to_c() for l in d.layers])
        start, stop, times = d.loop or (0, 0, 1)
        cfg = _lib.StackConfig(vocab_size=d.vocab_size, width=d.width, max_positions=d.max_positions, cache_positions=int(cache_positions or 0),
                               num_layers=len(d.layers), loop_start=start, loop_stop=stop, loop_times=times, compute=COMPUTE[dtype],
                               norm_eps=d.norm_eps, logit_softcap=d.logit_softcap, layers=layers, norm=d.norm,
                               position_table=int(d.position_table), parallel=int(d.parallel), depth_average=int(d.depth_average))
        h = C.c_void_p()
        ctx.check(ctx.lib.axq_model_create_stack(ctx.handle, C.byref(cfg), C.byref(h)))
        super().__init__(ctx, h, d.vocab_size, d.width)
        self.can_rewind = all(l.mixer in (ATTENTION, SOFTMAX) for l in d.layers)

    def set_tensor(self, layer, name, data):
        """A weight by its name; layer -1 for those outside the layers."""
        a = np.ascontiguousarray(data, dtype=np.float32)
        rows, cols = (1, a.size) if a.ndim < 2 else a.shape
        self.ctx.check(self.ctx.lib.axq_model_set_tensor(self.handle, int(layer), name.encode(), a.ctypes.data, rows, cols))

    def random_init(self, std=0.02, seed=1):
        self.ctx.check(self.ctx.lib.axq_model_random_init(self.handle, 0, std, seed))


def bench_rates(model, weights, bytes_per_weight, prompt, new_tokens):
    """Median of three: prompt and generation throughput of a model whose token passes `weights` linear weights."""
    model.generate(prompt, 4)
    model.reset()
    pre, dec = [], []
    for _ in range(3):
        _, p, d = model.generate(prompt, new_tokens)
        model.reset()
        pre.append(p)
        dec.append(d)
    pre_ms, dec_ms = sorted(pre)[1], sorted(dec)[1]
    tok_s = (new_tokens - 1) / (dec_ms * 1e-3)
    return {"prefill_tokens_per_s": len(prompt) / (pre_ms * 1e-3), "prefill_tflops": 2.0 * weights * len(prompt) / (pre_ms * 1e-3) / 1e12,
            "decode_tokens_per_s": tok_s, "decode_ms_per_token": 1e3 / tok_s, "decode_weight_gbps": weights * bytes_per_weight * tok_s / 1e9}


def bench_beside(ctx, width, weights, vocab, prompt, new_tokens):
    """The LLaMA-shape model of this width with as many layers as come nearest to `weights`, BF16 and Q4_K."""
    from .decode import QuantizedLlama
    from .quant import QuantType

    heads, ff = width // 128, width * 7 // 2
    kv = max(1, heads // 4)
    per_layer = width * (2 * width + 2 * kv * 128 + 3 * ff)
    n = max(1, round((weights - vocab * width) / per_layer))
    cfg = dict(vocab_size=vocab, hidden_size=width, intermediate_size=ff, num_hidden_layers=n, num_attention_heads=heads, num_key_value_heads=kv,
               head_dim=128, max_position_embeddings=len(prompt) + new_tokens, rms_norm_eps=1e-5, rope_theta=10000.0)
    lw, out = n * per_layer + vocab * width, {}
    for qt, bpw in ((QuantType.BF16, 2.0), (QuantType.Q4_K, 0.5625)):
        lm = QuantizedLlama(ctx, **cfg)
        lm.random_init(qt, 0.02, 1)
        out[f"llama_{str(qt).lower()}"] = dict(bench_rates(lm, lw, bpw, prompt, new_tokens), layers=n, linear_weights=lw)
        lm.close()
    return out
