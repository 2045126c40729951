"""Models of described layers (`axq_model_create_stack`): a `DecoderModel` whose layers are a list of descriptions, each
with a mixer of its own kind, its sizes and an optional feed-forward, some of them possibly run several times.

A design is a function from its configuration to `StackDescription` (see `axonml_amd/lakulix.py`); the stepping, the
sampling and the generation are those of every decode model.
"""
import ctypes as C
import dataclasses
from typing import List, Optional

import numpy as np

from . import _lib
from .decode import DecoderModel
from .quant import default_context

ATTENTION, LIGHTNING, WKV = 0, 1, 2
COMPUTE = {"bfloat16": 0, "float32": 1}


@dataclasses.dataclass
class LayerDescription:
    mixer: int
    heads: int
    dim: int
    vdim: int
    kv_heads: int = 1            # attention
    ff: int = 0                  # 0: no feed-forward sublayer
    bias_rows: int = 0           # attention: buckets of the distance bias, 0 for none
    bias_max: int = 0
    scale: float = 1.0           # attention
    q_temp_every: int = 0        # attention: 0 for no query factor
    q_temp_coef: float = 0.0
    decay_rank: int = 0          # wkv

    def to_c(self):
        return _lib.LayerConfig(mixer=self.mixer, heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, ff=self.ff,
                                bias_rows=self.bias_rows, bias_max=self.bias_max, q_temp_every=self.q_temp_every,
                                q_temp_coef=self.q_temp_coef, scale=self.scale, decay_rank=self.decay_rank)


@dataclasses.dataclass
class StackDescription:
    vocab_size: int
    width: int
    max_positions: int
    layers: List[LayerDescription]
    norm_eps: float
    logit_softcap: float = 0.0
    loop: Optional[tuple] = None  # (start, stop, times)


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
                               norm_eps=d.norm_eps, logit_softcap=d.logit_softcap, layers=layers)
        h = C.c_void_p()
        ctx.check(ctx.lib.axq_model_create_stack(ctx.handle, C.byref(cfg), C.byref(h)))
        super().__init__(ctx, h, d.vocab_size, d.width)
        self.can_rewind = all(l.mixer == ATTENTION for l in d.layers)

    def set_tensor(self, layer, name, data):
        """A weight by its name; layer -1 for those outside the layers."""
        a = np.ascontiguousarray(data, dtype=np.float32)
        rows, cols = (1, a.size) if a.ndim < 2 else a.shape
        self.ctx.check(self.ctx.lib.axq_model_set_tensor(self.handle, int(layer), name.encode(), a.ctypes.data, rows, cols))

    def random_init(self, std=0.02, seed=1):
        self.ctx.check(self.ctx.lib.axq_model_random_init(self.handle, 0, std, seed))
