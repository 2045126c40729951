"""What the tests of models of described layers share: bfloat16-exact weights, the measure of error, checkpoints on disk."""
import json
import os
import struct

import numpy as np


def bf16(x):
    """Rounded to bfloat16 (nearest even), as f32."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32).astype(np.uint64)
    return (((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16).astype(np.uint32).view(np.float32).reshape(np.shape(x))


def error(got, want):
    """Per position: rms of the difference over the vocabulary (mean taken off), relative to the typical spread of the logits."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d -= d.mean(-1, keepdims=True)
    scale = np.sqrt(np.mean((want - want.mean(-1, keepdims=True)) ** 2))
    return np.sqrt((d * d).mean(-1)) / scale


# f32: accumulation noise of a few layers over some hundred terms.  bf16: rounding of the products' inputs to 8 bits.
LIMIT = {"float32": 2e-5, "bfloat16": 3e-2}


def write_checkpoint(path, cfg, t):
    """config.json and model.safetensors (bfloat16) in the directory `path`."""
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, a in t.items():
        b = (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    head = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(blobs))


def close(got, want, dtype, layers=1):
    """f32: every position.  bfloat16: nearly all of them, and none far off (sums over many keys can nearly cancel, and then a
    position answers to rounding with several times the usual error)."""
    e, limit = error(got, want), LIMIT[dtype] * layers
    return e.max() < limit if dtype == "float32" else np.quantile(e, 0.97) < limit and e.max() < 3 * limit


def tokens_of(cfg, n, seed=5):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n)


def feed(model, tokens, cuts):
    """All logits, the tokens cut into portions."""
    at, out = 0, []
    for n in cuts:
        out.append(model.feed(tokens[at:at + n], list(range(n))))
        at += n
    assert at == len(tokens)
    return np.concatenate(out)
