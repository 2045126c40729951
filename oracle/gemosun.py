"""Plain numpy float64 forward of a Gemosun model, one function per mechanism, one query at a time where attention is
concerned.  TEST INFRASTRUCTURE: shares nothing with the product path, not even its reading of config.json; `tensors` is a
dict of plain arrays under the checkpoint's names.
"""
import math

import numpy as np


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return np.maximum(z, 0.0) ** 2


def layer_norm(x, w, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w


def rotation(rot):
    """(frequency per pair, factor on cos and sin)."""
    n, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = np.array([base ** (-2.0 * i / n) for i in range(n // 2)])
    if not sc:
        return f, 1.0

    def where(turns):
        """The (real) dimension whose pair turns this often over the original length."""
        return n * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(where(sc["fast"])), 0), min(math.ceil(where(sc["slow"])), n - 1)
    ramp = np.clip((np.arange(n // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [T, heads, dim]: neighbours (2i, 2i + 1) of the first rot.dims dimensions turned by position times frequency."""
    if not rot:
        return x
    f, m = rotation(rot)
    a = np.asarray(positions, np.float64)[:, None, None] * f
    c, s = np.cos(a) * m, np.sin(a) * m
    n = rot["dims"]
    out = x.copy()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


def visible(i, mask):
    """(tokens, pooled blocks) that position i sees."""
    size, pool = mask["size"], mask["pool"]
    return [j for j in range(i + 1) if i - j < size], [b for b in range((i + 1) // pool + 1) if b * pool + pool - 1 <= i - size]


def pooled(x, b, pool):
    return x[b * pool:(b + 1) * pool].mean(axis=0)


def attention(h, mix, t, pre, past=None):
    """Softmax attention over a window of tokens and the means of the blocks before it; the values are the keys before
    rotation.  h [T, width]; past: (keys, values) of earlier tokens.  Returns (output, (keys, values) of everything so far)."""
    H, G, d = mix["heads"], mix["kv_heads"], mix["dim"]
    T = h.shape[0]
    n0 = 0 if past is None else past[0].shape[0]
    positions = n0 + np.arange(T)
    q = rotate((h @ t[pre + "q"].T).reshape(T, H, d), positions, mix.get("rot"))
    v = (h @ t[pre + "k"].T).reshape(T, G, d)
    k = rotate(v, positions, mix.get("rot"))
    if past is not None:
        k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
    gate = sigmoid(h @ t[pre + "g"].T)
    pool = mix["mask"]["pool"]
    nb = k.shape[0] // pool
    kp = np.array([pooled(k, b, pool) for b in range(nb)]).reshape(nb, G, d)
    vp = np.array([pooled(v, b, pool) for b in range(nb)]).reshape(nb, G, d)
    out = np.zeros((T, H, d))
    for i in range(T):
        tok, blk = visible(n0 + i, mix["mask"])
        ks, vs = np.concatenate([kp[blk], k[tok]]), np.concatenate([vp[blk], v[tok]])
        for hd in range(H):
            g = hd // (H // G)
            s = ks[:, g] @ q[i, hd] * mix["scale"]
            w = np.exp(s - s.max())
            out[i, hd] = (w / w.sum()) @ vs[:, g] * gate[i, hd]
    return out.reshape(T, H * d) @ t[pre + "o"].T, (k, v)


def choose(s, router):
    """Experts of one token, from its scores: the `top` best within the `keep` best groups."""
    n, groups = len(s), router.get("groups") or {"count": 1, "keep": 1}
    per = n // groups["count"]
    group_score = [np.sort(s[g * per:(g + 1) * per])[-2:].sum() for g in range(groups["count"])]
    kept = np.argsort(group_score)[::-1][:groups["keep"]]
    allowed = [e for e in range(n) if e // per in kept]
    return sorted(allowed, key=lambda e: -s[e])[:router["top"]]


def dense_ff(h, t, pre):
    return (gelu_tanh(h @ t[pre + "gate"].T) * (h @ t[pre + "up"].T)) @ t[pre + "down"].T


def expert(h, t, pre):
    return relu_squared(h @ t[pre + "up"].T) @ t[pre + "down"].T


def moe_ff(h, mlp, t, pre):
    s = sigmoid(h @ t[pre + "router"].T)
    out = np.zeros_like(h)
    for i in range(h.shape[0]):
        chosen = choose(s[i], mlp["router"])
        total = sum(s[i, e] for e in chosen) + 1e-20
        for e in chosen:
            out[i] += s[i, e] / total * expert(h[i], t, f"{pre}e{e}.")
    if mlp.get("shared"):
        out = out + sigmoid(h @ t[pre + "shared.sg"].T) * expert(h, t, pre + "shared.")
    return out


def depth_average(results, weights):
    """The embedding output and every layer's result so far, weighted."""
    return sum(w * x for w, x in zip(np.asarray(weights).reshape(-1), results))


class Model:
    """`forward` feeds tokens behind those already fed."""

    def __init__(self, config, tensors):
        self.c = config
        self.t = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.reset()

    def reset(self):
        self.state = [None] * len(self.c["layers"])
        self.n = 0

    def forward(self, tokens):
        """Returns (logits [T, vocab], residual stream after every layer [layers, T, width])."""
        c, t, eps = self.c, self.t, self.c["norm"]["eps"]
        x = t["embed"][tokens]
        results, stream = [x], []
        for i, layer in enumerate(c["layers"]):
            pre = f"l{i}."
            y, self.state[i] = attention(layer_norm(x, t[pre + "norm1"], eps), layer["mixer"], t, pre + "mix.", self.state[i])
            mlp = layer["mlp"]
            if mlp is not None:
                h = layer_norm(x, t[pre + "norm2"], eps)
                y = y + (moe_ff(h, mlp, t, pre + "mlp.") if mlp["kind"] == "moe" else dense_ff(h, t, pre + "mlp."))
            results.append(x + y)
            x = depth_average(results, t[pre + "dwa"])
            stream.append(x)
        self.n += len(tokens)
        return layer_norm(x, t["final.norm"], eps) @ t["head"].T, np.stack(stream)
