"""Plain numpy float64 forward of a Lakulix model, one function per mechanism, one token at a time where
the mechanism is a recurrence.  TEST INFRASTRUCTURE: shares nothing with the product path, not even its
reading of config.json; `tensors` is a dict of plain arrays under the checkpoint's names.
"""
import math

import numpy as np


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def silu(z):
    return z * sigmoid(z)


def rms_norm(x, eps):
    """x divided by its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def dynamic_tanh(x, alpha, w, b):
    return np.tanh(alpha * x) * w + b


def poly_norm(z, coef, eps):
    a, b, c, e = (float(v) for v in np.asarray(coef).reshape(-1))
    return a * rms_norm(z, eps) + b * rms_norm(z * z, eps) + c * rms_norm(z * z * z, eps) + e


def distance_bucket(n, rows, dmax):
    """Row of the learned distance table for a key `n` tokens back: exact below rows/2, then logarithmic up to `dmax`."""
    half = rows // 2
    if n < half:
        return n
    v = math.log(n / half) / math.log(dmax / half) * (rows - half)
    near = round(v)
    return min(rows - 1, half + (near if abs(v - near) < 1e-9 else math.floor(v)))


def query_temperature(p, coef, every):
    return 1.0 + coef * math.log(math.floor((p + 1) / every) + 1.0)


def attention(h, mix, t, pre, eps, past=None):
    """Causal attention whose weights are sigmoids of the scores, not normalised over the keys.  h: [T, width], the
    layer's normed input; `past`: (k, v) of earlier tokens.  Returns (output, (k, v) of everything so far)."""
    H, G, d, dv = mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]
    T = h.shape[0]
    q = (h @ t[pre + "q"].T).reshape(T, H, d)
    k = (h @ t[pre + "k"].T).reshape(T, G, d)
    v = (h @ t[pre + "v"].T).reshape(T, G, dv)
    q = rms_norm(q, eps) * t[pre + "q.norm"]
    k = rms_norm(k, eps) * t[pre + "k.norm"]
    if past is not None:
        k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
    n0 = k.shape[0] - T
    rel, pb = t[pre + "rel"], t[pre + "pb"]
    bucket = np.array([distance_bucket(n, rel.shape[0], mix["bias_max"]) for n in range(k.shape[0])])
    temp = mix.get("q_temp")
    out = np.zeros((T, H, dv))
    for i in range(T):
        p = n0 + i
        qi = q[i] * (query_temperature(p, temp["coef"], temp["every"]) if temp else 1.0)
        for hd in range(H):
            g = hd // (H // G)
            s = k[:p + 1, g] @ qi[hd] * mix["scale"] + rel[bucket[p - np.arange(p + 1)], hd]
            out[i, hd] = sigmoid(s + pb[hd]) @ v[:p + 1, g]
    return out.reshape(T, H * dv) @ t[pre + "o"].T, (k, v)


def lightning(h, mix, t, pre, eps, S=None):
    """Linear attention with one constant decay per head; returns (output, state [heads, dim, vdim])."""
    H, d, dv = mix["heads"], mix["dim"], mix["vdim"]
    T = h.shape[0]
    q = silu(h @ t[pre + "q"].T).reshape(T, H, d)
    k = silu(h @ t[pre + "k"].T).reshape(T, H, d)
    v = silu(h @ t[pre + "v"].T).reshape(T, H, dv)
    decay = np.asarray(mix["decay"], np.float64)
    S = np.zeros((H, d, dv)) if S is None else S.copy()
    o = np.zeros((T, H, dv))
    for i in range(T):
        S = decay[:, None, None] * S + k[i][:, :, None] * v[i][:, None, :]
        o[i] = np.einsum("hkv,hk->hv", S, q[i])
    o = rms_norm(o.reshape(T, H * dv), eps) * t[pre + "norm"] * sigmoid(h @ t[pre + "g"].T)
    return o @ t[pre + "o"].T, S


def wkv(h, mix, t, pre, eps, state=None):
    """Time mixing with a decay per token, head and key channel; state: (S [heads, dim, dim], the previous token's h)."""
    H, d = mix["heads"], mix["dim"]
    T = h.shape[0]
    S, prev = (np.zeros((H, d, d)), np.zeros(h.shape[1])) if state is None else (state[0].copy(), state[1])
    shifted = np.concatenate([prev[None], h[:-1]])
    m = {s: h + (shifted - h) * t[pre + "mu." + s] for s in "rkvgw"}
    r, k, v = ((m[s] @ t[pre + s].T).reshape(T, H, d) for s in "rkv")
    gate = silu(m["g"] @ t[pre + "g"].T)
    w = np.exp(-np.exp(np.tanh(m["w"] @ t[pre + "w1"].T) @ t[pre + "w2"].T + t[pre + "w0"])).reshape(T, H, d)
    u = t[pre + "u"]
    o = np.zeros((T, H, d))
    for i in range(T):
        kv = k[i][:, :, None] * v[i][:, None, :]
        o[i] = np.einsum("hkv,hk->hv", S + u[:, :, None] * kv, r[i])
        S = w[i][:, :, None] * S + kv
    o = rms_norm(o, eps).reshape(T, H * d) * t[pre + "norm"] * gate
    return o @ t[pre + "o"].T, (S, h[-1].copy())


MIXERS = {"attention": attention, "lightning": lightning, "wkv": wkv}


def layer_order(config):
    """Indices of the layers in the order they run."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


class Model:
    """`forward` feeds tokens behind those already fed; every layer run has a state of its own."""

    def __init__(self, config, tensors):
        self.c = config
        self.t = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.order = layer_order(config)
        self.reset()

    def reset(self):
        self.state = [None] * len(self.order)
        self.n = 0

    def norm(self, x, name):
        return dynamic_tanh(x, self.t[name + ".alpha"], self.t[name], self.t[name + ".b"])

    def forward(self, tokens):
        """Returns (logits [T, vocab], residual stream after every layer run [runs, T, width])."""
        c, t, eps = self.c, self.t, self.c["norm"]["eps"]
        x = t["embed"][tokens] + t["pos"][self.n:self.n + len(tokens)]
        runs = []
        for run, l in enumerate(self.order):
            layer, pre = c["layers"][l], f"l{l}."
            y, self.state[run] = MIXERS[layer["type"]](self.norm(x, pre + "norm1"), layer["mixer"], t, pre + "mix.", eps, self.state[run])
            x = x + y
            if layer["mlp"] is not None:
                z = self.norm(x, pre + "norm2") @ t[pre + "mlp.up"].T
                x = x + poly_norm(z, t[pre + "mlp.act"], eps) @ t[pre + "mlp.down"].T
            runs.append(x)
        self.n += len(tokens)
        logits = self.norm(x, "final.norm") @ t["head"].T
        cap = c.get("logit_softcap")
        if cap:
            logits = cap * np.tanh(logits / cap)
        return logits, np.stack(runs)
