"""Random Lakulix models for the tests: configurations as config.json spells them and weights as plain arrays, bfloat16
exact, for the product (`axonml_amd.lakulix.build`) and for the plain forward (`oracle.lakulix.Model`) alike."""
import numpy as np

from .stack_common import LIMIT, bf16, error, write_checkpoint  # noqa: F401
from oracle import lakulix as plain


def attention(heads=4, kv_heads=2, dim=24, vdim=16, ff=0, bias_max=40, scale=0.2, coef=0.4, every=9):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "bias_max": bias_max, "scale": scale,
                      "q_temp": {"coef": coef, "every": every}}}


def lightning(heads=3, dim=20, vdim=12, ff=0, decay=None):
    decay = decay if decay is not None else [float(np.exp(-2.0 ** -(i + 0.5))) for i in range(heads)]
    return {"type": "lightning", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}}


def wkv(heads=3, dim=20, ff=0):
    return {"type": "wkv", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": {"heads": heads, "dim": dim}}


def config(layers, width=72, vocab=101, max_positions=400, loop=None, softcap=12.0, eps=1e-5):
    return {"architecture": "Lakulix", "layers": layers, "width": width, "vocab": vocab, "max_positions": max_positions, "loop": loop,
            "logit_softcap": softcap, "norm": {"eps": eps}}


def tensors(cfg, seed, bias_rows=12, rank=5, pb=-3.0):
    rng = np.random.default_rng(seed)
    W, t = cfg["width"], {}

    def lin(n, k, gain=1.0):
        return rng.standard_normal((n, k)) * (gain / np.sqrt(k))

    def norm(name):
        t[name] = 1.0 + 0.3 * rng.standard_normal(W)
        t[name + ".b"] = 0.15 * rng.standard_normal(W)
        t[name + ".alpha"] = np.asarray(rng.uniform(0.4, 0.8))

    t["embed"] = rng.standard_normal((cfg["vocab"], W))
    t["pos"] = 0.4 * rng.standard_normal((cfg["max_positions"], W))
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        H, d = m["heads"], m["dim"]
        norm(f"l{i}.norm1")
        if layer["type"] == "attention":
            dv, G = m["vdim"], m["kv_heads"]
            t[p + "q"], t[p + "k"], t[p + "v"] = lin(H * d, W), lin(G * d, W), lin(G * dv, W)
            t[p + "q.norm"], t[p + "k.norm"] = 1.0 + 0.4 * rng.standard_normal(d), 1.0 + 0.4 * rng.standard_normal(d)
            t[p + "rel"] = rng.standard_normal((bias_rows, H))
            t[p + "pb"] = pb + 0.5 * rng.standard_normal(H)
            out = H * dv
        elif layer["type"] == "lightning":
            dv = m["vdim"]
            t[p + "q"], t[p + "k"] = lin(H * d, W, 1.5), lin(H * d, W, 1.5)
            t[p + "v"], t[p + "g"] = lin(H * dv, W, 1.5), lin(H * dv, W)
            t[p + "norm"] = 1.0 + 0.3 * rng.standard_normal(H * dv)
            out = H * dv
        else:
            out = H * d
            for s in "rkvgw":
                t[p + "mu." + s] = rng.uniform(0.0, 0.9, W)
            for s in "rkvg":
                t[p + s] = lin(out, W)
            t[p + "w1"], t[p + "w2"] = lin(rank, W), lin(out, rank)
            t[p + "w0"] = rng.uniform(-6.0, 1.5, out)
            t[p + "u"] = 0.6 * rng.standard_normal((H, d))
            t[p + "norm"] = 1.0 + 0.3 * rng.standard_normal(out)
        t[p + "o"] = lin(W, out, 0.7)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            norm(f"l{i}.norm2")
            t[f"l{i}.mlp.up"], t[f"l{i}.mlp.down"] = lin(ff, W), lin(W, ff, 0.7)
            t[f"l{i}.mlp.act"] = rng.uniform(0.3, 0.9, 4)
    norm("final.norm")
    t["head"] = lin(cfg["vocab"], W, 3.0)
    return {k: bf16(v) for k, v in t.items()}


def oracle(cfg, t):
    return plain.Model(cfg, t)


def product(cfg, t, dtype, ctx, cache_positions=None):
    from axonml_amd import lakulix

    return lakulix.build(cfg, lambda n: t[n], lambda n: list(t[n].shape) if n in t else None, dtype, cache_positions, ctx)
