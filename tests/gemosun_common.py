"""Random Gemosun models for the tests: configurations as config.json spells them and weights as plain arrays, bfloat16
exact, for the product (`axonml_amd.gemosun.build`) and for the plain forward (`oracle.gemosun.Model`) alike.

A mixture's choice is a jump: two right evaluations may differ where two experts score nearly alike.  So the first CLASSES
channels of the stream hold a token's class, no layer writes to them, and routers read little else: the gaps between scores are
far larger than rounding, and `margin` says how large they were."""
import numpy as np

from .stack_common import LIMIT, bf16, error  # noqa: F401
from oracle import gemosun as plain

CLASSES = 8
YARN = {"factor": 3.0, "original": 80, "fast": 9.0, "slow": 0.5}


def rot(dims=12, base=3000.0, scaling=YARN):
    return {"dims": dims, "base": base, "scaling": scaling} if scaling else {"dims": dims, "base": base}


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=20, groups=(3, 2), shared=28):
    router = {"experts": experts, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared:
        mlp["shared"] = {"ff": shared}
    return mlp


DEFAULT = object()


def attention(heads=4, kv_heads=2, dim=20, size=23, pool=5, scale=0.25, turn=DEFAULT, mlp=None):
    mix = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": size, "pool": pool}, "scale": scale,
           "rot": rot() if turn is DEFAULT else turn}
    return {"type": "attention", "mixer": mix, "mlp": mlp}


def config(layers, width=72, vocab=101, eps=1e-5):
    return {"architecture": "Gemosun", "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps}}


def _gaps(s, router):
    """(scores of the chosen experts above the others that could be chosen, of the kept groups above the others), plainly."""
    groups = router.get("groups") or {"count": 1, "keep": 1}
    per = len(s) // groups["count"]
    score = np.array([np.sort(s[g * per:(g + 1) * per])[-2:].sum() for g in range(groups["count"])])
    order = np.sort(score)[::-1]
    by_group = order[groups["keep"] - 1] - order[groups["keep"]] if groups["keep"] < groups["count"] else np.inf
    usable = np.sort([s[e] for e in range(len(s)) if score[e // per] >= order[groups["keep"] - 1]])[::-1]
    return usable[router["top"] - 1] - usable[router["top"]] if router["top"] < len(usable) else np.inf, by_group


def _router_classes(rng, router):
    """Per expert and class: evenly spaced where they are few, in an order of its own for every class, without close calls."""
    n = router["experts"]
    if n > 16:  # too many for even spacing: `top` of them high, in as many groups as are kept
        groups = router.get("groups") or {"count": 1, "keep": 1}
        out = []
        for _ in range(CLASSES):
            r, kept = rng.uniform(-0.45, -0.2, n), rng.permutation(groups["count"])[:groups["keep"]]
            for i in range(router["top"]):
                r[kept[i % len(kept)] * (n // groups["count"]) + 1 + 2 * (i // len(kept))] = rng.uniform(0.2, 0.45)
            out.append(r)
        return np.stack(out, axis=1)
    spaced, out = np.linspace(-0.45, 0.45, n) if n > 1 else np.zeros(1), []
    while len(out) < CLASSES:
        r = rng.permutation(spaced)
        if min(min(_gaps(plain.sigmoid(r * f), router)) for f in (1.5, 2.0, 3.0, 4.0, 5.0)) > 0.02:
            out.append(r)
    return np.stack(out, axis=1)


def tensors(cfg, seed):
    rng = np.random.default_rng(seed)
    W, t = cfg["width"], {}

    def lin(n, k, gain=1.0):
        return rng.standard_normal((n, k)) * (gain / np.sqrt(k))

    def out(n, k, gain):  # writes to the stream, but not to the class
        w = lin(n, k, gain)
        w[:CLASSES] = 0.0
        return w

    def norm(name):
        t[name] = 1.0 + 0.3 * rng.standard_normal(W)
        t[name][:CLASSES] = 1.0

    t["embed"] = rng.standard_normal((cfg["vocab"], W))
    t["embed"][:, :CLASSES] = 5.0 * np.eye(CLASSES)[rng.integers(0, CLASSES, cfg["vocab"])]
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        H, G, d = m["heads"], m["kv_heads"], m["dim"]
        norm(f"l{i}.norm1")
        t[p + "q"], t[p + "k"] = lin(H * d, W, 1.3), lin(G * d, W, 1.3)
        t[p + "g"] = lin(H, W, 1.5)
        t[p + "o"] = out(W, H * d, 1.5)
        mlp, p = layer["mlp"], f"l{i}.mlp."
        if mlp is not None:
            norm(f"l{i}.norm2")
            if mlp["kind"] == "dense":
                t[p + "gate"], t[p + "up"], t[p + "down"] = lin(mlp["ff"], W, 1.5), lin(mlp["ff"], W, 1.5), out(W, mlp["ff"], 0.9)
            else:
                E = mlp["router"]["experts"]
                router = 0.004 * rng.standard_normal((E, W))
                router[:, :CLASSES] = _router_classes(rng, mlp["router"])
                t[p + "router"] = router
                for e in range(E):
                    t[p + f"e{e}.up"], t[p + f"e{e}.down"] = lin(mlp["expert"]["ff"], W, 1.2), out(W, mlp["expert"]["ff"], 0.9)
                if mlp.get("shared"):
                    ff = mlp["shared"]["ff"]
                    t[p + "shared.up"], t[p + "shared.down"], t[p + "shared.sg"] = lin(ff, W, 1.2), out(W, ff, 0.9), lin(1, W, 1.5)
        w = 0.15 * rng.standard_normal(i + 2)
        w[0] += 0.4
        w[-1] += 0.8
        t[f"l{i}.dwa"] = w
    t["final.norm"] = 1.0 + 0.3 * rng.standard_normal(W)
    t["head"] = lin(cfg["vocab"], W, 3.0)
    return {k: bf16(v) for k, v in t.items()}


def oracle(cfg, t):
    return plain.Model(cfg, t)


def margin(cfg, t, tokens):
    """The smallest gap of any choice that the tokens' mixtures make."""
    real, least = plain.choose, [np.inf]

    def watched(s, router):
        least.extend(_gaps(s, router))
        return real(s, router)

    plain.choose = watched
    try:
        oracle(cfg, t).forward(tokens)
    finally:
        plain.choose = real
    return min(least)


def product(cfg, t, dtype, ctx, positions=400):
    from axonml_amd import gemosun

    return gemosun.build(cfg, lambda n: t[n], dtype, positions, ctx)
