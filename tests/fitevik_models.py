"""Small random Fitevik models for the tests, and the measure by which their logits are compared."""
import numpy as np

from lozedra_models import LIMIT, error  # noqa: F401
from oracle import fitevik as fv


def states(heads=3, dim=20, vdim=24):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def attention(heads=4, kv_heads=2, dim=12, vdim=28, size=37, scale=None, kv_from=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "mask": {"size": size}}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "attention", "mixer": mx}


def dense(ff=50):
    return {"kind": "dense", "ff": ff}


def moe(experts=12, top=3, ff=24):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(layers, width=88, vocab=149, eps=1e-5, logit_scale=0.7, max_positions=600):
    """layers: [(layer, feed-forward or None)]"""
    return {"architecture": "Fitevik", "layers": [dict(l, mlp=f) for l, f in layers], "norm": {"eps": eps}, "vocab": vocab, "width": width,
            "logit_scale": logit_scale, "max_positions": max_positions}


def margin(z, top):
    """By how much a row's choice is clear: between the last expert chosen and the next. z: [rows, experts]"""
    s = -np.sort(-z, -1)
    return s[:, top - 1] - s[:, top] if top < z.shape[1] else np.full(len(z), np.inf)


def tensors(cfg, seed, qk_gain=2.0, sink=0.5, keep=1.0):
    """Random weights, already on the bfloat16 grid. qk_gain: how far attention is from uniform; keep: mean of the gates' bias, above 0
    they forget slowly. The stream's first dimensions belong to the routers alone: nothing adds to them behind the embedding, whose code
    for a token is such that no choice is a close call."""
    rng = np.random.default_rng(seed)
    W, V, P, out = cfg["width"], cfg["vocab"], cfg["max_positions"], {}
    routers = {i: l["mlp"]["router"] for i, l in enumerate(cfg["layers"]) if l["mlp"] and l["mlp"]["kind"] == "moe"}
    code = max([r["experts"] for r in routers.values()], default=0)
    code = code if code < W else 0                              # (no room in the smallest models)

    def mat(name, n, k, gain=1.0):
        out[name] = fv.bf16_round(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, mean=0.0, std=0.2):
        out[name] = fv.bf16_round(mean + std * rng.standard_normal(n))

    def norm(name):
        vec(name, W, 1.0)
        vec(name + ".b", W)

    for i, r in routers.items():
        out["l%d.mlp.router.b" % i] = fv.bf16_round(rng.choice([-0.5, -0.25, 0.0, 0.4], r["experts"]))
    emb, pos, scales = rng.standard_normal((V, W)), 0.6 * rng.standard_normal((P, W)), np.linspace(0.6, 1.2, 100)  # (what the norm may make of a code)
    for t in range(V if code else 0):
        for _ in range(2000):
            c = fv.bf16_round(rng.permutation(np.linspace(-1.6, 1.6, code)))
            if all(margin(np.outer(scales, c[:r["experts"]]) + out["l%d.mlp.router.b" % i], r["top"]).min() > 0.015 for i, r in routers.items()):
                break
        else:
            raise ValueError("no code keeps every choice clear")
        emb[t, :code] = c
    pos[:, :code] = 0
    out["embed"], out["pos"] = fv.bf16_round(emb), fv.bf16_round(pos)
    norm("embed.norm")
    out["embed.norm"][:code], out["embed.norm.b"][:code] = 1, 0
    for i, layer in enumerate(cfg["layers"]):
        l, m, mx = "l%d." % i, "l%d.mix." % i, layer["mixer"]
        H, D, X = mx["heads"], mx["dim"], mx["vdim"]
        for n in ("norm1", "norm2") if layer["mlp"] else ("norm1",):
            norm(l + n)
            out[l + n][:code], out[l + n + ".b"][:code] = 0, 0
        if layer["type"] == "hgrn2":
            for n, size in (("q", D), ("f", D), ("v", X)):
                mat(m + n, H * size, W, 1.5)
            vec(m + "f.b", H * D, keep, 1.5)
            out[m + "lower"] = fv.bf16_round(rng.choice([0.0, 0.1, 0.5, 0.9, 0.98], H * D))
            vec(m + "norm", X, 1.0)
        else:
            G = mx["kv_heads"]
            mat(m + "q", H * D, W)
            vec(m + "q.norm", H * D, np.sqrt(qk_gain), 0.3)
            if "kv_from" not in mx:
                mat(m + "k", G * D, W)
                mat(m + "v", G * X, W)
                vec(m + "k.norm", G * D, np.sqrt(qk_gain), 0.3)
            out[m + "talk"] = fv.bf16_round(np.eye(H) + 0.5 * rng.standard_normal((H, H)) / np.sqrt(H))
            vec(m + "sink", H, sink, 1.0)
        mat(m + "o", W, H * X)
        if not layer["mlp"]:
            continue
        mlp, p = layer["mlp"], l + "mlp."
        if mlp["kind"] == "dense":
            mat(p + "up", mlp["ff"], W, 1.2)
            vec(p + "up.b", mlp["ff"])
            mat(p + "down", W, mlp["ff"])
            vec(p + "down.b", W)
            continue
        r = np.zeros((mlp["router"]["experts"], W))
        if code:
            r[np.arange(len(r)), np.arange(len(r))] = 1.0
        else:
            r = rng.standard_normal(r.shape) / np.sqrt(W)
        out[p + "router"] = fv.bf16_round(r)
        for e in range(len(r)):
            mat(p + "e%d.up" % e, mlp["expert"]["ff"], W, 1.2)
            mat(p + "e%d.down" % e, W, mlp["expert"]["ff"])
    norm("final.norm")
    mat("head", V, W)
    return out


# other sizes than round ones, every branch: both mixers, keys of another layer (with another mask), dense and routed feed-forwards and
# none, windows no multiple of a block, also last in the list
SMALL = config([(attention(), dense()), (states(), moe()), (attention(heads=6, kv_heads=2, size=50, kv_from=0), moe(experts=7, top=2, ff=33)),
                (attention(heads=5, kv_heads=1, dim=9, vdim=7, size=3), None), (states(heads=2, dim=7, vdim=33), dense(21)),
                (attention(heads=10, kv_heads=2, dim=30, vdim=18, size=64), dense(130)), (states(heads=1, dim=40, vdim=16), None)])
# everything that can be one is one (the norm of a single number is its sign, but for a large eps)
TINY = config([(attention(heads=1, kv_heads=1, dim=1, vdim=1, size=1, scale=1.0), moe(1, 1, 1)), (states(heads=1, dim=1, vdim=1), dense(1)),
               (attention(heads=1, kv_heads=1, dim=1, vdim=1, size=1, scale=1.0, kv_from=0), None)], width=5, vocab=7, eps=0.5, logit_scale=1.0, max_positions=230)
# whole tiles: the matrix-core kernels
EVEN = config([(attention(heads=8, kv_heads=2, dim=32, vdim=64, size=80), moe(16, 4, 64)), (states(heads=2, dim=64, vdim=48), dense(128)),
               (attention(heads=8, kv_heads=2, dim=32, vdim=64, size=48, kv_from=0), dense(64)), (states(heads=3, dim=128, vdim=32), moe(8, 1, 32)),
               (attention(heads=16, kv_heads=16, dim=64, vdim=64, size=90), None)], width=128, vocab=256)
# wider heads than those kernels take, many query heads to a key head, more heads than a wave's tile, more than two tiles a wave
WIDE = config([(attention(heads=3, kv_heads=1, dim=144, vdim=160, size=70), dense(40)), (attention(heads=20, kv_heads=1, dim=96, vdim=128, size=100), None),
               (attention(heads=40, kv_heads=8, dim=16, vdim=16, size=61), moe(4, 4, 16)), (states(heads=1, dim=160, vdim=144), None),
               (attention(heads=24, kv_heads=24, dim=8, vdim=24, size=33), None), (attention(heads=66, kv_heads=3, dim=8, vdim=8, size=40), None)], width=96, vocab=199)


def limit(dtype, cfg, t, toks, want):
    """The largest error allowed: fixed for float32, three times what rounding operands to bfloat16 does to the same tokens in
    the plain implementation otherwise."""
    if dtype == "float32":
        return LIMIT[dtype]
    return 3 * max(5e-3, error(fv.forward(cfg, t, toks, rounded=True), want).max())
