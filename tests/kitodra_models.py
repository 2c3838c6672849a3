"""Small random Kitodra models for the tests, and the measure by which their logits are compared."""
import numpy as np

from lozedra_models import LIMIT, error  # noqa: F401
from oracle import kitodra as kt


def lightning(heads=3, dim=20, vdim=24, decay=None):
    decay = decay or [float(d) for d in 1.0 - np.geomspace(0.5, 0.002, heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}}


def differential(heads=4, kv_heads=2, dim=12, vdim=28, size=37, scale=None, cap=9.0, diff=0.35):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "diff": diff, "mask": {"size": size}}
    if cap:
        mx["softcap"] = cap
    return {"type": "attention", "mixer": mx}


def key_value(heads=3, kv_heads=1, dim=22, size=29, rot=(8, 700.0), scale=None):
    return {"type": "attention_2", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale or 2.0 * dim ** -0.5,
                                             "mask": {"size": size}, "rot": {"dims": rot[0], "base": rot[1]}}}


def moe(experts=12, top=3, groups=(3, 2), ff=24, limit=0.8, shared=(40, 1.3)):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if groups:
        m["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def config(layers, width=88, vocab=149, eps=1e-5, pair=(211, 31, 17)):
    """layers: [(layer, feed-forward or None)], or the number of an earlier entry whose weights are used again"""
    entries = []
    for l in layers:
        entries.append(dict(entries[l], weights_of=l) if isinstance(l, int) else dict(l[0], mlp=l[1]))
    c = {"architecture": "Kitodra", "layers": entries, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if pair:
        c["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), pair))}
    return c


def margin(c, router):
    """By how much a row's choice is clear: between the last expert chosen and the next, and between the last group kept and the next.
    c: [rows, experts] choice scores"""
    def gap(v, n):
        v = -np.sort(-v, -1)
        return v[:, n - 1] - v[:, n] if n < v.shape[1] else np.full(len(v), np.inf)

    g, out = router.get("groups"), np.full(len(c), np.inf)
    if g:
        per = c.reshape(len(c), g["count"], -1)
        score = np.sort(per, -1)[..., -2:].sum(-1)
        out = gap(score, g["keep"])
        best = np.argsort(-score, -1)[:, :g["keep"]]
        kept = np.zeros((len(c), g["count"]), dtype=bool)
        np.put_along_axis(kept, best, True, -1)
        c = np.where(np.repeat(kept, c.shape[1] // g["count"], -1), c, -1e9)
    return np.minimum(out, gap(c, router["top"]))


def tensors(cfg, seed, qk_gain=2.0):
    """Random weights, already on the bfloat16 grid. qk_gain: how far attention is from uniform. The stream's first dimensions belong to
    the routers alone: nothing writes to them behind the embedding, whose code for a token is such that no choice is a close call."""
    rng = np.random.default_rng(seed)
    W, V, out = cfg["width"], cfg["vocab"], {}
    routers = {}
    for i, l in enumerate(cfg["layers"]):
        if l["mlp"] and "weights_of" not in l:
            routers[i] = l["mlp"]["router"]
    code = max([r["experts"] for r in routers.values()], default=0)
    code = code if code < W else 0                              # (no room in the smallest models)

    def mat(name, n, k, gain=1.0, writes=False):
        a = rng.standard_normal((n, k)) * gain / np.sqrt(k)
        if writes:
            a[:code] = 0
        out[name] = kt.bf16_round(a)

    def vec(name, n, mean=0.0, std=0.2):
        out[name] = kt.bf16_round(mean + std * rng.standard_normal(n))

    for i, r in routers.items():
        out["l%d.mlp.correction" % i] = kt.bf16_round(rng.choice([-0.9, -0.6, 0.0, 0.25], r["experts"]))
    emb, scales = rng.standard_normal((V, W)), np.linspace(0.25, 1.1, 180)    # (what norms may make of the code)
    for t in range(V if code else 0):
        for _ in range(2000):
            c = kt.bf16_round(rng.permutation(np.linspace(-1.6, 1.6, code)))
            if all(margin(kt.sigmoid(np.outer(scales, c[:r["experts"]])) + out["l%d.mlp.correction" % i], r).min() > 0.004
                   for i, r in routers.items()):
                break
        else:
            raise ValueError("no code keeps every choice clear")
        emb[t, :code] = c
    out["embed"] = kt.bf16_round(emb)
    pair = (cfg.get("embedding") or {}).get("bigram")
    if pair:
        b = rng.standard_normal((pair["buckets"] + 1, W)) * 0.7
        b[:, :code] = 0
        out["bigram"] = kt.bf16_round(b)
    for i, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            continue
        l, m, mx = "l%d." % i, "l%d.mix." % i, layer["mixer"]
        H, D, X = mx["heads"], mx["dim"], mx["vdim"]
        vec(l + "norm1", W, 1.0)
        out[l + "norm1"][:code] = 1.0
        if layer["type"] == "lightning":
            for n, size in (("q", D), ("k", D), ("v", X), ("g", X)):
                mat(m + n, H * size, W, 1.5)
            vec(m + "norm", H * X, 1.0)
        else:
            G, maps = mx["kv_heads"], 2 if layer["type"] == "attention" else 1
            for n, size in (("q", H * maps * D), ("k", G * maps * D)) + ((("v", G * X),) if maps == 2 else ()):
                mat(m + n, size, W)
                vec(m + n + ".b", size, 0.0, 0.4)
            vec(m + "o.b", W)
            out[m + "o.b"][:code] = 0
            if maps == 2:
                for n in ("q.norm", "k.norm"):
                    vec(m + n, D, np.sqrt(qk_gain), 0.3)
                for n in ("lq1", "lk1", "lq2", "lk2"):
                    vec(m + n, D, 0.0, 0.8 * D ** -0.25)
        mat(m + "o", W, H * X, 0.7, True)
        if layer["mlp"]:
            mlp, p = layer["mlp"], l + "mlp."
            r = np.zeros((mlp["router"]["experts"], W))
            if code:
                r[np.arange(len(r)), np.arange(len(r))] = 1.0
            else:
                r = rng.standard_normal(r.shape) / np.sqrt(W)
            out[p + "router"] = kt.bf16_round(r)
            named = [("e%d" % e, mlp["expert"]["ff"]) for e in range(len(r))] + ([("shared", mlp["shared"]["ff"])] if mlp.get("shared") else [])
            for name, ff in named:
                mat(p + name + ".gate", ff, W, 1.2)
                mat(p + name + ".up", ff, W, 1.2)
                mat(p + name + ".down", W, ff, 0.7, True)
    vec("final.norm", W, 1.0)
    return out


# other sizes than round ones, every branch: three mixers, layers without experts, without groups, without a shared expert, weights used
# again (also those of a layer that comes later in the list of mixers), chunks and windows no multiple of a block
SMALL = config([(lightning(), moe()), (differential(), moe(experts=8, top=2, groups=None, ff=33, shared=(17, 0.6))), (key_value(), None),
                (differential(heads=6, kv_heads=1, dim=9, vdim=7, size=50, cap=None, diff=0.7), None), 0, 1, 2,
                (key_value(heads=4, kv_heads=4, dim=10, size=3, rot=(10, 90.0)), moe(shared=None)),
                (lightning(heads=2, dim=7, vdim=33, decay=[0.0, 1.0]), moe(experts=9, top=4, groups=(9, 6), ff=1))])
# everything that can be one is one
TINY = config([(lightning(heads=1, dim=1, vdim=1, decay=[0.5]), moe(1, 1, (1, 1), 1, 1.0, (1, 1.0))),
               (differential(heads=1, kv_heads=1, dim=1, vdim=1, size=1, scale=1.0, cap=1.0), moe(1, 1, None, 1, 1.0, None)),
               (key_value(heads=1, kv_heads=1, dim=2, size=1, rot=(2, 1.0), scale=1.0), None), 0], width=5, vocab=7, pair=(1, 1, 1))
# whole tiles: the matrix-core kernels
EVEN = config([(lightning(heads=2, dim=64, vdim=48), moe(16, 4, (4, 2), 64, 1.5, (64, 1.5))),
               (differential(heads=8, kv_heads=2, dim=32, vdim=64, size=80), moe(16, 4, (4, 2), 64, 1.5, (128, 1.0))),
               (key_value(heads=8, kv_heads=2, dim=64, size=64, rot=(32, 1e4)), moe(16, 4, (4, 2), 64, 1.5, (64, 1.5)))], width=128, vocab=256)
# wider heads than those, many query heads to a key head
WIDE = config([(lightning(heads=1, dim=160, vdim=144, decay=[0.97]), None), (differential(heads=3, kv_heads=1, dim=128, vdim=256, size=90), moe(4, 1, None, 16)),
               (key_value(heads=20, kv_heads=1, dim=136, size=100, rot=(64, 1e5)), moe(4, 4, (2, 2), 16))], width=96, vocab=199)


def limit(dtype, cfg, t, toks, want):
    """The largest error allowed: fixed for float32, three times what rounding operands to bfloat16 does to the same tokens in
    the plain implementation otherwise."""
    if dtype == "float32":
        return LIMIT[dtype]
    return 3 * max(5e-3, error(kt.forward(cfg, t, toks, rounded=True), want).max())
