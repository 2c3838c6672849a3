"""Small random Tulipel models for the tests, and the measure by which their logits are compared."""
import numpy as np

from lozedra_models import LIMIT, error  # noqa: F401
from oracle import tulipel as tl


def first(heads=3, dim=20, rot_dim=12, vdim=24, kv_rank=40, q_rank=28, base=900.0, scale=None):
    """A layer with a query latent and neighbouring rotated pairs."""
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "rot": {"base": base, "dims": rot_dim}, "scale": scale or (dim + rot_dim) ** -0.5}}


def second(heads=2, dim=16, rot_dim=8, vdim=40, kv_rank=72, base=5000.0, scaling=(3.0, 96, 4.0, 0.5), kv_from=None, scale=None):
    """A layer with direct queries, rotated halves, YaRN or not, perhaps on another layer's latents."""
    mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
          "rot": {"base": base, "dims": rot_dim}, "scale": scale or (dim + rot_dim) ** -0.5}
    if scaling:
        mx["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "latent_attention_2", "mixer": mx}


def config(layers, width=88, vocab=149, eps=1e-5, alpha=1.7, cap=12.0):
    """layers: [(layer, feed-forward size or None)]"""
    return {"architecture": "Tulipel", "layers": [dict(l, mlp={"kind": "dense", "ff": ff} if ff else None) for l, ff in layers],
            "norm": {"eps": eps}, "postln_alpha": alpha, "logit_softcap": cap, "vocab": vocab, "width": width}


def tensors(cfg, seed, qk_gain=2.0):
    """Random weights, already on the bfloat16 grid. qk_gain: how far attention is from uniform."""
    rng = np.random.default_rng(seed)
    W, V, out = cfg["width"], cfg["vocab"], {}

    def mat(name, n, k, gain=1.0):
        out[name] = tl.bf16_round(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, mean=0.0, std=0.2):
        out[name] = tl.bf16_round(mean + std * rng.standard_normal(n))

    out["embed"] = tl.bf16_round(rng.standard_normal((V, W)))
    for i, layer in enumerate(cfg["layers"]):
        l, m, mx = "l%d." % i, "l%d.mix." % i, layer["mixer"]
        H, D, R, C = mx["heads"], mx["dim"], mx["rot_dim"], mx["kv_rank"]
        vec(l + "norm1", W)
        if layer["type"] == "latent_attention":
            mat(m + "dq", mx["q_rank"], W)
            vec(m + "dq.norm", mx["q_rank"], 1.0)
            mat(m + "uq", H * (D + R), mx["q_rank"], qk_gain)
        else:
            mat(m + "q", H * (D + R), W, qk_gain)
        if "kv_from" not in mx:
            mat(m + "dkv", C + R, W)
            vec(m + "dkv.norm", C, 1.0)
        mat(m + "uk", H * D, C, qk_gain)
        mat(m + "uv", H * mx["vdim"], C)
        vec(m + "sink", H, 1.0, 1.0)
        mat(m + "o", W, H * mx["vdim"])
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            vec(l + "norm2", W)
            mat(l + "mlp.up", ff, W)
            mat(l + "mlp.down", W, ff)
            out[l + "mlp.act"] = tl.bf16_round(rng.uniform(0.2, 0.8, 4) * np.array([1, -1, 1, 1]))
        d = rng.uniform(-0.4, 0.4, i + 2)
        d[-1] = rng.uniform(0.6, 1.0)
        out[l + "dwa"] = tl.bf16_round(d)
    vec("final.norm", W)
    mat("head", V, W, 3.0)
    return out


# other sizes than round ones, every branch: both kinds, YaRN and none, shared latents, a layer without feed-forward
SMALL = config([(first(), 60), (second(), 41), (second(heads=5, dim=11, vdim=9, kv_from=1), None), (second(rot_dim=2, kv_rank=33, scaling=None), 24),
                (first(heads=1, rot_dim=20, vdim=7, q_rank=9, kv_rank=18, base=40.0), 77),
                (second(heads=3, dim=30, vdim=17, kv_rank=33, rot_dim=2, scaling=None, kv_from=3), 50)])
# everything that can be one is one
TINY = config([(first(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, q_rank=1, scale=1.0), 1),
               (second(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, scaling=(1.0, 1, 1.0, 1.0), scale=1.0), None)], width=5, vocab=7, alpha=1.0, cap=1.0)
# whole tiles; keys and values of portions of SPELL rows are spelled out in bfloat16
EVEN = config([(first(heads=8, dim=32, rot_dim=32, vdim=32, kv_rank=128, q_rank=64), 192), (second(heads=8, dim=64, rot_dim=64, vdim=16, kv_rank=256), 128),
               (second(heads=4, dim=64, rot_dim=64, vdim=64, kv_rank=256, kv_from=1), 128)], width=128, vocab=256)
# real latents: one 512 wide beside 64 rotated dimensions, more heads than a query tile holds
WIDE = config([(first(heads=20, dim=16, rot_dim=64, vdim=16, kv_rank=512, q_rank=48), 64), (second(heads=40, dim=16, rot_dim=64, vdim=16, kv_rank=300), 64)],
              width=96, vocab=199)


def limit(dtype, cfg, t, toks, want):
    """The largest error allowed: fixed for float32, three times what rounding operands to bfloat16 does to the same tokens in
    the plain implementation otherwise."""
    if dtype == "float32":
        return LIMIT[dtype]
    return 3 * max(5e-3, error(tl.forward(cfg, t, toks, rounded=True), want).max())
