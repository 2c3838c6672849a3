"""Small random Lozedra models for the tests, and the measure by which their logits are compared."""
import numpy as np

from oracle import lozedra as lz


def mixer(heads=3, kv_heads=1, dim=24, vdim=16, bias_max=70, temp=(0.4, 16), inner=48, state=6, dt_rank=5, conv=3,
          left_scale=0.8, right_scale=0.55, scale=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "bias_max": bias_max,
            "scale": scale or dim ** -0.5}
    if temp:
        left["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return {"left": left, "right": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv},
            "left_scale": left_scale, "right_scale": right_scale}


def config(layers, width=80, vocab=151, loop=None, eps=1e-5, mult=0.6):
    """layers: [(mixer, feed-forward size or None)]; loop: (start, stop, times)"""
    return {"architecture": "Lozedra",
            "layers": [{"type": "parallel", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None} for m, ff in layers],
            "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None,
            "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab, "width": width}


def tensors(cfg, seed, bias_rows=12, qk_gain=2.0):
    """Random weights, already on the bfloat16 grid. qk_gain: how far attention is from uniform."""
    rng = np.random.default_rng(seed)
    W, V, out = cfg["width"], cfg["vocab"], {}

    def mat(name, n, k, gain=1.0):
        out[name] = lz.bf16_round(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, mean=1.0, std=0.1):
        out[name] = lz.bf16_round(mean + std * rng.standard_normal(n))

    out["embed"] = lz.bf16_round(rng.standard_normal((V, W)))
    for i, layer in enumerate(cfg["layers"]):
        l, mx = "l%d." % i, layer["mixer"]
        a, s = mx["left"], mx["right"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if layer["mlp"] else ()):
            vec(l + n, W)
        p = l + "mix.left."
        mat(p + "q", a["heads"] * a["dim"], W, qk_gain)
        mat(p + "k", a["kv_heads"] * a["dim"], W, qk_gain)
        mat(p + "v", a["kv_heads"] * a["vdim"], W)
        mat(p + "g", a["heads"] * a["vdim"], W)
        mat(p + "o", W, a["heads"] * a["vdim"])
        out[p + "rel"] = lz.bf16_round(2.0 * rng.standard_normal((bias_rows, a["heads"])))
        p = l + "mix.right."
        n = s["inner"]
        mat(p + "in", 2 * n, W)
        out[p + "conv"] = lz.bf16_round(rng.standard_normal((n, s["conv"])) * 0.6)
        vec(p + "conv.b", n, 0.0, 0.2)
        mat(p + "x", s["dt_rank"] + 2 * s["state"], n, 1.5)
        mat(p + "dt", n, s["dt_rank"])
        vec(p + "dt.b", n, -2.5, 1.0)            # steps from slow to fast: some states last for hundreds of tokens
        out[p + "A_log"] = lz.bf16_round(np.log(rng.uniform(0.05, 4.0, (n, s["state"]))))
        vec(p + "D", n)
        mat(p + "o", W, n)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            mat(l + "mlp.gate", ff, W)
            mat(l + "mlp.up", ff, W)
            mat(l + "mlp.down", W, ff)
    vec("final.norm", W)
    mat("head", V, W)
    return out


# other sizes than round ones, layers that differ, a layer without feed-forward, a loop that runs three times
SMALL = config([(mixer(), 96), (mixer(heads=4, kv_heads=2, dim=16, vdim=40, temp=None, bias_max=33, inner=56, state=17, dt_rank=9,
                                      conv=5), None), (mixer(heads=2, kv_heads=2, dim=33, vdim=7, inner=37, state=1, dt_rank=1,
                                                             conv=1, bias_max=7), 41)], width=72, vocab=131, loop=(1, 3, 3))
# one plain layer, everything that can be one is one, no loop
TINY = config([(mixer(heads=1, kv_heads=1, dim=1, vdim=1, inner=1, state=1, dt_rank=1, conv=1, bias_max=2, temp=(1.0, 1),
                      left_scale=1.0, right_scale=1.0), 1)], width=5, vocab=7, mult=1.0)
# whole tiles everywhere
EVEN = config([(mixer(heads=8, kv_heads=2, dim=64, vdim=64, inner=128, state=16, dt_rank=16, conv=4, bias_max=128, temp=(0.3, 32)),
                192), (mixer(heads=8, kv_heads=2, dim=64, vdim=64, inner=128, state=16, dt_rank=16, conv=4, bias_max=128,
                             temp=(0.3, 32)), 192)], width=128, vocab=256, loop=(0, 1, 2))


def error(got, want):
    """rms over the vocabulary of the difference, mean taken off, by the spread of the expected logits, per row"""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    d = got - want
    d -= d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / want.std(-1).mean()


LIMIT = {"float32": 1e-4}


def limit(dtype, cfg, t, toks, want):
    """The largest error allowed: fixed for float32, three times what rounding activations to bfloat16 does to the same
    tokens in the plain implementation otherwise."""
    if dtype == "float32":
        return LIMIT[dtype]
    return 3 * max(5e-3, error(lz.forward(cfg, t, toks, rounded=True), want).max())
