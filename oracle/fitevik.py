"""Plain, slow Fitevik forward pass over a whole sequence (TEST INFRASTRUCTURE ONLY).

numpy in float64, one function per mechanism, no cache, no batch, no kernels. Fitevik is a decoder with learned positions whose
sublayers read the stream itself and are layer-normed before they are added to it. Mixers: HGRN2 (states with a forget gate per
channel, whose complement writes) and attention over a sliding window with a slope per head, scores mixed across heads and a sink.
Feed-forwards: squared relu, dense or routed. Keys are seen or not by a mask over all pairs, the recurrence runs token by token,
every expert is computed for every token.
"""
import numpy as np

from oracle.lozedra import bf16_round, read_tensors, sigmoid, silu, sub, write_model  # noqa: F401

F = np.float64

# What an implementation with 16-bit activations rounds: operands of matrix products. forward(.., rounded=True) sets it.
_round = lambda a: a


def rms(x, eps):
    """x divided by its root mean square"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w + b


def linear(w, h, b=None):
    """w [out, in], h [tokens, in]"""
    y = _round(h) @ w.T
    return y if b is None else y + b


def relu2(z):
    return np.maximum(z, 0.0) ** 2


def embedding(tokens, T, eps):
    x = T["embed"][np.asarray(tokens)] + T["pos"][:len(tokens)]
    return layer_norm(x, T["embed.norm"], T["embed.norm.b"], eps)


# ---------------------------------------------------------------- states
def forget(z, bias, lower):
    """The forget gate from its projection, never below `lower`"""
    return lower + (1.0 - lower) * sigmoid(z + bias)


def gated_states(q, f, v, state=None):
    """q, f [tokens, heads, dim], v [tokens, heads, vdim] -> (outputs [tokens, heads, vdim], final state [heads, dim, vdim])"""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2])) if state is None else state.copy()
    o = np.zeros_like(v, dtype=F)
    for i in range(len(q)):
        S = f[i][:, :, None] * S + (1.0 - f[i])[:, :, None] * v[i][:, None, :]
        o[i] = (q[i][:, :, None] * S).sum(1)
    return o, S


def hgrn2(h, t, cfg, eps):
    T, H, D, V = len(h), cfg["heads"], cfg["dim"], cfg["vdim"]
    q = _round(silu(linear(t["q"], h))).reshape(T, H, D)
    v = _round(linear(t["v"], h)).reshape(T, H, V)
    f = forget(linear(t["f"], h), t["f.b"], t["lower"]).reshape(T, H, D)
    o, _ = gated_states(q, f, v)
    return linear(t["o"], (rms(o, eps) * t["norm"]).reshape(T, H * V))


# ---------------------------------------------------------------- attention
def slopes(heads):
    return 2.0 ** (-8.0 * (np.arange(heads) + 1) / heads)


def in_window(i, j, size):
    return (i - j >= 0) & (i - j < size)


def mix_heads(talk, s):
    """s [heads, ..]: every head's scores become a weighted sum of all heads'"""
    return np.tensordot(talk, s, axes=(1, 0))


def softmax(s, sink):
    """Weights over the last axis; the denominator also holds exp(sink)."""
    m = np.maximum(s.max(-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - m))


def keys_values(h, t, cfg, eps):
    T, G = len(h), cfg["kv_heads"]
    k = _round(rms(linear(t["k"], h), eps) * t["k.norm"]).reshape(T, G, cfg["dim"])
    return k, _round(linear(t["v"], h)).reshape(T, G, cfg["vdim"])


def attention(h, t, cfg, eps, kv):
    """kv: keys [tokens, kv_heads, dim] and values, the layer's own or another's"""
    T, H, G, D = len(h), cfg["heads"], cfg["kv_heads"], cfg["dim"]
    k, v = kv
    q = _round(rms(linear(t["q"], h), eps) * t["q.norm"]).reshape(T, H, D)
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    s = np.stack([q[:, n] @ k[:, n // (H // G)].T * cfg["scale"] for n in range(H)])
    s = mix_heads(t["talk"], s - slopes(H)[:, None, None] * (i - j))
    mask = cfg.get("mask")
    seen = in_window(i, j, mask["size"]) if mask else i >= j
    out = np.stack([softmax(np.where(seen, s[n], -np.inf), t["sink"][n]) @ v[:, n // (H // G)] for n in range(H)], 1)
    return linear(t["o"], out.reshape(T, -1))


# ---------------------------------------------------------------- feed-forward
def dense(h, t):
    return linear(t["down"], relu2(linear(t["up"], h, t["up.b"])), t["down.b"])


def choose(z, top):
    """Router logits [tokens, experts] -> weights [tokens, experts], 0 where an expert is not chosen"""
    best = np.argsort(-z, -1, kind="stable")[:, :top]
    c = np.take_along_axis(z, best, -1)
    e = np.exp(c - c.max(-1, keepdims=True))
    w = np.zeros_like(z)
    np.put_along_axis(w, best, e / e.sum(-1, keepdims=True), -1)
    return w


def mixture(h, t, cfg):
    r = cfg["router"]
    w = choose(linear(t["router"], h, t["router.b"]), r["top"])
    return sum(w[:, e:e + 1] * linear(t["e%d.down" % e], relu2(linear(t["e%d.up" % e], h))) for e in range(r["experts"]))


def feed_forward(h, t, cfg):
    return dense(h, t) if cfg["kind"] == "dense" else mixture(h, t, cfg)


# ---------------------------------------------------------------- model
def forward(cfg, tensors, tokens, residuals=None, rounded=False):
    """-> logits [tokens, vocab]; residuals: a list that receives the stream behind every layer"""
    global _round
    if rounded:
        _round = lambda a: bf16_round(a).astype(F)
        try:
            return forward(cfg, tensors, tokens, residuals)
        finally:
            _round = lambda a: a
    T = {k: np.asarray(v, dtype=F) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = embedding(tokens, T, eps)
    cached = {}
    for i, c in enumerate(cfg["layers"]):
        t, mx = sub(T, "l%d." % i), c["mixer"]
        if c["type"] == "hgrn2":
            y = hgrn2(x, sub(t, "mix."), mx, eps)
        else:
            if mx.get("kv_from") is None:
                cached[i] = keys_values(x, sub(t, "mix."), mx, eps)
            y = attention(x, sub(t, "mix."), mx, eps, cached[i if mx.get("kv_from") is None else mx["kv_from"]])
        x = x + layer_norm(y, t["norm1"], t["norm1.b"], eps)
        if c.get("mlp"):
            x = x + layer_norm(feed_forward(x, sub(t, "mlp."), c["mlp"]), t["norm2"], t["norm2.b"], eps)
        if residuals is not None:
            residuals.append(x)
    return linear(T["head"], layer_norm(x, T["final.norm"], T["final.norm.b"], eps)) * cfg["logit_scale"]
