"""Plain, slow Tulipel forward pass over a whole sequence (TEST INFRASTRUCTURE ONLY).

numpy in float64, one function per mechanism, no cache, no batch, no kernels. Tulipel is a decoder of latent-attention
layers (keys and values come from a small normed vector per token; one rotated key part serves all heads; a learned sink
per head in the softmax), with the norm behind every residual sum, a polynomial feed-forward activation normed over its
row, and a weighted sum of all earlier layer results in front of the next layer. Nothing here absorbs, pages or batches:
every head's keys and values are spelled out.
"""
import math

import numpy as np

from oracle.lozedra import bf16_round, read_tensors, write_model  # noqa: F401  (the file formats)

F = np.float64

# What an implementation with 16-bit activations rounds: operands of matrix products. forward(.., rounded=True) sets it.
_round = lambda a: a


def rms(x, eps):
    """x divided by its root mean square"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def model_norm(x, w, eps):
    """The weight is stored around zero."""
    return rms(x, eps) * (1.0 + w)


def linear(w, h):
    """w [out, in], h [tokens, in]"""
    return _round(h) @ w.T


def frequencies(rot):
    """-> (radians per position of every pair, factor of both cosine and sine)"""
    n, base = rot["dims"], rot["base"]
    i = np.arange(n // 2)
    f = base ** (-2.0 * i / n)
    s = rot.get("scaling")
    if not s:
        return f, 1.0
    turn = lambda t: n * math.log(s["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo, hi = max(math.floor(turn(s["fast"])), 0), min(math.ceil(turn(s["slow"])), n - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, pos, rot, halves):
    """x [tokens, .., width]: the first rot.dims of the last axis turn by the token's position. Pairs are (2i, 2i + 1), or
    (i, i + dims / 2) with halves."""
    f, m = frequencies(rot)
    n = rot["dims"]
    a = np.asarray(pos)[:, None] * f[None, :]
    shape = (len(pos),) + (1,) * (x.ndim - 2) + (n // 2,)
    c, s = (np.cos(a) * m).reshape(shape), (np.sin(a) * m).reshape(shape)
    y = np.array(x, dtype=F)
    iu, iv = (slice(0, n // 2), slice(n // 2, n)) if halves else (slice(0, n, 2), slice(1, n, 2))
    u, v = x[..., iu], x[..., iv]
    y[..., iu], y[..., iv] = u * c - v * s, v * c + u * s
    return y


def sink_softmax(s, sink):
    """Weights over the last axis when the denominator also holds exp(sink)."""
    m = np.maximum(s.max(-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(-1, keepdims=True) + np.exp(sink - m))


def latent(h, pos, t, cfg, halves, eps):
    """-> (normed latent [tokens, kv_rank], rotated key part [tokens, rot_dim]): all that a cache has to hold"""
    y = linear(t["dkv"], h)
    R = cfg["kv_rank"]
    return rms(y[:, :R], eps) * t["dkv.norm"], rotate(y[:, R:], pos, cfg["rot"], halves)


def queries(h, t, cfg, eps):
    if "dq" in t:
        return linear(t["uq"], rms(linear(t["dq"], h), eps) * t["dq.norm"])
    return linear(t["q"], h)


def latent_attention(h, t, cfg, kind, eps, shared=None):
    """shared: another layer's (latent, rotated key part). -> (output, this layer's pair)"""
    T, H, D, R, V = len(h), cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"]
    halves = kind == "latent_attention_2"
    pos = np.arange(T)
    c, kr = shared if shared is not None else latent(h, pos, t, cfg, halves, eps)
    c, kr = _round(c), _round(kr)
    q = queries(h, t, cfg, eps).reshape(T, H, D + R)
    qn, qr = _round(q[..., :D]), _round(rotate(q[..., D:], pos, cfg["rot"], halves))
    k = _round(linear(t["uk"], c)).reshape(T, H, D)
    v = _round(linear(t["uv"], c)).reshape(T, H, V)
    seen = pos[:, None] >= pos[None, :]
    out = np.zeros((T, H, V))
    for g in range(H):
        s = (qn[:, g] @ k[:, g].T + qr[:, g] @ kr.T) * cfg["scale"]
        out[:, g] = sink_softmax(np.where(seen, s, -np.inf), t["sink"][g]) @ v[:, g]
    return linear(t["o"], out.reshape(T, H * V)), (c, kr)


def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z * z, eps) + c * rms(z * z * z, eps) + e


def dense_mlp(h, t, eps):
    return linear(t["down"], poly_norm(linear(t["up"], h), t["act"], eps))


def depth_average(weights, results):
    """results: the embedding output, then every layer's result so far"""
    return sum(w * r for w, r in zip(weights, results))


def softcap(logits, cap):
    return cap * np.tanh(logits / cap) if cap else logits


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(cfg, tensors, tokens, residuals=None, rounded=False):
    """-> logits [tokens, vocab]; residuals: a list that receives what every layer passes on"""
    global _round
    if rounded:
        _round = lambda a: bf16_round(a).astype(F)
        try:
            return forward(cfg, tensors, tokens, residuals)
        finally:
            _round = lambda a: a
    T = {k: np.asarray(v, dtype=F) for k, v in tensors.items()}
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = T["embed"][np.asarray(tokens)]
    results, caches = [x], []
    for i, layer in enumerate(cfg["layers"]):
        t, mx = sub(T, "l%d." % i), layer["mixer"]
        src = mx.get("kv_from")
        y, cache = latent_attention(x, sub(t, "mix."), mx, layer["type"], eps, None if src is None else caches[src])
        caches.append(cache)
        x = model_norm(alpha * x + y, t["norm1"], eps)
        if layer.get("mlp"):
            x = model_norm(alpha * x + dense_mlp(x, sub(t, "mlp."), eps), t["norm2"], eps)
        results.append(x)
        x = depth_average(t["dwa"], results)
        if residuals is not None:
            residuals.append(x)
    return softcap(linear(T["head"], model_norm(x, T["final.norm"], eps)), cfg.get("logit_softcap"))
