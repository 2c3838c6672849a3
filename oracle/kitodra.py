"""Plain, slow Kitodra forward pass over a whole sequence (TEST INFRASTRUCTURE ONLY).

numpy in float64, one function per mechanism, no cache, no batch, no kernels. Kitodra is a decoder whose layers add a mixer and
a mixture of experts, both reading one normed input, to the stream. Mixers: differential attention inside chunks, attention over a
sliding window whose values are the unrotated keys, and linear attention with a decay per head. Keys are seen or not by a mask over
all pairs, the recurrence runs token by token, every expert is computed for every token.
"""
import numpy as np

from oracle.lozedra import bf16_round, read_tensors, sigmoid, silu, sub, write_model  # noqa: F401

F = np.float64

# What an implementation with 16-bit activations rounds: operands of matrix products. forward(.., rounded=True) sets it.
_round = lambda a: a


def rms(x, eps):
    """x divided by its root mean square"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def linear(w, h, b=None):
    """w [out, in], h [tokens, in]"""
    y = _round(h) @ w.T
    return y if b is None else y + b


def bigram_rows(tokens, cfg):
    """The row of the pair table for every token; the row behind the buckets for a sequence's first one."""
    t = np.asarray(tokens, dtype=np.int64)
    rows = np.full(len(t), cfg["buckets"])
    rows[1:] = (t[:-1] * cfg["mul_prev"] + t[1:] * cfg["mul_cur"]) % cfg["buckets"]
    return rows


def embedding(tokens, T, cfg):
    x = T["embed"][np.asarray(tokens)]
    pair = (cfg.get("embedding") or {}).get("bigram")
    return x + T["bigram"][bigram_rows(tokens, pair)] if pair else x


def rotate_halves(x, pos, dims, base):
    """x [tokens, heads, width]: dimensions i and i + dims / 2 turn together by pos * base^(-2 i / dims)"""
    n = dims // 2
    a = np.asarray(pos)[:, None, None] * (float(base) ** (-2.0 * np.arange(n) / dims))
    y = np.array(x, dtype=F)
    u, v = x[..., :n], x[..., n:dims]
    y[..., :n], y[..., n:dims] = u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)
    return y


def in_window(i, j, size):
    return (i - j >= 0) & (i - j < size)


def in_chunk(i, j, size):
    return (i - j >= 0) & (i // size == j // size)


def softcap(s, cap):
    return cap * np.tanh(s / cap) if cap else s


def softmax(s, sink=None):
    """Weights over the last axis; with a sink the denominator also holds exp(sink)."""
    m = s.max(-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink)
    e = np.exp(s - m)
    return e / (e.sum(-1, keepdims=True) + (0.0 if sink is None else np.exp(sink - m)))


def difference_weight(t, diff):
    return np.exp((t["lq1"] * t["lk1"]).sum()) - np.exp((t["lq2"] * t["lk2"]).sum()) + diff


def difference(a1, a2, lam, diff, eps):
    """Two maps' results per head -> their difference, normed over the head"""
    return rms(a1 - lam * a2, eps) * (1.0 - diff)


def differential_attention(h, t, cfg, eps):
    T, H, G, D, V = len(h), cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = linear(t["q"], h, t["q.b"]).reshape(T, H, 2, D)
    k = linear(t["k"], h, t["k.b"]).reshape(T, G, 2, D)
    v = _round(linear(t["v"], h, t["v.b"]).reshape(T, G, V))
    q, k = _round(rms(q, eps) * t["q.norm"]), _round(rms(k, eps) * t["k.norm"])
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = in_chunk(i, j, cfg["mask"]["size"])
    lam = difference_weight(t, cfg["diff"])
    out = np.zeros((T, H, V))
    for n in range(H):
        g = n // (H // G)
        a = []
        for m in range(2):
            s = softcap(q[:, n, m] @ k[:, g, m].T * cfg["scale"], cfg.get("softcap"))
            a.append(softmax(np.where(seen, s, -np.inf)) @ v[:, g])
        out[:, n] = difference(a[0], a[1], lam, cfg["diff"], eps)
    return linear(t["o"], out.reshape(T, H * V), t["o.b"])


def key_value_attention(h, t, cfg, eps):
    """Values are the keys before they turn and are normed."""
    T, H, G, D = len(h), cfg["heads"], cfg["kv_heads"], cfg["dim"]
    pos, rot = np.arange(T), cfg["rot"]
    q = linear(t["q"], h, t["q.b"]).reshape(T, H, D)
    v = linear(t["k"], h, t["k.b"]).reshape(T, G, D)
    q = _round(rms(rotate_halves(q, pos, rot["dims"], rot["base"]), eps))
    k = _round(rms(rotate_halves(v, pos, rot["dims"], rot["base"]), eps))
    v = _round(v)
    seen = in_window(pos[:, None], pos[None, :], cfg["mask"]["size"])
    out = np.zeros((T, H, D))
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].T * cfg["scale"]
        out[:, n] = softmax(np.where(seen, s, -np.inf), sink=0.0) @ v[:, g]
    return linear(t["o"], out.reshape(T, H * D), t["o.b"])


def decayed_states(q, k, v, decay, state=None):
    """q, k [tokens, heads, dim], v [tokens, heads, vdim], decay [heads] -> (outputs [tokens, heads, vdim], final state)"""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2])) if state is None else state.copy()
    o = np.zeros_like(v, dtype=F)
    for i in range(len(q)):
        S = np.asarray(decay)[:, None, None] * S + k[i][:, :, None] * v[i][:, None, :]
        o[i] = (q[i][:, :, None] * S).sum(1)
    return o, S


def gated_norm(o, w, gate, eps):
    return rms(o, eps) * w * sigmoid(gate)


def lightning(h, t, cfg, eps):
    T, H, D, V = len(h), cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k = (_round(silu(linear(t[n], h))).reshape(T, H, D) for n in "qk")
    v = _round(silu(linear(t["v"], h))).reshape(T, H, V)
    o, _ = decayed_states(q, k, v, cfg["decay"])
    return linear(t["o"], gated_norm(o.reshape(T, H * V), t["norm"], linear(t["g"], h), eps))


def expert(h, t, limit):
    g, u = np.minimum(linear(t["gate"], h), limit), np.clip(linear(t["up"], h), -limit, limit)
    return linear(t["down"], g * sigmoid(1.702 * g) * (u + 1.0))


def choose(z, correction, router):
    """Router logits z [tokens, experts] -> weights [tokens, experts], 0 where an expert is not chosen"""
    s = sigmoid(z)
    c = s + correction
    n, E = z.shape
    groups = router.get("groups")
    if groups:
        per = c.reshape(n, groups["count"], -1)
        score = np.sort(per, -1)[..., -2:].sum(-1)
        best = np.argsort(-score, -1, kind="stable")[:, :groups["keep"]]
        kept = np.zeros((n, groups["count"]), dtype=bool)
        np.put_along_axis(kept, best, True, -1)
        c = np.where(np.repeat(kept, E // groups["count"], -1), c, -np.inf)
    top = np.argsort(-c, -1, kind="stable")[:, :router["top"]]
    w = np.zeros((n, E))
    np.put_along_axis(w, top, np.take_along_axis(s, top, -1), -1)
    return w


def mixture(h, t, cfg):
    r = cfg["router"]
    w = choose(linear(t["router"], h), t["correction"], r)
    y = sum(w[:, e:e + 1] * expert(h, sub(t, "e%d." % e), cfg["expert"]["limit"]) for e in range(r["experts"]))
    if cfg.get("shared"):
        y = y + expert(h, sub(t, "shared."), cfg["shared"]["limit"])
    return y


MIXERS = {"attention": differential_attention, "attention_2": key_value_attention, "lightning": lightning}


def layer(x, t, cfg, eps):
    h = rms(x, eps) * t["norm1"]
    y = MIXERS[cfg["type"]](h, sub(t, "mix."), cfg["mixer"], eps)
    return x + (y + mixture(h, sub(t, "mlp."), cfg["mlp"]) if cfg.get("mlp") else y)


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
    x = embedding(tokens, T, cfg)
    for i, c in enumerate(cfg["layers"]):
        own = c.get("weights_of")
        x = layer(x, sub(T, "l%d." % (i if own is None else own)), c, eps)
        if residuals is not None:
            residuals.append(x)
    return linear(T["embed"], rms(x, eps) * T["final.norm"])
