"""Plain, slow Lozedra forward pass over a whole sequence (TEST INFRASTRUCTURE ONLY).

numpy in float64, one function per mechanism, no cache, no batch, no kernels: a token's row is computed from all the
tokens before it each time. Lozedra is a decoder whose layers run two mixers side by side over the same input, grouped
attention without rotation (a learned bias per head and distance bucket, a query temperature, an output gate) and a
selective scan, with a norm before and after every sublayer and a range of layers that is run several times.
"""
import json
import math
import struct

import numpy as np

F = np.float64


def rms_norm(x, w, eps):
    x = x.astype(F)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def silu(z):
    return z / (1.0 + np.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


# What an implementation with 16-bit activations rounds: the inputs of linear maps and the operands of attention. The
# default keeps everything as it is; forward(.., rounded=True) uses bfloat16, to measure what that rounding alone does.
_round = lambda a: a


def linear(w, h):
    """w [out, in], h [tokens, in]"""
    return _round(h) @ w.T


def distance_bucket(n, rows, bias_max):
    """Bucket of a distance n >= 0: its own for the first half of the table, logarithmic beyond, the last one from
    bias_max on. Where the logarithm is a whole number (n = half * ratio^(i / (rows - half))) it counts as reached."""
    half = rows // 2
    if n < half:
        return n
    v = math.log(n / half) / math.log(bias_max / half) * (rows - half)
    near = round(v)
    v = near if abs(v - near) < 1e-9 else math.floor(v)
    return min(rows - 1, half + int(v))


def distance_bias(rel, bias_max, n_max):
    """[heads, n_max + 1]: what is added to a score at every distance"""
    b = [distance_bucket(n, rel.shape[0], bias_max) for n in range(n_max + 1)]
    return rel[b].T


def query_temperature(pos, coef, every):
    return 1.0 + coef * np.log(np.floor((pos + 1) / every) + 1.0)


def attention(h, t, cfg):
    """t: tensors q, k, v, g, o, rel of one layer; positions 0 .. len(h) - 1"""
    T, H, G, D, V = len(h), cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = linear(t["q"], h).reshape(T, H, D)
    k = _round(linear(t["k"], h)).reshape(T, G, D)
    v = _round(linear(t["v"], h)).reshape(T, G, V)
    q = _round(q)
    pos = np.arange(T)
    qt = cfg.get("q_temp")
    if qt:
        q = q * query_temperature(pos, qt["coef"], qt["every"])[:, None, None]
    bias = distance_bias(t["rel"], cfg["bias_max"], max(T - 1, 0))
    out = np.zeros((T, H, V))
    dist = pos[:, None] - pos[None, :]
    for hd in range(H):
        g = hd // (H // G)
        s = q[:, hd] @ k[:, g].T * cfg["scale"] + bias[hd][np.maximum(dist, 0)]
        s = np.where(dist >= 0, s, -np.inf)
        s = np.exp(s - s.max(-1, keepdims=True))
        out[:, hd] = s / s.sum(-1, keepdims=True) @ v[:, g]
    o = out.reshape(T, H * V) * sigmoid(linear(t["g"], h))
    return linear(t["o"], o)


def causal_conv(x, w, b):
    """x [tokens, channels], w [channels, taps] with the last column the current token's"""
    T, taps = len(x), w.shape[1]
    p = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(p[i:i + T] * w[:, i] for i in range(taps)) + b


def selective_scan(x, dt, A, B, C, D, state=None):
    """x, dt [tokens, channels]; A [channels, state]; B, C [tokens, state] -> (y, final state)"""
    s = np.zeros(A.shape) if state is None else state.copy()
    y = np.zeros_like(x)
    for i in range(len(x)):
        s = np.exp(dt[i][:, None] * A) * s + (dt[i] * x[i])[:, None] * B[i][None, :]
        y[i] = s @ C[i] + D * x[i]
    return y, s


def mamba(h, t, cfg):
    n, r, s = cfg["inner"], cfg["dt_rank"], cfg["state"]
    xz = linear(t["in"], h)
    x, z = xz[:, :n], xz[:, n:]
    x = silu(causal_conv(x, t["conv"], t["conv.b"]))
    p = linear(t["x"], x)
    dt = softplus(linear(t["dt"], p[:, :r]) + t["dt.b"])
    y, _ = selective_scan(x, dt, -np.exp(t["A_log"]), p[:, r:r + s], p[:, r + s:], t["D"])
    return linear(t["o"], y * silu(z))


def dense_mlp(h, t):
    return linear(t["down"], silu(linear(t["gate"], h)) * linear(t["up"], h))


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def layer(x, t, cfg, eps, mult):
    mx = cfg["mixer"]
    h = rms_norm(x, t["norm1"], eps)
    y = mx["left_scale"] * attention(h, sub(t, "mix.left."), mx["left"]) + \
        mx["right_scale"] * mamba(h, sub(t, "mix.right."), mx["right"])
    x = x + mult * rms_norm(y, t["norm1b"], eps)
    if cfg["mlp"] is not None:
        h = rms_norm(x, t["norm2"], eps)
        x = x + mult * rms_norm(dense_mlp(h, sub(t, "mlp.")), t["norm2b"], eps)
    return x


def layer_order(cfg):
    """[(layer, whether the embedding output is added first)]"""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    body = range(lp["start"], lp["stop"])
    runs = [(i, False) for i in range(lp["start"])]
    for p in range(lp["times"]):
        runs += [(i, p > 0 and i == lp["start"]) for i in body]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def forward(cfg, tensors, tokens, residuals=None, rounded=False):
    """-> logits [tokens, vocab]; residuals: a list that receives the stream after every layer run"""
    global _round
    if rounded:
        _round = lambda a: bf16_round(a).astype(F)
        try:
            return forward(cfg, tensors, tokens, residuals)
        finally:
            _round = lambda a: a
    T = {k: np.asarray(v, dtype=F) for k, v in tensors.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    emb = T["embed"][np.asarray(tokens)]
    x = emb
    for i, again in layer_order(cfg):
        if again:
            x = x + emb
        x = layer(x, sub(T, "l%d." % i), cfg["layers"][i], eps, mult)
        if residuals is not None:
            residuals.append(x)
    return linear(T["head"], rms_norm(x, T["final.norm"], eps))


# ---- files (the same format the product reads, by code of its own)
def bf16_round(a):
    """float32 values nearest in bfloat16 (ties to even)"""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    return (((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16).astype(np.uint32).view(np.float32)


def write_model(folder, cfg, tensors):
    """config.json + model.safetensors with every tensor in bfloat16"""
    import os
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {}, [], 0
    for name, a in tensors.items():
        raw = (bf16_round(a).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    js = json.dumps(head).encode()
    js += b" " * (-len(js) % 8)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(js)) + js)
        for b in blobs:
            f.write(b)


def read_tensors(path):
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        head = json.loads(f.read(n))
        base = f.read()
    out = {}
    for name, d in head.items():
        if name == "__metadata__":
            continue
        lo, hi = d["data_offsets"]
        assert d["dtype"] == "BF16"
        u = np.frombuffer(base[lo:hi], dtype="<u2").astype(np.uint32) << 16
        out[name] = u.view(np.float32).reshape(d["shape"])
    return out
