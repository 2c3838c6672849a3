"""Kitodra on the GPU: each kernel alone against the plain implementation, then models through the engine's loader, block
pool, step, scheduler and graph replay."""
import json
import os
import subprocess

import numpy as np
import pytest

from kitodra_models import (EVEN, LIMIT, SMALL, TINY, WIDE, config, differential, error, key_value, lightning, limit, margin, moe, tensors)
from mixed_batches import ACTS, BF16, BS, F32, Batch, blank, close, down, grid, lin_out, packed, prompt, run_portions, up
from oracle import kitodra as kt

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
pad = lambda n, m: -(-n // m) * m


@pytest.fixture(scope="module")
def be():
    from vexel_amd.backend import HipBackend
    b = HipBackend(0)
    yield b
    b.close()


@pytest.fixture(autouse=True)
def fresh_pool(be):
    be.reset_pool()


# prompts, later portions, single tokens; at the edges of blocks (16), of groups of keys (32) and of pieces
MIXED = ([0, 5, 300, 31, 62, 15, 127, 255, 0, 63], [70, 2, 1, 1, 3, 40, 1, 2, 1, 2])
SINGLE = ([0, 1, 15, 16, 63, 64, 127, 128, 255, 256, 257, 400], [1] * 12)


# ---------------------------------------------------------------- embedding
@pytest.mark.parametrize("cols", [3, 64, 200])
def test_pair_embedding(be, cols):
    """Mixed batches and single tokens; the token before a portion comes from the pool's slots, whatever else they hold."""
    from vexel_amd.backend import VxPairEmbeddingArgs
    rng = np.random.default_rng(cols)
    V, cfg = 50, {"buckets": 37, "mul_prev": 2147483647, "mul_cur": 131}
    emb, pairs = rng.standard_normal((V, cols)).astype(np.float32), rng.standard_normal((38, cols)).astype(np.float32)
    for batch in (MIXED, SINGLE):
        bt = Batch(be, *batch, seed=cols)
        seqs = [rng.integers(0, V, n) for n in bt.kv]
        pool = rng.integers(0, V, bt.pool_blocks * BS).astype(np.int32)
        for i, s in enumerate(seqs):
            for t in range(bt.start[i]):
                pool[bt.slot(i, t)] = s[t]
        tokens = np.concatenate([s[bt.start[i]:] for i, s in enumerate(seqs)]).astype(np.int32)
        p = VxPairEmbeddingArgs()
        p.cols, p.vocab, p.buckets, p.mul_prev, p.mul_cur = cols, V, 37, cfg["mul_prev"], cfg["mul_cur"]
        p.tokens, p.embed, p.pairs = be.upload(tokens), be.upload(emb), be.upload(pairs)
        p.token_pool, p.out = be.upload(pool), blank(be, (bt.rows, cols), F32)
        be.pair_embedding(bt.c, p)
        want = np.concatenate([(emb[s] + pairs[kt.bigram_rows(s, cfg)])[bt.start[i]:] for i, s in enumerate(seqs)])
        assert np.array_equal(down(be, p.out, (bt.rows, cols), F32), want)
        after = be.download(p.token_pool, (len(pool),), np.int32)
        for i, s in enumerate(seqs):
            assert all(after[bt.slot(i, t)] == s[t] for t in range(bt.kv[i]))
        be.reset_pool()


# ---------------------------------------------------------------- heads to their places
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", [(6, 2, 2, 12, 28, 0), (3, 1, 1, 22, 22, 4), (4, 4, 2, 64, 128, 0), (8, 2, 2, 128, 128, 32), (2, 2, 2, 200, 200, 100), (1, 1, 1, 300, 300, 7),
                                  (5, 5, 5, 2, 2, 1), (2, 1, 1, 40, 8, 4)])
def test_heads_store(be, act, geom):
    """Slices and biases, rotation of a part or all of a head, norms with and without a weight, values apart or from the keys."""
    from vexel_amd.backend import VxHeadsArgs
    HQ, HK, HV, D, X, pairs = geom
    rng = np.random.default_rng(D)
    eps = 1e-3
    for batch in (MIXED, SINGLE):
        for own, norm, weighted, biased, slices in ((True, 1, True, True, 3), (False, 1, False, False, 1), (True, 0, False, True, 1), (False, 0, False, True, 2)):
            if not own and (HV != HK or X != D):
                continue
            bt = Batch(be, *batch, seed=D)
            qc, kc = 16, 16 + pad(HQ * D, 16)
            vc = kc + pad(HK * D, 16)
            ld = vc + pad(HV * X, 16) + 16
            y = (rng.standard_normal((slices, bt.rows, ld)) * rng.uniform(0.02, 3, (bt.rows, 1))).astype(np.float32)
            bias = rng.standard_normal(ld).astype(np.float32)
            wq, wk = (1 + 0.3 * rng.standard_normal((2, D))).astype(np.float32)
            ang = bt.pos[:, None] * 50.0 ** (-np.arange(max(pairs, 1)) / max(pairs, 1))
            p = VxHeadsArgs()
            p.q_heads, p.k_heads, p.v_heads, p.dim, p.v_dim = HQ, HK, HV, D, X
            p.y, p.y_slices, p.ldy, p.y_stride = be.upload(y), slices, ld, bt.rows * ld
            p.q_col, p.k_col, p.v_col, p.rot_pairs, p.norm, p.eps = qc, kc, vc if own else -1, pairs, norm, eps
            if biased:
                p.bias = be.upload(bias)
            if pairs:
                p.rot_tab = be.upload(np.stack([np.cos(ang), np.sin(ang)], -1).astype(np.float32))
            if weighted:
                p.w_q, p.w_k = be.upload(wq), be.upload(wk)
            ldq, kp = pad(HQ * D, 8) + 8, pad(D, 8)
            per = BS * (HK * kp + HV * X)
            assert be.lib_call("vx_kv_block_elems2", BS, HK, D, HV, X) == per
            p.q, p.ldq, p.pool = blank(be, (bt.rows, ldq), act), ldq, blank(be, (bt.pool_blocks, per), act)
            be.heads_store(act, bt.c, p)
            s = y.astype(np.float64).sum(0) + (bias if biased else 0)
            q, k = s[:, qc:qc + HQ * D].reshape(-1, HQ, D), s[:, kc:kc + HK * D].reshape(-1, HK, D)
            v = s[:, vc:vc + HV * X].reshape(-1, HV, X) if own else k

            def want(x, w):
                if pairs:
                    u, z = x[..., :pairs].copy(), x[..., pairs:2 * pairs].copy()
                    x = x.copy()
                    c, n = np.cos(ang)[:, None], np.sin(ang)[:, None]
                    x[..., :pairs], x[..., pairs:2 * pairs] = u * c - z * n, z * c + u * n
                return (kt.rms(x, eps) if norm else x) * (w if weighted else 1)

            got = down(be, p.q, (bt.rows, ldq), act)
            close(got[:, :HQ * D].reshape(-1, HQ, D), want(q, wq), act, geom)
            assert np.isnan(got[:, HQ * D:]).all()
            pool = down(be, p.pool, (bt.pool_blocks, per), act)
            kk = pool[:, :BS * HK * kp].reshape(-1, HK, BS, kp).transpose(0, 2, 1, 3).reshape(-1, HK, kp)
            vv = pool[:, BS * HK * kp:].reshape(-1, HV, X, BS).transpose(0, 3, 1, 2).reshape(-1, HV, X)
            close(kk[bt.slot_map][..., :D], want(k, wk), act, geom)
            close(vv[bt.slot_map], v, act, geom)
            assert np.isnan(np.delete(kk, bt.slot_map, 0)).all() and np.isnan(np.delete(vv, bt.slot_map, 0)).all()
            be.reset_pool()


# ---------------------------------------------------------------- attention
def run_attn(be, act, bt, H, G, D, X, maps=1, window=0, chunk=0, cap=0.0, sinks=False, seed=0, lam=0.7, diff=0.4, scale=None, change=None, min_rows=0):
    """vx_attn_ragged against masked softmax over every pair; tokens outside the sequences hold large numbers."""
    from vexel_amd.backend import VxAttnArgs
    rng = np.random.default_rng(seed)
    q = rng.standard_normal((bt.rows, H, maps, D))
    ks = [rng.standard_normal((n, G, maps, D)) for n in bt.kv]
    vs = [rng.standard_normal((n, G, X)) for n in bt.kv]
    if change:
        change(q, ks, vs)
    q, ks, vs = grid(q, act), [grid(k, act) for k in ks], [grid(v, act) for v in vs]
    scale = scale or 1.5 / D ** 0.5
    kp = pad(D, 8)
    pool = rng.standard_normal((bt.pool_blocks, BS * G * (maps * kp + X))) * 60
    kk, vv = pool[:, :BS * G * maps * kp].reshape(-1, G * maps, BS, kp), pool[:, BS * G * maps * kp:].reshape(-1, G, X, BS)
    kk[..., D:] = 0
    for i, n in enumerate(bt.kv):
        for t in range(n):
            s = bt.slot(i, t)
            kk[s // BS, :, s % BS, :D], vv[s // BS, :, :, s % BS] = ks[i][t].reshape(G * maps, D), vs[i][t]
    sink = (rng.standard_normal(H * maps) * 2).astype(np.float32)
    p = VxAttnArgs()
    p.heads, p.kv_heads, p.k_dim, p.v_dim, p.scale, p.out_scale, p.min_rows = H, G, D, X, scale, 1.0, min_rows
    p.window, p.chunk, p.softcap, p.maps, p.diff_lambda, p.diff_scale, p.diff_eps = window, chunk, cap, maps, lam, 1 - diff, 1e-5
    p.q, p.ldq, p.pool, p.out, p.ldo = up(be, q, act), H * maps * D, up(be, pool, act), blank(be, (bt.rows, H, X), act), H * X
    if sinks:
        p.sink = be.upload(sink)
    be.attn_ragged(act, bt.c, p)
    got = down(be, p.out, (bt.rows, H, X), act)
    for i in range(len(bt.lens)):
        r = slice(bt.cu[i], bt.cu[i + 1])
        if bt.lens[i] < min_rows:
            assert np.isnan(got[r]).all()
            continue
        a, b = bt.pos[r][:, None], np.arange(bt.kv[i])[None, :]
        seen = a >= b
        if window:
            seen = seen & kt.in_window(a, b, window)
        if chunk:
            seen = seen & kt.in_chunk(a, b, chunk)
        for h in range(H):
            g, o = h // (H // G), []
            for m in range(maps):
                s = kt.softcap(q[r, h, m].astype(np.float64) @ ks[i][:, g, m].T.astype(np.float64) * scale, cap)
                o.append(kt.softmax(np.where(seen, s, -np.inf), sink[h * maps + m] if sinks else None) @ vs[i][:, g].astype(np.float64))
            want = o[0] if maps == 1 else kt.difference(o[0], o[1], lam, diff, 1e-5)
            close(got[r, h], want, act, (i, bt.start[i], bt.lens[i], h))
    return got


# (heads, K/V heads, key size, value size, maps): each matrix-core geometry, narrower heads than it holds, and some that only the plain
# kernel takes
GEOMETRIES = [(4, 2, 12, 28, 2), (8, 2, 64, 64, 2), (6, 1, 48, 96, 2), (4, 4, 64, 128, 2), (8, 1, 100, 120, 2), (2, 1, 128, 256, 2), (2, 1, 200, 40, 2), (17, 1, 30, 20, 2),
              (1, 1, 1, 1, 2), (3, 1, 22, 22, 1), (8, 2, 128, 128, 1), (20, 1, 136, 136, 1), (2, 2, 256, 256, 1), (2, 1, 270, 9, 1)]


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", GEOMETRIES)
def test_attention_geometries(be, act, geom):
    H, G, D, X, maps = geom
    for batch in (MIXED, SINGLE):
        bt = Batch(be, *batch, seed=D)
        for kw in (dict(window=50), dict(chunk=64, cap=6.0), dict(sinks=True, cap=3.0, lam=-0.5)):  # (no difference that nearly vanishes)
            run_attn(be, act, bt, H, G, D, X, maps, **kw)
        be.reset_pool()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("size", [1, 2, 15, 16, 17, 31, 32, 33, 64, 100, 255, 256, 257, 401, 5000])
def test_windows_and_chunks_of_every_size(be, act, size):
    for batch in (MIXED, SINGLE):
        bt = Batch(be, *batch, seed=size)
        for maps in (1, 2):
            for kw in (dict(window=size), dict(chunk=size), dict(window=size, chunk=2 * size)):
                run_attn(be, act, bt, 4, 2, 16, 24, maps, sinks=maps == 1, seed=size, **kw)
        be.reset_pool()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("pos", [0, 1, 30, 63, 64, 65, 127, 128, 300, 700])
@pytest.mark.parametrize("maps", [1, 2])
def test_keys_at_the_edges_stand_out(be, act, pos, maps):
    """One key with a score far above the others', just inside and just outside the edge of what the last row sees: in prompts, in
    short portions and decoded alone."""
    for size in (1, 37, 64, 130):
        for kind in ("window", "chunk"):
            first = max(0, pos - size + 1) if kind == "window" else pos - pos % size
            for key in {first, first - 1, pos, 0}:
                if key < 0:
                    continue

                def stand_out(q, ks, vs):
                    q[-1, ..., 3] = 6.0
                    ks[0][..., 3] = 0.0
                    ks[0][key, ..., 3] = 10.0
                    vs[0][key] *= 4

                for rows in {1, min(2, pos + 1), min(40, pos + 1)}:
                    run_attn(be, act, Batch(be, [pos + 1 - rows], [rows], seed=pos), 2, 1, 16, 16, maps, change=stand_out, scale=0.5, seed=pos, **{kind: size})
                be.reset_pool()


@pytest.mark.parametrize("maps", [1, 2])
@pytest.mark.parametrize("start,lens", [(0, [700]), (900, [33]), (0, [2200]), (1500, [64, 1])])
def test_attention_of_long_portions(be, maps, start, lens):
    """Each arrangement of waves of the prompt kernel, with windows and chunks that begin inside a tile of rows."""
    for kw in (dict(window=200), dict(chunk=333), dict()):
        run_attn(be, BF16, Batch(be, [start] * len(lens), lens, seed=1), 16, 2, 32, 32, maps, **kw)
        be.reset_pool()


def test_attention_of_many_decoding_sequences(be):
    """Enough sequences that pieces come from the step's list."""
    rng = np.random.default_rng(6)
    bt = Batch(be, rng.integers(0, 900, 130).tolist(), [1] * 130, seed=6)
    for maps in (1, 2):
        for kw in (dict(), dict(window=300), dict(chunk=512), dict(chunk=4096)):
            run_attn(be, BF16, bt, 8, 4, 32, 32, maps, seed=2, **kw)


def test_rows_left_out(be):
    for act in ACTS:
        for least in (2, 40):
            run_attn(be, act, Batch(be, *MIXED, seed=4), 4, 2, 24, 24, 2, min_rows=least, window=30)


# ---------------------------------------------------------------- decaying states
def run_decay(be, act, bt, H, D, X, decay, seed=0, calls=1):
    from vexel_amd.backend import VxDecayArgs
    rng = np.random.default_rng(seed)
    slots = max(bt.slots) + 2
    ldq, ldv = H * D + 16, H * X + 8
    q, k = (grid(rng.standard_normal((bt.rows, H, D)), act) for _ in range(2))
    v = grid(rng.standard_normal((bt.rows, H, X)), act)
    state = rng.standard_normal((slots, H, D, X)).astype(np.float32)
    wide = lambda a, ld: np.concatenate([a.reshape(bt.rows, -1), np.full((bt.rows, ld - a[0].size), np.nan)], 1)
    p = VxDecayArgs()
    p.heads, p.dim, p.vdim = H, D, X
    d = np.asarray(decay, dtype=np.float64)
    p.decay = be.upload(np.stack([d - 1, np.maximum(np.log2(np.maximum(d, 1e-300)), -1e4)], 1).astype(np.float32))
    p.q, p.k, p.v, p.ldq, p.ldk, p.ldv = up(be, wide(q, ldq), act), up(be, wide(k, ldq), act), up(be, wide(v, ldv), act), ldq, ldq, ldv
    p.state, p.out, p.ldo = be.upload(state), blank(be, (bt.rows, H * X + 4), F32), H * X + 4
    be.decay_attn(act, bt.c, p)
    got = down(be, p.out, (bt.rows, H * X + 4), F32)
    after = down(be, p.state, state.shape, F32)
    assert np.isnan(got[:, H * X:]).all()
    used = set()
    for i in range(len(bt.lens)):
        r, s = slice(bt.cu[i], bt.cu[i + 1]), bt.slots[i]
        o, S = kt.decayed_states(q[r].astype(np.float64), k[r].astype(np.float64), v[r].astype(np.float64), d, state[s].astype(np.float64) if bt.start[i] else None)
        tol = F32 if act == F32 else BF16                       # (two bfloat16 parts: far below 1.2e-2)
        close(got[r, :H * X].reshape(-1, H, X), o, tol, (i, bt.start[i], bt.lens[i]))
        assert np.abs(got[r, :H * X].reshape(-1, H, X) - o).max() < 2e-4 * np.abs(o).max()
        close(after[s], S, F32 if act == F32 or bt.lens[i] <= 16 else BF16)
        assert np.abs(after[s] - S).max() < 2e-4 * np.abs(S).max()
        used.add(s)
    for s in range(slots):
        if s not in used:
            assert np.array_equal(after[s], state[s])          # nobody else's state moves


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", [(3, 32, 16), (2, 64, 48), (1, 160, 144), (4, 128, 128), (2, 96, 272), (1, 512, 512), (2, 256, 32)])
def test_decaying_states(be, act, geom):
    H, D, X = geom
    rng = np.random.default_rng(D)
    decay = [0.0, 1.0, 0.999, 0.6][:H] if H > 1 else [0.98]
    for batch in (MIXED, SINGLE, ([0, 40, 7], [300, 1, 17]), ([5, 0], [16, 129])):
        run_decay(be, act, Batch(be, *batch, seed=D), H, D, X, decay, seed=D)
        be.reset_pool()


@pytest.mark.parametrize("rows", [2, 8, 9, 16, 17, 63, 64, 65, 127, 128, 129, 191, 192, 193, 256, 257])
def test_portions_of_decaying_states(be, rows):
    """Around every border of sub-chunks and chunks, from nothing and from an earlier state."""
    for start in (0, 3):
        run_decay(be, BF16, Batch(be, [start, 9], [rows, 1], seed=rows), 2, 64, 64, [0.9, 0.999], seed=rows)
        be.reset_pool()


def test_long_portions_of_decaying_states(be):
    """Enough rows and heads for chunks of two sub-chunks, several sequences, a last chunk with one sub-chunk and a short one."""
    run_decay(be, BF16, Batch(be, [0, 50, 4], [1300, 800, 1], seed=1), 32, 32, 32, np.linspace(0.5, 0.9995, 32), seed=1)
    be.reset_pool()
    run_decay(be, BF16, Batch(be, [0], [2100], seed=2), 32, 32, 16, np.linspace(0.5, 0.9995, 32), seed=2)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("cols,count", [(5, 5), (48, 40), (96, 96), (4096, 4096), (9000, 8999), (20000, 20000)])
def test_gated_norm(be, act, cols, count):
    rng = np.random.default_rng(cols)
    for rows in (1, 9, 300):
        if rows * cols > 2_000_000:
            continue
        x = (rng.standard_normal((rows, cols)) * rng.uniform(1e-3, 30, (rows, 1))).astype(np.float32)
        x[:, count:] = 0
        g, w = rng.standard_normal((rows, cols + 8)).astype(np.float32) * 3, (1 + 0.3 * rng.standard_normal(cols)).astype(np.float32)
        ldo = pad(cols, 64)
        out = blank(be, (rows, ldo), act)
        be.gated_norm(act, up(be, x), cols, up(be, g), cols + 8, up(be, w), 1e-3, rows, cols, count, out, ldo)
        got = down(be, out, (rows, ldo), act)
        xs = x.astype(np.float64)
        close(got[:, :cols], xs / np.sqrt((xs * xs).sum(-1, keepdims=True) / count + 1e-3) * w * kt.sigmoid(g[:, :cols]), act)
        assert np.all(got[:, cols:] == 0)
        be.reset_pool()


# ---------------------------------------------------------------- experts
def route(be, z, correction, top, groups, keep, shared, tile):
    from vexel_amd.backend import VxRouteArgs
    slices, rows, E = z.shape
    ld = E + 3
    zz = np.full((slices, rows, ld), np.nan, dtype=np.float32)
    zz[..., :E] = z
    p = VxRouteArgs()
    p.rows, p.experts, p.top, p.groups, p.keep, p.shared, p.tile_rows = rows, E, top, groups, keep, shared, tile
    p.z, p.z_slices, p.ldz, p.z_stride = be.upload(zz), slices, ld, rows * ld
    if correction is not None:
        p.correction = be.upload(correction.astype(np.float32))
    most = be.lib_call("vx_route_max_tiles", rows, E, top, shared, tile)
    p.weights, p.places = blank(be, (rows, top), F32), be.upload(np.full((rows, top), -1, dtype=np.int32))
    p.order, p.tiles = be.upload(np.full(rows * (top + shared), -1, dtype=np.int32)), be.upload(np.full(4 + 4 * most, -1, dtype=np.int32))
    be.route(p)
    return (p, be.download(p.weights, (rows, top), np.float32), be.download(p.places, (rows, top), np.int32),
            be.download(p.order, (rows * (top + shared),), np.int32), be.download(p.tiles, (1 + most, 4), np.int32))


@pytest.mark.parametrize("experts,top,groups,keep", [(1, 1, 1, 1), (9, 4, 9, 6), (12, 3, 3, 2), (16, 4, 4, 2), (64, 6, 8, 4), (65, 8, 1, 1), (130, 5, 10, 3), (256, 8, 8, 4),
                                                     (1024, 10, 32, 5), (8, 8, 2, 2), (8, 4, 2, 1)])
def test_routing(be, experts, top, groups, keep):
    rng = np.random.default_rng(experts)
    for rows in (1, 7, 32, 64, 65, 300):
        for slices, corrected, shared, tile in ((1, True, 1, 64), (3, False, 0, 128), (2, True, 0, 5)):
            z = (rng.standard_normal((slices, rows, experts)) * 1.5).astype(np.float32)
            c = rng.uniform(-1.5, 0.5, experts) if corrected else None
            p, w, places, order, tiles = route(be, z, c, top, groups, keep, shared, tile)
            zs = z.astype(np.float64).sum(0)
            r = {"top": top, "groups": {"count": groups, "keep": keep} if groups > 1 else None}
            c32 = np.zeros(experts) if c is None else c.astype(np.float32).astype(np.float64)
            want = kt.choose(zs, c32, r)
            clear = margin(kt.sigmoid(zs) + c32, r) > 1e-5
            assert clear.mean() > 0.7
            # the places are the pairs sorted by expert, each once
            pairs = rows * top
            assert np.array_equal(np.sort(places.ravel()), np.arange(pairs))
            assert np.array_equal(order[places.ravel()], np.repeat(np.arange(rows), top))
            if shared:
                assert np.array_equal(order[pairs:], np.arange(rows))
            n_tiles = tiles[0, 0]
            expert_of, at = np.full(rows * (top + shared), -1), 0
            for e, first, n, _ in tiles[1:1 + n_tiles]:
                assert first == at and 1 <= n <= tile
                expert_of[first:first + n] = e
                at += n
            assert at == rows * (top + shared) and np.all(np.diff(expert_of) >= 0) and (not shared or np.all(expert_of[pairs:] == experts))
            assert np.all(expert_of[:pairs] < experts)
            chosen = expert_of[places]
            got = np.zeros((rows, experts))
            np.put_along_axis(got, chosen, w, -1)
            assert np.abs(got - want)[clear].max() < 1e-6
            assert all(len(set(x)) == top for x in chosen.tolist())
            be.reset_pool()


def test_routing_of_equal_scores(be):
    """Equal choice scores go by number, so that every row has its experts."""
    for rows in (3, 100):
        z = np.zeros((1, rows, 70), dtype=np.float32)
        z[:, 1::2, 69] = 1.0
        _, w, places, order, tiles = route(be, z, None, 3, 1, 1, 0, 64)
        expert_of = np.concatenate([np.full(n, e) for e, _, n, _ in tiles[1:1 + tiles[0, 0]]])
        got = np.sort(expert_of[places], -1)
        assert np.array_equal(got[0], [0, 1, 2]) and np.array_equal(got[1], [0, 1, 69])


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("E,top,W,ff,shared_ff", [(5, 2, 40, 24, 0), (12, 3, 88, 33, 70), (16, 4, 128, 64, 64), (4, 4, 200, 100, 17), (1, 1, 64, 1, 1), (40, 1, 96, 130, 200)])
def test_experts(be, act, E, top, W, ff, shared_ff):
    """Both maps of every expert over rows that were sorted, and the weighted sum in the seam; few rows, many, and many to one expert."""
    from vexel_amd.backend import VxExpertsArgs, VxResidualNormArgs
    rng = np.random.default_rng(E)
    shared, limits = int(shared_ff > 0), (0.7, 1.1)
    t = {"e%d.%s" % (e, n): kt.bf16_round(rng.standard_normal(s) / np.sqrt(s[1]) * 1.5) for e in range(E) for n, s in
         (("gate", (ff, W)), ("up", (ff, W)), ("down", (W, ff)))}
    if shared:
        t.update({"shared." + n: kt.bf16_round(rng.standard_normal(s) / np.sqrt(s[1]) * 1.5) for n, s in
                  (("gate", (shared_ff, W)), ("up", (shared_ff, W)), ("down", (W, shared_ff)))})
    wk, wn = pad(W, 64), pad(W, 32)

    def pack(names, f):
        fp = pad(f, 64)
        gu, dn = be.alloc(len(names) * 2 * fp * wk * 2), be.alloc(len(names) * wn * fp * 2)
        be.fill_zero(gu, len(names) * 2 * fp * wk * 2), be.fill_zero(dn, len(names) * wn * fp * 2)
        for i, n in enumerate(names):
            packed(be, t[n + ".gate"], len(names) * 2 * fp, wk, i * 2 * fp // 16, 2, dst=gu)
            packed(be, t[n + ".up"], len(names) * 2 * fp, wk, i * 2 * fp // 16 + 1, 2, dst=gu)
            packed(be, t[n + ".down"], len(names) * wn, fp, i * wn // 16, 1, dst=dn)
        return gu, dn, fp

    for rows in (1, 16, 17, 32, 33, 64, 65, 200, 700):
        be.reset_pool()
        gu, dn, fp = pack(["e%d" % e for e in range(E)], ff)
        sgu, sdn, sfp = pack(["shared"], shared_ff) if shared else (0, 0, 0)
        h = grid(rng.standard_normal((rows, W)), act)
        hp = np.zeros((rows, wk))
        hp[:, :W] = h
        z = (rng.standard_normal((1, rows, E)) * 2).astype(np.float32)
        if rows % 2:
            z[:, :, 0] += 9                                     # one expert that nearly every row takes
        tile = be.lib_call("vx_route_tile_rows", act, rows, E, top)
        r, w, places, order, tiles = route(be, z, None, top, 1, 1, shared, tile)
        n_places, ldo = rows * (top + shared), max(fp, sfp)
        g = VxExpertsArgs()
        g.kind, g.rows, g.experts, g.shared, g.tile_rows = 1, rows, E, shared, tile
        g.max_tiles = be.lib_call("vx_route_max_tiles", rows, E, top, shared, tile)
        g.tiles, g.a_rows, g.a, g.lda = r.tiles, r.order, up(be, hp, act), wk
        g.w, g.n, g.k, g.w_shared, g.n_shared, g.k_shared = gu, 2 * fp, wk, sgu, 2 * sfp, wk
        g.glu_limit, g.shared_limit, g.glu_alpha, g.glu_add = limits[0], limits[1], 1.702, 1.0
        mid = blank(be, (n_places, ldo), act)
        g.out, g.ldo, g.cols, g.cols_shared = mid, ldo, fp, sfp
        be.linear_experts(act, g)
        g.kind, g.a, g.lda, g.a_rows = 0, mid, ldo, None
        g.w, g.n, g.k, g.w_shared, g.n_shared, g.k_shared = dn, wn, fp, sdn, wn, sfp
        out = blank(be, (n_places, wn), act)
        g.out, g.ldo, g.cols, g.cols_shared = out, wn, wn, wn
        be.linear_experts(act, g)
        got = down(be, out, (n_places, wn), act)
        expert_of = np.concatenate([np.full(n, e) for e, _, n, _ in tiles[1:1 + tiles[0, 0]]])
        assert np.all(got[:, W:] == 0)
        with np.errstate(over="ignore"):
            for e in range(E + shared):
                at = np.flatnonzero(expert_of == e)
                if len(at):
                    name, lim = ("e%d" % e, limits[0]) if e < E else ("shared", limits[1])
                    x = h[order[at]].astype(np.float64)
                    close(got[at, :W], kt.expert(x, {n: v.astype(np.float64) for n, v in kt.sub(t, name + ".").items()}, lim), act, (rows, e))
        # the seam adds them up
        x = rng.standard_normal((rows, W)).astype(np.float32)
        y = rng.standard_normal((2, rows, wn)).astype(np.float32)
        b, nw = rng.standard_normal(W).astype(np.float32), (1 + 0.3 * rng.standard_normal(W)).astype(np.float32)
        for idx in (None, rng.integers(0, rows, 3).astype(np.int32)):
            n = rows if idx is None else len(idx)
            s = VxResidualNormArgs()
            s.rows, s.cols, s.x_in, s.mult, s.eps = n, W, up(be, x), 1.0, 1e-4
            s.y, s.y_slices, s.ldy, s.y_stride, s.y_bias = up(be, y), 2, wn, rows * wn, up(be, b)
            s.e_rows, s.lde, s.e_top, s.e_shared, s.e_places, s.e_weights = out, wn, top, rows * top if shared else -1, r.places, r.weights
            s.w_pre, s.ldo, s.out = up(be, nw), wk, blank(be, (n, wk), act)
            if idx is None:
                s.x_out = blank(be, (rows, W), F32)
            else:
                s.row_idx = be.upload(idx)
            be.residual_norm(act, s)
            want = x.astype(np.float64) + y.astype(np.float64).sum(0)[:, :W] + b + (w[..., None] * got[places][..., :W]).sum(1)
            if shared:
                want = want + got[rows * top:, :W]
            if idx is None:
                close(down(be, s.x_out, (rows, W), F32), want, F32)
            else:
                want = want[idx]
            o = down(be, s.out, (n, wk), act)
            close(o[:, :W], kt.rms(want, 1e-4) * nw, act)
            assert np.all(o[:, W:] == 0)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [1, 20, 50, 70, 300])
def test_linear_with_silu_on_a_part(be, act, rows):
    """Columns below the split through SiLU, the others as they are in float32; whole, and in slices where the map is deep."""
    rng = np.random.default_rng(rows)
    for n, k, split in ((80, 100, 48), (64, 2200, 32)):
        w = kt.bf16_round(rng.standard_normal((n, k)) / np.sqrt(k) * 2)
        dst, n_pad, k_pad = packed(be, w)
        a = np.zeros((rows, k_pad))
        a[:, :k] = grid(rng.standard_normal((rows, k)), act)
        out, out2 = blank(be, (rows, split), act), blank(be, (rows, n - split), F32)
        be.linear(act, up(be, a, act), k_pad, dst, n_pad, k_pad, rows, lin_out(kind=7, out=out, ldo=split, cols=split, split=split, out2=out2, ldo2=n - split))
        y = a[:, :k] @ w.T.astype(np.float64)
        close(down(be, out, (rows, split), act), kt.silu(y[:, :split]), act)
        close(down(be, out2, (rows, n - split), F32), y[:, split:], F32)
        be.reset_pool()


# ---------------------------------------------------------------- models
def load(be, tmp_path, cfg, seed=1, dtype="float32", **kw):
    from vexel_amd.runtime import ModelRuntime
    t = tensors(cfg, seed)
    folder = str(tmp_path / "model")
    kt.write_model(folder, cfg, t)
    kw = {**dict(pool_blocks=64, max_seqs=6, max_batch=32), **kw}
    return ModelRuntime.load(be, folder, dtype=dtype, **kw), t


MODELS = {"SMALL": SMALL, "TINY": TINY, "EVEN": EVEN, "WIDE": WIDE}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MODELS))
def test_prompts_portions_and_decoding(be, tmp_path, dtype, name):
    """The whole prompt, token by token, and portions of several sizes, down to two tokens: the plain implementation's logits at
    every position, in the blocks and the slot of the run before."""
    cfg = MODELS[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=1, pool_blocks=13)
    for n in (1, 2, 3, 16, 17, 203):
        toks = prompt(cfg, n, n)
        want = kt.forward(cfg, t, toks)
        top = limit(dtype, cfg, t, toks, want)
        for sizes in ([n], [1], [2], [2, 3, 1], [16], [17], [7, 63, 1], [65, 1], [64, 128], [80, 2, 37, 1]):
            if sizes[0] > n:
                continue
            err = error(run_portions(mr, 3, toks, sizes), want).max()
            assert err < top, (n, sizes, err)
            mr.delete_sequence(3)
    mr.close()


@pytest.mark.parametrize("dtype,name", [("float32", "SMALL"), ("bfloat16", "SMALL"), ("bfloat16", "EVEN")])
def test_mixed_batches_equal_each_alone(be, tmp_path, dtype, name):
    """Sequences of unequal lengths: prompts' portions beside single tokens, a sequence left out of steps in between, ends and
    new sequences in the freed blocks and slots; every position's logits are the plain implementation's."""
    cfg = MODELS[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=3, pool_blocks=32)
    rng = np.random.default_rng(8)
    todo = [(i, prompt(cfg, n, 100 + i)) for i, n in enumerate((90, 3, 150, 130, 1, 17, 64, 200, 33))]
    want = {i: kt.forward(cfg, t, p) for i, p in todo}
    top = max(limit(dtype, cfg, t, p, want[i]) for i, p in todo if len(p) > 10)
    toks, at, live, seen = dict(todo), {}, [], set()
    waiting = [i for i, _ in todo]
    while waiting or live:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
            at[live[-1]] = 0
        entries, rows, want_rows, row = [], [], [], 0
        for i in live:
            if len(live) > 1 and rng.random() < 0.25:
                continue                                       # left out of this step
            left = len(toks[i]) - at[i]
            n = int(min(left, rng.choice([1, 1, 2, 3, 16, 17, 40, 75, 100])))
            entries.append((i, toks[i][at[i]:at[i] + n]))
            for r in range(n):
                if rng.random() < 0.7 or r == n - 1:
                    want_rows.append(row + r)
                    rows.append((i, at[i] + r))
            row += n
            at[i] += n
        if not entries:
            continue
        lg, am = mr.step(entries, want_rows)
        for j, (i, p) in enumerate(rows):
            assert error(lg[j:j + 1], want[i][p:p + 1])[0] < top, (i, p)
            assert am[j] == lg[j].argmax()
            seen.add((i, p))
        assert mr.device_matches_host()
        for i in [i for i in live if at[i] == len(toks[i])]:
            mr.delete_sequence(i)
            live.remove(i)
    assert len(seen) > 400
    total, free, _ = mr.block_stats()
    assert total == free
    mr.close()


@pytest.mark.parametrize("dtype,name", [("float32", "SMALL"), ("bfloat16", "EVEN")])
def test_long_decoding(be, tmp_path, dtype, name):
    """300 tokens one by one after a prompt of 5, beside another sequence, past the edges of windows and chunks; then another in its
    place."""
    cfg = MODELS[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=2, pool_blocks=40)
    for seed in (1, 2):
        a, b = prompt(cfg, 305, seed), prompt(cfg, 305, seed + 10)
        wa, wb = kt.forward(cfg, t, a), kt.forward(cfg, t, b)
        mr.step([(0, a[:5]), (1, b[:5])], [])
        ga, gb = [], []
        for i in range(5, 305):
            lg, _ = mr.step([(1, b[i:i + 1]), (0, a[i:i + 1])], [0, 1])
            ga.append(lg[1]), gb.append(lg[0])
        assert error(np.array(ga), wa[5:]).max() < limit(dtype, cfg, t, a, wa)
        assert error(np.array(gb), wb[5:]).max() < limit(dtype, cfg, t, b, wb)
        mr.delete_sequence(0), mr.delete_sequence(1)
    mr.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_keys_of_a_model(be, tmp_path, dtype):
    """Sharp attention over wide windows and chunks, and slow decays: tokens that repeat far back, in the middle of prompts, at their ends
    and decoded, in whole prompts and in portions."""
    from vexel_amd.runtime import ModelRuntime
    cfg = config([(differential(heads=4, dim=32, vdim=64, size=500, cap=40.0), moe()), (key_value(heads=4, dim=64, size=480, rot=(16, 1e5), scale=0.9), None),
                  (lightning(heads=2, dim=32, vdim=32, decay=[0.9995, 0.98]), moe())], width=96, vocab=400)
    t = tensors(cfg, 4, qk_gain=3.0)
    kt.write_model(str(tmp_path / "model"), cfg, t)
    mr = ModelRuntime.load(be, str(tmp_path / "model"), dtype=dtype, pool_blocks=40, max_seqs=2, max_batch=32)
    toks = prompt(cfg, 560, 9)
    for at in (130, 257, 400, 479, 480, 486, 487, 499, 500, 558, 559):
        toks[at] = toks[at % 7]
    want = kt.forward(cfg, t, toks)
    top = limit(dtype, cfg, t, toks, want)
    for sizes in ([560], [500, 1], [129, 128, 1]):
        assert error(run_portions(mr, 0, toks, sizes), want).max() < top, sizes
        mr.delete_sequence(0)
    mr.close()


def greedy(cfg, t, toks, n):
    toks, out = list(toks), []
    for _ in range(n):
        lg = kt.forward(cfg, t, toks)[-1]
        top = np.sort(lg)
        assert top[-1] - top[-2] > 1e-3                        # (no near tie that rounding could turn)
        out.append(int(lg.argmax()))
        toks.append(out[-1])
    return out


@pytest.mark.parametrize("chunk", [0, 2, 7])
def test_greedy_generation_through_the_scheduler(be, tmp_path, chunk):
    from vexel_amd.runtime import Scheduler
    cfg = SMALL
    mr, t = load(be, tmp_path, cfg, max_seqs=4, pool_blocks=40)
    assert mr.mixed_batches
    prompts = {i: prompt(cfg, n, 40 + i) for i, n in enumerate((3, 20, 1, 33))}
    want = {i: greedy(cfg, t, p, 6) for i, p in prompts.items()}
    for _ in range(2):                                         # the second time in used blocks and slots
        s = Scheduler(mr, max_batch_size=4, max_tokens=6, eos_token=-1, prefill_chunk=chunk)
        s.add_sequence(0, prompts[0])
        s.step()
        for i in (1, 2, 3):
            s.add_sequence(i, prompts[i])
        for _ in range(60):
            s.step()
            if all(s.state(i) == 3 for i in prompts):
                break
        assert {i: s.generated(i) for i in prompts} == want
        for i in prompts:
            s.remove_sequence(i)
        s.close()
    mr.close()


@pytest.mark.parametrize("name,dtype", [("SMALL", "float32"), ("EVEN", "bfloat16"), ("WIDE", "bfloat16")])
def test_graph_replay_equals_eager_steps(be, tmp_path, name, dtype):
    """Device-driven greedy decoding: captured and replayed several times with the engine's own steps in between, the same
    tokens as eager steps up to where two tokens are too close to call."""
    cfg = MODELS[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=8, pool_blocks=80)
    prompts = {i: prompt(cfg, n, 60 + i) for i, n in enumerate((5, 140, 14))}

    def eager(base):
        out, gaps = [], []
        lg, am = mr.step([(base + i, p) for i, p in prompts.items()], np.cumsum([len(p) for p in prompts.values()]) - 1)
        start = last = am.copy()
        for _ in range(24):
            lg, am = mr.step([(base + i, [int(last[i])]) for i in prompts], [0, 1, 2])
            out.append(am.tolist())
            top = np.sort(lg, -1)
            gaps.append(((top[:, -1] - top[:, -2]) / lg.std(-1)).tolist())
            last = am
        for i in prompts:
            mr.delete_sequence(base + i)
        return start, out, np.array(gaps)

    start, want, gaps = eager(0)
    lens = [len(p) for p in prompts.values()]
    mr.step([(10 + i, p) for i, p in prompts.items()], [])
    got, _ = mr.decode_graph(start, [10, 11, 12], lens, 6)
    rows = got.tolist()
    for n in (1, 7, 10):
        assert eager(100)[1] == want                           # other work between the replays
        got, _ = mr.decode_graph(None, None, None, n, batch=3)
        rows += got.tolist()
        assert mr.device_matches_host()
    compared = 0
    for i in range(3):
        for step in range(24):
            if gaps[step, i] < (1e-4 if dtype == "float32" else 0.015):
                break
            assert rows[step][i] == want[step][i], (step, i)
            compared += 1
    assert compared > (70 if dtype == "float32" else 20)
    mr.close()


def test_sequences_without_states(be, tmp_path):
    """Without decaying states a sequence is its blocks and the tokens in them: it can be cut to any length, and another can start from
    its first blocks. With them it cannot."""
    from vexel_amd.backend import VexelError
    cfg = config([(differential(size=20), moe()), (key_value(size=11), None)])
    mr, t = load(be, tmp_path, cfg, max_seqs=3, pool_blocks=20)
    a, b = prompt(cfg, 60, 1), prompt(cfg, 60, 2)
    mr.step([(0, a[:50])], [])
    mr.truncate_sequence(0, 21)
    toks = a[:21] + b[21:50]
    want = kt.forward(cfg, t, toks)
    lg, _ = mr.step([(0, toks[21:])], list(range(29)))
    assert error(lg, want[21:]).max() < LIMIT["float32"]
    mr.create_sequence(1)
    mr.share_blocks(0, 1, 32)                                  # two whole blocks
    toks = toks[:32] + a[32:60]
    want = kt.forward(cfg, t, toks)
    lg, _ = mr.step([(1, toks[32:])], list(range(28)))
    assert error(lg, want[32:]).max() < LIMIT["float32"]
    with pytest.raises(VexelError, match="fragment"):
        mr.cache_fragment("a", 0)
    mr.close()
    mr, t = load(be, tmp_path, SMALL, max_seqs=3, pool_blocks=20)
    mr.step([(0, a[:50])], [])
    with pytest.raises(VexelError, match="recurrent"):
        mr.truncate_sequence(0, 21)
    mr.close()


def test_loader_errors(be, tmp_path):
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import ModelRuntime
    cfg = config([(lightning(), moe(experts=3, top=1, groups=None)), (differential(), None), (key_value(), None), 0])
    t = tensors(cfg, 1)
    folder = str(tmp_path / "m")
    for change, text in ((lambda d: d.pop("l0.mix.norm"), "l0.mix.norm is missing"), (lambda d: d.pop("l1.mix.v"), "l1.mix.v is missing"),
                         (lambda d: d.pop("l2.mix.k.b"), "l2.mix.k.b is missing"), (lambda d: d.update({"bigram": d["bigram"][:-1]}), "bigram: shape"),
                         (lambda d: d.pop("l0.mlp.e2.up"), "l0.mlp.e2.up is missing"), (lambda d: d.pop("l0.mlp.shared.down"), "shared.down is missing"),
                         (lambda d: d.update({"l0.mlp.router": d["l0.mlp.router"][:-1]}), "router: shape"), (lambda d: d.pop("l0.mlp.correction"), "correction"),
                         (lambda d: d.update({"l1.mix.lq2": d["l1.mix.lq2"][:-1]}), "lq2: shape")):
        d = dict(t)
        change(d)
        kt.write_model(folder, cfg, d)
        with pytest.raises(VexelError, match=text):
            ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1)
    kt.write_model(folder, cfg, t)                             # (what the last layer does not have, it does not ask for)
    assert "l3.norm1" not in t and "l2.mix.v" not in t
    ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1).close()


def test_generation_from_the_command_line(be, tmp_path, capsys):
    from vexel_amd.__main__ import main
    cfg = SMALL
    t = tensors(cfg, 2)
    kt.write_model(str(tmp_path / "m"), cfg, t)
    prompts = [prompt(cfg, 9, 1), prompt(cfg, 30, 2)]
    args = ["generate", "--model", str(tmp_path / "m"), "--dtype", "float32", "--max-new", "5", "--prefill-chunk", "8"]
    for p in prompts:
        args += ["--tokens", ",".join(map(str, p))]
    assert main(args) == 0
    got = [[int(x) for x in line.split()] for line in capsys.readouterr().out.splitlines()]
    assert got == [greedy(cfg, t, p, 5) for p in prompts]


def test_trace_replay(be, tmp_path):
    """bin/trace_run in a process of its own: steps in, logits out, blocks given back at the end of requests."""
    cfg = SMALL
    t = tensors(cfg, 6)
    kt.write_model(str(tmp_path / "m"), cfg, t)
    a, b, c = (prompt(cfg, n, 80 + n) for n in (50, 30, 47))
    steps = [{"entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:1], "want": []}], "end": []},
             {"entries": [{"id": "b", "tokens": b[1:], "want": [28]}, {"id": "a", "tokens": a[20:], "want": [29, 3]}], "end": ["a", "b"]},
             {"entries": [{"id": "c", "tokens": c, "want": [46]}], "end": ["c"]}]
    want = {n: kt.forward(cfg, t, toks) for n, toks in (("a", a), ("b", b), ("c", c))}
    text = "".join(json.dumps({"step": i, **s}) + "\n" for i, s in enumerate(steps))
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    read = lambda i: np.fromfile(str(out / ("%d.f32" % i)), dtype="<f4").reshape(-1, cfg["vocab"])
    assert error(read(0), want["a"][[0, 19]]).max() < LIMIT["float32"]
    assert error(read(1), np.stack([want["b"][29], want["a"][49], want["a"][23]])).max() < LIMIT["float32"]
    assert error(read(2), want["c"][46:]).max() < LIMIT["float32"]
