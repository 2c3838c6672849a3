"""Fitevik on the GPU: each kernel alone against the plain implementation, then models through the engine's loader, block
pool, step, scheduler and graph replay."""
import json
import os
import subprocess

import numpy as np
import pytest

from fitevik_models import EVEN, LIMIT, SMALL, TINY, WIDE, attention, config, dense, error, limit, margin, moe, states, tensors
from mixed_batches import ACTS, BF16, BS, F32, Batch, blank, close, down, grid, lin_out, packed, prompt, run_portions, up
from oracle import fitevik as fv

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


# ---------------------------------------------------------------- heads to their places, normed over the row
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", [(6, 2, 12, 28), (3, 1, 21, 7), (8, 2, 128, 128), (40, 8, 128, 128), (1, 1, 1, 1), (64, 4, 130, 64), (4, 0, 24, 16)])
def test_heads_normed_over_the_row(be, act, geom):
    """One norm over all query heads of a row and one over its key heads, with a weight of that size; values as projected; queries alone."""
    from vexel_amd.backend import VxHeadsArgs
    H, G, D, X = geom
    rng = np.random.default_rng(D)
    for batch in (MIXED, SINGLE):
        for slices in (1, 3):
            bt = Batch(be, *batch, seed=D)
            qc, kc = 16, 16 + pad(H * D, 16)
            vc = kc + pad(G * D, 16)
            ld = vc + pad(G * X, 16) + 16
            y = (rng.standard_normal((slices, bt.rows, ld)) * rng.uniform(0.02, 3, (bt.rows, 1))).astype(np.float32)
            wq, wk = (1 + 0.3 * rng.standard_normal(H * D)).astype(np.float32), (1 + 0.3 * rng.standard_normal(max(G * D, 1))).astype(np.float32)
            p = VxHeadsArgs()
            p.q_heads, p.k_heads, p.v_heads, p.dim, p.v_dim = H, G, G, D, X
            p.y, p.y_slices, p.ldy, p.y_stride = be.upload(y), slices, ld, bt.rows * ld
            p.q_col, p.k_col, p.v_col, p.norm, p.eps, p.w_q, p.w_k = qc, kc, vc, 2, 1e-3, be.upload(wq), be.upload(wk)
            ldq, kp = pad(H * D, 8) + 8, pad(D, 8)
            per = BS * (G * kp + G * X)
            p.q, p.ldq = blank(be, (bt.rows, ldq), act), ldq
            if G:
                p.pool = blank(be, (bt.pool_blocks, per), act)
            be.heads_store(act, bt.c, p)
            s = y.astype(np.float64).sum(0)
            got = down(be, p.q, (bt.rows, ldq), act)
            close(got[:, :H * D], fv.rms(s[:, qc:qc + H * D], 1e-3) * wq, act, geom)
            assert np.isnan(got[:, H * D:]).all()
            if G:
                pool = down(be, p.pool, (bt.pool_blocks, per), act)
                kk = pool[:, :BS * G * kp].reshape(-1, G, BS, kp).transpose(0, 2, 1, 3).reshape(-1, G, kp)
                vv = pool[:, BS * G * kp:].reshape(-1, G, X, BS).transpose(0, 3, 1, 2).reshape(-1, G, X)
                close(kk[bt.slot_map][..., :D], (fv.rms(s[:, kc:kc + G * D], 1e-3) * wk).reshape(-1, G, D), act, geom)
                close(vv[bt.slot_map], s[:, vc:vc + G * X].reshape(-1, G, X), act, geom)
                assert np.isnan(np.delete(kk, bt.slot_map, 0)).all() and np.isnan(np.delete(vv, bt.slot_map, 0)).all()
            be.reset_pool()


# ---------------------------------------------------------------- attention
def run_attn(be, act, bt, H, G, D, X, window=0, talk=True, slopes=True, sinks=True, seed=0, scale=None, change=None, min_rows=0):
    """vx_attn_ragged against masked softmax over every pair; tokens outside the sequences hold large numbers."""
    from vexel_amd.backend import VxAttnArgs
    rng = np.random.default_rng(seed)
    q = rng.standard_normal((bt.rows, H, D))
    ks = [rng.standard_normal((n, G, D)) for n in bt.kv]
    vs = [rng.standard_normal((n, G, X)) for n in bt.kv]
    mix = fv.bf16_round(np.eye(H) + 0.6 * rng.standard_normal((H, H)) / np.sqrt(H))
    slope = (fv.slopes(H) * rng.uniform(0.2, 1.0, H)).astype(np.float32) if slopes else np.zeros(H, dtype=np.float32)
    if change:
        change(q, ks, vs, mix, slope)
    q, ks, vs = grid(q, act), [grid(k, act) for k in ks], [grid(v, act) for v in vs]
    scale = scale or 1.5 / D ** 0.5
    kp = pad(D, 8)
    pool = rng.standard_normal((bt.pool_blocks, BS * G * (kp + X))) * 60
    kk, vv = pool[:, :BS * G * kp].reshape(-1, G, BS, kp), pool[:, BS * G * kp:].reshape(-1, G, X, BS)
    kk[..., D:] = 0
    for i, n in enumerate(bt.kv):
        for t in range(n):
            s = bt.slot(i, t)
            kk[s // BS, :, s % BS, :D], vv[s // BS, :, :, s % BS] = ks[i][t], vs[i][t]
    sink = (rng.standard_normal(H) * 2).astype(np.float32)
    p = VxAttnArgs()
    p.heads, p.kv_heads, p.k_dim, p.v_dim, p.scale, p.out_scale, p.min_rows, p.window = H, G, D, X, scale, 1.0, min_rows, window
    p.q, p.ldq, p.pool, p.out, p.ldo = up(be, q, act), H * D, up(be, pool, act), blank(be, (bt.rows, H, X), act), H * X
    if talk:
        p.talk = up(be, mix, BF16)
    if slopes:
        p.slopes = be.upload(slope)
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
        seen = fv.in_window(a, b, window) if window else a >= b
        s = np.stack([q[r, h].astype(np.float64) @ ks[i][:, h // (H // G)].T.astype(np.float64) * scale for h in range(H)])
        if talk:
            s = fv.mix_heads(mix.astype(np.float64), s)
        s = s - slope.astype(np.float64)[:, None, None] * (a - b)
        for h in range(H):
            w = fv.softmax(np.where(seen, s[h], -np.inf), sink[h] if sinks else -1e30)
            close(got[r, h], w @ vs[i][:, h // (H // G)].astype(np.float64), act, (i, bt.start[i], bt.lens[i], h))
    return got


# (heads, K/V heads, key size, value size): each matrix-core geometry, narrower heads than it holds, groups of every kind, and some that
# only the plain kernel takes
GEOMETRIES = [(4, 4, 96, 80), (4, 2, 12, 28), (8, 2, 64, 64), (16, 4, 128, 128), (12, 4, 72, 40), (5, 1, 16, 24), (1, 1, 1, 1), (17, 1, 30, 20), (32, 8, 48, 128),
              (32, 32, 24, 16), (20, 20, 100, 100), (40, 8, 16, 33), (64, 4, 32, 8), (2, 1, 200, 40), (66, 2, 8, 8), (10, 2, 128, 9)]


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", GEOMETRIES)
def test_attention_geometries(be, act, geom):
    H, G, D, X = geom
    for batch in (MIXED, SINGLE):
        bt = Batch(be, *batch, seed=D)
        for kw in (dict(window=50), dict(sinks=False), dict(window=130, slopes=False)):
            run_attn(be, act, bt, H, G, D, X, **kw)
        be.reset_pool()


def test_which_kernel_takes_which_geometry(be):
    fast = lambda *a: be.lib_call("vx_attn_talk_fast", *a)
    assert all(fast(BF16, BS, *g) for g in GEOMETRIES if g[0] <= 64 and max(g[2:]) <= 128)
    assert not any(fast(F32, BS, *g) for g in GEOMETRIES) and not fast(BF16, 32, 4, 4, 64, 64)
    assert not fast(BF16, BS, 66, 2, 8, 8) and not fast(BF16, BS, 4, 2, 136, 64) and not fast(BF16, BS, 36, 36, 64, 64)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("size", [1, 2, 15, 16, 17, 31, 32, 33, 64, 100, 255, 256, 257, 401, 5000])
def test_windows_of_every_size(be, act, size):
    for batch in (MIXED, SINGLE):
        bt = Batch(be, *batch, seed=size)
        for talk in (True, False):
            run_attn(be, act, bt, 8, 2, 16, 24, talk=talk, window=size, seed=size)
        be.reset_pool()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", [(4, 2, 40, 24), (16, 2, 128, 128), (2, 1, 200, 40)])
def test_slopes_without_mixed_heads(be, act, geom):
    """The slopes of the kernels that take heads one by one."""
    for batch in (MIXED, SINGLE):
        for kw in (dict(), dict(window=77, sinks=False)):
            run_attn(be, act, Batch(be, *batch, seed=2), *geom, talk=False, **kw)
        be.reset_pool()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("pos", [0, 1, 30, 63, 64, 65, 127, 128, 300, 700])
def test_keys_at_the_window_edge_stand_out(be, act, pos):
    """One key that one head scores far above the others, and that another head sees only through the mixing, just inside and just outside
    the window of the last row: in prompts, in short portions and decoded alone."""
    for size in (1, 37, 64, 130):
        first = max(0, pos - size + 1)
        for key in {first, first - 1, pos, 0}:
            if key < 0:
                continue

            def stand_out(q, ks, vs, mix, slope):
                q[-1, 1, 3] = 8.0
                q[-1, 0, 3] = 0.0
                ks[0][..., 3] = 0.0
                ks[0][key, ..., 3] = 8.0
                vs[0][key] *= 4
                mix[:] = 0
                mix[0] = (0.125, 1.0)
                mix[1, 1] = 0.5
                slope[:] = 0.01

            for rows in {1, min(2, pos + 1), min(40, pos + 1)}:
                run_attn(be, act, Batch(be, [pos + 1 - rows], [rows], seed=pos), 2, 1, 16, 16, window=size, change=stand_out, scale=0.5, seed=pos)
            be.reset_pool()


def test_a_row_of_the_mixing_counts_for_its_own_head(be):
    """A matrix that is no symmetric one, moving every head's scores one head on."""
    def shift(q, ks, vs, mix, slope):
        mix[:] = np.roll(np.eye(len(mix)), 1, 1)

    for act in ACTS:
        for H, G in ((8, 2), (6, 6), (40, 8)):
            run_attn(be, act, Batch(be, *MIXED, seed=3), H, G, 24, 16, window=60, change=shift, seed=H)
        be.reset_pool()


@pytest.mark.parametrize("start,lens", [(0, [700]), (900, [33]), (0, [2200]), (1500, [64, 1]), (100, [3000])])
def test_attention_of_long_portions(be, start, lens):
    """Few rows, whose keys are cut into pieces, and enough of them that they are not; windows that begin inside a tile of rows."""
    for geom in ((16, 2, 32, 32), (8, 8, 16, 24)):
        for kw in (dict(window=200), dict(window=1000), dict()):
            run_attn(be, BF16, Batch(be, [start] * len(lens), lens, seed=1), *geom, **kw)
            be.reset_pool()


def test_attention_of_many_decoding_sequences(be):
    rng = np.random.default_rng(6)
    bt = Batch(be, rng.integers(0, 900, 130).tolist(), [1] * 130, seed=6)
    for kw in (dict(), dict(window=300), dict(window=64)):
        run_attn(be, BF16, bt, 8, 4, 32, 32, seed=2, **kw)


def test_rows_left_out(be):
    for act in ACTS:
        for least in (2, 40):
            run_attn(be, act, Batch(be, *MIXED, seed=4), 4, 2, 24, 24, min_rows=least, window=30)


def test_attention_errors(be):
    from vexel_amd.backend import VexelError
    bt = Batch(be, [0], [3])
    from vexel_amd.backend import VxAttnArgs
    z = be.alloc(1 << 16)
    for change, text in ((dict(softcap=1.0), "no cap"), (dict(maps=2), "one map"), (dict(bias=z, bias_len=4, slopes=z), "bias table")):
        p = VxAttnArgs()
        p.heads, p.kv_heads, p.k_dim, p.v_dim, p.scale, p.out_scale, p.q, p.ldq, p.pool, p.out, p.ldo, p.talk = 2, 1, 8, 8, 1.0, 1.0, z, 32, z, z, 16, z
        for k, v in change.items():
            setattr(p, k, v)
        with pytest.raises(VexelError, match=text):
            be.attn_ragged(F32, bt.c, p)


# ---------------------------------------------------------------- states with forget gates
def run_forget(be, act, bt, H, D, X, gates, seed=0):
    """gates(rng, shape) -> 1 - f"""
    from vexel_amd.backend import VxForgetArgs
    rng = np.random.default_rng(seed)
    slots = max(bt.slots) + 2
    ldq, ldv, ldg = H * D + 16, H * X + 8, H * D + 3
    q, v = grid(rng.standard_normal((bt.rows, H, D)), act), grid(rng.standard_normal((bt.rows, H, X)), act)
    g = gates(rng, (bt.rows, H, D)).astype(np.float32)
    state = rng.standard_normal((slots, H, D, X)).astype(np.float32)
    wide = lambda a, ld: np.concatenate([a.reshape(bt.rows, -1), np.full((bt.rows, ld - a[0].size), np.nan)], 1)
    p = VxForgetArgs()
    p.heads, p.dim, p.vdim = H, D, X
    p.q, p.v, p.g, p.ldq, p.ldv, p.ldg = up(be, wide(q, ldq), act), up(be, wide(v, ldv), act), up(be, wide(g, ldg)), ldq, ldv, ldg
    p.state, p.out, p.ldo = be.upload(state), blank(be, (bt.rows, H * X + 4), F32), H * X + 4
    be.forget_attn(act, bt.c, p)
    got = down(be, p.out, (bt.rows, H * X + 4), F32)
    after = down(be, p.state, state.shape, F32)
    assert np.isnan(got[:, H * X:]).all()
    used = set()
    for i in range(len(bt.lens)):
        r, s = slice(bt.cu[i], bt.cu[i + 1]), bt.slots[i]
        o, S = fv.gated_states(q[r].astype(np.float64), 1.0 - g[r].astype(np.float64), v[r].astype(np.float64), state[s].astype(np.float64) if bt.start[i] else None)
        tol = 2e-5 if act == F32 or bt.lens[i] <= 16 else 2e-4  # (two bfloat16 parts)
        assert np.abs(got[r, :H * X].reshape(-1, H, X) - o).max() < tol * np.abs(o).max(), (i, bt.start[i], bt.lens[i])
        assert np.abs(after[s] - S).max() < tol * np.abs(S).max(), (i, bt.start[i], bt.lens[i])
        used.add(s)
    for s in range(slots):
        if s not in used:
            assert np.array_equal(after[s], state[s])          # nobody else's state moves


sigma = lambda z: 1.0 / (1.0 + np.exp(-z))
GATES = {"mixed": lambda rng, s: sigma(rng.standard_normal(s) * 3 - 1), "slow": lambda rng, s: 10.0 ** rng.uniform(-5, -2, s),
         "fast": lambda rng, s: 1.0 - 10.0 ** rng.uniform(-6, -1, s), "all or nothing": lambda rng, s: rng.choice([0.0, 1.0, 0.5], s),
         "by channel": lambda rng, s: np.broadcast_to(10.0 ** np.linspace(-6, 0, s[-1]), s)}


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", [(3, 32, 16), (2, 64, 48), (1, 160, 144), (4, 128, 128), (2, 96, 272), (1, 512, 512), (2, 256, 32)])
def test_forgetting_states(be, act, geom):
    for batch in (MIXED, SINGLE):
        run_forget(be, act, Batch(be, *batch, seed=geom[1]), *geom, GATES["mixed"], seed=geom[1])
        be.reset_pool()


@pytest.mark.parametrize("gates", list(GATES))
@pytest.mark.parametrize("rows", [2, 8, 9, 16, 17, 63, 64, 65, 127, 128, 129, 191, 192, 193, 256, 257])
def test_portions_of_forgetting_states(be, rows, gates):
    """Around every border of blocks and chunks, from the start and later, beside others; gates that keep nearly all and nothing."""
    for act, geom in ((BF16, (2, 64, 32)), (BF16, (1, 128, 16)), (F32, (1, 32, 16))):
        run_forget(be, act, Batch(be, [0, 77, 3, 0], [rows, rows, 1, 33], seed=rows), *geom, GATES[gates], seed=rows)
        be.reset_pool()


def test_long_portions_of_forgetting_states(be):
    for gates in ("slow", "by channel"):
        run_forget(be, BF16, Batch(be, [0, 400], [1500, 700], seed=1), 4, 64, 64, GATES[gates], seed=1)
        be.reset_pool()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("heads,vdim,count", [(3, 16, 10), (5, 48, 48), (4, 64, 60), (32, 128, 128), (2, 272, 270), (1, 512, 512), (7, 4, 1)])
def test_head_norm(be, act, heads, vdim, count):
    rng = np.random.default_rng(vdim)
    for rows in (1, 33, 700):
        ldx, ldo = heads * vdim + 8, pad(heads * vdim, 64) + 8
        x = (rng.standard_normal((rows, heads, vdim)) * rng.uniform(0.01, 5, (rows, heads, 1))).astype(np.float32)
        x[..., count:] = 0
        w = (1 + 0.3 * rng.standard_normal(vdim)).astype(np.float32)
        wide = np.full((rows, ldx), np.nan, dtype=np.float32)
        wide[:, :heads * vdim] = x.reshape(rows, -1)
        out = blank(be, (rows, ldo), act)
        be.head_norm(act, be.upload(wide), ldx, be.upload(w), 1e-3, rows, heads, vdim, count, out, ldo)
        got = down(be, out, (rows, ldo), act)
        want = x / np.sqrt((x.astype(np.float64) ** 2).sum(-1, keepdims=True) / count + 1e-3) * w
        close(got[:, :heads * vdim].reshape(want.shape), want, act)
        assert np.all(got[:, heads * vdim:] == 0)
        be.reset_pool()


# ---------------------------------------------------------------- norms of what joins the stream
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("cols", [1, 5, 88, 256, 1000, 4096, 9000, 12290])
def test_branch_norm(be, act, cols):
    """Slices, bias and experts' rows through a layer norm into the stream; the last one with the final norm, for some of the rows."""
    from vexel_amd.backend import VxBranchNormArgs
    rng = np.random.default_rng(cols)
    eps, top = 1e-4, 3
    for rows in (1, 40, 300):
        ldy, ldo, lde = pad(cols, 16), pad(cols, 64), pad(cols, 32)
        x = rng.standard_normal((rows, cols)).astype(np.float32)
        y = (rng.standard_normal((2, rows, ldy)) * 3 + 2).astype(np.float32)
        er = grid(rng.standard_normal((rows * top, lde)), act)
        places, weights = rng.permutation(rows * top).astype(np.int32).reshape(rows, top), rng.uniform(0, 1, (rows, top)).astype(np.float32)
        yb, w, b, wf, bf = ((m + 0.3 * rng.standard_normal(cols)).astype(np.float32) for m in (0, 1, 0, 1, 0))
        for slices, experts, last in ((2, False, False), (1, True, False), (0, True, True), (2, False, True)):
            idx = rng.integers(0, rows, 3).astype(np.int32) if last else None
            n = 3 if last else rows
            p = VxBranchNormArgs()
            p.rows, p.cols, p.eps, p.x_in, p.w, p.b = n, cols, eps, up(be, x), up(be, w), up(be, b)
            v = np.zeros((rows, cols))
            if slices:
                p.y, p.y_bias, p.y_slices, p.ldy, p.y_stride = up(be, y), up(be, yb), slices, ldy, rows * ldy
                v = v + y[:slices].astype(np.float64).sum(0)[:, :cols] + yb
            if experts:
                p.e_rows, p.lde, p.e_top, p.e_places, p.e_weights = up(be, er, act), lde, top, be.upload(places), up(be, weights)
                v = v + (weights[..., None] * er[places][..., :cols].astype(np.float64)).sum(1)
            want = x + fv.layer_norm(v, w, b, eps)
            p.out, p.ldo = blank(be, (n, ldo), act), ldo
            if last:
                p.row_idx, p.w_pre, p.b_pre = be.upload(idx), up(be, wf), up(be, bf)
            else:
                p.x_out = blank(be, (rows, cols), F32)
            be.branch_norm(act, p)
            if last:
                want = fv.layer_norm(want, wf, bf, eps)[idx]
            else:
                close(down(be, p.x_out, (rows, cols), F32), want, F32)
            got = down(be, p.out, (n, ldo), act)
            close(got[:, :cols], want, act)
            assert np.all(got[:, cols:] == 0)
            be.reset_pool()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("cols", [1, 5, 88, 1000, 4096])
def test_embedding_with_positions(be, act, cols):
    from vexel_amd.backend import VxBranchNormArgs
    rng = np.random.default_rng(cols)
    for rows in (1, 300):
        T = {"embed": rng.standard_normal((50, cols)).astype(np.float32), "pos": rng.standard_normal((400, cols)).astype(np.float32),
             "embed.norm": (1 + 0.3 * rng.standard_normal(cols)).astype(np.float32), "embed.norm.b": rng.standard_normal(cols).astype(np.float32)}
        tok, pos = rng.integers(0, 50, rows).astype(np.int32), rng.integers(0, 400, rows).astype(np.int32)
        ldo = pad(cols, 64)
        p = VxBranchNormArgs()
        p.rows, p.cols, p.eps, p.x_in, p.tokens, p.token_pos = rows, cols, 1e-4, up(be, T["embed"]), be.upload(tok), be.upload(pos)
        p.positions, p.w_pre, p.b_pre = up(be, T["pos"]), up(be, T["embed.norm"]), up(be, T["embed.norm.b"])
        p.x_out, p.out, p.ldo = blank(be, (rows, cols), F32), blank(be, (rows, ldo), act), ldo
        be.branch_norm(act, p)
        x = T["embed"][tok].astype(np.float64) + T["pos"][pos]
        want = fv.layer_norm(x, T["embed.norm"], T["embed.norm.b"], 1e-4)
        close(down(be, p.x_out, (rows, cols), F32), want, F32)
        got = down(be, p.out, (rows, ldo), act)
        close(got[:, :cols], want, act)
        assert np.all(got[:, cols:] == 0)
        be.reset_pool()


# ---------------------------------------------------------------- experts
def route(be, z, bias, top, tile):
    from vexel_amd.backend import VxRouteArgs
    slices, rows, E = z.shape
    ld = E + 3
    zz = np.full((slices, rows, ld), np.nan, dtype=np.float32)
    zz[..., :E] = z
    p = VxRouteArgs()
    p.rows, p.experts, p.top, p.groups, p.keep, p.tile_rows, p.softmax = rows, E, top, 1, 1, tile, 1
    p.z, p.z_slices, p.ldz, p.z_stride = be.upload(zz), slices, ld, rows * ld
    if bias is not None:
        p.bias = be.upload(bias.astype(np.float32))
    most = be.lib_call("vx_route_max_tiles", rows, E, top, 0, tile)
    p.weights, p.places = blank(be, (rows, top), F32), be.upload(np.full((rows, top), -1, dtype=np.int32))
    p.order, p.tiles = be.upload(np.full(rows * top, -1, dtype=np.int32)), be.upload(np.full(4 + 4 * most, -1, dtype=np.int32))
    be.route(p)
    tiles = be.download(p.tiles, (1 + most, 4), np.int32)
    expert_of = np.concatenate([np.full(n, e) for e, _, n, _ in tiles[1:1 + tiles[0, 0]]])
    places = be.download(p.places, (rows, top), np.int32)
    assert np.array_equal(np.sort(places.ravel()), np.arange(rows * top))
    return p, be.download(p.weights, (rows, top), np.float32), places, be.download(p.order, (rows * top,), np.int32), expert_of


@pytest.mark.parametrize("experts,top", [(1, 1), (9, 4), (16, 1), (64, 6), (65, 8), (130, 130), (1024, 10), (8, 8)])
def test_routing_by_softmax(be, experts, top):
    """The largest logits with their bias, weighted by the softmax over the chosen ones; large logits as well."""
    rng = np.random.default_rng(experts)
    for rows in (1, 7, 64, 65, 300):
        for slices, biased, spread in ((1, True, 1.5), (3, False, 1.5), (2, True, 60.0)):
            z = (rng.standard_normal((slices, rows, experts)) * spread).astype(np.float32)
            b = rng.uniform(-1.5, 0.5, experts).astype(np.float32) if biased else None
            p, w, places, order, expert_of = route(be, z, b, top, 64)
            zs = z.astype(np.float64).sum(0) + (0 if b is None else b)
            want = fv.choose(zs, top)
            got = np.zeros((rows, experts))
            np.put_along_axis(got, expert_of[places], w, -1)
            clear = margin(zs, top) > 1e-4
            assert clear.mean() > 0.7
            assert np.abs(got - want)[clear].max() < (2e-6 if spread < 2 else 1e-4)
            assert np.abs(got.sum(-1) - 1).max() < 1e-5
            assert np.array_equal(order[places.ravel()], np.repeat(np.arange(rows), top))
            be.reset_pool()


def test_routing_of_equal_logits(be):
    """Equal logits go by number, so that every row has its experts and its weights add up to one."""
    for rows in (3, 100):
        z = np.zeros((1, rows, 70), dtype=np.float32)
        z[:, 1::2, 69] = 1.0
        _, w, places, _, expert_of = route(be, z, None, 3, 64)
        got = np.sort(expert_of[places], -1)
        assert np.array_equal(got[0], [0, 1, 2]) and np.array_equal(got[1], [0, 1, 69])
        assert np.allclose(w[0], 1 / 3, atol=1e-6) and np.allclose(np.sort(w[1]), np.array([1, 1, np.e]) / (2 + np.e), atol=1e-6)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("E,top,W,ff", [(5, 2, 40, 24), (12, 3, 88, 33), (16, 4, 128, 64), (1, 1, 64, 1), (40, 1, 96, 130)])
def test_experts_of_one_map(be, act, E, top, W, ff):
    """Squared relu between both maps of every expert over rows that were sorted; few rows, many, and many to one expert."""
    from vexel_amd.backend import VxExpertsArgs
    rng = np.random.default_rng(E)
    t = {(e, n): fv.bf16_round(rng.standard_normal(s) / np.sqrt(s[1]) * 1.5) for e in range(E) for n, s in (("up", (ff, W)), ("down", (W, ff)))}
    wk, wn, fp = pad(W, 64), pad(W, 32), pad(ff, 64)
    for rows in (1, 16, 17, 33, 64, 65, 200, 700):
        be.reset_pool()
        u, d = be.alloc(E * fp * wk * 2), be.alloc(E * wn * fp * 2)
        be.fill_zero(u, E * fp * wk * 2), be.fill_zero(d, E * wn * fp * 2)
        for e in range(E):
            packed(be, t[e, "up"], E * fp, wk, e * fp // 16, 1, dst=u)
            packed(be, t[e, "down"], E * wn, fp, e * wn // 16, 1, dst=d)
        h = grid(rng.standard_normal((rows, W)), act)
        hp = np.zeros((rows, wk))
        hp[:, :W] = h
        z = (rng.standard_normal((1, rows, E)) * 2).astype(np.float32)
        if rows % 2:
            z[:, :, 0] += 9                                     # one expert that nearly every row takes
        tile = be.lib_call("vx_route_tile_rows", act, rows, E, top)
        r, w, places, order, expert_of = route(be, z, None, top, tile)
        g = VxExpertsArgs()
        g.kind, g.rows, g.experts, g.tile_rows = 9, rows, E, tile
        g.max_tiles = be.lib_call("vx_route_max_tiles", rows, E, top, 0, tile)
        g.tiles, g.a_rows, g.a, g.lda = r.tiles, r.order, up(be, hp, act), wk
        g.w, g.n, g.k = u, fp, wk
        mid = blank(be, (rows * top, fp), act)
        g.out, g.ldo, g.cols = mid, fp, fp
        be.linear_experts(act, g)
        g.kind, g.a, g.lda, g.a_rows = 0, mid, fp, None
        g.w, g.n, g.k = d, wn, fp
        out = blank(be, (rows * top, wn), act)
        g.out, g.ldo, g.cols = out, wn, wn
        be.linear_experts(act, g)
        got = down(be, out, (rows * top, wn), act)
        assert np.all(got[:, W:] == 0)
        for e in range(E):
            at = np.flatnonzero(expert_of == e)
            if len(at):
                x = h[order[at]].astype(np.float64)
                close(got[at, :W], fv.linear(t[e, "down"].astype(np.float64), fv.relu2(fv.linear(t[e, "up"].astype(np.float64), x))), act, (rows, e))


# ---------------------------------------------------------------- linear maps
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [1, 20, 50, 70, 300])
def test_linear_epilogues(be, act, rows):
    """Gates with a lower bound behind SiLU and plain columns, squared relu with a bias, a factor; whole, and in slices where the map is deep."""
    rng = np.random.default_rng(rows)
    for n, k, split, silu in ((80, 100, 48, 32), (64, 2200, 32, 0), (64, 70, 32, 32)):
        w = fv.bf16_round(rng.standard_normal((n, k)) / np.sqrt(k) * 2)
        dst, n_pad, k_pad = packed(be, w)
        a = np.zeros((rows, k_pad))
        a[:, :k] = grid(rng.standard_normal((rows, k)), act)
        y = a[:, :k] @ w.T.astype(np.float64)
        da = up(be, a, act)
        bias, keep = rng.standard_normal(n).astype(np.float32), rng.choice([0.0, 0.02, 0.5, 1.0], n).astype(np.float32)
        out, out2 = blank(be, (rows, split), act), blank(be, (rows, n - split), F32)
        be.linear(act, da, k_pad, dst, n_pad, k_pad, rows, lin_out(kind=8, out=out, ldo=split, cols=split, split=split, out2=out2, ldo2=n - split, silu_cols=silu,
                                                                   bias=up(be, bias), keep=up(be, keep)))
        close(down(be, out, (rows, split), act), np.concatenate([fv.silu(y[:, :silu]), y[:, silu:split]], 1), act)
        f = fv.forget(y[:, split:], bias[:n - split], 1.0 - keep[:n - split].astype(np.float64))
        got = down(be, out2, (rows, n - split), F32)
        assert np.abs(got - (1.0 - f)).max() < 3e-6 and np.all((got >= 0) & (got <= 1))
        for b in (None, bias):
            out = blank(be, (rows, n), act)
            be.linear(act, da, k_pad, dst, n_pad, k_pad, rows, lin_out(kind=9, out=out, ldo=n, cols=n, bias=up(be, b) if b is not None else None))
            close(down(be, out, (rows, n), act), fv.relu2(y if b is None else y + b), act)
        out = blank(be, (rows, n), F32)
        be.linear(act, da, k_pad, dst, n_pad, k_pad, rows, lin_out(kind=0, out_f32=1, out=out, ldo=n, cols=n, slices=1, mult=0.37))
        close(down(be, out, (rows, n), F32), 0.37 * y, F32)
        be.reset_pool()


# ---------------------------------------------------------------- models
def load(be, tmp_path, cfg, seed=1, dtype="float32", **kw):
    from vexel_amd.runtime import ModelRuntime
    t = tensors(cfg, seed)
    folder = str(tmp_path / "model")
    fv.write_model(folder, cfg, t)
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
        want = fv.forward(cfg, t, toks)
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
    want = {i: fv.forward(cfg, t, p) for i, p in todo}
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
    """300 tokens one by one after a prompt of 5, beside another sequence, past the edges of windows; then another in its place."""
    cfg = MODELS[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=2, pool_blocks=40)
    for seed in (1, 2):
        a, b = prompt(cfg, 305, seed), prompt(cfg, 305, seed + 10)
        wa, wb = fv.forward(cfg, t, a), fv.forward(cfg, t, b)
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
    """Sharp attention over wide windows, and states that forget slowly: tokens that repeat far back, in the middle of prompts, at their
    ends and decoded, in whole prompts and in portions."""
    from vexel_amd.runtime import ModelRuntime
    cfg = config([(attention(heads=4, dim=32, vdim=64, size=500), moe()), (attention(heads=4, dim=32, vdim=64, size=480, scale=0.4, kv_from=0), None),
                  (states(heads=2, dim=32, vdim=32), dense())], width=96, vocab=400)
    t = tensors(cfg, 4, qk_gain=4.0, sink=2.0, keep=6.0)
    for i in (0, 1):                                           # (the steepest slopes would hide what is far)
        t["l%d.mix.talk" % i][:, :2] *= 2.0 ** -6
    fv.write_model(str(tmp_path / "model"), cfg, t)
    mr = ModelRuntime.load(be, str(tmp_path / "model"), dtype=dtype, pool_blocks=40, max_seqs=2, max_batch=32)
    toks = prompt(cfg, 560, 9)
    for at in (130, 257, 400, 479, 480, 486, 487, 499, 500, 558, 559):
        toks[at] = toks[at % 7]
    want = fv.forward(cfg, t, toks)
    top = limit(dtype, cfg, t, toks, want)
    for sizes in ([560], [500, 1], [129, 128, 1]):
        assert error(run_portions(mr, 0, toks, sizes), want).max() < top, sizes
        mr.delete_sequence(0)
    mr.close()


def greedy(cfg, t, toks, n):
    toks, out = list(toks), []
    for _ in range(n):
        lg = fv.forward(cfg, t, toks)[-1]
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
    assert mr.mixed_batches and mr.max_positions == cfg["max_positions"]
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


def test_the_last_position(be, tmp_path):
    """A sequence holds as many tokens as there are positions: the scheduler ends it there, steps and replays beyond are refused, and the
    last position's logits are right."""
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import Scheduler
    cfg = config([(attention(size=9), dense()), (states(), None)], max_positions=40)
    mr, t = load(be, tmp_path, cfg, max_seqs=3, pool_blocks=12)
    toks = prompt(cfg, 41, 1)
    want = fv.forward(cfg, t, toks[:40])
    assert error(mr.step([(0, toks[:40])], list(range(40)))[0], want).max() < LIMIT["float32"]
    with pytest.raises(VexelError, match="40 positions"):
        mr.step([(0, toks[40:])], [0])
    with pytest.raises(VexelError, match="40 positions"):
        mr.step([(1, toks)], [])
    mr.step([(1, toks[:35])], [])
    with pytest.raises(VexelError, match="40 positions"):
        mr.decode_graph(np.array([3], dtype=np.int32), [1], [35], 6)
    mr.delete_sequence(0), mr.delete_sequence(1)
    s = Scheduler(mr, max_batch_size=2, max_tokens=100, eos_token=-1, prefill_chunk=0)
    with pytest.raises(VexelError, match="40 positions"):
        s.add_sequence(7, toks)
    s.add_sequence(0, toks[:36])
    s.add_sequence(1, toks[:40])
    for _ in range(30):
        s.step()
        if s.state(0) == 3 and s.state(1) == 3:
            break
    assert s.state(0) == 3 and len(s.generated(0)) == 5 and s.state(1) == 3 and len(s.generated(1)) == 1
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
    """Without states a sequence is its blocks: it can be cut to any length, and another can start from its first blocks. With them
    it cannot."""
    from vexel_amd.backend import VexelError
    cfg = config([(attention(size=20), moe()), (attention(size=11, kv_from=0), None)])
    mr, t = load(be, tmp_path, cfg, max_seqs=3, pool_blocks=20)
    a, b = prompt(cfg, 60, 1), prompt(cfg, 60, 2)
    mr.step([(0, a[:50])], [])
    mr.truncate_sequence(0, 21)
    toks = a[:21] + b[21:50]
    want = fv.forward(cfg, t, toks)
    lg, _ = mr.step([(0, toks[21:])], list(range(29)))
    assert error(lg, want[21:]).max() < LIMIT["float32"]
    mr.create_sequence(1)
    mr.share_blocks(0, 1, 32)                                  # two whole blocks
    toks = toks[:32] + a[32:60]
    want = fv.forward(cfg, t, toks)
    lg, _ = mr.step([(1, toks[32:])], list(range(28)))
    assert error(lg, want[32:]).max() < LIMIT["float32"]
    mr.close()
    mr, t = load(be, tmp_path, SMALL, max_seqs=3, pool_blocks=20)
    mr.step([(0, a[:50])], [])
    with pytest.raises(VexelError, match="recurrent"):
        mr.truncate_sequence(0, 21)
    mr.close()


def test_loader_errors(be, tmp_path):
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import ModelRuntime
    cfg = config([(states(), moe(experts=3, top=1)), (attention(), dense()), (attention(kv_from=1), None)])
    t = tensors(cfg, 1)
    folder = str(tmp_path / "m")
    for change, text in ((lambda d: d.pop("l0.mix.norm"), "l0.mix.norm is missing"), (lambda d: d.pop("l0.mix.lower"), "l0.mix.lower is missing"),
                         (lambda d: d.pop("l1.mix.talk"), "l1.mix.talk is missing"), (lambda d: d.update({"l1.mix.sink": d["l1.mix.sink"][:-1]}), "sink: shape"),
                         (lambda d: d.pop("l2.mix.q.norm"), "l2.mix.q.norm is missing"), (lambda d: d.pop("l0.mlp.e2.up"), "l0.mlp.e2.up is missing"),
                         (lambda d: d.update({"l0.mlp.router": d["l0.mlp.router"][:-1]}), "router: shape"), (lambda d: d.pop("l0.mlp.router.b"), "router.b"),
                         (lambda d: d.pop("l1.mlp.down.b"), "down.b is missing"), (lambda d: d.pop("l0.norm2.b"), "norm2.b is missing"),
                         (lambda d: d.update({"pos": d["pos"][:-1]}), "pos: shape"), (lambda d: d.pop("embed.norm.b"), "embed.norm.b is missing")):
        d = dict(t)
        change(d)
        fv.write_model(folder, cfg, d)
        with pytest.raises(VexelError, match=text):
            ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1)
    fv.write_model(folder, cfg, t)                             # (what the last layer does not have, it does not ask for)
    assert "l2.mix.k" not in t and "l2.norm2" not in t
    ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1).close()


def test_generation_from_the_command_line(be, tmp_path, capsys):
    from vexel_amd.__main__ import main
    cfg = SMALL
    t = tensors(cfg, 2)
    fv.write_model(str(tmp_path / "m"), cfg, t)
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
    fv.write_model(str(tmp_path / "m"), cfg, t)
    a, b, c = (prompt(cfg, n, 80 + n) for n in (50, 30, 47))
    steps = [{"entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:1], "want": []}], "end": []},
             {"entries": [{"id": "b", "tokens": b[1:], "want": [28]}, {"id": "a", "tokens": a[20:], "want": [29, 3]}], "end": ["a", "b"]},
             {"entries": [{"id": "c", "tokens": c, "want": [46]}], "end": ["c"]}]
    want = {n: fv.forward(cfg, t, toks) for n, toks in (("a", a), ("b", b), ("c", c))}
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
