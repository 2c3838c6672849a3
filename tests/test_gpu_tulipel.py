"""Tulipel on the GPU: each kernel alone against the plain implementation, then models through the engine's loader, block
pool, step, scheduler and graph replay."""
import json
import os
import subprocess

import numpy as np
import pytest

from mixed_batches import ACTS, BF16, BS, F32, Batch, blank, close, down, grid, lin_out, packed, prompt, run_portions, up
from oracle import tulipel as tl
from tulipel_models import EVEN, LIMIT, SMALL, TINY, WIDE, config, error, first, limit, second, tensors

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def be():
    from vexel_amd.backend import HipBackend
    b = HipBackend(0)
    yield b
    b.close()


@pytest.fixture(autouse=True)
def fresh_pool(be):
    be.reset_pool()


# ---------------------------------------------------------------- linear maps
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [1, 5, 40, 70, 200])
def test_linear_in_groups(be, act, rows):
    """Independent maps over column ranges that overlap where a map's inputs are padded; a chosen row order; a cap on the result."""
    rng = np.random.default_rng(rows)
    groups, n, k, a_group, out_group = 5, 48, 40, 56, 64
    ws = [tl.bf16_round(rng.standard_normal((n, k))) for _ in range(groups)]
    dst = be.alloc(groups * n * 64 * 2)
    be.fill_zero(dst, groups * n * 64 * 2)
    for g, w in enumerate(ws):
        packed(be, w, n_pad=groups * n, k_pad=64, tile0=g * n // 16, dst=dst)
    lda = (groups - 1) * a_group + 64 + 8
    a = grid(rng.standard_normal((rows, lda)), act)
    da = up(be, a, act)
    out = blank(be, (rows, groups * out_group), act)
    be.linear(act, da, lda, dst, n, 64, rows, lin_out(kind=0, out=out, ldo=groups * out_group, cols=n, groups=groups, a_group=a_group, out_group=out_group))
    got = down(be, out, (rows, groups, out_group), act)
    for g, w in enumerate(ws):
        close(got[:, g, :n], a[:, g * a_group:g * a_group + k].astype(np.float64) @ w.T, act, g)
    assert np.isnan(got[..., n:]).all()
    order = rng.integers(0, rows, 90).astype(np.int32)
    out = blank(be, (90, n), F32)
    be.linear(act, da, lda, dst, n, 64, 90, lin_out(kind=0, out_f32=1, out=out, ldo=n, cols=n, a_rows=be.upload(order), softcap=2.5))
    close(down(be, out, (90, n), F32), tl.softcap(a[order][:, :k].astype(np.float64) @ ws[0].T, 2.5), F32)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [1, 20, 64, 130])
@pytest.mark.parametrize("k", [128, 4096])
def test_linear_rotary(be, act, rows, k):
    """Heads whose last part is turned, float32 columns behind them; deep maps in slices; the same without columns behind."""
    rng = np.random.default_rng(rows)
    heads, plain, pairs, stride, rest = 3, 20, 5, 32, 40
    w = tl.bf16_round(rng.standard_normal((heads * stride + rest, k)) / k ** 0.5)
    dst, n_pad, _ = packed(be, w)
    a = grid(rng.standard_normal((rows, k)), act)
    tab = rng.standard_normal((rows, pairs, 2)).astype(np.float32)
    y = a.astype(np.float64) @ w.T
    want = y[:, :heads * stride].reshape(rows, heads, stride).copy()
    u, v = want[..., plain:plain + 2 * pairs:2].copy(), want[..., plain + 1:plain + 2 * pairs:2].copy()
    c, s = (tab[:, None, :, i] for i in (0, 1))
    want[..., plain:plain + 2 * pairs:2], want[..., plain + 1:plain + 2 * pairs:2] = u * c - v * s, v * c + u * s
    split = heads * stride
    o1, o2 = blank(be, (rows, split), act), blank(be, (rows, n_pad - split), F32)
    kw = dict(kind=5, ldo=split, cols=split, split=split, rot_stride=stride, rot_first=plain, rot_pairs=pairs, rot_tab=be.upload(tab))
    be.linear(act, up(be, a, act), k, dst, n_pad, k, rows, lin_out(out=o1, out2=o2, ldo2=n_pad - split, **kw))
    close(down(be, o1, (rows, split), act), want.reshape(rows, -1), act)
    close(down(be, o2, (rows, n_pad - split), F32)[:, :rest], y[:, split:], F32)
    o1 = blank(be, (rows, split), act)
    be.linear(act, up(be, a, act), k, dst, split, k, rows, lin_out(out=o1, **kw))
    close(down(be, o1, (rows, split), act), want.reshape(rows, -1), act)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [16, 48, 80, 272])
@pytest.mark.parametrize("heads,kd,used,vd", [(3, 24, 16, 16), (2, 80, 64, 48), (5, 10, 9, 32)])
def test_linear_keys_and_values_for_a_pool(be, act, rows, heads, kd, used, vd):
    """Keys that fill only the first part of a head, values stored transposed, four slots at a time where they are neighbours."""
    rng = np.random.default_rng(rows)
    kp = -(-kd // 8) * 8
    per = heads * BS * (kp + vd)
    wk, wv = (tl.bf16_round(rng.standard_normal((n, 64)) / 8) for n in (heads * used, heads * vd))
    a = grid(rng.standard_normal((rows, 64)), act)
    for mapping in (None, rng.permutation(rows), np.roll(np.arange(rows), 1), np.roll(np.arange(rows), 4)):
        slots = np.arange(rows) if mapping is None else mapping
        pool = blank(be, (rows // BS, per), act)
        sm = None if mapping is None else be.upload(mapping.astype(np.int32))
        kw = dict(kv_heads=heads, k_dim=kd, v_dim=vd, block_size=BS, pool=pool, slot_mapping=sm)
        dk, nk, _ = packed(be, wk)
        dv, nv, _ = packed(be, wv)
        da = up(be, a, act)
        scratch = be.alloc(rows * 512 * 4)
        be.linear(act, da, 64, dk, nk, 64, rows, lin_out(kind=2, out=scratch, ldo=nk, cols=nk, k_used=used, v_col=nk, **kw))
        be.linear(act, da, 64, dv, nv, 64, rows, lin_out(kind=6, out=scratch, ldo=nv, cols=nv, **kw))
        got = down(be, pool, (rows // BS, per), act)
        k = got[:, :heads * BS * kp].reshape(-1, heads, BS, kp)
        v = got[:, heads * BS * kp:].reshape(-1, heads, vd, BS)
        assert np.isnan(k[..., used:]).all()
        k = k[slots // BS, :, slots % BS, :used]
        v = v[slots // BS, :, :, slots % BS]
        close(k.reshape(rows, -1), a.astype(np.float64) @ wk.T, act)
        close(v.reshape(rows, -1), a.astype(np.float64) @ wv.T, act)


# ---------------------------------------------------------------- angles and latents
def test_rotary_table(be):
    """Angles at far positions, with a factor."""
    pos = np.array([0, 1, 15, 4097, 100003, 2 ** 24 + 1, 2 ** 31 - 1], dtype=np.int32)
    for rot in ({"dims": 2, "base": 9.0}, {"dims": 64, "base": 1e4}, {"dims": 30, "base": 3.0, "scaling": {"factor": 8.0, "original": 64, "fast": 4.0, "slow": 1.0}}):
        f, m = tl.frequencies(rot)
        n = len(f)
        out = blank(be, (len(pos), n, 2), F32)
        be.rotary_table(be.upload(pos), len(pos), n, be.upload(f.astype(np.float64)), m, out)
        a = pos[:, None].astype(np.float64) * f
        assert np.abs(down(be, out, (len(pos), n, 2), F32) - m * np.stack([np.cos(a), np.sin(a)], -1)).max() < 1e-6 * m


def latent_row(be, rank, rot):
    pad, row = be.lib_call("vx_latent_pad", rank), be.lib_call("vx_latent_row", rank, rot)
    assert pad >= rank and pad % 64 == 0 and row >= pad + rot and row % 64 == 0
    return pad, row


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rank,rot,q_rank", [(1, 2, 1), (40, 12, 28), (512, 64, 768), (100, 64, 0), (0, 0, 96), (64, 32, 2500), (700, 130, 13)])
def test_latent_store(be, act, rank, rot, q_rank):
    from vexel_amd.backend import VxLatentStoreArgs
    rng = np.random.default_rng(rank + q_rank)
    bt = Batch(be, [0, 17, 40], [3, 1, 20], seed=2)
    eps, slices = 1e-3, 3
    pad16 = lambda n: -(-n // 16) * 16
    ld = pad16(q_rank) + pad16(rank) + pad16(rot)
    y = rng.standard_normal((slices, bt.rows, ld)).astype(np.float32) * rng.uniform(1e-2, 5, (1, bt.rows, 1)).astype(np.float32)
    wc, wq = ((1 + 0.3 * rng.standard_normal(max(n, 1))).astype(np.float32) for n in (rank, q_rank))
    tab = rng.standard_normal((bt.rows, max(rot // 2, 1), 2)).astype(np.float32)
    p = VxLatentStoreArgs()
    p.rank, p.rot_dim, p.q_rank, p.y, p.y_slices, p.ldy, p.y_stride = rank, rot, q_rank, up(be, y), slices, ld, bt.rows * ld
    p.q_col, p.c_col, p.kr_col, p.eps = 0, pad16(q_rank), pad16(q_rank) + pad16(rank), eps
    p.w_c, p.w_q, p.rot_tab = be.upload(wc), be.upload(wq), be.upload(tab)
    ldq = -(-max(q_rank, 1) // 64) * 64
    qo = blank(be, (bt.rows, ldq), act)
    p.q_out, p.ldq = qo, ldq
    if rank:
        pad, row = latent_row(be, rank, rot)
        pool = blank(be, (bt.pool_blocks * BS, row), act)
        p.pool = pool
    be.latent_store(act, bt.c, p)
    ys = y.astype(np.float64).sum(0)
    if rank:
        got = down(be, pool, (bt.pool_blocks * BS, row), act)
        at = got[bt.slot_map]
        close(at[:, :rank], tl.rms(ys[:, p.c_col:p.c_col + rank], eps) * wc, act)
        u, v = ys[:, p.kr_col:p.kr_col + rot:2], ys[:, p.kr_col + 1:p.kr_col + rot:2]
        kr = at[:, pad:pad + rot]
        close(kr[:, ::2], u * tab[..., 0] - v * tab[..., 1], act)
        close(kr[:, 1::2], v * tab[..., 0] + u * tab[..., 1], act)
        assert np.isnan(at[:, rank:pad]).all() and np.isnan(at[:, pad + rot:]).all()      # nothing else is written
        assert np.isnan(np.delete(got, bt.slot_map, 0)).all()
    if q_rank:
        got = down(be, qo, (bt.rows, ldq), act)
        close(got[:, :q_rank], tl.rms(ys[:, :q_rank], eps) * wq, act)
        assert np.all(got[:, q_rank:] == 0)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rank,rot,heads,kd,first_col", [(40, 12, 3, 96, 64), (512, 64, 4, 192, 128), (10, 2, 2, 20, 6), (64, 32, 5, 40, 8)])
def test_latent_spread(be, act, rank, rot, heads, kd, first_col):
    rng = np.random.default_rng(rot)
    pad, row = latent_row(be, rank, rot)
    src = grid(rng.standard_normal((200, row)), act)
    rows, vd, kp = 96, 16, -(-kd // 8) * 8
    order = rng.integers(0, 200, rows).astype(np.int32)
    per = heads * BS * (kp + vd)
    pool = blank(be, (rows // BS, per), act)
    be.latent_spread(act, up(be, src, act), rank, rot, be.upload(order), rows, pool, heads, kd, vd, BS, first_col)
    got = down(be, pool, (rows // BS, per), act)
    k = got[:, :heads * BS * kp].reshape(-1, heads, BS, kp).transpose(0, 2, 1, 3).reshape(rows, heads, kp)
    assert np.array_equal(k[..., first_col:first_col + rot], np.repeat(src[order][:, None, pad:pad + rot], heads, 1))
    assert np.isnan(k[..., :first_col]).all() and np.isnan(k[..., first_col + rot:]).all() and np.isnan(got[:, heads * BS * kp:]).all()


# ---------------------------------------------------------------- seams and activation
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("cols", [5, 72, 90, 256, 4096, 8200])
def test_post_norm(be, act, cols):
    from vexel_amd.backend import VxPostNormArgs
    rng = np.random.default_rng(cols)
    eps, alpha, slices, depth = 1e-3, 1.9, 3, 4
    ld, ldo = -(-cols // 16) * 16, -(-cols // 64) * 64
    for rows in (1, 9, 300):
        x = (rng.standard_normal((rows, cols)) * rng.uniform(1e-3, 30, (rows, 1))).astype(np.float32)   # rows where eps matters and others
        y = (rng.standard_normal((slices, rows, ld)) * rng.uniform(1e-3, 30, (rows, 1))).astype(np.float32)
        w, wn = (1 + 0.3 * rng.standard_normal((2, cols))).astype(np.float32)
        hist = rng.standard_normal((depth, rows, cols)).astype(np.float32)
        avg = rng.standard_normal(depth).astype(np.float32)
        dx, dy, dw, dn, da = (up(be, v) for v in (x, y, w, wn, avg))

        def run(**kw):
            p = VxPostNormArgs()
            p.rows, p.cols, p.alpha, p.eps, p.x_in, p.y, p.y_slices, p.ldy, p.y_stride = rows, cols, alpha, eps, dx, dy, slices, ld, rows * ld
            p.ldo, p.hist_stride, p.avg = ldo, rows * cols, da
            for name, v in kw.items():
                setattr(p, name, v)
            be.post_norm(act, p)

        v = tl.rms(alpha * x.astype(np.float64) + y.astype(np.float64).sum(0)[:, :cols], eps) * w
        out, xo = blank(be, (rows, ldo), act), blank(be, (rows, cols), F32)
        run(w=dw, x_out=xo, out=out)
        close(down(be, xo, (rows, cols), F32), v, F32)
        got = down(be, out, (rows, ldo), act)
        close(got[:, :cols], v, act)
        assert np.all(got[:, cols:] == 0)
        for keep in (0, 1):
            dh = up(be, hist)
            out, xo = blank(be, (rows, ldo), act), blank(be, (rows, cols), F32)
            run(w=dw, x_out=xo, out=out, hist=dh, n_avg=depth, keep=keep, w_pre=dn)
            mixed = tl.depth_average(avg.astype(np.float64), list(hist[:-1].astype(np.float64)) + [v])
            close(down(be, xo, (rows, cols), F32), mixed, F32)
            close(down(be, out, (rows, ldo), act)[:, :cols], tl.rms(mixed, eps) * wn, act)
            now = down(be, dh, hist.shape, F32)
            assert np.array_equal(now[:-1], hist[:-1])
            if keep:
                close(now[-1], v, F32)
            else:
                assert np.array_equal(now[-1], hist[-1])
        idx = rng.integers(0, rows, 4).astype(np.int32)        # chosen rows
        out = blank(be, (4, ldo), act)
        run(rows=4, row_idx=be.upload(idx), w=dw, out=out, hist=up(be, hist), n_avg=depth, w_pre=dn)
        close(down(be, out, (4, ldo), act)[:, :cols], (tl.rms(mixed, eps) * wn)[idx], act)
        out = blank(be, (rows, ldo), act)
        run(y=None, out=out)                                   # the stream as it is
        close(down(be, out, (rows, ldo), act)[:, :cols], x, act)
        run(w=dw, x_out=dx)                                    # in place
        close(down(be, dx, (rows, cols), F32), v, F32)
        be.reset_pool()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("cols", [1, 13, 24, 320, 5632, 14336, 40000])
def test_poly_norm(be, act, cols):
    rng = np.random.default_rng(cols)
    coef, eps = np.array([0.7, -0.4, 0.2, 0.3], dtype=np.float32), 1e-3
    ldo = -(-cols // 64) * 64
    for rows in (1, 30, 300):
        if rows * cols > 2_000_000:
            continue
        z = rng.standard_normal((rows, cols)) * rng.uniform(1e-3, 12, (rows, 1))
        zp = np.full((rows, ldo), np.nan)
        zp[:, :cols] = grid(z, act)
        out = blank(be, (rows, ldo), act)
        be.poly_norm(act, up(be, zp, act), ldo, rows, cols, be.upload(coef), eps, out, ldo)
        got = down(be, out, (rows, ldo), act)
        close(got[:, :cols], tl.poly_norm(zp[:, :cols].astype(np.float64), coef, eps), act)
        assert np.all(got[:, cols:] == 0)
        parts = rng.standard_normal((3, rows, ldo)).astype(np.float32)     # float32, in slices
        out = blank(be, (rows, ldo), act)
        be.poly_norm(act, up(be, parts), ldo, rows, cols, be.upload(coef), eps, out, ldo, 3, rows * ldo)
        close(down(be, out, (rows, ldo), act)[:, :cols], tl.poly_norm(parts.astype(np.float64).sum(0)[:, :cols], coef, eps), act)
        be.reset_pool()


# ---------------------------------------------------------------- attention over latents
def plain_latent(q, qr, c, kr, pos, scale, sink):
    """q [rows, H, rank], qr [rows, H, rot] at positions pos over c, kr [tokens, ..] -> [rows, H, rank]"""
    out = np.zeros(q.shape)
    for r, p in enumerate(pos):
        s = (q[r].astype(np.float64) @ c[:p + 1].T.astype(np.float64) + qr[r].astype(np.float64) @ kr[:p + 1].T.astype(np.float64)) * scale
        for h in range(q.shape[1]):
            out[r, h] = tl.sink_softmax(s[h], sink[h] if sink is not None else -1e30) @ c[:p + 1].astype(np.float64)
    return out


def run_latent(be, act, bt, H, rank, rot, seed=0, sinks=True, max_rows=0, change=None, scale=None):
    from vexel_amd.backend import VxLatentAttnArgs
    rng = np.random.default_rng(seed)
    pad, row = latent_row(be, rank, rot)
    cs = [grid(rng.standard_normal((n, rank)), act) for n in bt.kv]
    krs = [grid(rng.standard_normal((n, rot)), act) for n in bt.kv]
    q, qr = grid(rng.standard_normal((bt.rows, H, rank)), act), grid(rng.standard_normal((bt.rows, H, rot)), act)
    scale = scale or 1.5 / (rank + rot) ** 0.5
    if change:
        change(q, qr, cs, krs)
    # tokens that are no longer, or not yet, anyone's: large latents a kernel must not see
    pool = np.zeros((bt.pool_blocks * BS, row))
    pool[:, :rank], pool[:, pad:pad + rot] = rng.standard_normal((len(pool), rank)) * 50, rng.standard_normal((len(pool), rot)) * 50
    for i, n in enumerate(bt.kv):
        for t in range(n):
            s = bt.slot(i, t)
            pool[s, :rank], pool[s, pad:pad + rot] = cs[i][t], krs[i][t]
    qp = np.zeros((bt.rows, H, pad))
    qp[..., :rank] = q
    stride = 64 + -(-rot // 16) * 16                           # the rotated part behind 64 columns of something else
    qrp = rng.standard_normal((bt.rows, H, stride))
    qrp[..., 64:] = 0
    qrp[..., 64:64 + rot] = qr
    sink = (rng.standard_normal(H) * 2).astype(np.float32) if sinks else None
    out = blank(be, (bt.rows, H, pad), act)
    p = VxLatentAttnArgs()
    p.heads, p.rank, p.rot_dim, p.scale, p.max_rows = H, rank, rot, scale, max_rows
    p.q, p.ldq, p.qr, p.ldqr, p.qr_stride = up(be, qp, act), H * pad, up(be, qrp, act) + 64 * (4 if act == F32 else 2), H * stride, stride
    p.pool, p.out, p.ldo = up(be, pool, act), out, H * pad
    if sinks:
        p.sink = be.upload(sink)
    be.attn_latent(act, bt.c, p)
    got = down(be, out, (bt.rows, H, pad), act)
    for i in range(len(bt.lens)):
        r = slice(bt.cu[i], bt.cu[i + 1])
        if max_rows and bt.lens[i] > max_rows:
            assert np.isnan(got[r]).all()
            continue
        close(got[r, :, :rank], plain_latent(q[r], qr[r], cs[i], krs[i], bt.pos[r], scale, sink), act, (i, bt.start[i], bt.lens[i]))
        assert np.all(got[r, :, rank:] == 0)


# prompts, later portions, single tokens; at the edges of blocks (16), of key tiles (64, 128) and of pieces
MIXED = ([0, 5, 300, 31, 62, 15, 127, 255, 0, 63], [70, 2, 1, 1, 3, 40, 1, 2, 1, 2])
SINGLE = ([0, 1, 15, 16, 63, 64, 127, 128, 255, 256, 257, 400], [1] * 12)
LATENTS = [(4, 40, 12), (1, 1, 2), (16, 64, 64), (17, 100, 32), (33, 128, 16), (3, 256, 64), (20, 512, 64), (70, 300, 6), (2, 520, 64), (2, 64, 80)]


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", LATENTS)
def test_latent_attention_geometries(be, act, geom):
    H, rank, rot = geom
    assert be.lib_call("vx_attn_latent_fast", act, BS, rank, rot) == int(act == BF16 and rank <= 512 and rot <= 64)
    run_latent(be, act, Batch(be, *MIXED, seed=1), *geom)
    run_latent(be, act, Batch(be, *SINGLE, seed=2), *geom)


@pytest.mark.parametrize("act", ACTS)
def test_latent_attention_options(be, act):
    """No sinks; sequences left out by how many rows they bring; scores far apart."""
    for batch in (MIXED, SINGLE):
        run_latent(be, act, Batch(be, *batch, seed=3), 5, 72, 8, sinks=False)
        run_latent(be, act, Batch(be, *batch, seed=3), 5, 72, 8, scale=3.0)
    for most in (1, 2, 39, 40):
        run_latent(be, act, Batch(be, *MIXED, seed=4), 5, 72, 8, max_rows=most)


@pytest.mark.parametrize("heads,start,lens", [(2, 900, [7]), (2, 1500, [33]), (16, 700, [64]), (9, 0, [300]), (64, 40, [90]), (1, 5000, [1]), (40, 3000, [1])])
def test_latent_attention_pieces_and_tiles(be, heads, start, lens):
    """Few rows over many keys (in pieces) and many rows (one piece), each size of query tile, beside a single token."""
    run_latent(be, BF16, Batch(be, [start, 40], lens + [1], seed=5), heads, 64, 32, seed=1)


def test_latent_attention_many_sequences(be):
    rng = np.random.default_rng(6)
    run_latent(be, BF16, Batch(be, rng.integers(0, 700, 70).tolist(), [1] * 70, seed=6), 24, 130, 64, seed=2)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("length,back", [(1, 0), (17, 16), (65, 64), (130, 129), (130, 128), (257, 256), (700, 699), (700, 512), (700, 511), (700, 1)])
def test_latent_attention_far_key(be, act, length, back):
    """One key far back stands out, by its latent or by its rotated part: nearly all the weight is its."""
    for rotated in (False, True):
        for rows in {1, 2, min(length, 40)}:
            if rows > length:
                continue

            def stand_out(q, qr, cs, krs):
                x, k = (qr, krs) if rotated else (q, cs)
                x[-1], k[0][:, 3] = 0, np.minimum(k[0][:, 3], 0)
                x[-1, :, 3] = 8.0
                k[0][length - 1 - back, 3] = 40.0

            run_latent(be, act, Batch(be, [length - rows], [rows], seed=length), 4, 72, 24, change=stand_out)


@pytest.mark.parametrize("act", ACTS)
def test_sink_of_grouped_attention(be, act):
    """vx_attn_ragged with a sink per head, for single tokens, few and many rows, and with sequences that bring few rows left out."""
    from vexel_amd.backend import VxAttnArgs
    for batch, H, G, least in ((MIXED, 4, 2, 0), (SINGLE, 4, 2, 0), (MIXED, 4, 4, 40), (([7, 3], [500, 30]), 16, 16, 31), (([0, 300], [90, 1]), 64, 64, 2)):
        bt = Batch(be, *batch, seed=8)
        rng = np.random.default_rng(8)
        D, V = 24, 16
        kv = [(grid(rng.standard_normal((n, G, D)), act), grid(rng.standard_normal((n, G, V)), act)) for n in bt.kv]
        pool = np.zeros((bt.pool_blocks, G * BS * (D + V)))
        kk, vv = pool[:, :G * BS * D].reshape(-1, G, BS, D), pool[:, G * BS * D:].reshape(-1, G, V, BS)
        for i, (k, v) in enumerate(kv):
            for t in range(bt.kv[i]):
                s = bt.slot(i, t)
                kk[s // BS, :, s % BS], vv[s // BS, :, :, s % BS] = k[t], v[t]
        q, sink = grid(rng.standard_normal((bt.rows, H, D)), act), (rng.standard_normal(H) * 3).astype(np.float32)
        out = blank(be, (bt.rows, H, V), act)
        p = VxAttnArgs()
        p.heads, p.kv_heads, p.k_dim, p.v_dim, p.scale, p.out_scale, p.min_rows = H, G, D, V, 0.3, 1.0, least
        p.q, p.ldq, p.pool, p.out, p.ldo, p.sink = up(be, q, act), H * D, up(be, pool, act), out, H * V, be.upload(sink)
        be.attn_ragged(act, bt.c, p)
        got = down(be, out, (bt.rows, H, V), act)
        for i, (k, v) in enumerate(kv):
            r = slice(bt.cu[i], bt.cu[i + 1])
            if bt.lens[i] < least:
                assert np.isnan(got[r]).all()
                continue
            seen = bt.pos[r][:, None] >= np.arange(bt.kv[i])[None, :]
            for h in range(H):
                s = q[r, h].astype(np.float64) @ k[:, h // (H // G)].T.astype(np.float64) * 0.3
                close(got[r, h], tl.sink_softmax(np.where(seen, s, -np.inf), sink[h]) @ v[:, h // (H // G)].astype(np.float64), act, (i, h))


# ---------------------------------------------------------------- models
def load(be, tmp_path, cfg, seed=1, dtype="float32", **kw):
    from vexel_amd.runtime import ModelRuntime
    t = tensors(cfg, seed)
    folder = str(tmp_path / "model")
    tl.write_model(folder, cfg, t)
    kw = {**dict(pool_blocks=64, max_seqs=6, max_batch=32), **kw}
    return ModelRuntime.load(be, folder, dtype=dtype, **kw), t


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["SMALL", "TINY", "EVEN", "WIDE"])
def test_prompts_portions_and_decoding(be, tmp_path, dtype, name):
    """The whole prompt, token by token, and portions of several sizes (EVEN: around the sizes from which keys are spelled out): the
    plain implementation's logits at every position, in the blocks of the run before."""
    cfg = {"SMALL": SMALL, "TINY": TINY, "EVEN": EVEN, "WIDE": WIDE}[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=1, pool_blocks=13)
    for n in (1, 2, 3, 16, 17, 203):
        toks = prompt(cfg, n, n)
        want = tl.forward(cfg, t, toks)
        top = limit(dtype, cfg, t, toks, want)
        for sizes in ([n], [1], [2], [2, 3, 1], [16], [7, 63, 1], [65, 1], [72, 71, 60], [1, 72, 2, 128]):
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
    cfg = {"SMALL": SMALL, "EVEN": EVEN}[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=3, pool_blocks=32)
    rng = np.random.default_rng(8)
    todo = [(i, prompt(cfg, n, 100 + i)) for i, n in enumerate((90, 3, 150, 130, 1, 17, 64, 200, 33))]
    want = {i: tl.forward(cfg, t, p) for i, p in todo}
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
    """300 tokens one by one after a prompt of 5, beside another sequence; then another in its place."""
    cfg = {"SMALL": SMALL, "EVEN": EVEN}[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=2, pool_blocks=40)
    for seed in (1, 2):
        a, b = prompt(cfg, 305, seed), prompt(cfg, 305, seed + 10)
        wa, wb = tl.forward(cfg, t, a), tl.forward(cfg, t, b)
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
    """Sharp attention (queries and keys scaled up): tokens that repeat far back, in the middle of prompts, at their ends and decoded, in
    whole prompts and in portions."""
    cfg = config([(first(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=64, q_rank=40, base=1e5), 64), (second(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=64), 64)],
                 width=96, vocab=400)
    from vexel_amd.runtime import ModelRuntime
    t = tensors(cfg, 4, qk_gain=3.5)
    tl.write_model(str(tmp_path / "model"), cfg, t)
    mr = ModelRuntime.load(be, str(tmp_path / "model"), dtype=dtype, pool_blocks=40, max_seqs=2, max_batch=32)
    toks = prompt(cfg, 560, 9)
    for at in (130, 257, 400, 511, 512, 558, 559):
        toks[at] = toks[at % 7]
    want = tl.forward(cfg, t, toks)
    top = limit(dtype, cfg, t, toks, want)
    for sizes in ([560], [500, 1], [129, 128, 1]):
        assert error(run_portions(mr, 0, toks, sizes), want).max() < top, sizes
        mr.delete_sequence(0)
    mr.close()


def greedy(cfg, t, toks, n):
    toks, out = list(toks), []
    for _ in range(n):
        lg = tl.forward(cfg, t, toks)[-1]
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
    cfg = {"SMALL": SMALL, "EVEN": EVEN, "WIDE": WIDE}[name]
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


def test_a_sequence_goes_back_and_shares_blocks(be, tmp_path):
    """A sequence is its blocks alone here: it can be cut to any length, and another can start from its first blocks."""
    from vexel_amd.backend import VexelError
    cfg = SMALL
    mr, t = load(be, tmp_path, cfg, max_seqs=3, pool_blocks=20)
    a, b = prompt(cfg, 60, 1), prompt(cfg, 60, 2)
    mr.step([(0, a[:50])], [])
    mr.truncate_sequence(0, 21)
    toks = a[:21] + b[21:50]
    want = tl.forward(cfg, t, toks)
    lg, _ = mr.step([(0, toks[21:])], list(range(29)))
    assert error(lg, want[21:]).max() < LIMIT["float32"]
    mr.create_sequence(1)
    mr.share_blocks(0, 1, 32)                                  # two whole blocks
    toks = toks[:32] + a[32:60]
    want = tl.forward(cfg, t, toks)
    lg, _ = mr.step([(1, toks[32:])], list(range(28)))
    assert error(lg, want[32:]).max() < LIMIT["float32"]
    with pytest.raises(VexelError, match="fragment"):
        mr.cache_fragment("a", 0)
    with pytest.raises(VexelError, match="mixer program"):
        mr.verify_tree([0], [1], [50], [([], [])])
    with pytest.raises(VexelError, match="position"):
        mr.decode_with_paged_kv_batched([1], [0], [9])
    lg, _ = mr.decode_with_paged_kv_batched([b[50]], [0], [50])
    assert error(lg, tl.forward(cfg, t, a[:21] + b[21:51])[-1:]).max() < LIMIT["float32"]
    mr.close()


def test_loader_errors(be, tmp_path):
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import ModelRuntime
    cfg = config([(first(), 32), (second(), 16), (second(kv_from=1), None)])
    t = tensors(cfg, 1)
    folder = str(tmp_path / "m")
    for change, text in ((lambda d: d.pop("l0.mix.sink"), "l0.mix.sink is missing"), (lambda d: d.pop("l1.mix.q"), "l1.mix.q is missing"),
                         (lambda d: d.pop("l0.mix.dq.norm"), "l0.mix.dq.norm is missing"), (lambda d: d.update({"head": d["head"][:-1]}), "head: shape"),
                         (lambda d: d.update({"l2.dwa": d["l2.dwa"][:-1]}), "l2.dwa: shape"), (lambda d: d.update({"l2.mix.uk": d["l2.mix.uk"][:, :-1]}), "l2.mix.uk: shape"),
                         (lambda d: d.update({"l0.mlp.act": d["l0.mlp.act"][:3]}), "l0.mlp.act: shape")):
        d = dict(t)
        change(d)
        tl.write_model(folder, cfg, d)
        with pytest.raises(VexelError, match=text):
            ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1)
    tl.write_model(folder, cfg, t)                             # (what the third layer does not need, it does not ask for)
    assert "l2.mix.dkv" not in t and "l2.norm2" not in t
    ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1).close()


def test_generation_from_the_command_line(be, tmp_path, capsys):
    from vexel_amd.__main__ import main
    cfg = SMALL
    t = tensors(cfg, 2)
    tl.write_model(str(tmp_path / "m"), cfg, t)
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
    tl.write_model(str(tmp_path / "m"), cfg, t)
    a, b, c = (prompt(cfg, n, 80 + n) for n in (50, 30, 47))
    steps = [{"entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:1], "want": []}], "end": []},
             {"entries": [{"id": "b", "tokens": b[1:], "want": [28]}, {"id": "a", "tokens": a[20:], "want": [29, 3]}], "end": ["a", "b"]},
             {"entries": [{"id": "c", "tokens": c, "want": [46]}], "end": ["c"]}]
    want = {n: tl.forward(cfg, t, toks) for n, toks in (("a", a), ("b", b), ("c", c))}
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
