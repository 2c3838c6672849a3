"""Lozedra on the GPU: each mixed-batch kernel alone against the plain implementation, then models through the engine's
loader, block pool, step, scheduler and graph replay."""
import ctypes as C
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import lozedra as lz
from mixed_batches import ACTS, BF16, BS, F32, Batch, act_array, blank, close, down, grid, lin_out, packed, prompt, run_portions, up
from lozedra_models import EVEN, LIMIT, SMALL, TINY, config, error, limit, mixer, tensors

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
@pytest.mark.parametrize("rows", [1, 2, 16, 17, 33, 64, 65, 129, 300])
def test_linear_plain(be, act, rows):
    rng = np.random.default_rng(rows)
    for n, k in ((16, 64), (50, 77), (208, 448), (1040, 130)):
        w, a = lz.bf16_round(rng.standard_normal((n, k))), grid(rng.standard_normal((rows, k)), act)
        p, n_pad, k_pad = packed(be, w)
        a_pad = np.zeros((rows, k_pad))
        a_pad[:, :k] = a
        da, want = up(be, a_pad, act), a.astype(np.float64) @ w.T.astype(np.float64)
        out = blank(be, (rows, n), F32)
        be.linear(act, da, k_pad, p, n_pad, k_pad, rows, lin_out(kind=0, out_f32=1, out=out, ldo=n, cols=n))
        close(down(be, out, (rows, n), F32), want, F32, (n, k))
        out = blank(be, (rows, n_pad), act)
        be.linear(act, da, k_pad, p, n_pad, k_pad, rows, lin_out(kind=0, out=out, ldo=n_pad, cols=n))
        got = down(be, out, (rows, n_pad), act)
        close(got[:, :n], want, act, (n, k))
        assert np.isnan(got[:, n:]).all()                      # nothing beyond the columns asked for
        for slices in (2, 5):
            out = blank(be, (slices, rows, n_pad), F32)
            be.linear(act, da, k_pad, p, n_pad, k_pad, rows, lin_out(kind=0, out_f32=1, out=out, ldo=n_pad, cols=n_pad, slices=slices))
            close(down(be, out, (slices, rows, n_pad), F32).sum(0)[:, :n], want, F32, (n, k, slices))
        be.reset_pool()


def test_linear_rows_do_not_depend_on_the_batch(be):
    """A row is the same number whatever rows stand beside it (within one kernel: bit for bit)."""
    rng = np.random.default_rng(4)
    w = lz.bf16_round(rng.standard_normal((96, 256)))
    p, n_pad, k_pad = packed(be, w)
    a = rng.standard_normal((300, 256))
    res = {}
    for rows in (1, 5, 30, 64, 65, 300):
        out = blank(be, (rows, 96), F32)
        be.linear(BF16, up(be, a[:rows], BF16), k_pad, p, n_pad, k_pad, rows, lin_out(kind=0, out_f32=1, out=out, ldo=96, cols=96))
        res[rows] = down(be, out, (rows, 96), F32)
    for rows in (1, 5, 30):
        assert np.array_equal(res[rows], res[64][:rows])
    assert np.array_equal(res[65], res[300][:65])
    assert np.abs(res[64] - res[300][:64]).max() < 1e-4


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [3, 70])
def test_linear_concatenated_columns_and_rows(be, act, rows):
    """Two matrices stacked in the rows of one packed matrix, and two side by side in its columns at an odd column."""
    rng = np.random.default_rng(9)
    w1, w2 = (lz.bf16_round(rng.standard_normal((n, 90))) for n in (21, 40))
    dst, n_pad, k_pad = packed(be, w1, n_pad=32 + 48)
    packed(be, w2, n_pad=80, k_pad=k_pad, tile0=2, dst=dst)
    a = np.zeros((rows, k_pad))
    a[:, :90] = grid(rng.standard_normal((rows, 90)), act)
    out = blank(be, (rows, 80), F32)
    be.linear(act, up(be, a, act), k_pad, dst, 80, k_pad, rows, lin_out(kind=0, out_f32=1, out=out, ldo=80, cols=80))
    got = down(be, out, (rows, 80), F32)
    close(got[:, :21], a[:, :90] @ w1.T, F32)
    close(got[:, 32:72], a[:, :90] @ w2.T, F32)
    assert np.all(got[:, 21:32] == 0) and np.all(got[:, 72:] == 0)
    v1, v2 = lz.bf16_round(rng.standard_normal((32, 37))), lz.bf16_round(rng.standard_normal((32, 50)))
    dst, n_pad, k_pad = packed(be, v1, k_pad=128)
    packed(be, v2, k_pad=128, col0=37, dst=dst)
    a = np.zeros((rows, 128))
    a[:, :87] = grid(rng.standard_normal((rows, 87)), act)
    out = blank(be, (rows, 32), F32)
    be.linear(act, up(be, a, act), 128, dst, 32, 128, rows, lin_out(kind=0, out_f32=1, out=out, ldo=32, cols=32))
    close(down(be, out, (rows, 32), F32), a[:, :37] @ v1.T + a[:, 37:87] @ v2.T, F32)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows", [1, 20, 64, 90])
def test_linear_fused_results(be, act, rows):
    """silu(gate) * up over alternating tiles; the split with its second half in float32, deep enough for slices; softplus."""
    rng = np.random.default_rng(rows)
    k, ff = 128, 70
    g, u = (lz.bf16_round(rng.standard_normal((ff, k)) * 0.2) for _ in range(2))
    dst, n_pad, k_pad = packed(be, g, n_pad=256, step=2)
    packed(be, u, n_pad=256, tile0=1, step=2, dst=dst)
    a = grid(rng.standard_normal((rows, k)), act)
    out = blank(be, (rows, 128), act)
    be.linear(act, up(be, a, act), k, dst, 256, k, rows, lin_out(kind=1, out=out, ldo=128, cols=128))
    got = down(be, out, (rows, 128), act)
    close(got[:, :ff], lz.silu(a.astype(np.float64) @ g.T) * (a.astype(np.float64) @ u.T), act)
    assert np.all(got[:, ff:] == 0)
    k = 4096
    w = lz.bf16_round(rng.standard_normal((112, k)))
    dst, n_pad, k_pad = packed(be, w)
    a = grid(rng.standard_normal((rows, k)), act)
    o1, o2 = blank(be, (rows, 64), act), blank(be, (rows, 48), F32)
    be.linear(act, up(be, a, act), k, dst, 112, k, rows, lin_out(kind=3, out=o1, ldo=64, cols=64, split=64, out2=o2, ldo2=48))
    want = a.astype(np.float64) @ w.T
    close(down(be, o1, (rows, 64), act), want[:, :64], act)
    close(down(be, o2, (rows, 48), F32), want[:, 64:], F32)
    w = lz.bf16_round(rng.standard_normal((37, 20)))
    bias = (rng.standard_normal(37) * 8).astype(np.float32)
    dst, n_pad, k_pad = packed(be, w)
    a = np.zeros((rows, 64))
    a[:, :20] = grid(rng.standard_normal((rows, 20)), act)
    out = blank(be, (rows, 48), F32)
    be.linear(act, up(be, a, act), 64, dst, 48, 64, rows, lin_out(kind=4, out_f32=1, out=out, ldo=48, cols=37, bias=be.upload(bias)))
    got = down(be, out, (rows, 48), F32)[:, :37]
    want = lz.softplus(a[:, :20] @ w.T + bias)
    assert np.all(np.abs(got - want) <= 1e-5 * np.abs(want) + 1e-9 + 2e-6 * np.abs(want).max())


# ---------------------------------------------------------------- seams
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("cols", [5, 72, 90, 256, 4096, 8200])
def test_residual_norm(be, act, cols):
    from vexel_amd.backend import VxResidualNormArgs
    rng = np.random.default_rng(cols)
    eps, mult, slices = 1e-3, 0.37, 3
    ld = -(-cols // 16) * 16
    ldo = -(-cols // 64) * 64
    for rows in (1, 9, 300):
        x, add = rng.standard_normal((2, rows, cols)).astype(np.float32)
        x *= rng.uniform(1e-3, 30, (rows, 1))                  # rows where eps matters and rows where it does not
        x = x.astype(np.float32)
        y = rng.standard_normal((slices, rows, ld)).astype(np.float32)
        wp, wn = (1 + 0.3 * rng.standard_normal((2, cols))).astype(np.float32)
        dx, da, dy, dp, dn = (up(be, v) for v in (x, add, y, wp, wn))

        def run(**kw):
            p = VxResidualNormArgs()
            p.rows, p.cols, p.mult, p.eps, p.ldy, p.y_stride, p.y_slices = rows, cols, mult, eps, ld, rows * ld, slices
            p.x_in = dx
            for name, v in kw.items():
                setattr(p, name, v)
            be.residual_norm(act, p)

        out, xo = blank(be, (rows, ldo), act), blank(be, (rows, cols), F32)
        run(y=dy, w_post=dp, add=da, x_out=xo, w_pre=dn, out=out, ldo=ldo)
        xn = x + mult * lz.rms_norm(y.astype(np.float64).sum(0)[:, :cols], wp, eps) + add
        close(down(be, xo, (rows, cols), F32), xn, F32)
        got = down(be, out, (rows, ldo), act)
        close(got[:, :cols], lz.rms_norm(xn, wn, eps), act)
        assert np.all(got[:, cols:] == 0)
        out = blank(be, (rows, ldo), act)
        run(w_pre=dn, out=out, ldo=ldo)                        # a plain norm; the stream stays as it is
        close(down(be, out, (rows, ldo), act)[:, :cols], lz.rms_norm(x, wn, eps), act)
        assert np.array_equal(down(be, dx, (rows, cols), F32), x)
        idx = rng.integers(0, rows, 4).astype(np.int32)        # chosen rows
        out = blank(be, (4, ldo), act)
        run(rows=4, row_idx=be.upload(idx), y=dy, w_post=dp, w_pre=dn, out=out, ldo=ldo)
        xn = x + mult * lz.rms_norm(y.astype(np.float64).sum(0)[:, :cols], wp, eps)
        close(down(be, out, (4, ldo), act)[:, :cols], lz.rms_norm(xn, wn, eps)[idx], act)
        run(y=dy, w_post=dp, x_out=dx)                         # in place
        close(down(be, dx, (rows, cols), F32), xn, F32)
        be.reset_pool()


# ---------------------------------------------------------------- convolution and scan
PORTIONS = [[90], [2] * 5 + [1] * 4, [1, 2, 3, 1, 64, 1], [65, 2, 130], [63, 1, 64, 64, 1], [1] * 7]


def feed(portions_by_seq, run):
    """Hands the sequences' portions to run(start, lens, which), one portion of each sequence a step, unequal counts."""
    at = [0] * len(portions_by_seq)
    for step in range(max(len(p) for p in portions_by_seq)):
        which = [i for i, p in enumerate(portions_by_seq) if step < len(p)]
        lens = [portions_by_seq[i][step] for i in which]
        run([at[i] for i in which], lens, which)
        for i, l in zip(which, lens):
            at[i] += l


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("taps,channels", [(1, 8), (2, 40), (4, 64), (4, 37), (7, 24)])
def test_convolution(be, act, taps, channels):
    from vexel_amd.backend import VxConvArgs
    rng = np.random.default_rng(taps)
    w, b = rng.standard_normal((channels, taps)).astype(np.float32), rng.standard_normal(channels).astype(np.float32)
    ldx, ldo = channels + 24 - channels % 8, -(-channels // 64) * 64
    xs = [grid(rng.standard_normal((sum(p), channels)), act) for p in PORTIONS]
    wants = [lz.silu(lz.causal_conv(x.astype(np.float64), w.astype(np.float64), b)) for x in xs]
    hist = taps - 1
    slots = rng.permutation(8)[:len(xs)].tolist()
    state = be.upload(act_array(np.full((8, max(hist, 1), channels), 1e3), act), permanent=True)   # an earlier owner's leavings

    def run(start, lens, which):
        bt = Batch(be, start, lens, slots=[slots[i] for i in which])
        x = np.full((bt.rows, ldx), np.nan)
        x[:, :channels] = np.concatenate([xs[i][s:s + l] for i, s, l in zip(which, start, lens)])
        out = blank(be, (bt.rows, ldo), act)
        p = VxConvArgs()
        p.channels, p.taps, p.x, p.ldx, p.out, p.ldo = channels, taps, up(be, x, act), ldx, out, ldo
        p.w, p.b, p.state = be.upload(np.ascontiguousarray(w.T)), be.upload(b), state
        be.conv_silu(act, bt.c, p)
        got = down(be, out, (bt.rows, ldo), act)
        for j, i in enumerate(which):
            close(got[bt.cu[j]:bt.cu[j + 1], :channels], wants[i][start[j]:start[j] + lens[j]], act, (i, start[j], lens[j]))
        assert np.all(got[:, channels:] == 0)
        be.reset_pool()

    feed(PORTIONS, run)
    be.free(state)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("states,channels", [(1, 5), (8, 64), (16, 130), (17, 33), (64, 20), (130, 12), (256, 9)])
def test_selective_scan(be, act, states, channels):
    from vexel_amd.backend import VxScanArgs
    pad = be.lib_call("vx_scan_state_pad", states)
    assert pad >= states and pad % 8 == 0
    rng = np.random.default_rng(states)
    A = -np.exp(rng.uniform(np.log(0.002), np.log(8.0), (channels, states)))   # states that last and states that do not
    D = rng.standard_normal(channels).astype(np.float32)
    n = [sum(p) for p in PORTIONS]
    xs = [grid(rng.standard_normal((t, channels)), act) for t in n]
    zs = [grid(rng.standard_normal((t, channels)), act) for t in n]
    dts = [np.exp(rng.uniform(-6, 1, (t, channels))).astype(np.float32) for t in n]
    Bs, Cs = ([rng.standard_normal((t, states)).astype(np.float32) for t in n] for _ in range(2))
    scale = 0.7
    wants = []
    for i in range(len(n)):
        y, _ = lz.selective_scan(xs[i].astype(np.float64), dts[i].astype(np.float64), A, Bs[i], Cs[i], D)
        wants.append(scale * y * lz.silu(zs[i].astype(np.float64)))
    a2 = np.zeros((channels, pad), dtype=np.float32)
    a2[:, :states] = A / np.log(2.0)
    slots = rng.permutation(8)[:len(n)].tolist()
    state = be.upload(np.full((8, channels, pad), 1e3, dtype=np.float32), permanent=True)
    ld, out_cols = channels + 3, channels + 5

    def run(start, lens, which):
        bt = Batch(be, start, lens, slots=[slots[i] for i in which])
        cat = lambda src: np.concatenate([src[i][s:s + l] for i, s, l in zip(which, start, lens)])
        wide = lambda a: np.concatenate([a, np.full((bt.rows, ld - channels), np.nan)], 1)
        bc = np.zeros((bt.rows, 2, pad), dtype=np.float32)
        bc[:, 0, :states], bc[:, 1, :states] = cat(Bs), cat(Cs)
        out = blank(be, (bt.rows, out_cols + 1), act)
        p = VxScanArgs()
        p.channels, p.states, p.a2, p.d = channels, states, be.upload(a2), be.upload(D)
        p.x, p.z, p.ldx, p.ldz = up(be, wide(cat(xs)), act), up(be, wide(cat(zs)), act), ld, ld
        p.dt, p.bc, p.lddt = up(be, wide(cat(dts))), be.upload(bc), ld
        p.state, p.out_scale, p.out, p.ldo, p.out_cols = state, scale, out, out_cols + 1, out_cols
        be.selective_scan(act, bt.c, p)
        got = down(be, out, (bt.rows, out_cols + 1), act)
        for j, i in enumerate(which):
            close(got[bt.cu[j]:bt.cu[j + 1], :channels], wants[i][start[j]:start[j] + lens[j]], act, (i, start[j], lens[j]))
        assert np.all(got[:, channels:out_cols] == 0) and np.isnan(got[:, out_cols:]).all()
        be.reset_pool()

    feed(PORTIONS, run)
    be.free(state)


# ---------------------------------------------------------------- attention
class Cache:
    """Random keys and values of every sequence, in the pool's layout on the device."""

    def __init__(self, be, bt, act, G, D, V, rng, k_scale=1.0):
        self.k = [grid(rng.standard_normal((n, G, D)) * k_scale, act) for n in bt.kv]
        self.v = [grid(rng.standard_normal((n, G, V)), act) for n in bt.kv]
        kp = -(-D // 8) * 8
        per = G * BS * (kp + V)
        assert be.lib_call("vx_kv_block_elems", BS, G, D, V) == per
        self.shape = (bt.pool_blocks, per)
        pool = np.zeros(self.shape, dtype=np.float32)
        # tokens that are no longer, or not yet, anyone's: large keys and values a kernel must not see
        pool[:] = rng.standard_normal(self.shape) * 50
        kk = pool[:, :G * BS * kp].reshape(-1, G, BS, kp)
        kk[..., D:] = 0
        vv = pool[:, G * BS * kp:].reshape(-1, G, V, BS)
        for i, n in enumerate(bt.kv):
            for p in range(n):
                s = bt.slot(i, p)
                kk[s // BS, :, s % BS, :D] = self.k[i][p]
                vv[s // BS, :, :, s % BS] = self.v[i][p]
        self.dev = up(be, pool, act)


def plain_attention(q, k, v, pos, scale, bias, temp, gate, out_scale):
    """q [rows, H, D] at positions pos over k, v [tokens, G, ..]; bias [H, n] -> [rows, H * V]"""
    H, G = q.shape[1], k.shape[1]
    qt = q.astype(np.float64) * (lz.query_temperature(pos, *temp) if temp else np.ones(len(pos)))[:, None, None]
    out = np.zeros((len(pos), H, v.shape[2]))
    for r, p in enumerate(pos):
        for h in range(H):
            s = k[:p + 1, h // (H // G)].astype(np.float64) @ qt[r, h] * scale
            if bias is not None:
                s = s + bias[h][np.minimum(p - np.arange(p + 1), bias.shape[1] - 1)]
            e = np.exp(s - s.max())
            out[r, h] = e / e.sum() @ v[:p + 1, h // (H // G)].astype(np.float64)
    out = out.reshape(len(pos), -1)
    return out_scale * out * (lz.sigmoid(gate.astype(np.float64)) if gate is not None else 1.0)


def run_attention(be, act, bt, H, G, D, V, seed=0, bias_len=40, temp=(0.5, 16), gated=True, change=None, k_scale=1.0):
    from vexel_amd.backend import VxAttnArgs
    rng = np.random.default_rng(seed)
    cache = Cache(be, bt, act, G, D, V, rng, k_scale)
    q = grid(rng.standard_normal((bt.rows, H, D)), act)
    if change:
        change(q, cache, bt)
    gate = grid(rng.standard_normal((bt.rows, H * V)), act) if gated else None
    bias = (rng.standard_normal((H, bias_len)) * 2).astype(np.float32) if bias_len else None
    ldq = -(-H * D // 8) * 8 + 8
    qp = np.full((bt.rows, ldq), np.nan)
    qp[:, :H * D] = q.reshape(bt.rows, -1)
    ldo = H * V + 3
    out = blank(be, (bt.rows, ldo), act)
    p = VxAttnArgs()
    p.heads, p.kv_heads, p.k_dim, p.v_dim, p.scale = H, G, D, V, D ** -0.5
    if temp:
        p.temp_coef, p.temp_every = temp
    if bias_len:
        p.bias, p.bias_len = be.upload(bias), bias_len
    p.q, p.ldq, p.pool, p.out_scale, p.out, p.ldo = up(be, qp, act), ldq, cache.dev, 0.8, out, ldo
    if gated:
        p.gate, p.ldg = up(be, gate, act), H * V
    be.attn_ragged(act, bt.c, p)
    got = down(be, out, (bt.rows, ldo), act)
    assert np.isnan(got[:, H * V:]).all()
    for i in range(len(bt.lens)):
        r = slice(bt.cu[i], bt.cu[i + 1])
        want = plain_attention(q[r], cache.k[i], cache.v[i], bt.pos[r], D ** -0.5, bias, temp, gate[r] if gated else None, 0.8)
        close(got[r, :H * V], want, act, (i, bt.start[i], bt.lens[i]))


# prompts, later portions, single tokens; at the edges of blocks (16), of groups of keys (32) and of pieces (128, 256)
MIXED = ([0, 5, 300, 31, 32, 15, 16, 255, 0, 127], [70, 2, 1, 1, 1, 40, 1, 2, 1, 3])
SINGLE = ([0, 1, 15, 16, 31, 32, 127, 128, 255, 256, 257, 400], [1] * 12)

GEOMETRIES = [(4, 2, 64, 64), (3, 1, 96, 40), (6, 6, 40, 96), (8, 1, 128, 128), (5, 1, 13, 9), (20, 1, 64, 32), (2, 1, 192, 160),
              (4, 2, 256, 256), (1, 1, 1, 1), (7, 7, 8, 120), (2, 2, 300, 270)]


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("geom", GEOMETRIES)
def test_attention_geometries(be, act, geom):
    H, G, D, V = geom
    assert be.lib_call("vx_attn_ragged_fast", act, BS, H, G, D, V) == int(act == BF16 and max(D, V) <= 256)
    run_attention(be, act, Batch(be, *MIXED, seed=1), *geom)
    run_attention(be, act, Batch(be, *SINGLE, seed=2), *geom)


@pytest.mark.parametrize("act", ACTS)
def test_attention_options(be, act):
    """No gate, no bias, no temperature, a temperature per position, bias tables of one entry and too long for LDS."""
    for batch in (MIXED, SINGLE):
        for kw in (dict(gated=False), dict(bias_len=0), dict(temp=None), dict(temp=(1.0, 1)), dict(bias_len=1), dict(bias_len=9000),
                   dict(gated=False, bias_len=0, temp=None), dict(bias_len=300)):
            run_attention(be, act, Batch(be, *batch, seed=3), 4, 2, 32, 48, seed=5, **kw)


@pytest.mark.parametrize("heads,start,lens", [(128, 33, 400), (128, 0, 180), (16, 1000, 515), (64, 5, 402), (64, 0, 263)])
def test_attention_many_rows(be, heads, start, lens):
    """Enough rows for each way of dealing queries and keys to a workgroup's waves: one or two query tiles a wave, one, two or
    four waves to the same queries."""
    run_attention(be, BF16, Batch(be, [start, 40, 0], [lens, 1, 3], seed=4), heads, heads // 4, 16, 16, seed=1)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("length,back", [(1, 0), (17, 16), (33, 32), (130, 129), (257, 256), (700, 699), (700, 444), (700, 129), (700, 1)])
def test_attention_far_key(be, act, length, back):
    """One key far back stands out: nearly all the weight is its, for a decoded token and for the last rows of a portion."""
    for lens in ([1], [2], [min(length, 40)]):
        if lens[0] > length:
            continue

        def stand_out(q, cache, bt):
            key = length - 1 - back
            q[-1] = 0
            q[-1, :, 3] = 8.0
            cache.k[0][:, :, 3] = np.minimum(cache.k[0][:, :, 3], 0.0)
            cache.k[0][key, :, 3] = 40.0
            # (the device copy is rebuilt from the changed keys)
            pool = down(be, cache.dev, cache.shape, act)
            kk = pool[:, :2 * BS * 32].reshape(-1, 2, BS, 32)
            for p in range(length):
                sl = bt.slot(0, p)
                kk[sl // BS, :, sl % BS] = cache.k[0][p]
            cache.dev = up(be, pool, act)

        run_attention(be, act, Batch(be, [length - lens[0]], lens, seed=length), 4, 2, 32, 24, change=stand_out, bias_len=20)


# ---------------------------------------------------------------- models
def load(be, tmp_path, cfg, seed=1, dtype="float32", **kw):
    from vexel_amd.runtime import ModelRuntime
    t = tensors(cfg, seed, bias_rows=kw.pop("bias_rows", 6))
    folder = str(tmp_path / "model")
    lz.write_model(folder, cfg, t)
    kw = {**dict(pool_blocks=64, max_seqs=6, max_batch=32), **kw}
    return ModelRuntime.load(be, folder, dtype=dtype, **kw), t


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["SMALL", "TINY", "EVEN"])
def test_prompts_portions_and_decoding(be, tmp_path, dtype, name):
    """The whole prompt, token by token, and portions of several sizes: the plain implementation's logits at every position,
    with the blocks and the slot of the previous run used again each time."""
    cfg = {"SMALL": SMALL, "TINY": TINY, "EVEN": EVEN}[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=1, pool_blocks=13, bias_rows=2 if name == "TINY" else 6)
    for n in (1, 2, 3, 16, 17, 203):
        toks = prompt(cfg, n, n)
        want = lz.forward(cfg, t, toks)
        top = limit(dtype, cfg, t, toks, want)
        for sizes in ([n], [1], [2], [2, 3, 1], [16], [7, 64, 1], [65, 1]):
            if sizes[0] > n:
                continue
            err = error(run_portions(mr, 3, toks, sizes), want).max()
            assert err < top, (n, sizes, err)
            mr.delete_sequence(3)
    mr.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_equal_each_alone(be, tmp_path, dtype):
    """Sequences of unequal lengths: prompts' portions beside single tokens, a sequence left out of steps in between, ends and
    new sequences in the freed blocks and slots; every position's logits are the plain implementation's."""
    cfg = SMALL
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=3, pool_blocks=24)
    rng = np.random.default_rng(8)
    todo = [(i, prompt(cfg, n, 100 + i)) for i, n in enumerate((90, 3, 40, 130, 1, 17, 64, 33))]
    want = {i: lz.forward(cfg, t, p) for i, p in todo}
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
            n = int(min(left, rng.choice([1, 1, 2, 3, 16, 17, 40])))
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
    assert len(seen) > 250
    total, free, _ = mr.block_stats()
    assert total == free
    mr.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(be, tmp_path, dtype):
    """300 tokens one by one after a prompt of 5, beside another sequence; then another in its place."""
    cfg = EVEN
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=2, pool_blocks=40)
    for seed in (1, 2):
        a, b = prompt(cfg, 305, seed), prompt(cfg, 305, seed + 10)
        wa, wb = lz.forward(cfg, t, a), lz.forward(cfg, t, b)
        mr.step([(0, a[:5]), (1, b[:5])], [])
        ga, gb = [], []
        for i in range(5, 305):
            lg, _ = mr.step([(1, b[i:i + 1]), (0, a[i:i + 1])], [0, 1])
            ga.append(lg[1]), gb.append(lg[0])
        assert error(np.array(ga), wa[5:]).max() < limit(dtype, cfg, t, a, wa)
        assert error(np.array(gb), wb[5:]).max() < limit(dtype, cfg, t, b, wb)
        mr.delete_sequence(0), mr.delete_sequence(1)
    mr.close()


def greedy(cfg, t, toks, n):
    toks, out = list(toks), []
    for _ in range(n):
        lg = lz.forward(cfg, t, toks)[-1]
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


def test_scheduler_samples_and_stops(be, tmp_path):
    """A sampled request draws what vh_sample draws from the same logits; the stop token ends a greedy one."""
    from vexel_amd.runtime import Scheduler
    cfg = SMALL
    mr, t = load(be, tmp_path, cfg, max_seqs=4, pool_blocks=40)
    p = prompt(cfg, 12, 7)
    stop = greedy(cfg, t, p, 3)[2]
    s = Scheduler(mr, max_batch_size=2, max_tokens=8, eos_token=stop)
    s.add_sequence(0, p)
    s.add_sequence(1, p)
    s.set_sampling(1, 0.9, 20, 0.95, 1234)
    for _ in range(12):
        if s.state(0) == 3 and s.state(1) == 3:
            break
        s.step()
    first = [x for x in s.generated(0)]
    assert first[-1] == stop and first == greedy(cfg, t, p, len(first))
    drawn = s.generated(1)
    state = 1234

    def uniform():
        nonlocal state
        M = (1 << 64) - 1
        state = (state + 0x9E3779B97F4A7C15) & M
        z = state
        z = ((z ^ (z >> 30)) * 0xBF58476D1CE4E5B9) & M
        z = ((z ^ (z >> 27)) * 0x94D049BB133111EB) & M
        return ((z ^ (z >> 31)) >> 40) / 16777216.0

    mr.step([(50, p)], [])
    mr.delete_sequence(50)
    toks = list(p)
    for tok in drawn:
        lg = run_portions(mr, 60, toks, [len(toks)])[-1]
        mr.delete_sequence(60)
        assert s.sample(lg, 0.9, 20, 0.95, uniform()) == tok
        toks.append(tok)
    s.close()
    mr.close()


@pytest.mark.parametrize("name,dtype", [("SMALL", "float32"), ("EVEN", "bfloat16")])
def test_graph_replay_equals_eager_steps(be, tmp_path, name, dtype):
    """Device-driven greedy decoding: captured and replayed several times with the engine's own steps in between, the same
    tokens as eager steps."""
    cfg = {"SMALL": SMALL, "EVEN": EVEN}[name]
    mr, t = load(be, tmp_path, cfg, dtype=dtype, max_seqs=8, pool_blocks=80)
    prompts = {i: prompt(cfg, n, 60 + i) for i, n in enumerate((5, 31, 14))}

    def eager(base):
        out, last = [], None
        lg, am = mr.step([(base + i, p) for i, p in prompts.items()], np.cumsum([len(p) for p in prompts.values()]) - 1)
        first = last = am.copy()
        for _ in range(24):
            _, am = mr.step([(base + i, [int(last[i])]) for i in prompts], [0, 1, 2])
            out.append(am.tolist())
            last = am
        for i in prompts:
            mr.delete_sequence(base + i)
        return first, out

    first, want = eager(0)
    lens = [len(p) for p in prompts.values()]
    mr.step([(10 + i, p) for i, p in prompts.items()], [])
    got, _ = mr.decode_graph(first, [10, 11, 12], lens, 6)
    rows = got.tolist()
    for n in (1, 7, 10):
        assert eager(100)[1] == want                           # other work between the replays
        got, _ = mr.decode_graph(None, None, None, n, batch=3)
        rows += got.tolist()
        assert mr.device_matches_host()
    assert rows == want
    mr.close()


def test_pool_limits_and_unsupported_calls(be, tmp_path):
    from vexel_amd.backend import VexelError
    cfg = SMALL
    mr, t = load(be, tmp_path, cfg, max_seqs=2, pool_blocks=3, max_blocks_per_seq=2)
    toks = prompt(cfg, 33, 1)
    with pytest.raises(VexelError, match="max_blocks_per_seq"):
        mr.step([(0, toks)], [])
    mr.step([(0, toks[:30])], [])
    with pytest.raises(VexelError, match="no free blocks"):
        mr.step([(0, toks[30:31]), (1, toks[:17])], [])
    want = lz.forward(cfg, t, toks[:32])
    lg, _ = mr.step([(0, toks[30:32]), (1, toks[:2])], [0, 1, 3])   # the refused steps changed nothing
    assert error(lg[:2], want[30:32]).max() < LIMIT["float32"] and error(lg[2:], want[1:2]).max() < LIMIT["float32"]
    with pytest.raises(VexelError, match="live sequences"):
        mr.step([(2, toks[:1])], [])
    for bad in ([(0, [cfg["vocab"]])], [(0, [-1])], [(1, []), (0, [1])], [(1, [1]), (1, [2])]):
        with pytest.raises(VexelError):
            mr.step(bad, [])
    with pytest.raises(VexelError, match="wanted"):
        mr.step([(1, [1])], [1])
    with pytest.raises(VexelError, match="recurrent"):
        mr.truncate_sequence(0, 5)
    with pytest.raises(VexelError, match="recurrent"):
        mr.share_blocks(0, 1, 16)
    with pytest.raises(VexelError, match="recurrent"):
        mr.cache_fragment("a", 0)
    with pytest.raises(VexelError, match="recurrent"):
        mr.verify_tree([0], [1], [32], [([], [])])
    mr.truncate_sequence(0, 0)                                 # back to nothing is possible
    lg, _ = mr.step([(0, toks[:4])], [0, 3])
    assert error(lg, want[[0, 3]]).max() < LIMIT["float32"]
    with pytest.raises(VexelError, match="position"):
        mr.decode_with_paged_kv_batched([1], [0], [9])
    lg, _ = mr.decode_with_paged_kv_batched([toks[4]], [0], [4])
    assert error(lg, want[4:5]).max() < LIMIT["float32"]
    assert error(mr.prefill_with_paged_kv(toks[5:9], 0, 5, all_logits=True), want[5:9]).max() < LIMIT["float32"]
    mr.close()


def test_loader_errors(be, tmp_path):
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import ModelRuntime
    cfg = config([(mixer(), 32)])
    t = tensors(cfg, 1)
    folder = str(tmp_path / "m")
    for change, text in ((lambda d: d.pop("l0.mix.left.g"), "l0.mix.left.g is missing"),
                         (lambda d: d.update({"head": d["head"][:-1]}), "head: shape"),
                         (lambda d: d.update({"l0.mix.left.rel": d["l0.mix.left.rel"][:1]}), "bias table")):
        d = dict(t)
        change(d)
        lz.write_model(folder, cfg, d)
        with pytest.raises(VexelError, match=text):
            ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1)
    lz.write_model(folder, cfg, t)
    path = os.path.join(folder, "model.safetensors")
    raw = open(path, "rb").read()
    for cut in (4, 100, len(raw) - 10):
        open(path, "wb").write(raw[:cut])
        with pytest.raises(VexelError):
            ModelRuntime.load(be, folder, pool_blocks=4, max_seqs=1, max_batch=1)
    with pytest.raises(VexelError):
        ModelRuntime.load(be, str(tmp_path / "nothing"))


def test_generation_from_the_command_line(be, tmp_path, capsys):
    from vexel_amd.__main__ import main
    cfg = SMALL
    t = tensors(cfg, 2)
    lz.write_model(str(tmp_path / "m"), cfg, t)
    prompts = [prompt(cfg, 9, 1), prompt(cfg, 30, 2)]
    args = ["generate", "--model", str(tmp_path / "m"), "--dtype", "float32", "--max-new", "5", "--prefill-chunk", "8"]
    for p in prompts:
        args += ["--tokens", ",".join(map(str, p))]
    assert main(args) == 0
    got = [[int(x) for x in line.split()] for line in capsys.readouterr().out.splitlines()]
    assert got == [greedy(cfg, t, p, 5) for p in prompts]


def test_trace_replay(be, tmp_path):
    """bin/trace_run in a process of its own: steps in, logits out, blocks and slots given back at the end of requests."""
    cfg = SMALL
    t = tensors(cfg, 6)
    lz.write_model(str(tmp_path / "m"), cfg, t)
    a, b, c = (prompt(cfg, n, 80 + n) for n in (50, 30, 47))
    steps = [{"entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:1], "want": []}], "end": []},
             {"entries": [{"id": "b", "tokens": b[1:3], "want": []}], "end": []},
             {"entries": [{"id": "b", "tokens": b[3:], "want": [26]}, {"id": "a", "tokens": a[20:], "want": [29, 3]}], "end": ["a"]},
             {"entries": [{"id": "c", "tokens": c, "want": [46]}], "end": ["b", "c"]}]
    want = {n: lz.forward(cfg, t, toks) for n, toks in (("a", a), ("b", b), ("c", c))}
    text = "".join(json.dumps({"step": i, **s}) + "\n" for i, s in enumerate(steps))
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert r.stdout.split() == "done 0 done 1 done 2 done 3".split()
    read = lambda i: np.fromfile(str(out / ("%d.f32" % i)), dtype="<f4").reshape(-1, cfg["vocab"])
    assert not (out / "1.f32").exists()
    assert error(read(0), want["a"][[0, 19]]).max() < LIMIT["float32"]
    assert error(read(2), np.stack([want["b"][29], want["a"][49], want["a"][23]])).max() < LIMIT["float32"]
    assert error(read(3), want["c"][46:]).max() < LIMIT["float32"]


def test_steps_of_the_llama_family(be):
    """vh_step on a LLaMA-family model: the logits of vh_prefill and vh_decode_batched on another copy of the sequences."""
    from oracle import model as om, numerics as nx
    from helpers import gpu_model_from_oracle
    cfg = om.ModelConfig(num_layers=2, hidden=256, num_heads=4, num_kv_heads=2, head_dim=64, ffn=512, vocab=300)
    mr = gpu_model_from_oracle(be, om.random_model(cfg, 0, nx.FMT_Q4_0, nx.FMT_Q8_0, max_blocks=32), pool_blocks=32, max_seqs=8,
                               max_blocks_per_seq=8, max_batch=4)
    assert not mr.mixed_batches
    rng = np.random.default_rng(1)
    a, b = rng.integers(0, 300, 20).tolist(), rng.integers(0, 300, 9).tolist()
    mr.step([(0, a[:12]), (1, b[:5])], [])
    lg, am = mr.step([(0, a[12:13]), (1, b[5:8])], [0, 3, 1])
    want_a = mr.prefill_with_paged_kv(a[:12], 10, 0)
    want_a, arg_a = mr.decode_with_paged_kv_batched([a[12]], [10], [12])
    mr.prefill_with_paged_kv(b[:5], 11, 0)
    want_b = mr.prefill_with_paged_kv(b[5:8], 11, 5, all_logits=True)
    assert np.allclose(lg[0], want_a[0], atol=1e-5) and am[0] == arg_a[0]
    assert np.allclose(lg[1], want_b[2], atol=1e-5) and np.allclose(lg[2], want_b[0], atol=1e-5)
    mr.close()
