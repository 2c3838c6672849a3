"""What the tests of mixed-batch kernels and models share: device arrays of either activation type, batches over a small paged
pool, packed matrices, portions."""
import numpy as np

from oracle.lozedra import bf16_round

F32, BF16 = 0, 1
ACTS = [F32, BF16]
BS = 16


def act_array(a, act):
    """numpy array -> what the device holds (float32, or bfloat16 as uint16)"""
    a = np.ascontiguousarray(a, dtype=np.float32)
    return a if act == F32 else (bf16_round(a).view(np.uint32) >> 16).astype(np.uint16)


def grid(a, act):
    """the values a device array of that type holds"""
    return np.asarray(a, dtype=np.float32) if act == F32 else bf16_round(a)


def up(be, a, act=F32):
    return be.upload(act_array(a, act))


def down(be, p, shape, act):
    if act == F32:
        return be.download(p, shape, np.float32)
    return (be.download(p, shape, np.uint16).astype(np.uint32) << 16).view(np.float32)


def blank(be, shape, act, fill=np.nan):
    return be.upload(act_array(np.full(shape, fill), act))


def close(got, want, act, what=""):
    want = np.asarray(want, dtype=np.float64)
    tol = 2e-5 if act == F32 else 1.2e-2
    err = np.abs(got - want).max() / (np.abs(want).max() + 1e-30)
    assert np.all(np.isfinite(got)) and err < tol, (what, err)


class Batch:
    """A mixed batch over a small paged pool: lens[i] new rows of a sequence that holds start[i] tokens already."""

    def __init__(self, be, start, lens, seed=0, max_blocks=None, slots=None):
        rng = np.random.default_rng(seed)
        n = len(lens)
        self.start, self.lens = list(start), list(lens)
        self.kv = [s + l for s, l in zip(start, lens)]
        need = [(k + BS - 1) // BS for k in self.kv]
        self.max_blocks = max_blocks or max(need) + 1
        self.pool_blocks = sum(need) + 3
        perm = rng.permutation(self.pool_blocks)
        self.slots = list(slots) if slots is not None else rng.permutation(n + 2)[:n].tolist()
        self.table = np.full((max(self.slots) + 1, self.max_blocks), -1, dtype=np.int32)
        at = 0
        for s, m in zip(self.slots, need):
            self.table[s, :m] = perm[at:at + m]
            at += m
        self.cu = np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)
        self.pos = np.concatenate([np.arange(s, s + l) for s, l in zip(start, lens)]).astype(np.int32)
        self.rows = int(self.cu[-1])
        self.seq = np.repeat(np.arange(n), lens)
        self.slot_map = np.array([self.slot(i, p) for i, p in zip(self.seq, self.pos)], dtype=np.int32)
        from vexel_amd.backend import VxRagged
        self.q_host = np.array(lens, dtype=np.int32)
        b = VxRagged()
        b.rows, b.n_seqs = self.rows, n
        b.q_lens = None if all(l == 1 for l in lens) else self.q_host.ctypes.data
        b.max_kv_len, b.max_blocks, b.block_size = max(self.kv), self.max_blocks, BS
        b.cu_seqlens, b.token_pos, b.slot_mapping = be.upload(self.cu), be.upload(self.pos), be.upload(self.slot_map)
        b.table_rows = be.upload(np.array(self.slots, dtype=np.int32))
        b.kv_lens, b.block_tables = be.upload(np.array(self.kv, dtype=np.int32)), be.upload(self.table)
        self.c = b

    def slot(self, i, p):
        return int(self.table[self.slots[i], p // BS]) * BS + p % BS


def packed(be, w, n_pad=None, k_pad=None, tile0=0, step=1, col0=0, dst=None):
    n, k = w.shape
    n_pad, k_pad = n_pad or -(-n // 16) * 16, k_pad or -(-k // 64) * 64
    if dst is None:
        dst = be.alloc(n_pad * k_pad * 2)
        be.fill_zero(dst, n_pad * k_pad * 2)
    be.linear_pack(up(be, w, BF16), n, k, dst, n_pad, k_pad, tile0, step, col0)
    return dst, n_pad, k_pad


def lin_out(**kw):
    from vexel_amd.backend import VxLinearOut
    o = VxLinearOut()
    for name, v in kw.items():
        setattr(o, name, v)
    return o


def prompt(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def run_portions(mr, sid, toks, sizes):
    """All logits of a sequence fed in portions of the given sizes, again and again."""
    at, got, i = 0, [], 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        got.append(mr.step([(sid, toks[at:at + n])], list(range(n)))[0])
        at += n
        i += 1
    return np.concatenate(got)
