"""Kitodra without a GPU: the plain implementation's mechanisms on cases worked out by hand, mistakes planted in it, and the
product's reading of configurations."""
import json
import math

import numpy as np
import pytest

from kitodra_models import EVEN, LIMIT, SMALL, TINY, WIDE, config, differential, error, key_value, lightning, margin, moe, tensors
from oracle import kitodra as kt


def test_pairs_by_hand():
    cfg = {"buckets": 10, "mul_prev": 3, "mul_cur": 4}
    assert kt.bigram_rows([5, 2, 0, 9], cfg).tolist() == [10, (15 + 8) % 10, 6, 36 % 10]
    T = {"embed": np.eye(3), "bigram": 100.0 * np.arange(3)[:, None] * np.ones((1, 3))}
    x = kt.embedding([1, 1], T, {"embedding": {"bigram": {"buckets": 2, "mul_prev": 1, "mul_cur": 0}}})
    assert np.allclose(x, [[200, 201, 200], [100, 101, 100]])
    assert np.allclose(kt.embedding([1, 1], T, {}), np.eye(3)[[1, 1]])


def test_rotation_by_hand():
    """Dimensions 0 and 2 turn by p, 1 and 3 by p / 2 (4^(-2 / 4)), 4 stays."""
    x = np.array([[[1.0, 0.0, 0.0, 2.0, 7.0]]] * 2)
    y = kt.rotate_halves(x, [0, 1], 4, 4.0)
    assert np.allclose(y[0], x[0])
    assert np.allclose(y[1, 0], [math.cos(1), -2 * math.sin(0.5), math.sin(1), 2 * math.cos(0.5), 7.0])


def test_masks_by_hand():
    i, j = np.arange(7)[:, None], np.arange(7)[None, :]
    assert [np.flatnonzero(r).tolist() for r in kt.in_window(i, j, 3)] == [[0], [0, 1], [0, 1, 2], [1, 2, 3], [2, 3, 4], [3, 4, 5], [4, 5, 6]]
    assert [np.flatnonzero(r).tolist() for r in kt.in_chunk(i, j, 3)] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]


def test_softmax_and_cap_by_hand():
    s = np.log(np.array([2.0, 2.0]))
    assert np.allclose(kt.softmax(s), 0.5) and np.allclose(kt.softmax(s, 0.0), 2 / 5) and np.allclose(kt.softmax(s - 800, 0.0), 0)
    assert np.allclose(kt.softcap(np.array([1e9, -1e9, 0.0, 1e-3]), 5.0), [5, -5, 0, 1e-3]) and kt.softcap(7.0, None) == 7.0


def test_difference_by_hand():
    t = {"lq1": np.array([1.0, 2.0]), "lk1": np.array([0.5, -0.25]), "lq2": np.array([1.0, 0.0]), "lk2": np.array([math.log(3), 5.0])}
    assert math.isclose(kt.difference_weight(t, 0.25), 1.0 - 3.0 + 0.25)
    assert np.allclose(kt.difference(np.array([[5.0, 1.0]]), np.array([[1.0, -1.5]]), 2.0, 0.75, 0.0), np.array([[3.0, 4.0]]) / math.sqrt(12.5) / 4)


def test_decaying_state_by_hand():
    """dim 1, vdim 1: o_t = q_t (v_t k_t + d k_(t-1) v_(t-1) + ..)"""
    q, k, v = (np.array(x, dtype=float)[:, None, None] for x in ([1, 10, 2], [2, 3, 1], [1, 1, 4]))
    o, S = kt.decayed_states(q, k, v, [0.5])
    assert np.allclose(o[:, 0, 0], [2, 10 * (1 + 3), 2 * (2 + 4)]) and np.allclose(S, 6)
    o2, _ = kt.decayed_states(q[1:], k[1:], v[1:], [0.5], np.full((1, 1, 1), 2.0))
    assert np.allclose(o2, o[1:])
    o, S = kt.decayed_states(q, k, v, [0.0])
    assert np.allclose(o[:, 0, 0], [2, 30, 8])
    assert np.allclose(kt.gated_norm(np.array([[3.0, 4.0]]), np.array([1.0, 2.0]), np.array([0.0, 100.0]), 0.0), [[1.5 / math.sqrt(12.5), 8 / math.sqrt(12.5)]])


def test_expert_by_hand():
    """gate cut above alone, up on both sides"""
    t = {"gate": np.array([[1.0]]), "up": np.array([[1.0]]), "down": np.array([[2.0]])}
    f = lambda g, u: 2 * g / (1 + math.exp(-1.702 * g)) * (u + 1)
    assert np.allclose(kt.expert(np.array([[0.25], [3.0], [-3.0]]), t, 0.5)[:, 0], [f(0.25, 0.25), f(0.5, 0.5), f(-3.0, -0.5)])


def test_choice_by_hand():
    logit = lambda s: np.log(np.array(s) / (1 - np.array(s)))
    z = logit([[0.9, 0.1, 0.6, 0.5, 0.4, 0.3]])
    w = kt.choose(z, np.zeros(6), {"top": 2})
    assert np.allclose(w, [[0.9, 0, 0.6, 0, 0, 0]])
    # groups 1.0, 1.1, 0.7: the first one's 0.9 cannot be chosen
    w = kt.choose(z, np.zeros(6), {"top": 2, "groups": {"count": 3, "keep": 1}})
    assert np.allclose(w, [[0, 0, 0.6, 0.5, 0, 0]])
    # the correction moves the choice, not the weight; choice scores below 0 still come before those of other groups
    w = kt.choose(z, np.array([0, 0, -2.0, -2.0, -3.0, -3.0]), {"top": 3, "groups": {"count": 3, "keep": 2}})
    assert np.allclose(w, [[0.9, 0.1, 0.6, 0, 0, 0]])
    w = kt.choose(z, np.array([-5.0, -5.0, 0, 0, -2.0, 0]), {"top": 3, "groups": {"count": 3, "keep": 2}})
    assert np.allclose(w, [[0, 0, 0.6, 0.5, 0, 0.3]])
    # three to a group: the two largest count
    w = kt.choose(logit([[0.8, 0.1, 0.1, 0.5, 0.5, 0.5]]), np.zeros(6), {"top": 1, "groups": {"count": 2, "keep": 1}})
    assert w[0, 3:].sum() == 0.5 and w[0, :3].sum() == 0
    assert np.allclose(margin(np.array([[0.9, 0.5, 0.2, 0.1]]), {"top": 1, "groups": {"count": 2, "keep": 1}}), 0.4)


def test_prefix_does_not_depend_on_what_follows():
    t = tensors(SMALL, 3)
    toks = np.random.default_rng(0).integers(0, SMALL["vocab"], 60).tolist()
    whole = kt.forward(SMALL, t, toks)
    assert np.allclose(whole[:17], kt.forward(SMALL, t, toks[:17]), atol=1e-9)


@pytest.mark.parametrize("cfg", [SMALL, EVEN, WIDE])
def test_the_choices_of_the_random_models_are_clear(monkeypatch, cfg):
    """(so that rounding does not change an expert)"""
    least, right = [], kt.choose

    def seen(z, correction, router):
        least.append(margin(kt.sigmoid(z) + correction, router).min())
        return right(z, correction, router)

    monkeypatch.setattr(kt, "choose", seen)
    for seed in (1, 4):
        kt.forward(cfg, tensors(cfg, seed), np.random.default_rng(seed).integers(0, cfg["vocab"], 150).tolist())
    assert min(least) > 2e-3


def test_the_weights_show_every_mechanism(monkeypatch):
    """The random models of the tests are such that leaving out or changing any one mechanism moves the logits far beyond the
    tolerance of the comparisons (the mistakes are planted in the plain implementation, or in the configuration it gets)."""
    t = tensors(SMALL, 5)
    toks = np.random.default_rng(1).integers(0, SMALL["vocab"], 130).tolist()
    good = kt.forward(SMALL, t, toks)

    def planted(**mistakes):
        with monkeypatch.context() as m:
            for name, value in mistakes.items():
                if name in ("differential_attention", "key_value_attention", "lightning"):
                    m.setitem(kt.MIXERS, {"differential_attention": "attention", "key_value_attention": "attention_2"}.get(name, name), value)
                m.setattr(kt, name, value)
            return kt.forward(SMALL, t, toks)

    def weights(change):
        d = dict(t)
        change(d)
        return kt.forward(SMALL, d, toks)

    def changed(change):
        c = json.loads(json.dumps(SMALL))
        change(c)
        return kt.forward(c, t, toks)

    mixer = lambda c, i: c["layers"][i]["mixer"]
    soft, rot, win, chunk, diff, states, gnorm, ex, pick, mix, rows, kva, dat = (
        kt.softmax, kt.rotate_halves, kt.in_window, kt.in_chunk, kt.difference, kt.decayed_states, kt.gated_norm, kt.expert, kt.choose, kt.mixture,
        kt.bigram_rows, kt.key_value_attention, kt.differential_attention)

    def first_row_zero(tokens, cfg):
        r = rows(tokens, cfg)
        r[0] = 0
        return r

    def expert_as(f):
        return lambda h, t, limit: kt.linear(t["down"], f(kt.linear(t["gate"], h), kt.linear(t["up"], h), limit))

    def normed_before_rotation(h, t, cfg, eps):
        t = dict(t, k=t["k"] * 2.0)                             # (values of twice the size)
        t["k.b"] = t["k.b"] * 2.0
        return kva(h, t, cfg, eps)

    def sequential(x, t, cfg, eps):
        h = kt.rms(x, eps) * t["norm1"]
        x = x + kt.MIXERS[cfg["type"]](h, kt.sub(t, "mix."), cfg["mixer"], eps)
        return x + kt.mixture(kt.rms(x, eps) * t["norm1"], kt.sub(t, "mlp."), cfg["mlp"]) if cfg.get("mlp") else x

    sg = kt.sigmoid
    wrong = {
        "no pairs": changed(lambda c: c.pop("embedding")),
        "pairs the other way round": changed(lambda c: c["embedding"]["bigram"].update(mul_prev=17, mul_cur=31)),
        "the first token's pair row": planted(bigram_rows=first_row_zero),
        "no sink": planted(softmax=lambda s, sink=None: soft(s)),
        "a sink for all": planted(softmax=lambda s, sink=None: soft(s, 0.0)),
        "window one longer": planted(in_window=lambda i, j, n: win(i, j, n + 1)),
        "window one shorter": planted(in_window=lambda i, j, n: win(i, j, max(n - 1, 1))),
        "chunk one longer": planted(in_chunk=lambda i, j, n: chunk(i, j, n + 1)),
        "chunks counted from 1": planted(in_chunk=lambda i, j, n: (i >= j) & ((i + 1) // n == (j + 1) // n)),
        "neighbours turned": planted(rotate_halves=lambda x, p, d, b: rot(x[..., np.argsort(np.r_[0:d:2, 1:d:2, d:x.shape[-1]])], p, d, b)),
        "turned the other way": planted(rotate_halves=lambda x, p, d, b: rot(x, -np.asarray(p) + 0.3, d, b)),
        "frequencies of the whole head": planted(rotate_halves=lambda x, p, d, b: rot(x, p, x.shape[-1], b)),
        "values of another size": planted(key_value_attention=normed_before_rotation),
        "no cap": changed(lambda c: mixer(c, 1).pop("softcap")),
        "second map left out": planted(difference=lambda a, b, lam, d, e: diff(a, b, 0.0, d, e)),
        "without 1 - diff": planted(difference=lambda a, b, lam, d, e: diff(a, b, lam, 0.0, e)),
        "difference not normed": planted(difference=lambda a, b, lam, d, e: (a - lam * b) * (1 - d)),
        "query norm's weight": weights(lambda d: d.update({"l1.mix.q.norm": np.ones_like(d["l1.mix.q.norm"])})),
        "key bias": weights(lambda d: d.update({"l2.mix.k.b": 0 * d["l2.mix.k.b"]})),
        "output bias": weights(lambda d: d.update({"l1.mix.o.b": 0 * d["l1.mix.o.b"]})),
        "state lost at 64": planted(decayed_states=lambda q, k, v, d, s=None: (np.concatenate([states(q[:64], k[:64], v[:64], d)[0],
                                                                                             states(q[64:], k[64:], v[64:], d)[0]]), None)),
        "decay before the write alone": planted(decayed_states=lambda q, k, v, d, s=None: states(q, k * np.asarray(d)[:, None], v, d)),
        "heads normed apart": planted(gated_norm=lambda o, w, g, e: kt.rms(o.reshape(len(o), 3 if w.size % 3 == 0 else 2, -1), e).reshape(o.shape) * w * sg(g)),
        "gate with SiLU": planted(gated_norm=lambda o, w, g, e: kt.rms(o, e) * w * kt.silu(g)),
        "expert without the limit": planted(expert=lambda h, t, n: ex(h, t, 1e9)),
        "gate cut on both sides": planted(expert=expert_as(lambda g, u, n: np.clip(g, -n, n) * sg(1.702 * np.clip(g, -n, n)) * (np.clip(u, -n, n) + 1))),
        "plain SiLU": planted(expert=expert_as(lambda g, u, n: np.minimum(g, n) * sg(np.minimum(g, n)) * (np.clip(u, -n, n) + 1))),
        "up without its 1": planted(expert=expert_as(lambda g, u, n: np.minimum(g, n) * sg(1.702 * np.minimum(g, n)) * np.clip(u, -n, n))),
        "weights renormalized": planted(choose=lambda z, c, r: pick(z, c, r) / pick(z, c, r).sum(-1, keepdims=True)),
        "weights with the correction": planted(choose=lambda z, c, r: np.where(pick(z, c, r) > 0, kt.sigmoid(z) + c, 0)),
        "no correction": planted(choose=lambda z, c, r: pick(z, 0 * c, r)),
        "no groups": planted(choose=lambda z, c, r: pick(z, c, {"top": r["top"]})),
        "one expert fewer": planted(choose=lambda z, c, r: pick(z, c, dict(r, top=r["top"] - 1))),
        "no shared expert": planted(mixture=lambda h, t, c: mix(h, t, dict(c, shared=None))),
        "one sublayer after the other": planted(layer=sequential),
        "another layer's weights": changed(lambda c: c["layers"][5].update(c["layers"][2], weights_of=2)),
    }
    for what, lg in wrong.items():
        assert error(lg, good).max() > 5 * LIMIT["float32"], what


def test_architecture_registry_and_configurations():
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import architectures, check_config
    assert {"Kitodra", "Tulipel", "Lozedra"} <= set(architectures())
    for c in (SMALL, TINY, EVEN, WIDE):
        check_config(json.dumps(c))
    ok = config([(lightning(), moe()), (differential(), moe()), (key_value(), moe()), 0, (differential(), None)])
    mixer, mlp = lambda c, i: c["layers"][i]["mixer"], lambda c, i: c["layers"][i]["mlp"]
    for change in (lambda c: c["layers"][4].pop("mlp"), lambda c: c.pop("embedding"), lambda c: c["embedding"].update(bigram=None),
                   lambda c: mlp(c, 0)["router"].pop("groups"), lambda c: mlp(c, 1).pop("shared"), lambda c: mixer(c, 1).update(softcap=None),
                   lambda c: mixer(c, 2).pop("rot"), lambda c: mixer(c, 0).update(decay=[0, 1, 0.5]), lambda c: c["layers"][4].update(weights_of=None)):
        c = json.loads(json.dumps(ok))
        change(c)
        check_config(json.dumps(c))
    bad = [(lambda c: c.update(layers=[]), "no layers"), (lambda c: c["layers"][0].update(type="attention_3"), "attention_3"),
           (lambda c: mlp(c, 0).update(kind="dense"), "dense"), (lambda c: mixer(c, 0).update(decay=[0.5]), "1 numbers for 3 heads"),
           (lambda c: mixer(c, 0).update(decay=[0.5, 1.5, 0.1]), "between 0 and 1"), (lambda c: mixer(c, 0).pop("decay"), "decay"),
           (lambda c: mixer(c, 1).update(kv_heads=3), "no multiple"), (lambda c: mixer(c, 1).pop("diff"), "diff"), (lambda c: mixer(c, 1).pop("scale"), "scale"),
           (lambda c: mixer(c, 1).update(softcap=-1.0), "softcap"), (lambda c: mixer(c, 1)["mask"].update(size=0), "size"),
           (lambda c: mixer(c, 2).update(vdim=9), "values of 9"), (lambda c: mixer(c, 2)["rot"].update(dims=7), "dimensions"),
           (lambda c: mixer(c, 2)["rot"].update(dims=24), "dimensions"), (lambda c: mixer(c, 2)["rot"].pop("base"), "base"),
           (lambda c: mlp(c, 0)["router"]["groups"].update(count=5), "groups"), (lambda c: mlp(c, 0)["router"]["groups"].update(keep=4), "groups"),
           (lambda c: mlp(c, 0)["router"].update(top=9), "9 of 12 experts"), (lambda c: mlp(c, 0)["expert"].update(limit=0.0), "limit"),
           (lambda c: mlp(c, 0)["expert"].pop("ff"), "ff"), (lambda c: c["layers"][3].update(weights_of=1), "another kind"),
           (lambda c: c["layers"][3].update(weights_of=3), "circle"), (lambda c: c["layers"][3].update(weights_of=5), "weights_of"),
           (lambda c: c["embedding"]["bigram"].update(buckets=0), "buckets"), (lambda c: c["norm"].pop("eps"), "eps"), (lambda c: c.update(vocab=1.5), "whole number")]
    for change, text in bad:
        c = json.loads(json.dumps(ok))
        change(c)
        with pytest.raises(VexelError, match=text):
            check_config(json.dumps(c))


def test_tiles_of_the_experts():
    """No way to deal rows to experts makes more tiles than there is room for."""
    from vexel_amd import lib
    l = lib.load()
    rng = np.random.default_rng(0)
    for _ in range(300):
        rows, experts = int(rng.integers(1, 400)), int(rng.integers(1, 40))
        top, tile, shared = int(rng.integers(1, experts + 1)), int(rng.choice([1, 5, 64, 128])), int(rng.integers(0, 2))
        chosen = np.stack([rng.permutation(experts)[:top] for _ in range(rows)]) if rng.random() < 0.5 else np.tile(np.arange(top), (rows, 1))
        n = np.bincount(chosen.ravel(), minlength=experts)
        assert (-(-n // tile)).sum() + shared * -(-rows // tile) <= l.vx_route_max_tiles(rows, experts, top, shared, tile)
    assert l.vx_route_tile_rows(1, 64, 64, 6) == 64 and l.vx_route_tile_rows(0, 5000, 8, 2) == 64 and l.vx_route_tile_rows(1, 5000, 8, 2) == 128
