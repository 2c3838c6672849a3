"""Fitevik without a GPU: the plain implementation's mechanisms on cases worked out by hand, mistakes planted in it, and the
product's reading of configurations."""
import json
import math

import numpy as np
import pytest

from fitevik_models import EVEN, LIMIT, SMALL, TINY, WIDE, attention, config, dense, error, margin, moe, states, tensors
from oracle import fitevik as fv


def test_layer_norm_by_hand():
    y = fv.layer_norm(np.array([[1.0, 3.0, 5.0, 7.0]]), np.array([1.0, 2.0, 1.0, 1.0]), np.array([0.0, 0.0, 10.0, 0.0]), 0.0)
    assert np.allclose(y, [[-3 / math.sqrt(5), -2 / math.sqrt(5), 10 + 1 / math.sqrt(5), 3 / math.sqrt(5)]])
    assert np.allclose(fv.layer_norm(np.array([[1.0, -1.0]]), 1.0, 0.0, 3.0), [[0.5, -0.5]])


def test_embedding_by_hand():
    T = {"embed": np.array([[0.0, 0.0], [2.0, 0.0]]), "pos": np.array([[0.0, 0.0], [0.0, 6.0], [9.0, 9.0]]), "embed.norm": np.ones(2), "embed.norm.b": np.zeros(2)}
    assert np.allclose(fv.embedding([1, 1], T, 0.0), [[1, -1], [-1, 1]])   # (2, 0) and (2, 6)


def test_window_and_slopes_by_hand():
    i, j = np.arange(5)[:, None], np.arange(5)[None, :]
    assert [np.flatnonzero(r).tolist() for r in fv.in_window(i, j, 3)] == [[0], [0, 1], [0, 1, 2], [1, 2, 3], [2, 3, 4]]
    assert np.allclose(fv.slopes(8), [2.0 ** -n for n in range(1, 9)]) and np.allclose(fv.slopes(2), [1 / 16, 1 / 256])


def test_mixing_and_sink_by_hand():
    s = np.array([[[1.0, 2.0]], [[10.0, 20.0]]])                # [heads, queries, keys]
    assert np.allclose(fv.mix_heads(np.array([[1.0, 0.5], [0.0, -1.0]]), s), [[[6, 12]], [[-10, -20]]])
    s = np.log(np.array([2.0, 2.0]))
    assert np.allclose(fv.softmax(s, 0.0), 2 / 5) and np.allclose(fv.softmax(s, math.log(4)), 1 / 4) and np.allclose(fv.softmax(s - 800, 0.0), 0)


def test_attention_by_hand():
    """Two heads over one key head, width 1, scores that the norms make 1: out of the biases, the mixing and the sinks alone."""
    t = {"q": np.array([[1.0], [1.0]]), "k": np.array([[1.0]]), "v": np.array([[1.0]]), "q.norm": np.ones(2), "k.norm": np.ones(1),
         "talk": np.array([[1.0, 1.0], [0.0, 2.0]]), "sink": np.array([0.0, 1.0]), "o": np.eye(2)}
    cfg = {"heads": 2, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 0.5, "mask": {"size": 2}}
    h = np.array([[5.0], [1.0], [3.0]])
    got = fv.attention(h, t, cfg, 0.0, fv.keys_values(h, t, cfg, 0.0))
    near, far = 0.5, 0.5 - np.array([1 / 16, 1 / 256])          # this token's score and the one before's, ahead of the mixing
    for head, (a, b, s) in enumerate(((2 * near, far.sum(), 0.0), (2 * near, 2 * far[1], 1.0))):
        e = np.exp([a, b, s])
        assert math.isclose(got[0, head], 5 * e[0] / (e[0] + e[2]))
        assert math.isclose(got[2, head], (3 * e[0] + 1 * e[1]) / e.sum())


def test_forgetting_state_by_hand():
    """dim 1, vdim 1: S = f S + (1 - f) v"""
    q, f, v = (np.array(x, dtype=float)[:, None, None] for x in ([1, 10, 2], [0.5, 0.25, 1.0], [4, 8, 100]))
    o, S = fv.gated_states(q, f, v)
    assert np.allclose(o[:, 0, 0], [2, 10 * 6.5, 2 * 6.5]) and np.allclose(S, 6.5)
    o2, _ = fv.gated_states(q[1:], f[1:], v[1:], np.full((1, 1, 1), 2.0))
    assert np.allclose(o2, o[1:])
    # channels keep apart: the gate acts on the state's rows
    o, S = fv.gated_states(np.ones((2, 1, 2)), np.array([[[0.0, 0.0]], [[1.0, 0.0]]]), np.array([[[1.0, 2.0, 3.0]], [[10.0, 20.0, 30.0]]]))
    assert np.allclose(S[0], [[1, 2, 3], [10, 20, 30]]) and np.allclose(o[:, 0], [[2, 4, 6], [11, 22, 33]])
    assert np.allclose(fv.forget(np.array([0.0, -700.0, 700.0, 1.0]), np.array([0.0, 0, 0, -1.0]), np.array([0.0, 0.25, 0.25, 0.5])), [0.5, 0.25, 1.0, 0.75])


def test_feed_forward_by_hand():
    t = {"up": np.array([[1.0], [-1.0]]), "up.b": np.array([1.0, 0.0]), "down": np.array([[1.0, 10.0]]), "down.b": np.array([0.5])}
    assert np.allclose(fv.dense(np.array([[2.0], [-3.0]]), t), [[9.5], [90.5]])


def test_choice_by_hand():
    w = fv.choose(np.log(np.array([[2.0, 1.0, 6.0, 0.5]])), 2)
    assert np.allclose(w, [[0.25, 0, 0.75, 0]])
    assert np.allclose(fv.choose(np.array([[800.0, -800.0, 799.0]]), 1), [[1, 0, 0]])
    assert np.allclose(margin(np.array([[0.9, 0.5, 0.2, 0.1]]), 2), 0.3)


def test_prefix_does_not_depend_on_what_follows():
    t = tensors(SMALL, 3)
    toks = np.random.default_rng(0).integers(0, SMALL["vocab"], 60).tolist()
    whole = fv.forward(SMALL, t, toks)
    assert np.allclose(whole[:17], fv.forward(SMALL, t, toks[:17]), atol=1e-9)


@pytest.mark.parametrize("cfg", [SMALL, EVEN, WIDE])
def test_the_choices_of_the_random_models_are_clear(monkeypatch, cfg):
    """(so that rounding does not change an expert)"""
    least, right = [], fv.choose

    def seen(z, top):
        least.append(margin(z, top).min())
        return right(z, top)

    monkeypatch.setattr(fv, "choose", seen)
    for seed in (1, 4):
        fv.forward(cfg, tensors(cfg, seed), np.random.default_rng(seed).integers(0, cfg["vocab"], 150).tolist())
    assert min(least) > 1e-2


def test_the_weights_show_every_mechanism(monkeypatch):
    """The random models of the tests are such that leaving out or changing any one mechanism moves the logits far beyond the
    tolerance of the comparisons (the mistakes are planted in the plain implementation, or in the configuration it gets)."""
    t = tensors(SMALL, 5)
    toks = np.random.default_rng(1).integers(0, SMALL["vocab"], 130).tolist()
    good = fv.forward(SMALL, t, toks)

    def planted(**mistakes):
        with monkeypatch.context() as m:
            for name, value in mistakes.items():
                m.setattr(fv, name, value)
            return fv.forward(SMALL, t, toks)

    def weights(change):
        d = dict(t)
        change(d)
        return fv.forward(SMALL, d, toks)

    def changed(change):
        c = json.loads(json.dumps(SMALL))
        change(c)
        return fv.forward(c, t, toks)

    mixer = lambda c, i: c["layers"][i]["mixer"]
    soft, win, mix, sl, st, fg, r2, pick, kv, emb, rms, att = (fv.softmax, fv.in_window, fv.mix_heads, fv.slopes, fv.gated_states, fv.forget, fv.relu2, fv.choose,
                                                               fv.keys_values, fv.embedding, fv.rms, fv.attention)

    def heads_normed_apart(h, t, cfg, eps):
        k = rms(fv.linear(t["k"], h).reshape(len(h), cfg["kv_heads"], -1), eps).reshape(len(h), -1) * t["k.norm"]
        return k.reshape(len(h), cfg["kv_heads"], -1), kv(h, t, cfg, eps)[1]

    def bias_behind_the_mixing(h, t, cfg, eps, keys):
        with monkeypatch.context() as m:
            H = cfg["heads"]
            m.setattr(fv, "slopes", lambda n: np.linalg.solve(t["talk"], sl(H)))
            return att(h, t, cfg, eps, keys)

    def sink_mixed(h, t, cfg, eps, keys):
        return att(h, dict(t, sink=t["talk"] @ t["sink"]), cfg, eps, keys)

    def other_way_round(s_):
        return lambda q, f, v, s=None: st(q, 1.0 - f, v, s)

    wrong = {
        "no positions": planted(embedding=lambda k, T, e: emb(k, dict(T, pos=0 * T["pos"]), e)),
        "positions from 1": planted(embedding=lambda k, T, e: emb(k, dict(T, pos=T["pos"][1:]), e)),
        "embedding not normed": planted(embedding=lambda k, T, e: T["embed"][np.asarray(k)] + T["pos"][:len(k)]),
        "norms without their mean": planted(layer_norm=lambda x, w, b, e: rms(x, e) * w + b),
        "norms without their bias": planted(layer_norm=lambda x, w, b, e: (x - x.mean(-1, keepdims=True)) / np.sqrt(x.var(-1, keepdims=True) + e) * w),
        "window one longer": planted(in_window=lambda i, j, n: win(i, j, n + 1)),
        "window one shorter": planted(in_window=lambda i, j, n: win(i, j, max(n - 1, 1))),
        "the other layer's window": changed(lambda c: mixer(c, 2).update(mask={"size": 37})),
        "no sink": planted(softmax=lambda s, k: soft(s, -1e30)),
        "sink scaled": planted(softmax=lambda s, k: soft(s, 0.5 * k)),
        "sink mixed": planted(attention=sink_mixed),
        "no mixing": planted(mix_heads=lambda T, s: s),
        "mixing transposed": planted(mix_heads=lambda T, s: mix(T.T, s)),
        "bias behind the mixing": planted(attention=bias_behind_the_mixing),
        "no bias": planted(slopes=lambda n: np.zeros(n)),
        "slopes from head 0": planted(slopes=lambda n: 2.0 ** (-8.0 * np.arange(n) / n)),
        "query norm's weight": weights(lambda d: d.update({"l0.mix.q.norm": np.ones_like(d["l0.mix.q.norm"])})),
        "heads normed apart": planted(keys_values=heads_normed_apart),
        "state lost at 64": planted(gated_states=lambda q, f, v, s=None: (np.concatenate([st(q[:64], f[:64], v[:64])[0], st(q[64:], f[64:], v[64:])[0]]), None)),
        "gate and its complement exchanged": planted(gated_states=other_way_round(None)),
        "written before it is forgotten": planted(gated_states=lambda q, f, v, s=None: st(q, np.concatenate([f[1:], f[-1:]]), v)),
        "no lower bound": planted(forget=lambda z, b, l: fg(z, b, 0 * l)),
        "gate's bias": planted(forget=lambda z, b, l: fg(z, 0 * b, l)),
        "queries without SiLU": planted(silu=lambda z: z),
        "relu without its square": planted(relu2=lambda z: np.maximum(z, 0)),
        "square without relu": planted(relu2=lambda z: z * z),
        "up's bias": weights(lambda d: d.update({"l0.mlp.up.b": 0 * d["l0.mlp.up.b"]})),
        "down's bias": weights(lambda d: d.update({"l0.mlp.down.b": 0 * d["l0.mlp.down.b"]})),
        "router's bias": weights(lambda d: d.update({"l1.mlp.router.b": 0 * d["l1.mlp.router.b"]})),
        "one expert fewer": planted(choose=lambda z, n: pick(z, n - 1)),
        # (a factor common to a row's experts is taken off again by the norm behind them)
        "experts of equal weight": planted(choose=lambda z, n: (pick(z, n) > 0) / n),
        "weights of another temperature": planted(choose=lambda z, n: pick(2 * z, n)),
        "no factor of the logits": changed(lambda c: c.update(logit_scale=1.0)),
        "no last norm": weights(lambda d: d.update({"final.norm": np.ones_like(d["final.norm"])})),
    }
    for what, lg in wrong.items():
        assert error(lg, good).max() > 5 * LIMIT["float32"], what


def test_architecture_registry_and_configurations():
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import architectures, check_config
    assert {"Fitevik", "Kitodra", "Tulipel", "Lozedra"} <= set(architectures())
    for c in (SMALL, TINY, EVEN, WIDE):
        check_config(json.dumps(c))
    ok = config([(attention(), moe()), (states(), dense()), (attention(kv_from=0), None)])
    mixer, mlp = lambda c, i: c["layers"][i]["mixer"], lambda c, i: c["layers"][i]["mlp"]
    for change in (lambda c: c["layers"][2].pop("mlp"), lambda c: mixer(c, 2).update(kv_from=None), lambda c: mixer(c, 2).update(heads=8), lambda c: mixer(c, 0).pop("mask"),
                   lambda c: mixer(c, 2)["mask"].update(size=1)):
        c = json.loads(json.dumps(ok))
        change(c)
        check_config(json.dumps(c))
    bad = [(lambda c: c.update(layers=[]), "no layers"), (lambda c: c["layers"][0].update(type="attention_2"), "attention_2"),
           (lambda c: mlp(c, 0).update(kind="glu"), "glu"), (lambda c: mixer(c, 0).update(kv_heads=3), "no multiple"), (lambda c: mixer(c, 0).pop("scale"), "scale"),
           (lambda c: mixer(c, 0)["mask"].update(size=0), "size"), (lambda c: mixer(c, 1).update(dim=513), "dim"), (lambda c: mixer(c, 2).update(kv_from=1), "layer 1 holds no keys"),
           (lambda c: mixer(c, 2).update(kv_from=2), "layer 2 holds no keys"), (lambda c: mixer(c, 2).update(vdim=9), "another kind"),
           (lambda c: mixer(c, 2).update(kv_heads=4), "another kind"), (lambda c: mlp(c, 0)["router"].update(top=13), "13 of 12 experts"),
           (lambda c: mlp(c, 0)["expert"].pop("ff"), "ff"), (lambda c: mlp(c, 1).pop("ff"), "ff"), (lambda c: c.pop("max_positions"), "max_positions"),
           (lambda c: c.pop("logit_scale"), "logit_scale"), (lambda c: c["norm"].pop("eps"), "eps"), (lambda c: c.update(vocab=1.5), "whole number")]
    for change, text in bad:
        c = json.loads(json.dumps(ok))
        change(c)
        with pytest.raises(VexelError, match=text):
            check_config(json.dumps(c))
