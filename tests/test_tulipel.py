"""Tulipel without a GPU: the plain implementation's mechanisms on cases worked out by hand, mistakes planted in it, and the
product's reading of configurations and its frequencies."""
import ctypes as C
import json
import math

import numpy as np
import pytest

from oracle import tulipel as tl
from tulipel_models import EVEN, LIMIT, SMALL, TINY, WIDE, config, error, first, second, tensors


def test_norms_by_hand():
    x = np.array([[3.0, 4.0]])
    assert np.allclose(tl.model_norm(x, np.array([0.0, 1.0]), 0.0), [[3 / math.sqrt(12.5), 8 / math.sqrt(12.5)]])
    assert np.allclose(tl.rms(x, 12.5), x / 5.0)               # eps stands under the root


def test_rotation_by_hand():
    """A quarter turn per position for the first pair, half of one for the second: base^(-2i / 4) = 1, 1 / 2."""
    rot = {"dims": 4, "base": 4.0}
    x = np.array([[1.0, 0.0, 0.0, 2.0]] * 2)
    a = np.array([0.0, 1.0])
    c1, s1, c2, s2 = math.cos(1), math.sin(1), math.cos(0.5), math.sin(0.5)
    y = tl.rotate(x, a, rot, halves=False)                     # pairs (1, 0) and (0, 2)
    assert np.allclose(y[0], x[0]) and np.allclose(y[1], [c1, s1, -2 * s2, 2 * c2])
    y = tl.rotate(x, a, rot, halves=True)                      # pairs (1, 0) and (0, 2) again, at other places
    assert np.allclose(y[1], [c1, -2 * s2, s1, 2 * c2])


def test_rotation_leaves_later_dimensions():
    x = np.random.default_rng(0).standard_normal((3, 2, 7))
    for halves in (False, True):
        y = tl.rotate(x, np.arange(3), {"dims": 4, "base": 10.0}, halves)
        assert np.array_equal(y[..., 4:], x[..., 4:]) and not np.allclose(y[1:, :, :4], x[1:, :, :4])


def test_yarn_by_hand():
    """8 dimensions, base 16, original 2 pi 16: a pair makes t turns at dimension log2(16 / t), so that just under 8 turns (fast) and just
    over 1 / 2 (slow) give the ramp from 1 to 5."""
    f, m = tl.frequencies({"dims": 8, "base": 16.0, "scaling": {"factor": 2.0, "original": 32 * math.pi, "fast": 7.9, "slow": 0.51}})
    plain = 16.0 ** (-np.arange(4) / 4)
    ramp = np.array([0, 0, 1 / 4, 2 / 4])
    assert np.allclose(f, plain / 2 * ramp + plain * (1 - ramp)) and math.isclose(m, 0.1 * math.log(2) + 1)


def engine_frequencies(rot):
    from vexel_amd.runtime import load_host
    h = load_host()
    f, both = (C.c_double * (rot["dims"] // 2))(), C.c_double()
    s = rot.get("scaling") or {"factor": 0, "original": 0, "fast": 0, "slow": 0}
    assert h.vh_rotary_frequencies(rot["dims"], rot["base"], s["factor"], s["original"], s["fast"], s["slow"], f, C.byref(both)) == 0
    return np.array(f), both.value


def test_frequencies_of_the_engine():
    """With the ramp inside the pairs, cut off at either end, of no width and upside down."""
    for dims in (2, 8, 30, 64, 128):
        for base in (1.5, 40.0, 10000.0, 1e6):
            for s in (None, (2.0, 512, 32.0, 1.0), (40.0, 4096, 32.0, 1.0), (4.0, 64, 1000.0, 500.0), (1.0, 10, 3.0, 2.9), (8.0, 3, 1.0, 0.001),
                      (0.5, 1e6, 2.0, 2.0), (3.0, 100, 0.1, 20.0)):
                rot = {"dims": dims, "base": base}
                if s:
                    rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), s))
                want, m = tl.frequencies(rot)
                got, both = engine_frequencies(rot)
                assert np.allclose(got, want, rtol=1e-12) and math.isclose(both, m)


def test_when_keys_are_spelled_out():
    from vexel_amd.runtime import load_host
    h = load_host()
    assert h.vh_spell_out_rows(512, 128, 128) == 256           # 1.5 * 512 * 256 / (1024 - 256)
    assert h.vh_spell_out_rows(64, 64, 80) == 0                # the latents are the shorter way for any number of rows
    assert h.vh_spell_out_rows(128, 32, 32) == 64 and h.vh_spell_out_rows(256, 64, 16) == 72 and h.vh_spell_out_rows(0, 1, 1) == 0


def test_sink_by_hand():
    """Two equal scores ln 2 and a sink ln 4: 2 / (2 + 2 + 4) each; a sink far below changes nothing, one far above takes all."""
    s = np.log(np.array([2.0, 2.0]))
    assert np.allclose(tl.sink_softmax(s, math.log(4)), [0.25, 0.25])
    assert np.allclose(tl.sink_softmax(s, -800.0), [0.5, 0.5]) and np.allclose(tl.sink_softmax(s, 800.0), 0)


def test_attention_by_hand():
    """One head, a latent of one element that the norm makes 1 or -1, no rotation to speak of at position 0 and 1 (queries and keys of
    zero): weights 1 / (n + e^sink) each, values 3 c."""
    t = {"q": np.zeros((3, 1)), "dkv": np.array([[1.0], [0.0], [0.0]]), "dkv.norm": np.ones(1), "uk": np.zeros((1, 1)),
         "uv": np.array([[3.0]]), "sink": np.zeros(1), "o": np.ones((1, 1))}
    cfg = {"heads": 1, "dim": 1, "rot_dim": 2, "vdim": 1, "kv_rank": 1, "scale": 1.0, "rot": {"dims": 2, "base": 10.0}}
    y, (c, kr) = tl.latent_attention(np.array([[2.0], [-5.0], [7.0]]), t, cfg, "latent_attention_2", 0.0)
    assert np.allclose(c[:, 0], [1, -1, 1]) and np.allclose(kr, 0)
    assert np.allclose(y[:, 0], [3 / 2, 0, 3 / 4])


def test_rotated_scores_depend_on_the_distance():
    """Scores between rotated parts are the same for every pair of positions equally far apart, with either layout of pairs."""
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((2, 1, 6))
    for halves in (False, True):
        for scaling in (None, {"factor": 4.0, "original": 50, "fast": 8.0, "slow": 1.0}):
            rot = {"dims": 6, "base": 50.0, "scaling": scaling}
            at = lambda v, p: tl.rotate(v, np.array([p]), rot, halves)[0]
            assert np.isclose(at(q, 9) @ at(k, 4), at(q, 105) @ at(k, 100)) and not np.isclose(at(q, 9) @ at(k, 4), at(q, 9) @ at(k, 5))


def test_activation_by_hand():
    """z = (1, -1): every power has the root mean square 1."""
    assert np.allclose(tl.poly_norm(np.array([[1.0, -1.0]]), (2.0, 3.0, 5.0, 7.0), 0.0), [[2 + 3 + 5 + 7, -2 + 3 - 5 + 7]])
    z = np.array([[1.0, 3.0]])
    want = 1.0 / math.sqrt(5) + 2 / math.sqrt(41) + 4 / math.sqrt(365)
    assert np.isclose(tl.poly_norm(z, (1.0, 2.0, 4.0, 0.0), 0.0)[0, 0], want)


def test_depth_average_by_hand():
    r = [np.full((1, 2), v) for v in (1.0, 10.0, 100.0)]
    assert np.allclose(tl.depth_average([1, 2, 3], r), 321) and np.allclose(tl.softcap(np.array([1e9, 0.0]), 30.0), [30, 0])


def test_prefix_does_not_depend_on_what_follows():
    t = tensors(SMALL, 3)
    toks = np.random.default_rng(0).integers(0, SMALL["vocab"], 40).tolist()
    whole = tl.forward(SMALL, t, toks)
    assert np.allclose(whole[:17], tl.forward(SMALL, t, toks[:17]), atol=1e-9)


def test_the_weights_show_every_mechanism(monkeypatch):
    """The random models of the tests are such that leaving out or changing any one mechanism moves the logits far beyond the
    tolerance of the comparisons (the mistakes are planted in the plain implementation, or in the weights it gets)."""
    t = tensors(SMALL, 5)
    toks = np.random.default_rng(1).integers(0, SMALL["vocab"], 90).tolist()
    good = tl.forward(SMALL, t, toks)

    def planted(**mistakes):
        with monkeypatch.context() as m:
            for name, value in mistakes.items():
                m.setattr(tl, name, value)
            return tl.forward(SMALL, t, toks)

    def weights(change):
        d = dict(t)
        change(d)
        return tl.forward(SMALL, d, toks)

    def changed(change):
        c = json.loads(json.dumps(SMALL))
        change(c)
        return tl.forward(c, t, toks)

    soft, rot, freq, lat, att, mn, avg, act = (tl.sink_softmax, tl.rotate, tl.frequencies, tl.latent, tl.latent_attention, tl.model_norm,
                                               tl.depth_average, tl.poly_norm)

    def raw_latent(h, pos, t, cfg, halves, eps):
        y = tl.linear(t["dkv"], h)
        return y[:, :cfg["kv_rank"]] * t["dkv.norm"], rot(y[:, cfg["kv_rank"]:], pos, cfg["rot"], halves)

    def turned_again(h, t, cfg, kind, eps, shared=None):
        if shared is not None:
            shared = (shared[0], rot(shared[1], np.arange(len(h)), cfg["rot"], True))
        return att(h, t, cfg, kind, eps, shared)

    def last_key(s, sink):
        s = s.copy()
        s[np.arange(1, len(s)), np.arange(len(s) - 1)] = -np.inf
        return soft(s, sink)

    wrong = {
        "no sink": planted(sink_softmax=lambda s, k: soft(s, -1e9)),
        "the sink twice": planted(sink_softmax=lambda s, k: soft(s, k + math.log(2))),
        "the key before last not seen": planted(sink_softmax=last_key),
        "the other layout of pairs": planted(rotate=lambda x, p, r, h: rot(x, p, r, not h)),
        "positions from 1": planted(latent=lambda h, p, *a: lat(h, p + 1, *a)),
        "turned the other way": planted(rotate=lambda x, p, r, h: rot(x, -np.asarray(p), r, h)),
        "no YaRN": planted(frequencies=lambda r: freq({**r, "scaling": None})),
        "YaRN without its factor": planted(frequencies=lambda r: (freq(r)[0], 1.0)),
        "latent not normed": planted(latent=raw_latent),
        "query latent's weight left out": weights(lambda d: d.update({"l0.mix.dq.norm": np.ones_like(d["l0.mix.dq.norm"])})),
        "shared keys turned twice": planted(latent_attention=turned_again),
        "norm weights around one": planted(model_norm=lambda x, w, e: mn(x, w - 1, e)),
        "alpha 1": changed(lambda c: c.update(postln_alpha=1.0)),
        "no average over the depth": planted(depth_average=lambda w, r: r[-1]),
        "the embedding left out of it": planted(depth_average=lambda w, r: avg(w[1:], r[1:])),
        "activation without its constant": planted(poly_norm=lambda z, a, e: act(z, (a[0], a[1], a[2], 0.0), e)),
        "powers of the normed row": planted(poly_norm=lambda z, a, e: a[0] * tl.rms(z, e) + a[1] * tl.rms(z, e) ** 2 + a[2] * tl.rms(z, e) ** 3 + a[3]),
        "no cap on the logits": planted(softcap=lambda x, c: x),
        "scale of the unrotated part alone": changed(lambda c: c["layers"][0]["mixer"].update(scale=c["layers"][0]["mixer"]["dim"] ** -0.5)),
    }
    for what, lg in wrong.items():
        assert error(lg, good).max() > 5 * LIMIT["float32"], what


def test_architecture_registry_and_configurations():
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import architectures, check_config
    assert "Tulipel" in architectures() and "Lozedra" in architectures()
    for c in (SMALL, TINY, EVEN, WIDE):
        check_config(json.dumps(c))
    ok = config([(first(), 32), (second(), 32), (second(kv_from=1), 16)])
    mixers = lambda c, i: c["layers"][i]["mixer"]
    for change in (lambda c: c["layers"][0].pop("mlp"), lambda c: mixers(c, 1)["rot"].pop("scaling") and mixers(c, 2)["rot"].pop("scaling"),
                   lambda c: mixers(c, 2).update(kv_from=None), lambda c: c.pop("logit_softcap")):
        c = json.loads(json.dumps(ok))
        change(c)
        check_config(json.dumps(c))
    bad = [(lambda c: c.pop("postln_alpha"), "postln_alpha"), (lambda c: c.update(layers=[]), "no layers"), (lambda c: c.update(logit_softcap=-1.0), "softcap"),
           (lambda c: c["layers"][0].update(type="latent_attention_3"), "latent_attention_3"), (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "sparse"),
           (lambda c: mixers(c, 0).pop("q_rank"), "q_rank"), (lambda c: mixers(c, 0).update(rot_dim=11), "dimensions"),
           (lambda c: mixers(c, 0)["rot"].update(dims=6), "dimensions"), (lambda c: mixers(c, 0)["rot"].update(base=1.0), "base"),
           (lambda c: mixers(c, 1)["rot"]["scaling"].pop("slow"), "slow"), (lambda c: mixers(c, 1)["rot"]["scaling"].update(factor=0.0), "scaling"),
           (lambda c: mixers(c, 2).update(kv_from=2), "holds no latents"), (lambda c: mixers(c, 1).update(kv_from=2), "holds no latents"),
           (lambda c: mixers(c, 2).update(kv_from=0), "another kind"), (lambda c: mixers(c, 2).update(kv_rank=8), "another kind"),
           (lambda c: mixers(c, 2)["rot"].update(base=7.0), "another kind"), (lambda c: mixers(c, 2).update(kv_from=1.5), "whole number"),
           (lambda c: mixers(c, 0).pop("scale"), "scale"), (lambda c: mixers(c, 0).update(vdim=0), "vdim")]
    for change, text in bad:
        c = json.loads(json.dumps(ok))
        change(c)
        with pytest.raises(VexelError, match=text):
            check_config(json.dumps(c))
    chain = config([(second(), 8), (second(kv_from=0), 8), (second(kv_from=1), 8)])
    with pytest.raises(VexelError, match="holds no latents"):
        check_config(json.dumps(chain))
