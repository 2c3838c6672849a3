"""Lozedra without a GPU: the plain implementation's mechanisms on cases worked out by hand, the product's reading of
configurations, and its distance buckets against the plain ones."""
import json
import math

import numpy as np
import pytest

from oracle import lozedra as lz
from lozedra_models import SMALL, config, mixer, tensors


def test_distance_buckets_by_hand():
    """8 rows up to 64: 0..3 alone, then four buckets whose edges are 4 * 16^(i/4) = 4, 8, 16, 32."""
    want = {0: 0, 1: 1, 3: 3, 4: 4, 7: 4, 8: 5, 15: 5, 16: 6, 31: 6, 32: 7, 63: 7, 64: 7, 5000: 7}
    for n, b in want.items():
        assert lz.distance_bucket(n, 8, 64) == b


def test_distance_buckets_of_the_engine():
    from vexel_amd.runtime import load_host
    h = load_host()
    for rows in (2, 3, 7, 8, 12, 31, 64):
        for top in (rows // 2 + 1, rows, 33, 64, 97, 1000):
            if top <= rows // 2:
                assert h.vh_distance_bucket(0, rows, top) == -1
                continue
            for n in list(range(1100)) + [10 ** 6]:
                assert h.vh_distance_bucket(n, rows, top) == lz.distance_bucket(n, rows, top), (n, rows, top)
    assert h.vh_distance_bucket(-1, 8, 64) == -1 and h.vh_distance_bucket(0, 1, 64) == -1


def test_query_temperature_by_hand():
    """1 until the first `every` positions are full, then 1 + coef ln 2, ln 3, .."""
    t = lz.query_temperature(np.arange(40), 0.5, 16)
    assert np.all(t[:15] == 1.0) and np.allclose(t[15:31], 1 + 0.5 * math.log(2)) and np.allclose(t[31:], 1 + 0.5 * math.log(3))


def test_attention_by_hand():
    """Two tokens, one head of one dimension, values 1 and 3, equal scores but for the bias ln 3 at distance 1: the second
    token weighs the first with 3/4; the gate at 0 halves the result."""
    t = {"q": np.zeros((1, 1)), "k": np.zeros((1, 1)), "v": np.ones((1, 1)), "g": np.zeros((1, 1)), "o": np.ones((1, 1)),
         "rel": np.array([[0.0], [math.log(3.0)]])}
    cfg = {"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 1.0, "bias_max": 2}
    y = lz.attention(np.array([[1.0], [3.0]]), t, cfg)
    assert np.allclose(y[:, 0], [0.5, 0.5 * (0.75 * 1 + 0.25 * 3)])


def test_convolution_by_hand():
    x = np.array([[1.0], [2.0], [5.0]])
    y = lz.causal_conv(x, np.array([[10.0, 1.0]]), np.array([0.5]))
    assert np.allclose(y[:, 0], [1.5, 12.5, 25.5])


def test_scan_by_hand():
    """A state that halves per token (dt ln 2, A = -1) and takes dt x B in: y = S C + D x."""
    ln2 = math.log(2.0)
    x, dt = np.array([[1.0], [0.0], [0.0]]), np.full((3, 1), ln2)
    y, s = lz.selective_scan(x, dt, np.array([[-1.0]]), np.ones((3, 1)), 2 * np.ones((3, 1)), np.array([3.0]))
    assert np.allclose(y[:, 0], [2 * ln2 + 3, ln2, ln2 / 2]) and np.allclose(s, ln2 / 4)


def test_order_of_runs():
    assert lz.layer_order({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, False), (1, False), (2, False), (1, True), (2, False), (3, False)]
    assert lz.layer_order({"layers": [0] * 2, "loop": None}) == [(0, False), (1, False)]


def test_prefix_does_not_depend_on_what_follows():
    t = tensors(SMALL, 3)
    toks = np.random.default_rng(0).integers(0, SMALL["vocab"], 40).tolist()
    whole = lz.forward(SMALL, t, toks)
    assert np.allclose(whole[:17], lz.forward(SMALL, t, toks[:17]), atol=1e-9)


def test_the_weights_show_every_mechanism():
    """The random models of the tests are such that leaving out or shifting any one mechanism moves the logits far beyond
    the tolerance of the comparisons (the mistakes are planted in the plain implementation)."""
    from lozedra_models import LIMIT, error
    t = tensors(SMALL, 5)
    toks = np.random.default_rng(1).integers(0, SMALL["vocab"], 90).tolist()
    good = lz.forward(SMALL, t, toks)

    def planted(name, value):
        keep = getattr(lz, name)
        setattr(lz, name, value)
        try:
            return lz.forward(SMALL, t, toks)
        finally:
            setattr(lz, name, keep)

    bucket, temp, conv, order, scan = lz.distance_bucket, lz.query_temperature, lz.causal_conv, lz.layer_order, lz.selective_scan
    wrong = {
        "bucket of the next distance": planted("distance_bucket", lambda n, r, m: bucket(n + 1, r, m)),
        "last bucket one distance late": planted("distance_bucket", lambda n, r, m: bucket(n, r, m + 1)),
        "no temperature": planted("query_temperature", lambda p, c, e: np.ones(len(p))),
        "temperature one position late": planted("query_temperature", lambda p, c, e: temp(p - 1, c, e)),
        "convolution without its oldest tap": planted("causal_conv", lambda x, w, b: conv(x, np.concatenate([0 * w[:, :1], w[:, 1:]], 1)
                                                                                          if w.shape[1] > 1 else w, b)),
        "embedding not added again": planted("layer_order", lambda c: [(i, False) for i, _ in order(c)]),
        "state lost at token 40": planted("selective_scan", lambda x, dt, *r: (np.concatenate([scan(x[:40], dt[:40], r[0], r[1][:40], r[2][:40], r[3])[0],
                                                                                               scan(x[40:], dt[40:], r[0], r[1][40:], r[2][40:], r[3])[0]]), None)),
    }
    for what, lg in wrong.items():
        assert error(lg, good).max() > 5 * LIMIT["float32"], what
    assert error(wrong["state lost at token 40"], good)[:40].max() < 1e-9


def test_architecture_registry_and_configurations():
    from vexel_amd.backend import VexelError
    from vexel_amd.runtime import architectures, check_config
    assert "Lozedra" in architectures()
    check_config(json.dumps(SMALL))
    ok = config([(mixer(), 32)])
    for change in (lambda c: c.pop("loop"), lambda c: c.update(loop={"start": 0, "stop": 1, "times": 1}),
                   lambda c: c["layers"][0].pop("mlp"), lambda c: c["layers"][0]["mixer"]["left"].update(q_temp=None)):
        c = json.loads(json.dumps(ok))
        change(c)
        check_config(json.dumps(c))
    bad = [(lambda c: c.update(architecture="Other"), "unknown architecture"), (lambda c: c.pop("architecture"), "no architecture"),
           (lambda c: c.update(layers=[]), "no layers"), (lambda c: c.pop("vocab"), "vocab"),
           (lambda c: c["layers"][0].update(type="serial"), "serial"), (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "sparse"),
           (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=2), "multiple"),
           (lambda c: c["layers"][0]["mixer"]["right"].update(state=0), "state"),
           (lambda c: c["layers"][0]["mixer"]["right"].update(inner=2.5), "inner"),
           (lambda c: c["layers"][0]["mixer"].pop("right_scale"), "right_scale"),
           (lambda c: c.update(loop={"start": 1, "stop": 0, "times": 2}), "loop")]
    for change, text in bad:
        c = json.loads(json.dumps(ok))
        change(c)
        with pytest.raises(VexelError, match=text):
            check_config(json.dumps(c))
    for text in ("", "{", "[1, 2", "{\"architecture\": }", "nonsense"):
        with pytest.raises(VexelError, match="not JSON"):
            check_config(text)


def test_written_tensors_come_back(tmp_path):
    t = tensors(SMALL, 9)
    lz.write_model(str(tmp_path), SMALL, t)
    back = lz.read_tensors(str(tmp_path / "model.safetensors"))
    assert set(back) == set(t) and all(np.array_equal(back[n], t[n]) for n in t)


def test_command_line_lists_architectures(capsys):
    from vexel_amd.__main__ import main
    assert main(["architectures"]) == 0
    assert "Lozedra" in capsys.readouterr().out.split()
