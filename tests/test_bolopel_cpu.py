"""Bolopel without a GPU: the plain statement's own properties, the registry and config reader, the position tables."""
import copy
import ctypes as C
import json

import numpy as np

import bolopel_models as M
import plain_bolopel as P


def test_plain_prefix_does_not_see_the_future():
    cfg, w, t = M.MODELS["mixed"][0], M.arrays(M.weights("mixed")), None
    t = M.tokens(cfg, 40)
    assert np.allclose(P.forward(cfg, w, t)[:17], P.forward(cfg, w, t[:17]), atol=1e-9)


def test_plain_window_and_sink():
    m = P.window_mask(6, 3)
    assert m[5, 3] and not m[5, 2] and not m[2, 3] and m[1, 0] and P.window_mask(4, 1).sum() == 4
    s = np.array([[1.0, -np.inf, 0.0], [-900.0, -np.inf, -np.inf], [900.0, 900.0, -np.inf]])
    p = P.softmax_with_sink(s)
    assert np.allclose(p[0], [np.e / (2 + np.e), 0, 1 / (2 + np.e)]) and p[1].sum() < 1e-300 and np.allclose(p[2], [0.5, 0.5, 0])


def test_plain_delta_rule_recalls_and_overwrites():
    """a unit key written with step 1 is read back exactly; written again it holds the new value only; a decayed channel forgets"""
    k = np.eye(4)[[0, 1, 0, 1]]
    v = np.arange(8.0).reshape(4, 2) + 1
    one = np.ones((4, 4))
    o, S = P.delta_rule(k, k, v, one, np.ones(4))
    assert np.allclose(o, v) and np.allclose(S[0], v[2]) and np.allclose(S[1], v[3])
    g = one.copy()
    g[3, 0] = 0.25
    _, S = P.delta_rule(k, k, v, g, np.array([1.0, 1.0, 0.5, 0.0]))
    assert np.allclose(S[0], 0.25 * (v[0] + v[2]) / 2) and np.allclose(S[1], v[1])
    # a state carried over a cut
    r = np.random.default_rng(0)
    q, kk, vv, gg, b = r.normal(size=(9, 4)), P.unit(r.normal(size=(9, 4))), r.normal(size=(9, 3)), r.uniform(0.2, 1, (9, 4)), r.uniform(size=9)
    full, S = P.delta_rule(q, kk, vv, gg, b)
    a, s0 = P.delta_rule(q[:4], kk[:4], vv[:4], gg[:4], b[:4])
    c, s1 = P.delta_rule(q[4:], kk[4:], vv[4:], gg[4:], b[4:], s0)
    assert np.allclose(np.concatenate([a, c]), full) and np.allclose(s1, S)


def test_plain_decayed_sum_and_convolution_and_layer_norm():
    r = np.random.default_rng(1)
    q, k, v = r.normal(size=(7, 5)), r.normal(size=(7, 5)), r.normal(size=(7, 3))
    o, S = P.decayed_sum(q, k, v, 0.7)
    assert np.allclose(o[6], sum(0.7 ** (6 - j) * (q[6] @ k[j]) * v[j] for j in range(7)))
    x, w = r.normal(size=(6, 2)), r.normal(size=(2, 3))
    y = P.short_conv(x, w)
    assert np.allclose(y[0], w[:, 2] * x[0]) and np.allclose(y[4], w[:, 0] * x[2] + w[:, 1] * x[3] + w[:, 2] * x[4])
    z = P.layer_norm(x + 50.0, np.ones(2), 0.0)
    assert np.allclose(z.mean(-1), 0) and np.allclose((z ** 2).mean(-1), 1)


def test_position_tables_of_the_library_match_the_plain_sinusoid():
    from koifish_amd import lib as L
    hip, _ = L.load()
    for n, width in ((5, 1), (130, 7), (1000, 96), (9000, 64)):
        ld = (width + 63) // 64 * 64
        hi, lo = np.zeros(((n + 63) // 64, ld // 2, 2), dtype=np.float32), np.zeros((64, ld // 2, 2), dtype=np.float32)
        assert hip.kf_rb_sinusoid_tables_host(hi.ctypes.data_as(C.c_void_p), lo.ctypes.data_as(C.c_void_p), n, width, ld, 10000.0) == 0
        p = np.arange(n)
        a, b = hi[p // 64].astype(np.float64), lo[p % 64].astype(np.float64)
        got = np.stack([a[..., 0] * b[..., 1] + a[..., 1] * b[..., 0], a[..., 1] * b[..., 1] - a[..., 0] * b[..., 0]], axis=-1).reshape(n, ld)[:, :width]
        assert np.abs(got - P.sinusoid(p, width)).max() < 3e-7
    assert hip.kf_rb_sinusoid_tables_host(None, None, 4, 4, 64, 10000.0) == -20


def _create(cfg, shapes):
    from koifish_amd import lib as L
    _, host = L.load()
    rc = C.c_int(0)
    h = host.kfh_seq_create(json.dumps(dict(cfg, tensor_shapes={k: list(v) for k, v in shapes.items()})).encode(), 0, None, L.BF16, 64, C.byref(rc))
    if h:
        host.kfh_destroy(C.c_void_p(h))
    return rc.value, host.kfh_last_error().decode()


def test_config_reader_names_what_is_wrong():
    good, sh = M.MODELS["mixed"][0], M.shapes("mixed")
    left = lambda c: c["layers"][1]["mixer"]["left"]
    right = lambda c: c["layers"][1]["mixer"]["right"]
    for edit, word in ((lambda c: c.pop("width"), "width"), (lambda c: c["norm"].pop("eps"), "eps"), (lambda c: c.update(layers=[]), "layers"), (lambda c: c["layers"][1].update(type="attention"), "attention"),
                       (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"), (lambda c: c["layers"][0]["mixer"].update(conv=0), "conv"), (lambda c: c["layers"][0]["mixer"].pop("vdim"), "vdim"),
                       (lambda c: left(c).update(kv_heads=4), "kv_heads"), (lambda c: left(c).pop("mask"), "mask"), (lambda c: left(c)["mask"].update(size=0), "size"), (lambda c: left(c).pop("scale"), "scale"),
                       (lambda c: right(c).update(decay=[0.5]), "decay"), (lambda c: right(c).update(decay=[0.5, "x", 1]), "decay"), (lambda c: c["layers"][1]["mixer"].pop("left_scale"), "left_scale"),
                       (lambda c: c["layers"][1]["mixer"].pop("right"), "right"), (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "moe"), (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff")):
        c = copy.deepcopy(good)
        edit(c)
        rc, err = _create(c, sh)
        assert rc == -20 and word in err, (rc, err)
    rc, err = _create(good, {k: v for k, v in sh.items() if k != "l3.mix.g1"})
    assert rc == -20 and "l3.mix.g1" in err


def test_registry(tmp_path):
    from koifish_amd import models
    (tmp_path / "config.json").write_text(json.dumps(M.MODELS["odd"][0]))
    assert models.architecture(tmp_path) == "Bolopel"
