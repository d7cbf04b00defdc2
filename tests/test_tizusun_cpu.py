"""Tizusun without a GPU: the plain statement's own properties, the registry and config reader, the trace replayer's bookkeeping."""
import copy
import ctypes as C
import json

import numpy as np
import pytest

import plain_tizusun as P
import tizusun_models as M


def test_plain_prefix_does_not_see_the_future():
    cfg = M.CONFIGS["mixed"]
    w = M.arrays(M.weights(cfg))
    t = M.tokens(cfg, 40)
    full = P.forward(cfg, w, t)
    assert np.allclose(full[:17], P.forward(cfg, w, t[:17]), atol=1e-9)


def test_plain_chunks_are_independent_through_the_mixer():
    m = P.chunk_mask(10, 4)
    assert m[3, 0] and not m[4, 3] and m[7, 4] and not m[4, 5] and m.sum() == 10 + 10 + 3
    assert P.chunk_mask(3, 1).sum() == 3 and P.chunk_mask(5, 0).sum() == 15


def test_plain_rope_keeps_lengths_and_relative_angles():
    f = P.rope_frequencies(100.0, 8, None)
    x = np.random.default_rng(0).normal(size=(6, 1, 12))
    p = np.arange(6.0)
    y = P.rope(x, p, f)
    assert np.allclose((y ** 2).sum(-1), (x ** 2).sum(-1)) and np.array_equal(y[..., 8:], x[..., 8:])
    a, b = P.rope(x[:1], np.array([9.0]), f), P.rope(x[1:2], np.array([4.0]), f)
    c, d = P.rope(x[:1], np.array([5.0]), f), P.rope(x[1:2], np.array([0.0]), f)
    assert np.allclose((a * b).sum(), (c * d).sum())


def test_rope_table_of_the_library_matches_the_plain_frequencies():
    from koifish_amd import lib as L
    hip, _ = L.load()
    for base, dims, sc in ((1e4, 16, (8.0, 1.0, 4.0, 64)), (500.0, 10, (1.0, 1.0, 4.0, 64)), (7e5, 64, (3.0, 2.0, 16.0, 4096)), (50.0, 2, (4.0, 1.0, 4.0, 8))):
        t = np.zeros((300, dims // 2, 2), dtype=np.float32)
        assert hip.kf_rb_rope_table_host(t.ctypes.data_as(C.c_void_p), 300, dims, base, *sc) == 0
        a = np.arange(300.0)[:, None] * P.rope_frequencies(base, dims, dict(zip(("factor", "low", "high", "original"), sc)))[None]
        assert np.abs(t[..., 0] - np.cos(a)).max() < 1e-6 and np.abs(t[..., 1] - np.sin(a)).max() < 1e-6
    assert hip.kf_rb_rope_table_host(None, 3, 4, 1e4, 1.0, 1.0, 4.0, 8.0) == -20
    assert hip.kf_rb_rope_table_host(t.ctypes.data_as(C.c_void_p), 3, 5, 1e4, 1.0, 1.0, 4.0, 8.0) == -20


def _create(cfg):
    from koifish_amd import lib as L
    _, host = L.load()
    rc = C.c_int(0)
    h = host.kfh_seq_create(json.dumps(cfg).encode(), 0, None, L.BF16, 64, C.byref(rc))
    if h:
        host.kfh_destroy(C.c_void_p(h))
    return rc.value, host.kfh_last_error().decode()


def test_config_reader_names_what_is_wrong():
    good = M.CONFIGS["mixed"]

    def bad(edit):
        c = copy.deepcopy(good)
        edit(c)
        return _create(c)
    for edit, word in ((lambda c: c.update(architecture="Nothing"), "Nothing"), (lambda c: c.pop("width"), "width"), (lambda c: c["norm"].pop("eps"), "eps"), (lambda c: c.update(layers=[]), "layers"),
                       (lambda c: c["layers"][1].update(type="recurrent"), "recurrent"), (lambda c: c["layers"][2]["mixer"].update(heads=7, kv_heads=2), "heads"),
                       (lambda c: c["layers"][0]["mixer"].update(vdim=8), "values"), (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=34), "rotated"),
                       (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "top"), (lambda c: c["layers"][2]["mlp"].update(kind="sparse"), "sparse"),
                       (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size")):
        rc, err = bad(edit)
        assert rc == -20 and word in err, (rc, err)


def test_without_a_gpu_creation_fails_loudly():
    import torch
    if torch.cuda.is_available():
        pytest.skip("GPU present")
    rc, err = _create(M.CONFIGS["mixed"])
    assert rc == -1400 and "no HIP device" in err


def test_registry(tmp_path):
    from koifish_amd import lib as L
    from koifish_amd import models
    for cfg, want in ((dict(architecture="Tizusun"), "Tizusun"), (dict(model_type="qwen3"), "qwen3"), (dict(architectures=["Qwen3ForCausalLM"]), "Qwen3ForCausalLM")):
        (tmp_path / "config.json").write_text(json.dumps(cfg))
        assert models.architecture(tmp_path) == want
    (tmp_path / "config.json").write_text(json.dumps(dict(architecture="Other")))
    with pytest.raises(L.KFError, match="Other"):
        models.architecture(tmp_path)
    with pytest.raises(L.KFError, match="float32"):
        models._qwen3(tmp_path, "float32", 0, 0)


class FakeSlots:
    """records what a trace asks of the slots; logits = [slot, position] of the wanted row"""
    made = []

    def __init__(self, model, n):
        self.n, self.free, self.calls = n, list(range(n)), []
        FakeSlots.made.append(self)

    def acquire(self):
        return self.free.pop(0)

    def release(self, s):
        self.free.insert(0, s)

    def run(self, spans, want):
        self.calls.append(spans)
        return np.array([[spans[k][0], spans[k][1] + o] for k, o in want], dtype=np.float32).reshape(len(want), 2)

    def close(self):
        self.closed = True


def test_trace_replay_keeps_slots_positions_and_files(tmp_path):
    from koifish_amd import trace
    FakeSlots.made = []
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": [1, 2, 3], "want": [2, 0]}, {"id": "y", "tokens": [4], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": [5], "want": [0]}, {"id": "x", "tokens": [6], "want": [0]}], "end": ["x"]},
             {"step": 2, "entries": [{"id": "y", "tokens": [7], "want": []}], "end": ["y"]},
             {"step": 3, "entries": [{"id": "z%d" % i, "tokens": [8] * (i + 1), "want": [i]} for i in range(3)], "end": ["z0", "z1", "z2"]}]
    said = []
    trace.replay(None, FakeSlots, str(tmp_path), [json.dumps(s) + "\n" for s in steps] + ["\n"], lambda line, flush: said.append(line))
    assert said == ["done %d" % i for i in range(4)]
    rd = lambda i: np.fromfile(tmp_path / ("%d.f32" % i), dtype="<f4").reshape(-1, 2).tolist()
    assert rd(0) == [[0, 2], [0, 0]] and rd(1) == [[1, 1], [0, 3]] and rd(3) == [[0, 0], [1, 1], [2, 2]]
    assert not (tmp_path / "2.f32").exists()
    assert [f.n for f in FakeSlots.made] == [2, 3] and FakeSlots.made[0].closed and FakeSlots.made[1].closed
    assert [(s, p) for s, p, _ in FakeSlots.made[0].calls[1]] == [(1, 1), (0, 3)]
    with pytest.raises(ValueError, match="live"):
        t = trace.Trace(None, FakeSlots)
        t.step([{"id": "a", "tokens": [1], "want": []}], [])
        t.step([{"id": "a", "tokens": [1], "want": []}, {"id": "b", "tokens": [1], "want": []}], [])
