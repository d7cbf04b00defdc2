"""Bolopel through the framework -- loader, step, slots, queue, sampler, trace replay -- against the plain float64 statement (plain_bolopel.py) on small models of our own."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import bolopel_models as M
import layered_helpers
import plain_bolopel as P
from koifish_amd import lib as L
from layered_helpers import bf16_view, rel

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# relative rms error of a row of logits: bf16 roundings of a few layers; a wrong key, edge or state is an order of magnitude larger (the float32 runs of the same schedules hold 2e-4)
TOL = {"float32": 2e-4, "bfloat16": 0.1}


def make(name, dtype="float32", max_seq=400, seed=0, w=None):
    from koifish_amd.runtime import Bolopel
    model = M.MODELS[name] if isinstance(name, str) else name
    w = M.weights(model, seed) if w is None else w
    m = Bolopel(model[0], dtype, max_seq, shapes=M.shapes(model))
    for i, (k, v) in enumerate(w.items()):
        m.set_tensor(k, v.cuda() if i % 2 else v)
    return m, M.arrays(w)


def Seqs(m, w, cfg, n=4):
    return layered_helpers.Seqs(P, m, w, cfg, TOL, n)


@pytest.fixture(scope="module", params=[(c, d) for c in M.MODELS for d in ("float32", "bfloat16")], ids=lambda p: p[0] + "-" + p[1])
def served(request):
    name, dtype = request.param
    m, w = make(name, dtype)
    yield M.MODELS[name][0], m, w
    m.close()


def test_residual_stream_after_every_layer(served):
    cfg, m, w = served
    t = M.tokens(cfg, 75)
    s = Seqs(m, w, cfg, 1)
    tap = m.tap(75)
    s.open("a", t)
    s.feed({"a": 75})
    m.tap(0)
    _, ref = P.forward(cfg, w, t, True)
    err = np.abs(tap - ref).max(axis=(1, 2)) / np.abs(ref).max(axis=(1, 2))
    assert (err < (1e-4 if m.dtype == "float32" else 0.06)).all(), err


def test_prompts_portions_decoding_and_mixed_batches(served):
    cfg, m, w = served
    s = Seqs(m, w, cfg)
    s.open("a", M.tokens(cfg, 240, 1))
    s.feed({"a": 66})                                   # alone
    s.open("b", M.tokens(cfg, 110, 2))
    s.open("c", M.tokens(cfg, 50, 3))
    s.feed({"b": 79, "a": 2, "c": 1})                   # a prompt, a portion of two, a first token
    for n in (3, 2, 7):
        s.feed({"c": n, "a": n + 1})
    s.feed({"a": 64, "c": 2})
    for _ in range(12):                                 # decoded together, then unequal ends
        s.feed({"a": 1, "b": 1, "c": 1})
    s.close("c")
    s.open("d", M.tokens(cfg, 60, 4))                   # the slot used again: its rings and states still hold c's
    s.feed({"d": 20})
    for _ in range(9):
        s.feed({"d": 1, "a": 1})
    s.feed({"b": 1, "d": 5})                            # a single token and a portion in one batch
    s.close("b")
    s.open("e", M.tokens(cfg, 9, 5))                    # a first token alone, then decoded, in a used slot
    s.feed({"e": 1, "a": 3})
    for _ in range(8):
        s.feed({"e": 1})
    s.close("a"), s.close("d"), s.close("e")


def test_long_decoding_past_every_window(served):
    cfg, m, w = served
    n = max([L_["mixer"]["left"]["mask"]["size"] for L_ in cfg["layers"] if "left" in L_["mixer"]] + [40])
    n = min(2 * n + 8, 330)
    s = Seqs(m, w, cfg, 2)
    t = M.tokens(cfg, n, 7)
    ref = P.forward(cfg, w, t)
    s.open("p", t, ref)
    s.open("a", t, ref)
    s.feed({"p": n})
    s.feed({"a": 3})
    for _ in range(n - 3):
        s.feed({"a": 1})


def test_slots_give_the_same_whatever_else_runs(served):
    """the same request alone and among others, in another slot: the difference is rounding only (the batch size picks the kernels)"""
    cfg, m, w = served
    from koifish_amd.runtime import XcdReplicas
    t, other = M.tokens(cfg, 70, 11), M.tokens(cfg, 70, 12)
    x = XcdReplicas(m, 3)
    a = x.run([(0, 0, t[:40])], [(0, i) for i in range(40)])
    da = np.concatenate([x.run([(0, 40 + i, t[40 + i:41 + i])], [(0, 0)]) for i in range(10)])
    b = x.run([(1, 0, other[:63]), (2, 0, t[:40])], [(1, i) for i in range(40)])
    db = np.concatenate([x.run([(1, 63 + i, [5]), (2, 40 + i, t[40 + i:41 + i])], [(1, 0)]) for i in range(7)])
    tol = 2e-5 if m.dtype == "float32" else TOL["bfloat16"]   # (40 rows and 103 take different kernels: another set of bf16 roundings)
    assert rel(b, a).max() < tol and rel(db, da[:7]).max() < tol
    x.close()


WINDOW = 20


def edge_model():
    """a windowed layer whose decayed sum is switched off by its scale: one marked token's key and value outshine the rest"""
    cfg, ranks = M.model(64, 40, 1e-6, [M.parallel((2, 1, 32, 32), WINDOW, 0.4, (1, 8, 8), (0.9,), 1.0, 0.0)])
    raw = M.weights((cfg, ranks), 5)
    e, q, k, v = (raw[n].float() for n in ("embed", "l0.mix.left.q", "l0.mix.left.k", "l0.mix.left.v"))
    e[:, 60:] = 0.0                                     # the slowest of the position vector's columns: about 0 and 1
    e[39, 60] = 9.0                                     # the marked token
    k[31], q[31::32] = 0.0, 0.0
    k[31, 60], q[31::32, 61] = 8.0, 25.0
    v[:, 60] = 1.5 * torch.randn(32, generator=torch.Generator().manual_seed(1))
    raw.update({n: t.bfloat16() for n, t in zip(("embed", "l0.mix.left.q", "l0.mix.left.k", "l0.mix.left.v"), (e, q, k, v))})
    return (cfg, ranks), raw


@pytest.mark.parametrize("how", ["prompt", "portions", "decoded"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_edges_show_in_the_logits(dtype, how):
    """the logits of the last position that sees the marked token and of the first one that does not, prompt and decoded"""
    model, raw = edge_model()
    cfg = model[0]
    m, w = make(model, dtype, 100, w=raw)
    for at in (0, WINDOW - 1, WINDOW, WINDOW + 1, 2 * WINDOW - 1):
        t = M.tokens(cfg, at + WINDOW + 9, at) % 39
        t[at] = 39
        s = Seqs(m, w, cfg, 1)
        s.open("a", t)
        plain = t.copy()
        plain[at] = 3
        d = rel(s.ref["a"], P.forward(cfg, w, plain))
        assert all(d[i] > 0.3 for i in range(at + 1, at + WINDOW)) and all(d[i] < 1e-9 for i in range(at + WINDOW, len(t))), d
        if how == "prompt":
            s.feed({"a": len(t)})
        elif how == "portions":
            for n in ([at + 1] if at else [1]) + [2, 3, WINDOW - 6, 2, 2]:
                s.feed({"a": n})
            s.feed({"a": len(s.tok["a"][1])})
        else:
            s.feed({"a": 1})
            for _ in range(len(t) - 1):
                s.feed({"a": 1})
        s.x.close()
    m.close()


@pytest.mark.parametrize("kind", ["delta", "sum", "sink"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_tokens_and_the_sink_show_in_the_logits(dtype, kind):
    """one layer: a token hundreds of positions back that the state still holds (no decay to speak of), in a prompt, over cuts and decoded; a sink that outweighs the keys"""
    def mark(raw, mix, key):                            # the marked token alone writes and asks along channel 31 of every head
        e = raw["embed"].float()
        e[:, 56:], e[39] = 0.0, 0.0
        e[39, 56] = 12.0
        raw["embed"] = e.bfloat16()
        for n in "qk":
            x = raw[mix + n].float()
            x[:, 56:], x[31::32] = 0.0, 0.0
            x[31::32, 56] = key
            raw[mix + n] = x.bfloat16()
    if kind == "delta":
        model = M.model(64, 40, 1e-6, [M.delta(2, 1, 32, 32, 4, 8, 8)])
        raw = M.weights(model, 6)
        raw["l0.mix.dt_bias"] = torch.full((64,), -12.0).bfloat16()
        raw["l0.mix.b"] = (0.3 * raw["l0.mix.b"].float()).bfloat16()
        mark(raw, "l0.mix.", 4.0)
        for n in "qk":
            c = 0.3 * raw["l0.mix.%s.conv" % n].float()
            c[:, 3] = 1.0
            raw["l0.mix.%s.conv" % n] = c.bfloat16()
    elif kind == "sum":
        model = M.model(64, 40, 1e-6, [M.parallel((1, 1, 8, 8), 3, 0.2, (2, 32, 32), (1.0, 0.9995), 0.1, 1.0)])
        raw = M.weights(model, 7)
        mark(raw, "l0.mix.right.", 6.0)
    else:
        model = M.model(64, 40, 1e-6, [M.parallel((2, 1, 32, 32), 300, 0.9, (1, 8, 8), (0.5,), 1.0, 0.0)])
        raw = M.weights(model, 8)
        # q against k: unit vectors that point the other way, scores far below the sink's
        raw["l0.mix.left.q"] = (-torch.cat([raw["l0.mix.left.k"].float()] * 2) + 0.05 * raw["l0.mix.left.q"].float()).bfloat16()
        raw["embed"] = (0.3 * raw["embed"].float() + torch.linspace(-2, 2, 64)).bfloat16()
    cfg = model[0]
    m, w = make(model, dtype, 300, w=raw)
    t = M.tokens(cfg, 220, 9) % 39
    t[[3, 200]] = 39
    other = t.copy()
    other[3] = 7
    ref = P.forward(cfg, w, t)
    if kind == "sink":
        full, P.softmax_with_sink = P.softmax_with_sink, lambda s: np.exp(s - s.max(-1, keepdims=True)) / np.exp(s - s.max(-1, keepdims=True)).sum(-1, keepdims=True)
        try:
            without = P.forward(cfg, w, t)
        finally:
            P.softmax_with_sink = full
        assert np.median(rel(ref, without)) > 5 * TOL["bfloat16"]
    else:
        assert rel(ref, P.forward(cfg, w, other))[200] > 2 * TOL["bfloat16"]
    s = Seqs(m, w, cfg, 2)
    s.open("a", t, ref), s.open("b", t, ref)
    s.feed({"a": 220})
    for n in (2, 61, 5, 64, 2, 60):
        s.feed({"b": n})
    while s.tok["b"][1]:
        s.feed({"b": 1})
    m.close()


def test_greedy_generation_matches_the_plain_model():
    cfg = M.MODELS["mixed"][0]
    m, w = make("mixed")
    p = M.tokens(cfg, 30, 21)
    want = P.greedy(cfg, w, p, 24)
    assert m.generate(p, 24, use_graph=True) == want                 # token-serial prompt, captured steps
    assert m.generate(p, 24, use_graph=False) == want
    m.set_prefill_mode(1)
    assert m.generate(p, 24, use_graph=True) == want                 # batched prompt
    assert m.num_graphs() >= 1
    nxt, lg = m.prefill(p)
    assert nxt == want[0] and int(bf16_view(lg).argmax()) >= 0
    for _ in range(2):                                               # a step run twice on its position gives the same: the state after it has a side of its own
        r, lg = m.forward(int(want[0]), 30)
        assert r == want[1]
        ref = P.forward(cfg, w, list(p) + want[:1])[-1]
        assert rel(bf16_view(lg)[None], ref[None])[0] < 0.01         # kfh_logits is the bf16 view
    m.close()


def test_queue_of_prompts_through_the_slots():
    """more prompts than slots through the scheduler's queue: every answer is the plain model's; eos and per-request limits; prompts prefilled together or one by one"""
    from koifish_amd.runtime import XcdReplicas
    cfg = M.MODELS["mixed"][0]
    m, w = make("mixed")
    prompts = [M.tokens(cfg, n, 40 + n) for n in (5, 33, 1, 70, 18, 9)]
    want = [P.greedy(cfg, w, p, 10) for p in prompts]
    for batch in (1, 3):
        x = XcdReplicas(m, 3)
        x.set_prefill_batch(batch)
        got, st = x.chat(prompts, 10)
        assert got == want and st["prefills"] == 6
        got, _ = x.chat(prompts, 10, max_new_each=[1, 4, 10, 2, 7, 3])
        assert got == [a[:k] for a, k in zip(want, [1, 4, 10, 2, 7, 3])]
        eos = want[1][3]
        got, _ = x.chat(prompts, 10, eos=eos)
        assert got == [a[:a.index(eos) + 1] if eos in a else a for a in want]
        x.close()
    m.close()


@pytest.mark.parametrize("name", ["mixed", "heads"])
def test_every_replay_of_a_captured_step_equals_the_eager_one(name):
    cfg = M.MODELS[name][0]
    m, w = make(name, "bfloat16")
    t = M.tokens(cfg, 40, 5)
    m.set_forced(np.concatenate([t, np.full(360, -1)]))

    def walk(graph):
        out = []
        m.set_state(int(t[0]), 0)
        for i in range(40):
            m.run_steps(i, 1, use_graph=graph)
            m.sync()
            out.append(m.logits().copy())
            torch.zeros(1 << 16, device="cuda").add_(1)     # other work between the replays
        return np.array(out)
    assert np.array_equal(walk(False), walk(True)) and np.array_equal(walk(True), walk(False))
    ref = P.forward(cfg, w, t)
    assert rel(bf16_view(walk(True)[-1])[None], ref[-1:])[0] < TOL["bfloat16"]
    m.close()


@pytest.mark.parametrize("n", [9, 60, 70])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_many_slots_decode_together(n, dtype):
    """decode batches past the sizes the streaming products take; a third of the slots parked"""
    model = M.model(64, 60, 1e-6, [M.parallel((2, 1, 32, 32), 6, 0.5, (2, 16, 24), (0.6, 0.99), 1.0, 0.8, 48), M.delta(2, 2, 16, 32, 3, 6, 6)])
    cfg = model[0]
    m, w = make(model, dtype, 40)
    s = Seqs(m, w, cfg, n)
    for i in range(n):
        s.open("s%d" % i, M.tokens(cfg, 14, i))
    s.feed({"s%d" % i: 5 + i % 4 for i in range(n)})
    for _ in range(5):
        s.feed({"s%d" % i: 1 for i in range(n)})
    s.feed({"s%d" % i: 1 for i in range(n) if i % 3 and len(s.tok["s%d" % i][1])})
    s.x.close()
    m.close()


def test_sampler_draws_through_the_framework():
    cfg = M.MODELS["mixed"][0]
    m, w = make("mixed")
    p = M.tokens(cfg, 12, 31)
    m.set_sampler(temperature=0.8, top_p=0.9, top_k=20, seed=9, true_topk=True)
    a = m.generate(p, 16)
    m.set_sampler(temperature=0.8, top_p=0.9, top_k=20, seed=9, true_topk=True)
    assert a == m.generate(p, 16) and len(a) == 16
    seq = list(p)
    for i in a:     # every drawn id is among the 20 best of the plain model's logits there
        assert i in np.argsort(-P.forward(cfg, w, seq)[-1])[:21]
        seq.append(i)
    m.close()


def test_a_prompt_longer_than_a_pass_and_a_full_context():
    cfg = M.MODELS["mixed"][0]
    m, w = make("mixed", max_seq=90)
    m.set_prefill_mode(1, 16)                           # passes of 16 rows
    s = Seqs(m, w, cfg, 2)
    s.open("a", M.tokens(cfg, 90, 1)), s.open("b", M.tokens(cfg, 41, 2))
    s.feed({"a": 70, "b": 41})
    s.feed({"a": 20})
    p = M.tokens(cfg, 80, 3)
    assert m.generate(p, 11) == P.greedy(cfg, w, p, 11)
    with pytest.raises(L.KFError):
        s.x.run([(0, 89, [1, 1])], [])
    m.close()


def test_missing_or_misshapen_tensors_are_refused(tmp_path):
    from koifish_amd.runtime import Bolopel
    cfg, w = M.MODELS["odd"][0], M.weights("odd")
    m = Bolopel(cfg, "bfloat16", 64, shapes=M.shapes("odd"))
    assert m.tensors() == {k: (v.shape[0], v.shape[1] if v.dim() > 1 else 1) for k, v in w.items()}
    m.close()
    for edit, word in ((lambda d: d.pop("l0.mix.A_log"), "l0.mix.A_log"), (lambda d: d.pop("l0.mix.a1"), "l0.mix.a1"), (lambda d: d.update({"l0.mix.a2": d["l0.mix.a2"][:, :2]}), "l0.mix.a2")):
        d = dict(w)
        edit(d)
        M.write_dir(tmp_path, cfg, d)
        with pytest.raises(L.KFError, match=word):
            Bolopel.from_dir(tmp_path)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_from_a_checkpoint(tmp_path, dtype):
    """bin/trace_run on a directory written here: two batches, prompts of unequal length, decoding, an early end"""
    cfg, w = M.MODELS["odd"][0], M.weights("odd", 2)
    M.write_dir(tmp_path / "model", cfg, w)
    seqs = {"u": M.tokens(cfg, 45, 1).tolist(), "v": M.tokens(cfg, 9, 2).tolist(), "w": M.tokens(cfg, 3, 3).tolist()}
    ref = {k: P.forward(cfg, M.arrays(w), v) for k, v in seqs.items()}
    cuts = [("u", 36), ("v", 5)], [("v", 1), ("u", 1)], [("u", 1), ("v", 1)], [("v", 1), ("u", 1)], [("u", 1), ("v", 1)], [("u", 1)], [("w", 3)]
    at, lines, want = {k: 0 for k in seqs}, [], []
    for i, c in enumerate(cuts):
        entries, rows, end = [], [], []
        for k, n in c:
            entries.append({"id": k, "tokens": seqs[k][at[k]:at[k] + n], "want": [n - 1] + ([0] if n > 1 else [])})
            rows += [ref[k][at[k] + j] for j in entries[-1]["want"]]
            at[k] += n
            if at[k] == len(seqs[k]) or (k == "u" and i == 5):
                end.append(k)
        lines.append(json.dumps({"step": i, "entries": entries, "end": end}))
        want.append(np.array(rows))
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", dtype, "--out", str(out), "--max-tokens", "50"], input="\n".join(lines) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    for i, ref_rows in enumerate(want):
        got = np.fromfile(out / ("%d.f32" % i), dtype="<f4").reshape(ref_rows.shape)
        assert rel(got, ref_rows).max() < TOL[dtype], i
