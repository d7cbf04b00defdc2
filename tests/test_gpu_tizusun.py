"""Tizusun through the framework -- loader, step, slots, queue, sampler, trace replay -- against the plain float64 statement (plain_tizusun.py) on small models of our own."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import layered_helpers
import plain_tizusun as P
import tizusun_models as M
from koifish_amd import lib as L
from layered_helpers import bf16_view, rel

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# relative rms error of a row of logits.  bf16: the roundings of q, k and the products (2^-9 each) through a few layers of deliberately peaked attention; what a wrong key,
# edge or state does is an order of magnitude larger (the float32 runs of the same schedules hold 2e-4)
TOL = {"float32": 2e-4, "bfloat16": 0.1}


def make(cfg, dtype="float32", max_seq=400, seed=0, qk=1.5):
    from koifish_amd.runtime import Tizusun
    w = M.weights(cfg, seed, qk, settled=dtype == "bfloat16")
    m = Tizusun(cfg, dtype, max_seq)
    for i, (k, v) in enumerate(w.items()):
        m.set_tensor(k, v.cuda() if i % 2 else v)
    return m, M.arrays(w)


def Seqs(m, w, cfg, n=4):
    return layered_helpers.Seqs(P, m, w, cfg, TOL, n)


@pytest.fixture(scope="module", params=[(c, d) for c in M.CONFIGS for d in ("float32", "bfloat16")], ids=lambda p: p[0] + "-" + p[1])
def served(request):
    name, dtype = request.param
    m, w = make(M.CONFIGS[name], dtype)
    yield M.CONFIGS[name], m, w
    m.close()


def test_residual_stream_after_every_layer(served):
    cfg, m, w = served
    t = M.tokens(cfg, 60)
    s = Seqs(m, w, cfg, 1)
    tap = m.tap(60)
    s.open("a", t)
    s.feed({"a": 60})
    m.tap(0)
    _, ref = P.forward(cfg, w, t, True)
    err = np.abs(tap - ref).max(axis=(1, 2)) / np.abs(ref).max(axis=(1, 2))
    assert (err < (1e-4 if m.dtype == "float32" else 0.06)).all(), err


def test_prompts_portions_decoding_and_mixed_batches(served):
    cfg, m, w = served
    s = Seqs(m, w, cfg)
    s.open("a", M.tokens(cfg, 140, 1))
    s.feed({"a": 66})                                   # alone
    s.open("b", M.tokens(cfg, 110, 2))
    s.open("c", M.tokens(cfg, 50, 3))
    s.feed({"b": 79, "a": 2, "c": 1})                   # a prompt, a portion of two, a first token
    for n in (3, 2, 7):
        s.feed({"c": n, "a": n + 1})
    for _ in range(12):                                 # decoded together, then unequal ends
        s.feed({"a": 1, "b": 1, "c": 1})
    s.close("c")
    s.open("d", M.tokens(cfg, 60, 4))                   # the slot used again: its rings still hold c's rows
    s.feed({"d": 20})
    for _ in range(9):
        s.feed({"d": 1, "a": 1})
    s.feed({"b": 1, "d": 5})                            # a single token and a portion in one batch
    s.close("a"), s.close("b"), s.close("d")


def test_long_decoding_past_every_chunk(served):
    cfg, m, w = served
    n = max(L_["mixer"]["mask"]["size"] for L_ in cfg["layers"])
    n = min(2 * n + 8, 330)
    s = Seqs(m, w, cfg, 2)
    t = M.tokens(cfg, n, 7)
    s.open("p", t)
    s.open("a", t)
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
    db = np.concatenate([x.run([(1, 63 + i % 7, [5]), (2, 40 + i, t[40 + i:41 + i])], [(1, 0)]) for i in range(7)])
    tol = 1e-5 if m.dtype == "float32" else TOL["bfloat16"]   # (40 rows and 103 take different kernels: another set of bf16 roundings)
    assert rel(b, a).max() < tol and rel(db, da[:7]).max() < tol
    x.close()


@pytest.mark.parametrize("how", ["prompt", "portions", "decoded"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_chunk_edges_show_in_the_logits(dtype, how):
    """a one-layer model in which one marked token's key outshines the rest: the logits of the last position of its chunk and of the first one behind it, prompt and decoded"""
    chunk = 20
    cfg = dict(architecture="Tizusun", width=64, vocab=40, postln_alpha=0.5, norm={"eps": 1e-6}, layers=[M.layer(M.mixer(2, 1, 32, chunk, 8, scale=4.0), None)])
    m, w = make(cfg, dtype, 100, seed=5)
    raw = M.weights(cfg, 5)
    e = raw["embed"].float()
    e[:, :2] = torch.tensor([3.0, 0.0])
    e[39, :2] = torch.tensor([0.0, 9.0])                # the marked token
    q, k = raw["l0.mix.q"].float(), raw["l0.mix.k"].float()
    q[31::32], k[31] = 0.0, 0.0
    q[31::32, 0], q[31::32, 1], k[31, 1], k[31, 0] = 3.0, 1.0, 3.0, -1.0
    for n, t in (("embed", e), ("l0.mix.q", q), ("l0.mix.k", k)):
        raw[n] = t.bfloat16()
        m.set_tensor(n, raw[n])
    w = M.arrays(raw)
    for at in (0, chunk - 1, chunk, chunk + 1, 2 * chunk - 1):
        t = M.tokens(cfg, 2 * chunk + 8, at) % 39
        t[at] = 39
        s = Seqs(m, w, cfg, 1)
        s.open("a", t)
        plain = t.copy()
        plain[at] = 3
        far = P.forward(cfg, w, plain)
        d = rel(s.ref["a"], far)
        inside = [i for i in range(at + 1, len(t)) if i // chunk == at // chunk]
        assert all(d[i] > 0.3 for i in inside) and all(d[i] < 1e-9 for i in range(at + 1, len(t)) if i not in inside)
        if how == "prompt":
            s.feed({"a": len(t)})
        elif how == "portions":
            for n in ([at + 1] if at else [1]) + [2, 3]:
                s.feed({"a": n})
            s.feed({"a": len(s.tok["a"][1])})
        else:
            s.feed({"a": 1})
            for _ in range(len(t) - 1):
                s.feed({"a": 1})
        s.x.close()
    m.close()


def test_greedy_generation_matches_the_plain_model():
    cfg = M.CONFIGS["mixed"]
    m, w = make(cfg)
    p = M.tokens(cfg, 30, 21)
    want = P.greedy(cfg, w, p, 24)
    assert m.generate(p, 24, use_graph=True) == want                 # token-serial prompt, captured steps
    assert m.generate(p, 24, use_graph=False) == want
    m.set_prefill_mode(1)
    assert m.generate(p, 24, use_graph=True) == want                 # batched prompt
    assert m.num_graphs() >= 1
    nxt, lg = m.prefill(p)
    assert nxt == want[0] and int(bf16_view(lg).argmax()) >= 0
    r, lg = m.forward(int(want[0]), 30)
    assert r == want[1]
    ref = P.forward(cfg, w, list(p) + want[:1])[-1]
    assert rel(bf16_view(lg)[None], ref[None])[0] < 0.01                # kfh_logits is the bf16 view
    m.close()


def test_queue_of_prompts_through_the_slots():
    """more prompts than slots through the scheduler's queue: every answer is the plain model's; eos and per-request limits; prompts prefilled together or one by one"""
    from koifish_amd.runtime import XcdReplicas
    cfg = M.CONFIGS["mixed"]
    m, w = make(cfg)
    prompts = [M.tokens(cfg, n, 40 + n) for n in (5, 33, 1, 60, 18, 9)]
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


def test_every_replay_of_a_captured_step_equals_the_eager_one():
    from koifish_amd.runtime import XcdReplicas
    cfg = M.CONFIGS["mixed"]
    m, w = make(cfg, "bfloat16")
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
    x = XcdReplicas(m, 2)
    for s in range(2):
        x.set_state(s, int(t[s]), 0)
    x.run_steps(12)
    a = [x.tokens_out(s, 12).tolist() for s in range(2)]
    m.set_forced(np.full(400, -1))
    for s in range(2):
        m.set_state(int(t[s]), 0)
        m.run_steps(0, 12, use_graph=False)
        b = m.tokens_out(12).tolist()
        assert sum(p == q for p, q in zip(a[s], b)) >= 1    # (bf16: another batch size may round a near tie the other way)
    x.close()
    m.close()


@pytest.mark.parametrize("n", [9, 60, 70])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_many_slots_decode_together(n, dtype):
    """decode batches past the sizes the streaming products, their norms and the in-product expert sums take; a third of the slots parked"""
    cfg = dict(architecture="Tizusun", width=64, vocab=60, postln_alpha=1.2, norm={"eps": 1e-6}, layers=[M.layer(M.mixer(2, 1, 32, 12, 8), M.moe(16, 24, 20)), M.layer(M.mixer(2, 2, 32, 9, 32), M.dense(48))])
    m, w = make(cfg, dtype, 40)
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
    from koifish_amd.runtime import XcdReplicas
    cfg = M.CONFIGS["mixed"]
    m, w = make(cfg)
    p = M.tokens(cfg, 12, 31)
    m.set_sampler(temperature=0.8, top_p=0.9, top_k=20, seed=9, true_topk=True)
    a, b = m.generate(p, 16), m.generate(p, 16)
    m.set_sampler(temperature=0.8, top_p=0.9, top_k=20, seed=9, true_topk=True)
    c = m.generate(p, 16)
    assert a == c and len(a) == 16 and (a != b or len(set(a)) == 1)
    # every drawn id is among the 20 best of the plain model's logits there
    seq = list(p)
    for i in a:
        assert i in np.argsort(-P.forward(cfg, w, seq)[-1])[:21]
        seq.append(i)
    x = XcdReplicas(m, 2)
    x.set_sampler(temperature=0.8, top_p=0.9, top_k=20, seed=9, true_topk=True)
    got, _ = x.chat([p, p], 16)
    assert got[0] == a                                  # request r draws like the model alone under seed + r
    x.close()
    m.close()


def test_a_prompt_longer_than_a_pass_and_a_full_context():
    cfg = M.CONFIGS["mixed"]
    m, w = make(cfg, max_seq=90)
    m.set_prefill_mode(1, 16)                           # passes of 16 rows
    s = Seqs(m, w, cfg, 2)
    s.open("a", M.tokens(cfg, 90, 1)), s.open("b", M.tokens(cfg, 41, 2))
    s.feed({"a": 70, "b": 41})
    s.feed({"a": 20})
    p = M.tokens(cfg, 80, 3)
    assert m.generate(p, 11) == P.greedy(cfg, w, p, 11)
    with pytest.raises(L.KFError):
        s.x.run([(0, 89, [1, 1])], [])
    with pytest.raises(L.KFError):
        s.x.run([(0, 0, [cfg["vocab"]])], [])
    with pytest.raises(L.KFError):
        s.x.run([(0, 0, [1]), (0, 1, [1])], [])
    m.close()


def test_missing_or_misshapen_tensors_are_refused(tmp_path):
    from koifish_amd.runtime import Tizusun, XcdReplicas
    cfg = M.CONFIGS["odd"]
    w = M.weights(cfg)
    m = Tizusun(cfg, "bfloat16", 64)
    assert m.tensors() == {k: (v.shape[0], v.shape[1] if v.dim() > 1 else 1) for k, v in w.items()}
    with pytest.raises(L.KFError, match="has not been set"):
        XcdReplicas(m, 1)
    with pytest.raises(L.KFError):
        m.set_tensor("l0.mix.q", torch.zeros(3, 3, dtype=torch.bfloat16))
    m.close()
    for edit, word in ((lambda d: d.pop("l1.mlp.e2.up"), "l1.mlp.e2.up"), (lambda d: d.update({"head": d["head"][:5]}), "head")):
        d = dict(w)
        edit(d)
        M.write_dir(tmp_path, cfg, d)
        with pytest.raises(L.KFError, match=word):
            Tizusun.from_dir(tmp_path)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_from_a_checkpoint(tmp_path, dtype):
    """bin/trace_run on a directory written here: two batches, prompts of unequal length, decoding, an early end"""
    cfg = M.CONFIGS["mixed"]
    w = M.weights(cfg, 2, settled=dtype == "bfloat16")
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
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(len(cuts))]
    for i, ref_rows in enumerate(want):
        got = np.fromfile(out / ("%d.f32" % i), dtype="<f4").reshape(ref_rows.shape)
        assert rel(got, ref_rows).max() < TOL[dtype], i
