"""The recurrent row-batch operators and the variants of attention and norm that came with them (include/kf_rb.h), each alone, against plain_bolopel.py in float64."""
import ctypes as C

import numpy as np
import pytest
import torch

import plain_bolopel as P
from koifish_amd import lib as L
from test_gpu_rows import TYPES, dev, f64, pad, stored, up

pytestmark = pytest.mark.gpu


@pytest.fixture(params=list(TYPES))
def kind(request):
    return TYPES[request.param]


def store_type(a, dt):
    return f64(torch.as_tensor(a).to(dt))


@pytest.mark.parametrize("dim,n", [(64, 3), (75, 5), (200, 1), (1000, 2), (5000, 2)])
def test_norm_rows(ctx, kind, dim, n):
    typ, dt, tol = kind
    ld, g = up(dim), torch.Generator().manual_seed(dim)
    w = pad(dev(torch.rand(1, dim, generator=g) + 0.5, dt), 1, ld)
    z, add = pad(dev(torch.randn(n, dim, generator=g) + 3.0), n, ld), pad(dev(torch.randn(n, dim, generator=g)), n, ld)
    z[:, dim:] = 9.0                                                       # whatever the pad columns hold
    zz, ww = f64(z)[:, :dim], f64(w)[0, :dim]
    norms = {L.RB_LAYER: lambda v: P.layer_norm(v, ww, 1e-5), L.RB_RMS: lambda v: P.by_rms(v, 1e-5) * ww}
    hi, lo = np.zeros((4, ld // 2, 2), dtype=np.float32), np.zeros((64, ld // 2, 2), dtype=np.float32)
    assert ctx.hip.kf_rb_sinusoid_tables_host(hi.ctypes.data_as(C.c_void_p), lo.ctypes.data_as(C.c_void_p), 256, dim, ld, 10000.0) == 0
    hi, lo = dev(hi), dev(lo)
    pos = np.array([0, 63, 64, 200, 131])[:n]
    meta = dev(np.stack([pos] * 4, 1), torch.int32)
    for k, fn in norms.items():
        x, h = torch.full((n, ld), 7.0, device="cuda"), torch.full((n, ld), 7.0, dtype=dt, device="cuda")
        a = L.RbNorming(z=z.data_ptr(), w=w.data_ptr(), x_out=x.data_ptr(), h_out=h.data_ptr(), ld=ld, type=typ, kind=k, dim=dim, n=n, eps=1e-5)
        L.check(ctx.hip.kf_rb_norm_rows(ctx.h, C.byref(a)))
        assert np.abs(f64(x)[:, :dim] - fn(zz)).max() < 2e-5 and not f64(x)[:, dim:].any() and np.abs(f64(h)[:, :dim] - fn(zz)).max() < tol * 8
        r = add.clone()                                                    # added to the residual, in place
        a.add = a.x_out = r.data_ptr()
        L.check(ctx.hip.kf_rb_norm_rows(ctx.h, C.byref(a)))
        assert np.abs(f64(r)[:, :dim] - (f64(add)[:, :dim] + fn(zz))).max() < 2e-5
        a.add, a.x_out, a.pos_hi, a.pos_lo, a.meta = None, x.data_ptr(), hi.data_ptr(), lo.data_ptr(), meta.data_ptr()
        L.check(ctx.hip.kf_rb_norm_rows(ctx.h, C.byref(a)))
        assert np.abs(f64(x)[:, :dim] - fn(zz + P.sinusoid(pos, dim))).max() < 2e-5
        rows = torch.tensor([n - 1, 0], dtype=torch.int32, device="cuda")
        h2 = torch.zeros(2, ld, dtype=dt, device="cuda")
        a = L.RbNorming(z=z.data_ptr(), w=w.data_ptr(), rows=rows.data_ptr(), h_out=h2.data_ptr(), ld=ld, type=typ, kind=k, dim=dim, n=2, eps=1e-5)
        L.check(ctx.hip.kf_rb_norm_rows(ctx.h, C.byref(a)))
        assert np.abs(f64(h2)[:, :dim] - fn(zz)[[n - 1, 0]]).max() < tol * 8


@pytest.mark.parametrize("n", [1, 20, 70, 300])
def test_product_with_activated_columns(ctx, kind, n):
    typ, dt, tol = kind
    m, k, lo, hi = 192, 128, 37, 150
    w, x = dev(torch.randn(m, k) / k ** 0.5, dt), dev(torch.randn(n, k), dt)
    y, ws = torch.zeros(n, m, dtype=dt, device="cuda"), stored(w)
    p = L.RbProduct(ws.data_ptr(), x.data_ptr(), y.data_ptr(), None, k, m, 0, typ, m, k, n, L.RB_STORE, L.RB_SILU, L.RB_ALL, 0.0, None)
    p.act_lo, p.act_hi = lo, hi
    L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
    ref = f64(x) @ f64(w).T
    ref[:, lo:hi] = P.silu(ref[:, lo:hi])
    assert np.abs(f64(y) - ref).max() < tol * 4
    p.act_hi = m + 1
    assert ctx.hip.kf_rb_linear(ctx.h, C.byref(p)) < 0


class Layer:
    """a layer with n_slots states: sequences' raw rows in, outputs out; the reference keeps every sequence's whole raw history (a subclass builds the operator's struct and the reference)"""

    def __init__(self, ctx, kind, cols, n_slots, seed):
        self.ctx, (self.typ, self.dt, _) = ctx, kind
        self.cols, self.ldraw, self.n_slots, self.hist = cols, up(cols), n_slots, {}
        self.rng = np.random.default_rng(seed)

    def new(self, slot):
        self.hist[slot] = np.zeros((0, self.cols))

    def rows(self, n):
        return store_type(self.rng.normal(size=(n, self.cols)), self.dt)

    def batch(self, parts, decode):
        """the fed rows as launch()'s arguments"""
        order = list(parts) if not decode else list(range(self.n_slots))
        raw, meta, seqs, r0 = [], [], [], {}
        for s in order:
            if s not in parts:   # a decode batch has a row for every slot
                raw.append(np.zeros((1, self.cols)))
                meta.append([-1, s, 0, 0])
                continue
            pos0, x = len(self.hist[s]), parts[s]
            self.hist[s] = np.concatenate([self.hist[s], x])
            r0[s] = len(meta)
            seqs.append([len(meta), len(x), pos0, s])
            raw.append(x)
            meta += [[pos0 + t, s, pos0, pos0 + len(x) - 1] for t in range(len(x))]
        n, seqs = len(meta), np.array(seqs)
        raw = pad(dev(np.concatenate(raw), self.dt), n, self.ldraw)
        out = torch.full((n, up(self.out_cols)), 7.0, dtype=self.dt, device="cuda")
        self.r0 = r0
        return raw, out, dev(np.array(meta), torch.int32), n, None if decode else dev(seqs, torch.int32), len(seqs), int(seqs[:, 1].max()), max(len(self.hist[s]) for s in parts) - 1

    def feed(self, parts, decode=False):
        """parts: {slot: raw rows}; returns {slot: (got, reference)} for the fed rows"""
        args = self.batch(parts, decode)
        self.launch(*args)
        return self.compare(parts, args[1])

    def compare(self, parts, out):
        got, r0 = f64(out), self.r0
        assert (got[:, self.out_cols:] == 7.0).all()
        return {s: (got[r0[s]:r0[s] + len(x), :self.out_cols], self.reference(s)[-len(x):]) for s, x in parts.items()}

    def check(self, parts, decode=False, results=None):
        tol = 5e-5 if self.typ == L.F32 else 0.04
        for s, (a, b) in (results or self.feed(parts, decode)).items():
            err = np.abs(a - b).max(axis=1)
            assert err.max() < tol * max(1.0, np.abs(b).max()), (s, int(err.argmax()), err.max(), decode)


class Delta(Layer):
    def __init__(self, ctx, kind, H, G, D, V, taps, ra, rg, n_slots=3, seed=0, decay=None):
        self.s = (H, G, D, V, taps, ra, rg)
        qd, vd = G * D, H * V
        self.ch = 2 * qd + vd
        col_a = up(self.ch)
        col_g = col_a + up(ra)
        super().__init__(ctx, kind, col_g + up(rg) + H, n_slots, seed)
        self.ldraw, self.out_cols = up(self.cols), vd
        g = torch.Generator().manual_seed(seed)
        t = lambda *shape: torch.randn(shape, generator=g)
        w = dict(conv=t(self.ch, taps) / taps ** 0.5, a2=t(H * D, ra) / ra ** 0.5, g2=t(vd, rg) / rg ** 0.5, A_log=t(H) - 0.5, dt_bias=2.5 * t(H * D) - 3.0 if decay is None else torch.full((H * D,), decay), norm=1 + 0.2 * t(V))
        self.w = {k: dev(v, self.dt) for k, v in w.items()}
        self.wa, self.wg = pad(self.w["a2"], up(H * D), up(ra)), pad(self.w["g2"], up(vd), up(rg))
        self.was, self.wgs = stored(self.wa), stored(self.wg)
        vs = (V + 3) // 4 * 4
        self.state = torch.full((n_slots * 2 * H * D * vs,), 3.0, device="cuda")
        if V % 4:
            self.state.zero_()                                             # pad columns hold zeros
        hist_slot = (taps * self.ch + 7) // 8 * 8
        self.hbuf = torch.full((n_slots * hist_slot,), 5.0, dtype=self.dt, device="cuda")
        self.a = L.RbDelta(conv=self.w["conv"].data_ptr(), w_a2=self.was.data_ptr(), w_g2=self.wgs.data_ptr(), a_log=self.w["A_log"].data_ptr(), dt_bias=self.w["dt_bias"].data_ptr(),
                           norm_w=self.w["norm"].data_ptr(), state=self.state.data_ptr(), hist=self.hbuf.data_ptr(), ldraw=self.ldraw, ldout=up(vd), hist_slot=hist_slot, type=self.typ, n_head=H, n_kv=G, dim=D,
                           vdim=V, taps=taps, col_b=col_g + up(rg), col_a=col_a, col_g=col_g, rank_a=ra, rank_g=rg, ld_a=up(ra), ld_g=up(rg), q_scale=D ** -0.5, unit_eps=1e-6, eps=1e-5)

    def rows(self, n):
        x = self.rng.normal(size=(n, self.cols))
        H, G, D, V, taps, ra, rg = self.s
        a = self.a
        x[:, self.ch:a.col_a] = x[:, a.col_a + ra:a.col_g] = x[:, a.col_g + rg:a.col_b] = 0.0
        return store_type(x, self.dt)

    def launch(self, raw, out, meta, n, seqs, n_seq, max_n, top):
        H, G, D, V, taps, ra, rg = self.s
        self.a.raw, self.a.out = raw.data_ptr(), out.data_ptr()
        if seqs is None:
            L.check(self.ctx.hip.kf_rb_delta_decode(self.ctx.h, C.byref(self.a), meta.data_ptr(), n))
            return
        az, gz = (raw[:, self.a.col_a:self.a.col_a + up(ra)].float() @ self.wa.float().T).contiguous(), (raw[:, self.a.col_g:self.a.col_g + up(rg)].float() @ self.wg.float().T).to(self.dt).contiguous()
        sc = torch.full((self.ctx.hip.kf_rb_delta_scratch(self.typ, n, n_seq, H, G, D, V) // 4,), 9.0, device="cuda")
        self.a.a_z, self.a.g_z, self.a.ld_az, self.a.ld_gz, self.a.scratch = az.data_ptr(), gz.data_ptr(), az.shape[1], gz.shape[1], sc.data_ptr()
        L.check(self.ctx.hip.kf_rb_delta_prefill(self.ctx.h, C.byref(self.a), meta.data_ptr(), n, seqs.data_ptr(), n_seq, max_n))
        self.ctx.sync()

    def reference(self, slot):
        H, G, D, V, taps, ra, rg = self.s
        r, a, w = self.hist[slot], self.a, {k: f64(v) for k, v in self.w.items()}
        T = len(r)
        y = P.silu(P.short_conv(r[:, :self.ch], w["conv"].reshape(self.ch, taps)))
        q, k, v = P.unit(y[:, :G * D].reshape(T, G, D)) * D ** -0.5, P.unit(y[:, G * D:2 * G * D].reshape(T, G, D)), y[:, 2 * G * D:].reshape(T, H, V)
        z = r[:, a.col_a:a.col_a + ra] @ w["a2"].T + w["dt_bias"]
        g = np.exp(-np.exp(w["A_log"])[None, :, None] * P.softplus(z).reshape(T, H, D))
        beta = P.sigmoid(r[:, a.col_b:a.col_b + H])
        o = np.stack([P.delta_rule(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], g[:, h], beta[:, h])[0] for h in range(H)], axis=1)
        return (P.by_rms(o, 1e-5) * w["norm"]).reshape(T, H * V) * P.sigmoid(r[:, a.col_g:a.col_g + rg] @ w["g2"].T)


class Decay(Layer):
    def __init__(self, ctx, kind, H, D, V, decay, n_slots=3, seed=0):
        self.s = (H, D, V)
        super().__init__(ctx, kind, 8 + 2 * H * D + H * V + H * V, n_slots, seed)
        self.out_cols, self.lam = H * V, np.asarray(decay, dtype=np.float32)
        self.nw, self.dec = dev(1 + 0.2 * torch.randn(H * V, generator=torch.Generator().manual_seed(seed)), self.dt), dev(self.lam)
        vs = (V + 3) // 4 * 4
        self.state = torch.full((n_slots * 2 * H * D * vs,), 3.0, device="cuda")
        if V % 4:
            self.state.zero_()
        self.a = L.RbDecay(norm_w=self.nw.data_ptr(), decay=self.dec.data_ptr(), state=self.state.data_ptr(), ldraw=self.ldraw, ldout=up(H * V), type=self.typ, n_head=H, dim=D, vdim=V, col_q=8,
                           col_g=8 + 2 * H * D + H * V, out_scale=0.7, eps=1e-5)
        self.step_scratch = torch.zeros(ctx.hip.kf_rb_decay_scratch(self.typ, n_slots, n_slots, H, D, V) // 4, device="cuda")   # zeroed once: its counters come back to zero

    def launch(self, raw, out, meta, n, seqs, n_seq, max_n, top):
        self.a.raw, self.a.out = raw.data_ptr(), out.data_ptr()
        if seqs is None:
            self.a.scratch = self.step_scratch.data_ptr()
            L.check(self.ctx.hip.kf_rb_decay_decode(self.ctx.h, C.byref(self.a), meta.data_ptr(), n))
            return
        sc = torch.zeros(self.ctx.hip.kf_rb_decay_scratch(self.typ, n, n_seq, *self.s) // 4, device="cuda")
        self.a.scratch = sc.data_ptr()
        L.check(self.ctx.hip.kf_rb_decay_prefill(self.ctx.h, C.byref(self.a), meta.data_ptr(), n, seqs.data_ptr(), n_seq, max_n))
        self.ctx.sync()

    def reference(self, slot):
        H, D, V = self.s
        r = self.hist[slot]
        q, k, v, g = r[:, 8:8 + H * D].reshape(-1, H, D), r[:, 8 + H * D:8 + 2 * H * D].reshape(-1, H, D), r[:, 8 + 2 * H * D:8 + 2 * H * D + H * V].reshape(-1, H, V), r[:, -H * V:]
        o = np.concatenate([P.decayed_sum(q[:, h], k[:, h], v[:, h], float(self.lam[h]))[0] for h in range(H)], axis=1)
        return 0.7 * P.by_rms(o, 1e-5) * f64(self.nw) * P.sigmoid(g)


def schedule(a):
    """prompts past chunk borders, portions down to two tokens, single tokens in both forms, unequal sequences in one batch, a slot used again, long decoding"""
    for s in range(3):
        a.new(s)
    a.check({1: a.rows(77)})
    a.check({0: a.rows(200), 2: a.rows(3), 1: a.rows(2)})
    a.check({2: a.rows(21), 1: a.rows(64), 0: a.rows(1)})
    a.check({2: a.rows(63), 1: a.rows(65), 0: a.rows(128)})
    for n in (2, 5, 2):
        a.check({2: a.rows(n), 0: a.rows(n + 1)})
    for i in range(9):
        a.check({s: a.rows(1) for s in ((0, 1, 2) if i % 3 else (2,))}, decode=True)
    a.check({1: a.rows(30)})
    a.new(1)                                   # the slot goes to another sequence; its state and last inputs are still the old one's
    a.check({1: a.rows(5)})
    a.new(2)
    a.check({2: a.rows(1), 1: a.rows(1)}, decode=True)
    for _ in range(25):
        a.check({1: a.rows(1), 2: a.rows(1)}, decode=True)


DELTAS = [(2, 1, 32, 48, 4, 10, 20), (4, 4, 64, 64, 4, 16, 16), (2, 2, 128, 128, 4, 128, 128), (3, 1, 18, 21, 1, 5, 7), (1, 1, 1, 1, 2, 1, 1), (2, 1, 256, 64, 3, 70, 9), (2, 1, 64, 256, 4, 33, 64),
          (6, 2, 16, 4, 9, 8, 8), (2, 1, 128, 32, 4, 64, 64), (1, 1, 320, 264, 4, 16, 16), (2, 2, 96, 80, 2, 24, 24)]


@pytest.mark.parametrize("shape", DELTAS, ids=lambda s: "x".join(map(str, s)))
def test_delta_prompts_portions_and_decoding(ctx, kind, shape):
    schedule(Delta(ctx, kind, *shape))


@pytest.mark.parametrize("decay", [-14.0, 4.0])
def test_delta_with_hardly_any_and_nearly_total_decay(ctx, kind, decay):
    """a state that keeps everything over hundreds of tokens; decays whose products over a chunk are far below the smallest float"""
    a = Delta(ctx, kind, 2, 2, 64, 64, 4, 16, 16, decay=decay, seed=3)
    a.new(0)
    a.check({0: a.rows(333)})
    a.check({0: a.rows(70)})
    for _ in range(5):
        a.check({0: a.rows(1)}, decode=True)


@pytest.mark.parametrize("form", ["prompt", "portions", "decode"])
def test_delta_reads_a_far_write(ctx, kind, form):
    """one marked key, written once and asked for 150 tokens later; the others' keys are kept orthogonal to it, so the read shows the write or nothing"""
    a = Delta(ctx, kind, 1, 1, 64, 64, 1, 16, 16, decay=-14.0, seed=4)
    x = a.rows(200)
    x[:, 63] = x[:, 127] = -30.0                # channel 63 of q and k: silu(-30 w) is about 0 where the tap is positive
    with torch.no_grad():
        a.w["conv"].abs_()
    x[7, 64:128], x[7, 127] = -30.0, 20.0       # the write
    x[7, 128:192] *= 5.0
    x[157, 0:64], x[157, 63] = -30.0, 20.0      # the read
    x = store_type(x, a.dt)
    a.new(0)
    if form == "prompt":
        a.check({0: x})
    elif form == "portions":
        for i in range(0, 200, 23):
            a.check({0: x[i:i + 23]})
    else:
        for i in range(200):
            if i < 150:
                a.feed({0: x[i:i + 1]}, decode=True) if i in (0,) else a.hist.__setitem__(0, np.concatenate([a.hist[0], x[i:i + 1]])) or a_step(a, x[i:i + 1], i)
            else:
                a.check({0: x[i:i + 1]}, decode=True)
    r = a.reference(0)
    x2 = x.copy()
    x2[7, 128:192] = 0.1
    a.hist[0] = x2
    assert np.abs(a.reference(0)[157] - r[157]).max() > 0.3


def a_step(a, row, pos):
    """a decode step without its reference (which walks the whole history)"""
    raw = pad(dev(np.concatenate([row] + [np.zeros((1, a.cols))] * (a.n_slots - 1)), a.dt), a.n_slots, a.ldraw)
    out = torch.zeros(a.n_slots, up(a.out_cols), dtype=a.dt, device="cuda")
    a.launch(raw, out, dev(np.array([[pos, 0, pos, pos]] + [[-1, s, 0, 0] for s in range(1, a.n_slots)]), torch.int32), a.n_slots, None, 1, 1, pos)
    a.ctx.sync()


DECAYS = [(3, 20, 36, (0.5, 0.9, 0.999)), (2, 64, 64, (0.8, 0.97)), (2, 128, 128, (0.95, 1.0)), (1, 9, 14, (0.3,)), (1, 128, 1, (1.0,)), (2, 256, 128, (0.05, 0.99)), (4, 64, 128, (0.1, 0.6, 0.98, 0.9995)),
          (2, 32, 256, (0.9, 0.0)), (1, 264, 300, (0.97,)), (3, 48, 40, (0.9, 0.99, 0.5))]


@pytest.mark.parametrize("shape", DECAYS, ids=lambda s: "x".join(map(str, s[:3])))
def test_decayed_sum_prompts_portions_and_decoding(ctx, kind, shape):
    schedule(Decay(ctx, kind, *shape))


def test_decayed_sum_reads_a_far_write(ctx, kind):
    a = Decay(ctx, kind, 1, 64, 64, (1.0,), seed=5)
    x = a.rows(400)
    x[:, 8 + 63] = x[:, 8 + 64 + 63] = 0.0      # channel 63 of q and k belongs to the marked pair
    x[5, 8 + 64 + 63], x[5, 136:200] = 8.0, 6.0 * x[5, 136:200]
    x[390, 8:72], x[390, 8 + 63] = 0.0, 4.0
    x = store_type(x, a.dt)
    a.new(0)
    for i in (0, 130, 260):
        a.check({0: x[i:min(i + 130, 389)]})
    a.check({0: x[389:390]}, decode=True)
    a.check({0: x[390:391]}, decode=True)
    a.check({0: x[391:]})


def test_refusals(ctx):
    a = Delta(ctx, TYPES["f32"], 2, 1, 32, 48, 4, 10, 20)
    raw, out, meta = torch.zeros(3, a.ldraw, device="cuda"), torch.zeros(3, 128, device="cuda"), torch.zeros(3, 4, dtype=torch.int32, device="cuda")
    a.a.raw, a.a.out = raw.data_ptr(), out.data_ptr()
    for k, v in (("dim", 600), ("n_kv", 3), ("taps", 0), ("col_b", 10), ("state", None), ("ld_a", 32), ("rank_g", 0), ("type", L.Q4)):
        old = getattr(a.a, k)
        setattr(a.a, k, v)
        assert ctx.hip.kf_rb_delta_decode(ctx.h, C.byref(a.a), meta.data_ptr(), 3) < 0, k
        setattr(a.a, k, old)
    assert ctx.hip.kf_rb_delta_prefill(ctx.h, C.byref(a.a), meta.data_ptr(), 3, None, 1, 3) < 0
    d = Decay(ctx, TYPES["f32"], 1, 9, 14, (0.3,))
    d.a.raw, d.a.out, d.a.scratch = raw.data_ptr(), out.data_ptr(), d.step_scratch.data_ptr()
    for k, v in (("dim", 513), ("decay", None), ("col_g", 10000), ("ldout", 8), ("vdim", 0)):
        old = getattr(d.a, k)
        setattr(d.a, k, v)
        assert ctx.hip.kf_rb_decay_decode(ctx.h, C.byref(d.a), meta.data_ptr(), 3) < 0, k
        setattr(d.a, k, old)


# ---- attention with values of their own, a window, unit q and k, a sink, a scale on the output
class Window(Layer):
    def __init__(self, ctx, kind, H, G, D, V, window, scale, sink=1, n_slots=3, n_ctx=640, seed=0):
        self.s = (H, G, D, V, window, scale, sink)
        v_col = up((H + G) * D, 8)
        super().__init__(ctx, kind, v_col + G * V, n_slots, seed)
        self.out_cols = H * V
        rows = min(window, n_ctx)
        hs = rows * max(D, V) + 40
        hs = (hs + 7) // 8 * 8
        self.kc, self.vc = (torch.full((n_slots * hs * G,), float("nan"), dtype=self.dt, device="cuda") for _ in range(2))   # a key that nobody wrote would show
        self.kc.nan_to_num_(2.0), self.vc.nan_to_num_(50.0)
        self.a = L.RbAttention(type=self.typ, n_head=H, n_kv=G, dim=D, cache_rows=rows, scale=scale, eps=1e-5, k_cache=self.kc.data_ptr(), v_cache=self.vc.data_ptr(), ldraw=self.ldraw, ldout=up(H * V),
                               slot_stride=hs * G, head_stride=hs, v_col=v_col, vdim=V, unit=1, window=window, sink=sink, scaled=1, out_scale=0.6)

    def launch(self, raw, out, meta, n, seqs, n_seq, max_n, top):
        H, G, D = self.s[:3]
        knew = torch.zeros(n, G * D, dtype=self.dt, device="cuda")
        sc = torch.zeros(self.ctx.hip.kf_rb_attention_scratch(n, H, self.s[3]) // 4, device="cuda")
        self.a.raw, self.a.out, self.a.k_new, self.a.scratch = raw.data_ptr(), out.data_ptr(), knew.data_ptr(), sc.data_ptr()
        if seqs is None:
            L.check(self.ctx.hip.kf_rb_attention_decode(self.ctx.h, C.byref(self.a), meta.data_ptr(), n, top))
        else:
            L.check(self.ctx.hip.kf_rb_attention_prefill(self.ctx.h, C.byref(self.a), meta.data_ptr(), n, seqs.data_ptr(), n_seq, max_n))
        self.ctx.sync()

    def reference(self, slot):
        H, G, D, V, window, scale, sink = self.s
        r, c = self.hist[slot], self.a.v_col
        q, k, v = r[:, :H * D].reshape(-1, H, D), r[:, H * D:(H + G) * D].reshape(-1, G, D), r[:, c:c + G * V].reshape(-1, G, V)
        full = P.softmax_with_sink
        if not sink:
            P.softmax_with_sink = lambda s: np.exp(s - s.max(-1, keepdims=True)) / np.exp(s - s.max(-1, keepdims=True)).sum(-1, keepdims=True)
        try:
            return 0.6 * P.attend(q, k, v, scale, window, 1e-5)
        finally:
            P.softmax_with_sink = full


WINDOWS = [(4, 2, 64, 64, 24, 0.1), (6, 1, 32, 16, 100, 0.3), (5, 5, 48, 80, 7, 0.2), (40, 1, 16, 32, 40, 0.5), (8, 2, 128, 64, 200, 0.05), (2, 1, 64, 192, 33, 0.1), (2, 2, 256, 256, 1, 0.02),
           (3, 1, 20, 9, 16, 0.3), (2, 1, 100, 30, 600, 0.1), (4, 1, 128, 128, 400, 0.12)]


@pytest.mark.parametrize("shape", WINDOWS, ids=lambda s: "x".join(map(str, s[:5])))
def test_window_attention_prompts_portions_and_decoding(ctx, kind, shape):
    schedule(Window(ctx, kind, *shape))


@pytest.mark.parametrize("sink", [0, 1])
@pytest.mark.parametrize("scale", [-0.5, 0.4])
def test_window_attention_scores_far_below_and_above_the_sink(ctx, kind, scale, sink):
    """long prompts of one sequence take two walks per column: their maxima meet the sink's score of 0.  Scores of both signs, peaked"""
    a = Window(ctx, kind, 2, 1, 64, 64, 90, scale, sink, seed=6)
    a.new(0)
    x = a.rows(420)
    x[:, 128:192] = x[:, 128:192] * 0.2 + 1.0   # keys that point one way, and queries that follow them
    x[:, :128] = x[:, :128] * 0.5 + 1.0
    a.check({0: store_type(x, a.dt)})
    for _ in range(4):
        a.check({0: store_type(x[:1], a.dt)}, decode=True)


@pytest.mark.parametrize("how", ["prompt", "portions", "decode"])
@pytest.mark.parametrize("window", [20, 64, 150])
def test_window_edges(ctx, kind, window, how):
    """a marked key outshines the rest: every row that sees it, and the first that does not"""
    a = Window(ctx, kind, 2, 1, 32, 32, window, 0.9, seed=7)
    for at in (0, 31, 64):
        n = at + window + 40
        x = a.rows(n)
        x[:, 31] = x[:, 63] = 6.0               # both heads look along dimension 31
        x[:, 95] = -1.0
        x[at, 64:96], x[at, 95] = 0.1, 8.0
        x[at, a.a.v_col:a.a.v_col + 32] += 3.0
        x = store_type(x, a.dt)
        a.new(0)
        if how == "prompt":
            a.check({0: x})
        elif how == "portions":
            i = 0
            for k in (at + 1, 2, 3, window - 7, 2, 2, 36):
                a.check({0: x[i:i + k]})
                i += k
        else:
            a.check({0: x[:at + window - 3]})
            for i in range(at + window - 3, at + window + 4):
                a.check({0: x[i:i + 1]}, decode=True)
        r = a.reference(0)
        e = a.hist[0].copy()
        e[at, a.a.v_col:a.a.v_col + 32] -= 6.0
        a.hist[0] = e
        d = np.abs(a.reference(0) - r).max(1)
        hi = min(at + window, len(d))
        assert (d[at:hi] > 0.5).all() and (d[at + window:] < 1e-12).all()


@pytest.mark.parametrize("sizes", [(3, (4, 2, 64, 64, 300, 0.1), (4, 64, 128, (0.1, 0.6, 0.98, 0.9995))), (3, (16, 2, 128, 128, 90, 0.08), (2, 128, 128, (0.95, 0.998))), (3, (2, 1, 64, 48, 24, 0.2), (1, 264, 300, (0.97,))),
                                   (24, (4, 1, 32, 64, 50, 0.1), (2, 64, 64, (0.8, 0.97)))], ids=["wide", "heads", "apart", "many"])
def test_attention_and_decayed_sum_in_one_launch(ctx, kind, sizes):
    n, w, d = sizes
    a, b = Window(ctx, kind, *w, n_slots=n), Decay(ctx, kind, *d, n_slots=n)
    for s in range(n):
        a.new(s), b.new(s)
    lens = {s: 5 + 7 * s for s in range(n) if s != 1}
    a.check({s: a.rows(k) for s, k in lens.items()}), b.check({s: b.rows(k) for s, k in lens.items()})
    for i in range(6):
        on = [s for s in range(n) if (s + i) % 3]
        pa, pb = {s: a.rows(1) for s in on}, {s: b.rows(1) for s in on}
        ra, rb = a.batch(pa, True), b.batch(pb, True)
        sc = torch.zeros(ctx.hip.kf_rb_attention_scratch(n, w[0], w[3]) // 4, device="cuda")
        a.a.raw, a.a.out, a.a.scratch = ra[0].data_ptr(), ra[1].data_ptr(), sc.data_ptr()
        b.a.raw, b.a.out, b.a.scratch = rb[0].data_ptr(), rb[1].data_ptr(), b.step_scratch.data_ptr()
        L.check(ctx.hip.kf_rb_attention_decay_decode(ctx.h, C.byref(a.a), C.byref(b.a), ra[2].data_ptr(), n, ra[7]))
        ctx.sync()
        a.check(pa, results=a.compare(pa, ra[1])), b.check(pb, results=b.compare(pb, rb[1]))
