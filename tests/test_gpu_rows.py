"""The row-batch operators (include/kf_rb.h), each alone, against numpy float64 / the plain functions of plain_tizusun.py."""
import ctypes as C

import numpy as np
import pytest
import torch

import plain_tizusun as P
from koifish_amd import lib as L

pytestmark = pytest.mark.gpu
TYPES = {"bf16": (L.BF16, torch.bfloat16, 2.0 ** -7), "f32": (L.F32, torch.float32, 2e-5)}


def up(n, m=64):
    return (n + m - 1) // m * m


def dev(a, dt=torch.float32):
    return torch.as_tensor(a).to(dt).cuda()


def pad(t, rows, cols):
    out = torch.zeros(rows, cols, dtype=t.dtype, device="cuda")
    out[:t.shape[0], :t.shape[1]] = t
    return out


def f64(t):
    return t.double().cpu().numpy()


def ptr(t):
    return None if t is None else t.data_ptr()


def stored(w):
    """a product's weight [..., m, k] as the library stores it: bf16 in 16 x 32 tiles, piece (row r, octet q) at number 16 q + r; fp32 as it is"""
    if w.dtype != torch.bfloat16:
        return w
    m, k = w.shape[-2:]
    return w.reshape(-1, m // 16, 16, k // 32, 4, 8).permute(0, 1, 3, 4, 2, 5).contiguous().reshape(w.shape)


@pytest.fixture(params=list(TYPES))
def kind(request):
    return TYPES[request.param]


def experts_of(n, E, top, tile, w_stride=0, ids=None, weight=None):
    nt = max(1, (n * top) // tile + min(n * top, E))
    bufs = dict(tile_expert=torch.full((nt,), -7, dtype=torch.int32, device="cuda"), list=torch.full((nt * tile,), -7, dtype=torch.int32, device="cuda"),
                ids=torch.full((n * top,), -7, dtype=torch.int32, device="cuda") if ids is None else ids, weight=torch.zeros(n * top, device="cuda") if weight is None else weight)
    e = L.RbExperts(E, top, tile, nt, bufs["tile_expert"].data_ptr(), bufs["list"].data_ptr(), bufs["ids"].data_ptr(), bufs["weight"].data_ptr(), w_stride)
    return e, bufs


def route(ctx, logits, bias, n, E, top, tile, typ, meta=None, w_stride=0):
    e, b = experts_of(n, E, top, tile, w_stride)
    assert e.n_tile == ctx.hip.kf_rb_list_tiles(n, top, E, tile)
    L.check(ctx.hip.kf_rb_route(ctx.h, typ, logits.data_ptr(), logits.shape[1], ptr(bias), n, ptr(meta), C.byref(e)), "route")
    return e, b


@pytest.mark.parametrize("dim,n", [(64, 3), (75, 5), (200, 1), (1000, 2), (5000, 2)])
def test_norm(ctx, kind, dim, n):
    typ, dt, tol = kind
    ld, top = up(dim), 3
    g = torch.Generator().manual_seed(dim)
    w = pad(dev(torch.rand(1, dim, generator=g) + 0.5, dt), 1, ld)
    res, z = pad(dev(torch.randn(n, dim, generator=g)), n, ld), pad(dev(torch.randn(n * top, dim, generator=g)), n * top, ld)
    zt = z.to(dt)
    x, h = torch.full((n, ld), 7.0, device="cuda"), torch.full((n, ld), 7.0, dtype=dt, device="cuda")
    L.check(ctx.hip.kf_rb_norm(ctx.h, typ, z.data_ptr(), None, 0.0, 0, w.data_ptr(), 1e-5, dim, ld, n, None, x.data_ptr(), h.data_ptr()))
    ref = P.rms_norm(f64(z)[:n, :dim], f64(w)[0, :dim], 1e-5)
    assert np.abs(f64(x)[:, :dim] - ref).max() < 1e-5 and not f64(x)[:, dim:].any() and np.abs(f64(h)[:, :dim] - ref).max() < tol * 8
    # the sum over a row's experts on the scaled residual, in place
    r0 = f64(res)[:, :dim]
    L.check(ctx.hip.kf_rb_norm(ctx.h, typ, zt.data_ptr(), res.data_ptr(), 1.7, top, w.data_ptr(), 1e-5, dim, ld, n, None, res.data_ptr(), h.data_ptr()))
    ref = P.rms_norm(1.7 * r0 + f64(zt)[:, :dim].reshape(n, top, dim).sum(1), f64(w)[0, :dim], 1e-5)
    assert np.abs(f64(res)[:, :dim] - ref).max() < 1e-5
    # rows picked from a list
    rows = torch.tensor([n - 1, 0], dtype=torch.int32, device="cuda")
    h2 = torch.zeros(2, ld, dtype=dt, device="cuda")
    L.check(ctx.hip.kf_rb_norm(ctx.h, typ, z.data_ptr(), None, 0.0, 0, w.data_ptr(), 1e-5, dim, ld, 2, rows.data_ptr(), None, h2.data_ptr()))
    ref = P.rms_norm(f64(z)[[n - 1, 0], :dim], f64(w)[0, :dim], 1e-5)
    assert np.abs(f64(h2)[:, :dim] - ref).max() < tol * 8


@pytest.mark.parametrize("n", [1, 7, 16, 17, 40, 64, 65, 130, 333])
@pytest.mark.parametrize("m,k", [(64, 64), (192, 320), (448, 128)])
def test_product_epilogues(ctx, kind, n, m, k):
    typ, dt, tol = kind
    g = torch.Generator().manual_seed(n * m + k)
    w, x, res = dev(torch.randn(m, k, generator=g) / k ** 0.5, dt), dev(torch.randn(n, k + 8, generator=g), dt), dev(torch.randn(n, m, generator=g))
    ref, ws = f64(x)[:, :k] @ f64(w).T, stored(w)
    for epi, y in ((L.RB_STORE, torch.zeros(n, m, dtype=dt, device="cuda")), (L.RB_STORE_F32, torch.zeros(n, m, device="cuda")), (L.RB_RESIDUAL, torch.zeros(n, m, device="cuda"))):
        p = L.RbProduct(ws.data_ptr(), x.data_ptr(), y.data_ptr(), res.data_ptr(), k + 8, m, m, typ, m, k, n, epi, 0, L.RB_ALL, -0.75, None)
        L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
        want = ref + (-0.75 * f64(res) if epi == L.RB_RESIDUAL else 0)
        assert np.abs(f64(y) - want).max() < (tol * 4 if epi == L.RB_STORE else 2e-5)
    # gate / up interleaved in blocks of 16 rows
    il = f64(w).reshape(m // 32, 2, 16, k)
    gate, upw = f64(x)[:, :k] @ il[:, 0].reshape(-1, k).T, f64(x)[:, :k] @ il[:, 1].reshape(-1, k).T
    gelu = lambda z: 0.5 * z * (1 + np.tanh(np.sqrt(2 / np.pi) * (z + 0.044715 * z ** 3)))
    for act, fn in ((L.RB_RELU, P.relu), (L.RB_SILU, P.silu), (L.RB_GELU_TANH, gelu)):
        y = torch.zeros(n, m // 2, dtype=dt, device="cuda")
        p = L.RbProduct(ws.data_ptr(), x.data_ptr(), y.data_ptr(), None, k + 8, m // 2, 0, typ, m, k, n, L.RB_GATED, act, L.RB_ALL, 0.0, None)
        L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
        assert np.abs(f64(y) - fn(gate) * upw).max() < tol * 8


@pytest.mark.parametrize("n,m,k,dim", [(1, 64, 64, 50), (3, 192, 320, 300), (4, 448, 1024, 1024), (2, 256, 4096, 4090)])
def test_norm_in_front_of_a_product(ctx, n, m, k, dim):
    assert ctx.hip.kf_rb_linear_norms(L.BF16, n, k) and not ctx.hip.kf_rb_linear_norms(L.F32, n, k) and not ctx.hip.kf_rb_linear_norms(L.BF16, 5, k)
    w, z = (torch.randn(m, k, device="cuda") / k ** 0.5).bfloat16(), torch.randn(n, k, device="cuda")
    z[:, dim:] = 0.0
    g = (torch.rand(k, device="cuda") + 0.5).bfloat16()
    g[dim:] = 0.0
    # the sums of squares come from the product in front: z = 0.5 res + W0 x0 with its epilogue's partial sums
    w0, x0, res = torch.zeros(k, 64, dtype=torch.bfloat16, device="cuda"), torch.zeros(n, 64, dtype=torch.bfloat16, device="cuda"), 2.0 * z
    ssq = torch.full((k // 16, 4), 7.0, device="cuda")
    p = L.RbProduct(w0.data_ptr(), x0.data_ptr(), z.data_ptr(), res.data_ptr(), 64, k, k, L.BF16, k, 64, n, L.RB_RESIDUAL, 0, L.RB_ALL, 0.5, None, ssq.data_ptr())
    L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
    assert np.abs(f64(ssq)[:, :n] - (f64(z) ** 2).reshape(n, k // 16, 16).sum(2).T).max() < 1e-4 and (ssq[:, n:] == 7.0).all()
    il, ws = f64(w).reshape(m // 32, 2, 16, k), stored(w)
    ref = P.rms_norm(f64(z)[:, :dim], f64(g)[:dim], 1e-5)
    for epi in (L.RB_STORE, L.RB_STORE_F32, L.RB_GATED):
        x, h = torch.full((n, k), 7.0, device="cuda"), torch.full((n, k), 7.0, dtype=torch.bfloat16, device="cuda")
        y = torch.zeros(n, m, dtype=torch.float32 if epi == L.RB_STORE_F32 else torch.bfloat16, device="cuda")
        p = L.RbProduct(ws.data_ptr(), h.data_ptr(), y.data_ptr(), None, k, m, 0, L.BF16, m, k, n, epi, L.RB_SILU, L.RB_ALL, 0.0, None, None, z.data_ptr(), ssq.data_ptr(), g.data_ptr(), x.data_ptr(), 1e-5, dim)
        L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
        assert np.abs(f64(x)[:, :dim] - ref).max() < 1e-5 and not f64(x)[:, dim:].any() and torch.equal(h, x.bfloat16())
        full = f64(h) @ f64(w).T
        if epi == L.RB_GATED:
            full = P.silu(f64(h) @ il[:, 0].reshape(-1, k).T) * (f64(h) @ il[:, 1].reshape(-1, k).T)
        got = f64(y).reshape(-1)[:n * m].reshape(n, m)[:, :full.shape[1]]
        assert np.abs(got - full).max() < (2e-5 if epi == L.RB_STORE_F32 else 0.04)


def test_product_many_tiles(ctx):
    """the larger tiles of the bf16 product (256 x 256, 128 x 128, 64 x 128)"""
    for m, n, k in ((2560, 4096, 128), (2048, 2048, 64), (1024, 1500, 192)):
        w, x = (torch.randn(m, k, device="cuda") / k ** 0.5).bfloat16(), torch.randn(n, k, device="cuda").bfloat16()
        y, ws = torch.zeros(n, m, device="cuda"), stored(w)
        p = L.RbProduct(ws.data_ptr(), x.data_ptr(), y.data_ptr(), None, k, m, m, L.BF16, m, k, n, L.RB_STORE_F32, 0, L.RB_ALL, 0.0, None)
        L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
        assert (y - x.float() @ w.float().T).abs().max().item() < 1e-4


def test_product_refuses_what_it_cannot_do(ctx):
    t = torch.zeros(64, 64, device="cuda")
    ok = dict(w=t.data_ptr(), x=t.data_ptr(), y=t.data_ptr(), res=t.data_ptr(), ldx=64, ldy=64, ldr=64, type=L.F32, m=64, k=64, n=2, epilogue=L.RB_STORE, act=0, mode=L.RB_ALL, alpha=1.0)
    for bad in (dict(m=60), dict(k=32), dict(ldx=60), dict(ldy=8), dict(type=L.Q4), dict(epilogue=9), dict(mode=L.RB_UP), dict(w=None), dict(epilogue=L.RB_RESIDUAL, res=None)):
        p = L.RbProduct(**dict(ok, **bad))
        assert ctx.hip.kf_rb_linear(ctx.h, C.byref(p)) < 0, bad


@pytest.mark.parametrize("n,E,top,tile", [(1, 4, 2, 16), (5, 7, 7, 16), (3, 200, 150, 16), (40, 3, 1, 48), (200, 70, 4, 64), (700, 130, 8, 128)])
def test_route(ctx, kind, n, E, top, tile):
    typ, dt, _ = kind
    g = torch.Generator().manual_seed(n + E)
    logits = pad(dev(torch.randn(n, E, generator=g)), n, up(E))
    bias = dev(torch.randn(E, generator=g), dt)
    meta = torch.zeros(n, 4, dtype=torch.int32, device="cuda")
    off = n > 4
    if off:
        meta[2, 0] = -1
    if n > 5 and E > 3:
        logits[4, :E] = -bias.float()      # all equal: the lowest experts
    e, b = route(ctx, logits, bias, n, E, top, tile, typ, meta)
    z = f64(logits)[:, :E] + f64(bias)
    ids, wt = b["ids"].cpu().numpy().reshape(n, top), b["weight"].cpu().numpy().reshape(n, top)
    z32 = (logits[:, :E] + bias.float()).cpu().numpy()
    for t in range(n):
        if off and t == 2:
            assert (ids[t] == -1).all()
            continue
        want = np.argsort(-z32[t], kind="stable")[:top]
        assert (ids[t] == want).all() and np.abs(wt[t] - P.softmax(z[t, want])).max() < 1e-5
    te, li = b["tile_expert"].cpu().numpy(), b["list"].cpu().numpy().reshape(-1, tile)
    seen = []
    used = int((te >= 0).sum())
    assert (te[:used] >= 0).all() and (np.diff(te[:used]) >= 0).all()
    for i in range(len(te)):
        pairs = li[i][li[i] >= 0]
        assert (te[i] >= 0) == (len(pairs) > 0)
        assert (ids.reshape(-1)[pairs] == te[i]).all()
        seen += pairs.tolist()
    assert sorted(seen) == [p for p in range(n * top) if ids.reshape(-1)[p] >= 0]


@pytest.mark.parametrize("n,E,top,tile", [(1, 5, 2, 16), (9, 4, 3, 16), (33, 6, 2, 48), (64, 3, 1, 64), (150, 4, 2, 64), (500, 3, 2, 128)])
def test_experts(ctx, kind, n, E, top, tile):
    typ, dt, tol = kind
    if typ == L.F32:
        tile = 64
    C_, ff, g = 128, 64, torch.Generator().manual_seed(n)
    gu, dn = dev(torch.randn(E, 2 * ff, C_, generator=g) / C_ ** 0.5, dt), dev(torch.randn(E, C_, ff, generator=g) / ff ** 0.5, dt)
    gus, dns = stored(gu), stored(dn)
    x, res = dev(torch.randn(n, C_, generator=g), dt), dev(torch.randn(n, C_, generator=g))
    logits = pad(dev(torch.randn(n, E, generator=g)), n, up(E))
    e, b = route(ctx, logits, None, n, E, top, tile, typ, w_stride=2 * ff * C_)
    act = torch.zeros(n * top, ff, dtype=dt, device="cuda")
    p = L.RbProduct(gus.data_ptr(), x.data_ptr(), act.data_ptr(), None, C_, ff, 0, typ, 2 * ff, C_, n, L.RB_GATED, L.RB_SILU, L.RB_UP, 0.0, C.pointer(e))
    L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
    ids, wt = b["ids"].cpu().numpy(), b["weight"].double().cpu().numpy()
    il = f64(gu).reshape(E, ff // 16, 2, 16, C_)
    A, y = np.zeros((n * top, ff)), np.zeros((n * top, C_))
    for q in range(n * top):
        xe, wg, wu = f64(x)[q // top], il[ids[q], :, 0].reshape(ff, C_), il[ids[q], :, 1].reshape(ff, C_)
        A[q] = wt[q] * P.silu(wg @ xe) * (wu @ xe)
        y[q] = f64(dn)[ids[q]] @ f64(act)[q]
    assert np.abs(f64(act) - A).max() < tol * 8
    e.w_stride = C_ * ff
    yd = torch.zeros(n * top, C_, dtype=dt, device="cuda")
    p = L.RbProduct(dns.data_ptr(), act.data_ptr(), yd.data_ptr(), None, ff, C_, 0, typ, C_, ff, n, L.RB_STORE, 0, L.RB_DOWN, 0.0, C.pointer(e))
    L.check(ctx.hip.kf_rb_linear(ctx.h, C.byref(p)))
    assert np.abs(f64(yd) - y).max() < tol * 4
    z = torch.zeros(n, C_, device="cuda")
    p = L.RbProduct(dns.data_ptr(), act.data_ptr(), z.data_ptr(), res.data_ptr(), ff, C_, C_, typ, C_, ff, n, L.RB_RESIDUAL, 0, L.RB_SUM, 1.25, C.pointer(e))
    rc = ctx.hip.kf_rb_linear(ctx.h, C.byref(p))
    if typ == L.F32 or n > 64:
        assert rc == -1000
    else:
        assert rc == 0 and np.abs(f64(z) - (1.25 * f64(res) + y.reshape(n, top, C_).sum(1))).max() < 2e-5


# ---- attention
def mix(H, G, D, chunk, rot, scale=None):
    return {"heads": H, "kv_heads": G, "dim": D, "mask": {"size": chunk} if chunk else None, "scale": D ** -0.5 if scale is None else scale,
            "rot": {"base": 300.0, "dims": rot, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}}}


class Attn:
    """one attention layer with n_slots rings: sequences' raw rows in, heads out; the reference keeps every sequence's whole raw history"""

    def __init__(self, ctx, mx, kind, n_slots=3, n_ctx=512, seed=0):
        self.ctx, self.mx, (self.typ, self.dt, _) = ctx, mx, kind
        H, G, D = mx["heads"], mx["kv_heads"], mx["dim"]
        g = torch.Generator().manual_seed(seed)
        self.qn, self.kn = (dev(torch.rand(up(D), generator=g) + 0.5, self.dt) for _ in range(2))
        chunk = mx["mask"]["size"] if mx["mask"] else 0
        rows = min(chunk, n_ctx) if chunk else n_ctx
        self.kc, self.vc = (torch.zeros(n_slots * (rows * D + 24) * G + 64, dtype=self.dt, device="cuda") for _ in range(2))
        self.tab = np.zeros((n_ctx, max(mx["rot"]["dims"], 2) // 2, 2), dtype=np.float32)
        if mx["rot"]["dims"]:
            s = mx["rot"]["scaling"]
            assert ctx.hip.kf_rb_rope_table_host(self.tab.ctypes.data_as(C.c_void_p), n_ctx, mx["rot"]["dims"], mx["rot"]["base"], s["factor"], s["low"], s["high"], s["original"]) == 0
        self.tab = dev(self.tab)
        self.ldraw, self.ldout = up(2 * H * D + G * D), up(H * D)
        self.n_slots, self.cols = n_slots, 2 * H * D + G * D
        self.a = L.RbAttention(type=self.typ, n_head=H, n_kv=G, dim=D, rot_dims=mx["rot"]["dims"], chunk=chunk, cache_rows=rows, gated=1, scale=mx["scale"], eps=1e-5, k_cache=self.kc.data_ptr(),
                               v_cache=self.vc.data_ptr(), q_norm=self.qn.data_ptr(), k_norm=self.kn.data_ptr(), rope=self.tab.data_ptr(), ldraw=self.ldraw, ldout=self.ldout,
                               slot_stride=(rows * D + 24) * G, head_stride=rows * D + 24)
        self.hist = {}
        self.rng = np.random.default_rng(seed)

    def new(self, slot):
        self.hist[slot] = np.zeros((0, self.cols))

    def rows(self, n):
        return f64(torch.as_tensor(self.rng.normal(size=(n, self.cols))).to(self.dt))

    def reference(self, slot):
        mx, r = self.mx, self.hist[slot]
        H, G, D = mx["heads"], mx["kv_heads"], mx["dim"]
        if mx["rot"]["dims"] == 0:
            mx = dict(mx, rot=dict(mx["rot"], dims=0))
        return P.attend(r[:, :H * D].reshape(-1, H, D), r[:, H * D:(H + G) * D].reshape(-1, G, D), r[:, (H + G) * D:], f64(self.qn)[:D], f64(self.kn)[:D], mx, 1e-5)

    def feed(self, parts, decode=False):
        """parts: {slot: raw rows}; returns {slot: (got, reference)} for the fed rows"""
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
        n = len(meta)
        raw = pad(dev(np.concatenate(raw), self.dt), n, self.ldraw)
        out, knew = torch.zeros(n, self.ldout, dtype=self.dt, device="cuda"), torch.zeros(n, self.mx["kv_heads"] * self.mx["dim"], dtype=self.dt, device="cuda")
        meta, seqs = dev(np.array(meta), torch.int32), dev(np.array(seqs), torch.int32)
        sc = torch.zeros(self.ctx.hip.kf_rb_attention_scratch(n, self.a.n_head, self.a.dim) // 4, device="cuda")
        self.a.raw, self.a.out, self.a.k_new, self.a.scratch = raw.data_ptr(), out.data_ptr(), knew.data_ptr(), sc.data_ptr()
        if decode:
            top = max(len(self.hist[s]) for s in parts) - 1
            L.check(self.ctx.hip.kf_rb_attention_decode(self.ctx.h, C.byref(self.a), meta.data_ptr(), n, top))
        else:
            L.check(self.ctx.hip.kf_rb_attention_prefill(self.ctx.h, C.byref(self.a), meta.data_ptr(), n, seqs.data_ptr(), len(seqs), max(len(x) for x in parts.values())))
        got = f64(out)[:, :self.mx["heads"] * self.mx["dim"]]
        return {s: (got[r0[s]:r0[s] + len(x)], self.reference(s)[-len(x):]) for s, x in parts.items()}

    def check(self, parts, decode=False):
        tol = 2e-5 if self.typ == L.F32 else 0.03
        for s, (a, b) in self.feed(parts, decode).items():
            err = np.abs(a - b).max(axis=1)
            assert err.max() < tol, (s, int(err.argmax()), err.max(), decode)


SHAPES = [(4, 2, 64, 24, 32), (6, 1, 32, 100, 8), (5, 5, 48, 7, 48), (3, 1, 80, 0, 16), (40, 1, 16, 40, 16), (8, 2, 128, 200, 64), (2, 1, 192, 33, 2), (2, 2, 256, 1, 256), (3, 1, 20, 16, 10),
          (2, 1, 100, 30, 0)]


@pytest.mark.parametrize("shape", SHAPES, ids=lambda s: "x".join(map(str, s)))
def test_attention_prompts_portions_and_decoding(ctx, kind, shape):
    """prompts that pass chunk edges, portions down to two tokens, single tokens in both forms, unequal sequences in one batch, a slot used again"""
    a = Attn(ctx, mix(*shape), kind)
    for s in range(3):
        a.new(s)
    a.check({1: a.rows(77)})
    a.check({0: a.rows(130), 2: a.rows(3), 1: a.rows(2)})
    a.check({2: a.rows(21), 1: a.rows(64), 0: a.rows(1)})
    for n in (2, 5, 2):
        a.check({2: a.rows(n), 0: a.rows(n + 1)})
    for i in range(9):
        a.check({s: a.rows(1) for s in ((0, 1, 2) if i % 3 else (2,))}, decode=True)
    a.check({1: a.rows(30)})
    a.new(1)                                   # the slot goes to another sequence; its ring still holds the old rows
    a.check({1: a.rows(5)})
    for _ in range(shape[3] % 40 + 3):
        a.check({1: a.rows(1)}, decode=True)


@pytest.mark.parametrize("shape", [(4, 2, 64, 24, 32), (6, 1, 128, 50, 32), (2, 1, 20, 24, 4)], ids=lambda s: "x".join(map(str, s)))
@pytest.mark.parametrize("how", ["prompt", "portions", "decoded"])
def test_attention_sees_exactly_its_chunk(ctx, kind, shape, how):
    """one key answers to everything (its score beats every other by far): queries of its chunk return that key's value, queries past the chunk's edge must not"""
    H, G, D, chunk, rot = shape
    for key in (0, 1, chunk - 1, chunk, 2 * chunk - 2):
        a = Attn(ctx, mix(H, G, D, chunk, rot, scale=25.0 / D), kind, seed=key)
        n = 2 * chunk + 3
        x = a.rows(n)
        q, k = x[:, :H * D], x[:, H * D:(H + G) * D]
        # every query and this one key aligned on an unrotated direction (the last dimension passes through)
        q[:, D - 1::D] = 8.0
        k[:, D - 1::D] = -3.0
        k[key, :] *= 0.1
        k[key, D - 1::D] = 8.0
        a.new(0)
        cuts = {"prompt": [n], "portions": [key + 1, 1, n - key - 2], "decoded": [max(key - 1, 1)] + [1] * (n - max(key - 1, 1))}[how]
        at = 0
        for c in cuts:
            if c < 1:
                continue
            got = a.feed({0: x[at:at + c]}, decode=how == "decoded" and at > 0)[0]
            assert np.abs(got[0] - got[1]).max() < (5e-5 if kind[0] == L.F32 else 0.1), (key, at)
            at += c
        ref = a.reference(0)
        near = [t for t in range(key, n) if t // chunk == key // chunk]
        away = [t for t in range(key + 1, n) if t // chunk != key // chunk]
        gate = P.sigmoid(x[:, (H + G) * D:])
        if near:      # the reference itself: that key's value comes back
            assert np.abs((ref / gate)[near[-1], D - 1] - 8.0) < 0.2
        if away:
            assert np.abs((ref / gate)[away[0], D - 1] - 8.0) > 1.0


def test_attention_long_range_in_key_ranges(ctx):
    """a decode row whose keys are cut into ranges for several workgroups (and no chunks)"""
    kind = TYPES["bf16"]
    a = Attn(ctx, mix(8, 2, 64, 0, 32), kind, n_slots=2, n_ctx=2100)
    a.new(0), a.new(1)
    a.check({0: a.rows(2000), 1: a.rows(700)})
    for _ in range(3):
        a.check({0: a.rows(1), 1: a.rows(1)}, decode=True)


def test_attention_refuses(ctx):
    a = Attn(ctx, mix(4, 2, 64, 24, 32), TYPES["bf16"])
    t = torch.zeros(4096, device="cuda")
    m = torch.zeros(4, dtype=torch.int32, device="cuda")
    for f in ("raw", "out", "k_new", "scratch"):
        setattr(a.a, f, t.data_ptr())
    for f, v in (("n_kv", 3), ("rot_dims", 66), ("rot_dims", 3), ("ldraw", 64), ("slot_stride", 8), ("head_stride", 8), ("cache_rows", 0), ("dim", 1024), ("type", L.Q4), ("raw", None)):
        old = getattr(a.a, f)
        setattr(a.a, f, v)
        assert ctx.hip.kf_rb_attention_prefill(ctx.h, C.byref(a.a), m.data_ptr(), 1, m.data_ptr(), 1, 1) < 0, f
        assert ctx.hip.kf_rb_attention_decode(ctx.h, C.byref(a.a), m.data_ptr(), 1, 0) < 0, f
        setattr(a.a, f, old)


@pytest.mark.parametrize("vocab", [5, 300, 5000, 1200000])
def test_pick(ctx, vocab):
    n, ld = 3, up(vocab)
    lg = torch.randn(n, ld, device="cuda")
    lg[:, vocab:] = 100.0                      # padding is not in the vocabulary
    lg[1, vocab // 2] = lg[1, vocab - 1] = 50.0  # the first of two equal maxima
    meta = torch.tensor([[4, 2, 0, 0], [0, 0, 0, 0], [-1, 1, 0, 0]], dtype=torch.int32, device="cuda")
    state, out = torch.zeros(3, 4, dtype=torch.int32, device="cuda"), torch.full((3, 8), -1, dtype=torch.int32, device="cuda")
    sc = torch.zeros(ctx.hip.kf_rb_pick_scratch(n) // 4, device="cuda")
    L.check(ctx.hip.kf_rb_pick(ctx.h, lg.data_ptr(), ld, vocab, n, meta.data_ptr(), state.data_ptr(), out.data_ptr(), 8, sc.data_ptr()))
    want = lg[:, :vocab].argmax(1).cpu().numpy()
    s, o = state.cpu().numpy(), out.cpu().numpy()
    assert s[2].tolist() == [want[0], 5, 0, 0] and s[0].tolist() == [vocab // 2, 1, 0, 0] and not s[1].any()
    assert o[2, 4] == want[0] and o[0, 0] == vocab // 2 and (o >= 0).sum() == 2
    b = torch.zeros(ld, dtype=torch.bfloat16, device="cuda")
    L.check(ctx.hip.kf_rb_to_bf16(ctx.h, lg.data_ptr(), b.data_ptr(), ld))
    assert torch.equal(b, lg[0].bfloat16())


def test_embed_and_pack(ctx, kind):
    typ, dt, _ = kind
    V, dim, ld = 11, 75, 128
    src = torch.randn(V, dim).bfloat16().cuda()
    tab = torch.zeros(64, ld, dtype=dt, device="cuda")
    L.check(ctx.hip.kf_rb_pack(ctx.h, typ, src.data_ptr(), V, dim, tab.data_ptr(), ld, 0, -1, 0))
    assert torch.equal(tab[:V, :dim].float(), src.float()) and not tab[:, dim:].any() and not tab[V:].any()
    tok = torch.tensor([3, 10, 0], dtype=torch.int32, device="cuda")
    x, h = torch.full((3, ld), 9.0, device="cuda"), torch.full((3, ld), 9.0, dtype=dt, device="cuda")
    L.check(ctx.hip.kf_rb_embed(ctx.h, typ, tab.data_ptr(), V, dim, ld, tok.data_ptr(), 3, x.data_ptr(), h.data_ptr()))
    assert torch.equal(x[:, :dim], src[tok.long()].float()) and not x[:, dim:].any() and torch.equal(h.float(), x)
    gu = torch.zeros(96, 64, dtype=dt, device="cuda")
    w = torch.randn(40, 50).bfloat16().cuda()
    L.check(ctx.hip.kf_rb_pack(ctx.h, typ, w.data_ptr(), 40, 50, gu.data_ptr(), 64, 0, 1, 0))
    for r in range(40):
        assert torch.equal(gu[32 * (r // 16) + 16 + r % 16, :50].float(), w[r].float())
    if typ == L.BF16:      # a product's weight, from a row no tile starts at
        pw, row = torch.zeros(64, 64, dtype=dt, device="cuda"), torch.zeros(64, 64, dtype=dt, device="cuda")
        row[21:61, :50] = w
        L.check(ctx.hip.kf_rb_pack(ctx.h, typ, w.data_ptr(), 40, 50, pw.data_ptr(), 64, 21, -1, 1))
        assert torch.equal(pw, stored(row))
    # states: forced ids, a parked slot, a position outside
    state = torch.tensor([[1, 2, 0, 0], [4, 0, 1, 0], [5, 8, 0, 0], [6, 7, 0, 0]], dtype=torch.int32, device="cuda")
    forced = torch.full((4, 8), -1, dtype=torch.int32, device="cuda")
    forced[3, 7] = 9
    x, h, meta = torch.zeros(4, ld, device="cuda"), torch.zeros(4, ld, dtype=dt, device="cuda"), torch.zeros(4, 4, dtype=torch.int32, device="cuda")
    L.check(ctx.hip.kf_rb_embed_state(ctx.h, typ, tab.data_ptr(), V, dim, ld, state.data_ptr(), forced.data_ptr(), 8, 8, 4, x.data_ptr(), h.data_ptr(), meta.data_ptr()))
    assert meta[:, 0].tolist() == [2, -1, -1, 7] and meta[:, 1].tolist() == [0, 1, 2, 3] and state[:, 3].tolist() == [0, 0, 64, 0]
    assert torch.equal(x[0, :dim], src[1].float()) and torch.equal(x[3, :dim], src[9].float())
