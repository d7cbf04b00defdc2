"""Python plumbing over the C ABI: device memory comes from torch tensors, every computation is a kf_* / kfh_* call.

Nothing here computes on the CPU and nothing imports oracle/.  bf16 tensors are torch.bfloat16 on the GPU;
packed weights are torch.uint8 blobs laid out `data || gama` exactly as the reference allocates them
(GTensor.cpp:456-510).
"""
import ctypes as C
import json
import os

import numpy as np
import torch

from . import lib as L

SLOTS = ("q", "k", "v", "o", "gate", "up", "down")
NORMS = ("norm_in", "norm_post", "qn", "kn")


def quant_range(type_, symmetric=False):
    """qMin, qMax, qBias as the GeQuant ctor sets them (GeQuant.cpp:107-124)."""
    if type_ == L.T_SIGN:
        return -1, 1, 1
    if type_ in (L.BOOL1, L.T_BINARY):
        return 0, 1, 0
    if type_ == L.Q4:
        return (-8, 7, 8) if symmetric else (0, 15, 0)
    return 0, 0, 0


class DevWeight:
    """A weight resident in HBM: blob = torch.uint8 [szData + szGama]."""

    def __init__(self, type_, ne0, ne1, blob, lGroup=128, symmetric=False):
        self.type, self.ne0, self.ne1, self.blob, self.lGroup = type_, ne0, ne1, blob, lGroup
        bits = L.BITS[type_]
        self.szData = ne0 * ne1 * bits // 8
        self.quantised = bits < 8
        self.nGroup = ne0 * ne1 // lGroup if self.quantised else 0
        self.szGama = (ne0 + ne1 + 2 * self.nGroup) * 2 if self.quantised else 0
        assert blob.numel() == self.szData + self.szGama, (blob.numel(), self.szData, self.szGama)
        self.qMin, self.qMax, self.qBias = quant_range(type_, symmetric)

    @staticmethod
    def blob_bytes(type_, ne0, ne1, lGroup=128):
        bits = L.BITS[type_]
        n = ne0 * ne1 * bits // 8
        if bits < 8:
            n += (ne0 + ne1 + 2 * (ne0 * ne1 // lGroup)) * 2
        return n

    def desc(self):
        p = self.blob.data_ptr()
        return L.Weight(p, (p + self.szData) if self.quantised else None, self.type, self.ne0, self.ne1, self.nGroup, self.lGroup, self.qMin, self.qMax,
                        self.qBias, None, None)

    def algorithmic_bytes(self):
        """what a mat-vec has to read: packed data + zero/step"""
        return self.szData + 4 * self.nGroup

    def zero_step(self):
        g = self.blob[self.szData:].view(torch.bfloat16)
        z0 = self.ne0 + self.ne1
        return g[z0:z0 + self.nGroup], g[z0 + self.nGroup:z0 + 2 * self.nGroup]


class LutDevWeight:
    """Row-codebook weight in HBM (KF_QUANT_ROW_LUT; GeQuant::RT_NormalF): blob = MSB-first `bits`-wide stream [ne0*ne1*bits/8] ‖ bf16 gama
    [ne0 + ne1 + (2^bits)*ne0]; bits 4 (the mat-vec format), 3 or 2 (dequant-only); rtn=True (bits 2): (zero, step) per row, KF_QUANT_ROW_RTN."""

    def __init__(self, ne0, ne1, blob, bits=4, rtn=False):
        self.type, self.ne0, self.ne1, self.blob, self.lGroup = {4: L.Q4, 3: L.Q3, 2: L.Q2}[bits], ne0, ne1, blob, 0
        self.bits, self.rtn = bits, rtn
        self.szData = ne0 * ne1 * bits // 8
        self.szGama = (ne0 + ne1 + (2 if rtn else 1 << bits) * ne0) * 2
        assert blob.numel() == self.szData + self.szGama, (blob.numel(), self.szData, self.szGama)

    @staticmethod
    def blob_bytes(ne0, ne1, bits=4):
        return ne0 * ne1 * bits // 8 + (ne0 + ne1 + (1 << bits) * ne0) * 2

    def desc(self):
        p = self.blob.data_ptr()
        return L.Weight(p, p + self.szData, self.type, self.ne0, self.ne1, 0, 0, 0, (1 << self.bits) - 1, 0, None, None,
                        L.QUANT_ROW_RTN if self.rtn else L.QUANT_ROW_LUT, 0)

    def algorithmic_bytes(self):
        """what a mat-vec has to read: the nibble stream + the rows' tables"""
        return self.szData + 32 * self.ne0

    def lut(self):
        g = self.blob[self.szData:].view(torch.bfloat16)
        return g[self.ne0 + self.ne1:].view(self.ne0, -1)


class AWQDevWeight:
    """Vendor AutoAWQ tensors in HBM: qweight int32 [in, out/8], qzeros int32 [in/128, out/8], scales fp16 [in/128, out]."""

    def __init__(self, n_out, n_in, qweight, qzeros, scales):
        self.type, self.ne0, self.ne1, self.lGroup = L.Q4, n_out, n_in, 128
        self.qweight, self.qzeros, self.scales = qweight.contiguous(), qzeros.contiguous(), scales.contiguous()

    def desc(self):
        return L.Weight(self.qweight.data_ptr(), None, L.Q4, self.ne0, self.ne1, self.ne0 * self.ne1 // 128, 128, 0, 15, 0, self.qzeros.data_ptr(),
                        self.scales.data_ptr())

    def algorithmic_bytes(self):
        return self.qweight.numel() * 4 + self.qzeros.numel() * 4 + self.scales.numel() * 2


def _ptr(t):
    return None if t is None else C.c_void_p(t.data_ptr())


_STREAM = {}


def stream(device=0):
    """One dedicated (non-default) HIP stream per device, made torch's current stream, so that torch's allocations /
    copies and the kf_* launches are ordered on the same queue and the queue can be captured into a hipGraph
    (the legacy default stream cannot)."""
    if device not in _STREAM:
        torch.cuda.set_device(device)
        _STREAM[device] = torch.cuda.Stream(device=device)
        torch.cuda.set_stream(_STREAM[device])
    return _STREAM[device]


# Test hook (Python side only; the library reads no environment): the summation order every Context / Qwen3 created from here on is switched to right after its
# creation.  None = the library's own default (canonical, kf_abi.h).  tests/conftest.py sets False: the tolerance tests were written against the v_dot2c order and keep
# covering it, the canonical order is asserted bit for bit by the tests that switch it on themselves.
DEFAULT_CANONICAL = None


class Context:
    """kf_ctx bound to torch's current stream on `device`."""

    def __init__(self, device=0):
        self.hip, self.host = L.load()
        if not torch.cuda.is_available():
            raise L.KFError("no GPU visible: koifish_amd runs on MI355X only (no CPU fallback)")
        torch.cuda.set_device(device)
        self.device = torch.device("cuda", device)
        self.h = C.c_void_p()
        L.check(self.hip.kf_init(device, C.c_void_p(stream(device).cuda_stream), C.byref(self.h)), "kf_init")
        self._attn_ws = None
        self._head_ws = torch.empty(self.hip.kf_head_scratch_bytes(), dtype=torch.uint8, device=self.device)
        self._lin_ws = None
        if DEFAULT_CANONICAL is not None:
            self.set_canonical(DEFAULT_CANONICAL)

    def close(self):
        if self.h:
            self.hip.kf_destroy(self.h)
            self.h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    def sync(self):
        L.check(self.hip.kf_sync(self.h), "kf_sync")

    def set_canonical(self, on):
        """1 (the library default): the decode kernels sum in the canonical order the CPU oracle shares (bit-exact); 0: the v_dot2c / fp32 forms"""
        L.check(self.hip.kf_set_canonical(self.h, int(bool(on))), "kf_set_canonical")

    # ---- weights
    def upload_blob(self, type_, ne0, ne1, blob_np, lGroup=128, symmetric=False):
        t = torch.from_numpy(np.ascontiguousarray(blob_np).view(np.uint8).reshape(-1).copy()).to(self.device)
        return DevWeight(type_, ne0, ne1, t, lGroup, symmetric)

    def quantize(self, w_bf16, type_, lGroup=128, symmetric=False):
        """w_bf16: torch.bfloat16 [ne0, ne1] on the GPU -> DevWeight (kf_quantize: GeQuant::RTN_x / YinYang on device)."""
        if type_ == L.NF4:
            return self.quantize_nf4(w_bf16)
        ne0, ne1 = w_bf16.shape
        w_bf16 = w_bf16.contiguous()
        if type_ == L.BF16:
            return DevWeight(L.BF16, ne0, ne1, w_bf16.view(torch.uint8).reshape(-1))
        if type_ == L.F8E5M2:
            # Float2T<f8e5> (g_float.hpp:433-443): float -> half (RNE) -> keep the high byte
            h = w_bf16.to(torch.float32).to(torch.float16).view(torch.int16)
            b = ((h.to(torch.int32) >> 8) & 0xFF).to(torch.uint8)
            return DevWeight(L.F8E5M2, ne0, ne1, b.reshape(-1).contiguous())
        blob = torch.zeros(DevWeight.blob_bytes(type_, ne0, ne1, lGroup), dtype=torch.uint8, device=self.device)
        dw = DevWeight(type_, ne0, ne1, blob, lGroup, symmetric)
        g = blob[dw.szData:].view(torch.bfloat16)
        g[:ne0 + ne1] = 1.0  # R_SCALE / C_SCALE (unused: rc_normal = 0)
        d = dw.desc()
        L.check(self.hip.kf_quantize(self.h, C.byref(d), _ptr(w_bf16), int(symmetric)), "kf_quantize")
        return dw

    def upload_lut_blob(self, ne0, ne1, blob_np, bits=4, rtn=False):
        t = torch.from_numpy(np.ascontiguousarray(blob_np).view(np.uint8).reshape(-1).copy()).to(self.device)
        return LutDevWeight(ne0, ne1, t, bits, rtn)

    def quantize_nf4(self, w_bf16, bits=4):
        """w_bf16: torch.bfloat16 [ne0, ne1] on the GPU -> LutDevWeight (kf_quantize in KF_QUANT_ROW_LUT mode: GeQuant::RT_NormalF on device; bits 4 or 3)."""
        ne0, ne1 = w_bf16.shape
        w_bf16 = w_bf16.contiguous()
        blob = torch.zeros(LutDevWeight.blob_bytes(ne0, ne1, bits), dtype=torch.uint8, device=self.device)
        dw = LutDevWeight(ne0, ne1, blob, bits)
        blob[dw.szData:].view(torch.bfloat16)[:ne0 + ne1] = 1.0  # R_SCALE / C_SCALE (unused: rc_normal = 0)
        d = dw.desc()
        L.check(self.hip.kf_quantize(self.h, C.byref(d), _ptr(w_bf16), 0), "kf_quantize")
        return dw

    # ---- operators (each one ABI call)
    def dequant(self, w):
        shape = (w.ne1, w.ne0) if isinstance(w, AWQDevWeight) else (w.ne0, w.ne1)   # AWQ: [in, out] (TransA = 0)
        out = torch.empty(*shape, dtype=torch.bfloat16, device=self.device)
        d = w.desc()
        L.check(self.hip.kf_dequant(self.h, C.byref(d), _ptr(out)), "kf_dequant")
        return out

    def linear_scratch(self, w, n_tok=1):
        """kernels never allocate: storages served by dequantise-then-multiply (AWQ, 3- / 2-bit row forms, row-codebook batches) get their workspace here"""
        d = w.desc() if not isinstance(w, L.Weight) else w
        need = self.hip.kf_linear_scratch_bytes(C.byref(d), int(n_tok))
        if need and (self._lin_ws is None or self._lin_ws.numel() < need):
            self.sync()   # earlier launches may still read the old buffer
            self._lin_ws = torch.empty(need, dtype=torch.uint8, device=self.device)
            L.check(self.hip.kf_set_scratch(self.h, C.c_void_p(self._lin_ws.data_ptr()), C.c_size_t(need)), "kf_set_scratch")
        return need

    def linear(self, w, x, bias=None, alpha=1.0, beta=0.0, residual=None, y=None):
        y = torch.zeros(w.ne0, dtype=torch.bfloat16, device=self.device) if y is None else y
        self.linear_scratch(w)
        d = w.desc()
        epi = L.KF_EPI_RESIDUAL if residual is not None else 0
        L.check(self.hip.kf_linear(self.h, C.byref(d), _ptr(x), _ptr(y), _ptr(bias), 1, alpha, beta, epi, _ptr(residual)), "kf_linear")
        return y

    def rmsnorm(self, x, w, eps=1e-6):
        y = torch.empty_like(x)
        rows = 1 if x.dim() == 1 else x.shape[0]
        L.check(self.hip.kf_rmsnorm(self.h, _ptr(x), _ptr(w), _ptr(y), rows, x.shape[-1], eps, None), "kf_rmsnorm")
        return y

    def rope_table(self, n_pos, hd, theta):
        t = np.zeros((n_pos, hd // 2, 2), dtype=np.float32)
        L.check(self.hip.kf_rope_table_host(t.ctypes.data_as(C.c_void_p), n_pos, hd, theta), "kf_rope_table_host")
        return torch.from_numpy(t).to(self.device)

    def qknorm_rope(self, q, k, wq, wk, table, pos, n_head, n_kv, hd, eps=1e-6):
        """in place on q and k"""
        L.check(self.hip.kf_qknorm_rope(self.h, _ptr(q), _ptr(k), _ptr(wq), _ptr(wk), _ptr(table), pos, None, n_head, n_kv, hd, eps), "kf_qknorm_rope")

    def _ws(self, n_head, hd):
        n = self.hip.kf_attn_scratch_bytes(n_head, hd)
        if self._attn_ws is None or self._attn_ws.numel() < n:
            self._attn_ws = torch.zeros(n, dtype=torch.uint8, device=self.device)  # arrival counters start at zero
        return self._attn_ws

    def attn_decode(self, q, kc, vc, pos, n_head, n_kv, hd, kv_stride=None):
        out = torch.empty(n_head * hd, dtype=torch.bfloat16, device=self.device)
        L.check(self.hip.kf_attn_decode(self.h, _ptr(q), _ptr(kc), _ptr(vc), _ptr(out), pos, None, n_head, n_kv, hd, kv_stride or n_kv * hd,
                                        _ptr(self._ws(n_head, hd))), "kf_attn_decode")
        return out

    def attn_block(self, q_raw, k_raw, kc, vc, wq, wk, table, pos, n_head, n_kv, hd, eps=1e-6, kv_stride=None):
        out = torch.empty(n_head * hd, dtype=torch.bfloat16, device=self.device)
        L.check(self.hip.kf_attn_block(self.h, _ptr(q_raw), _ptr(k_raw), _ptr(kc), _ptr(vc), _ptr(out), _ptr(wq), _ptr(wk), _ptr(table), pos, None, n_head,
                                       n_kv, hd, kv_stride or n_kv * hd, eps, _ptr(self._ws(n_head, hd))), "kf_attn_block")
        return out

    def swiglu(self, gate, up):
        out = torch.empty_like(gate)
        L.check(self.hip.kf_swiglu(self.h, _ptr(gate), _ptr(up), _ptr(out), gate.numel()), "kf_swiglu")
        return out

    def add(self, a, b):
        out = torch.empty_like(a)
        L.check(self.hip.kf_add(self.h, _ptr(a), _ptr(b), _ptr(out), a.numel()), "kf_add")
        return out

    def embed(self, w, token):
        out = torch.empty(w.ne1, dtype=torch.bfloat16, device=self.device)
        d = w.desc()
        L.check(self.hip.kf_embed(self.h, C.byref(d), int(token), None, _ptr(out)), "kf_embed")
        return out

    def lm_head(self, w, x):
        logits = torch.empty(w.ne0, dtype=torch.bfloat16, device=self.device)
        am = torch.zeros(1, dtype=torch.int32, device=self.device)
        d = w.desc()
        L.check(self.hip.kf_lm_head(self.h, C.byref(d), _ptr(x), _ptr(logits), _ptr(am), _ptr(self._head_ws)), "kf_lm_head")
        return logits, int(am.item())

    def norm_linear(self, x, norm_w, ws, eps=1e-6):
        ys = [torch.zeros(w.ne0, dtype=torch.bfloat16, device=self.device) for w in ws]
        descs = [w.desc() for w in ws]
        wp = (C.c_void_p * len(ws))(*[C.addressof(d) for d in descs])
        yp = (C.c_void_p * len(ws))(*[y.data_ptr() for y in ys])
        L.check(self.hip.kf_norm_linear(self.h, _ptr(x), _ptr(norm_w), eps, len(ws), wp, yp, None, 0, None), "kf_norm_linear")
        return ys

    def norm_gateup_swiglu(self, x, norm_w, gate, up, eps=1e-6):
        act = torch.zeros(gate.ne0, dtype=torch.bfloat16, device=self.device)
        dg, du = gate.desc(), up.desc()
        L.check(self.hip.kf_norm_gateup_swiglu(self.h, _ptr(x), _ptr(norm_w), eps, C.byref(dg), C.byref(du), _ptr(act)), "kf_norm_gateup_swiglu")
        return act

    # ---- HIP events on the ctx stream
    def event(self):
        e = C.c_void_p()
        L.check(self.hip.kf_event_create(C.byref(e)), "kf_event_create")
        return e

    def record(self, e):
        L.check(self.hip.kf_event_record(self.h, e), "kf_event_record")

    def elapsed_ms(self, a, b):
        ms = C.c_float()
        L.check(self.hip.kf_event_elapsed_ms(a, b, C.byref(ms)), "kf_event_elapsed_ms")
        return ms.value


class Qwen3:
    """The host-side Fish (koifish_amd/host/kf_host.cpp) for a Qwen3-shaped decoder."""

    def __init__(self, cfg, device=0, own_stream=False):
        """own_stream: this decoder launches on a HIP stream of its own (several decoders then overlap on the GPU); otherwise on the
        device's shared stream."""
        self.hip, self.host = L.load()
        if not torch.cuda.is_available():
            raise L.KFError("no GPU visible: koifish_amd runs on MI355X only (no CPU fallback)")
        torch.cuda.set_device(device)
        self.cfg, self.device = dict(cfg), torch.device("cuda", device)
        rc = C.c_int(0)
        shared = stream(device)
        self._stream = torch.cuda.Stream(device=device) if own_stream else shared
        self.h = self.host.kfh_create(device, C.c_void_p(self._stream.cuda_stream), cfg["dim"], cfg["n_layer"], cfg["n_head"], cfg["n_kv"],
                                      cfg["head_dim"], cfg["ffn"], cfg["vocab"], cfg["max_seq"], cfg.get("rms_eps", 1e-6), cfg.get("qk_eps", 1e-6),
                                      cfg.get("theta", 1e6), C.byref(rc))
        if not self.h:
            why = self.host.kfh_host_error().decode()
            if why:
                raise L.KFError("kfh_create failed with %d: %s" % (rc.value, why))
            L.check(rc.value or -1, "kfh_create")
        self.h = C.c_void_p(self.h)
        if DEFAULT_CANONICAL is not None:
            L.check(self.host.kfh_set_canonical(self.h, int(bool(DEFAULT_CANONICAL))), "kfh_set_canonical")
        self._keep = []
        self.weights = {}
        self._norms = {}

    @classmethod
    def from_hf(cls, path, layer_type=L.Q4, head_type=L.BF16, device=0, lGroup=128, max_seq=0):
        """Hugging Face directory (config.json + model.safetensors[.index.json]; dense BF16/F16/F32 tensors are quantised on the GPU to
        `layer_type` / `head_type`, AutoAWQ qweight/qzeros/scales triples are taken as they are) -> a ready model.  The C++ loader is
        koifish_amd/host/kf_safetensors.cpp (K_SafeTensors, Serialize.cpp:849-976 read side)."""
        self = cls.__new__(cls)
        self.hip, self.host = L.load()
        if not torch.cuda.is_available():
            raise L.KFError("no GPU visible: koifish_amd runs on MI355X only (no CPU fallback)")
        torch.cuda.set_device(device)
        rc = C.c_int(0)
        self.device = torch.device("cuda", device)
        self.h = self.host.kfh_load_hf(str(path).encode(), device, C.c_void_p(stream(device).cuda_stream), int(layer_type), int(head_type), int(lGroup), int(max_seq),
                                       C.byref(rc))
        if not self.h:
            raise L.KFError("kfh_load_hf(%s) failed with %d: %s" % (path, rc.value, self.host.kfh_last_error().decode()))
        self.h = C.c_void_p(self.h)
        if DEFAULT_CANONICAL is not None:
            L.check(self.host.kfh_set_canonical(self.h, int(bool(DEFAULT_CANONICAL))), "kfh_set_canonical")
        self._read_config()
        return self

    @classmethod
    def from_kun(cls, path, device=0, max_seq=0):
        """A `.kun` checkpoint (the reference's container: safetensors header, `data||gama` blobs, msgpack config tensor; Serialize.cpp:849-976)
        -> a ready model.  The blobs go to HBM as stored: nothing is re-quantised."""
        self = cls.__new__(cls)
        self.hip, self.host = L.load()
        if not torch.cuda.is_available():
            raise L.KFError("no GPU visible: koifish_amd runs on MI355X only (no CPU fallback)")
        torch.cuda.set_device(device)
        rc = C.c_int(0)
        self.device = torch.device("cuda", device)
        self.h = self.host.kfh_load_kun(str(path).encode(), device, C.c_void_p(stream(device).cuda_stream), int(max_seq), C.byref(rc))
        if not self.h:
            raise L.KFError("kfh_load_kun(%s) failed with %d: %s" % (path, rc.value, self.host.kfh_last_error().decode()))
        self.h = C.c_void_p(self.h)
        if DEFAULT_CANONICAL is not None:
            L.check(self.host.kfh_set_canonical(self.h, int(bool(DEFAULT_CANONICAL))), "kfh_set_canonical")
        self._read_config()
        return self

    def _read_config(self):
        iv = (C.c_int * 10)()
        fv = (C.c_float * 2)()
        L.check(self.host.kfh_get_config(self.h, iv, fv), "kfh_get_config")
        self.cfg = dict(dim=iv[0], n_layer=iv[1], n_head=iv[2], n_kv=iv[3], head_dim=iv[4], ffn=iv[5], vocab=iv[6], max_seq=iv[7], tied=bool(iv[8]),
                        theta=float(fv[1]))
        self.fuse_level = iv[9]
        self._keep, self.weights, self._norms = [], {}, {}
        self._ctx = None

    def save_kun(self, path):
        """Write every parameter of the model as its `data||gama` blob plus the config tensor (Fish::SAFETENSOR_Serialize, save branch)."""
        rc = self.host.kfh_save_kun(self.h, str(path).encode())
        if rc != 0:
            raise L.KFError("kfh_save_kun(%s) failed with %d: %s" % (path, rc, self.host.kfh_last_error().decode()))

    def close(self):
        """the objects built on this model (XcdReplicas / XcdTP: they read its context and weights when they go) are closed first"""
        for d in list(getattr(self, "_dependents", ())):
            try:
                d.close()
            except Exception:
                pass
        if getattr(self, "h", None):
            self.host.kfh_destroy(self.h)
            self.h = None

    def _depends(self, obj):
        import weakref
        if not hasattr(self, "_dependents"):
            self._dependents = weakref.WeakSet()
        self._dependents.add(obj)

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    def set_weight(self, layer, slot, w):
        """w: DevWeight (already in HBM)."""
        self._keep.append(w)
        self.weights[(layer, slot)] = w
        if isinstance(w, LutDevWeight):
            L.check(self.host.kfh_set_weight_lut(self.h, layer, slot, w.ne0, w.ne1, C.c_void_p(w.blob.data_ptr()), C.c_size_t(w.blob.numel()), C.c_size_t(w.szData), 1),
                    "kfh_set_weight_lut")
            return
        L.check(self.host.kfh_set_weight(self.h, layer, slot, w.type, w.ne0, w.ne1, C.c_void_p(w.blob.data_ptr()), w.blob.numel(), w.szData, 1, w.lGroup,
                                         w.qMin, w.qMax, w.qBias), "kfh_set_weight")

    def tie_head(self):
        L.check(self.host.kfh_tie_head(self.h), "kfh_tie_head")
        self.weights[(-1, 1)] = self.weights[(-1, 0)]

    def set_norm(self, layer, slot, w_bf16):
        w_bf16 = w_bf16.contiguous()
        self._keep.append(w_bf16)
        self._norms[(layer, slot)] = w_bf16
        L.check(self.host.kfh_set_norm(self.h, layer, slot, C.c_void_p(w_bf16.data_ptr()), w_bf16.numel(), 1), "kfh_set_norm")

    def set_fuse_level(self, lvl):
        self.host.kfh_set_fuse_level(self.h, lvl)

    def set_hot(self, layer, hot):
        """sparse forward (D_matmul_sparse / CS_Picker::hot): hot[ffn] int32 host array, 1 = the FFN row of gate / up is computed; None = dense"""
        if hot is None:
            L.check(self.host.kfh_set_hot(self.h, int(layer), None, 0), "kfh_set_hot")
            self._hot.pop(layer, None) if hasattr(self, "_hot") else None
            return
        a = np.ascontiguousarray(hot, dtype=np.int32)
        L.check(self.host.kfh_set_hot(self.h, int(layer), a.ctypes.data_as(C.c_void_p), a.size), "kfh_set_hot")
        if not hasattr(self, "_hot"):
            self._hot = {}
        self._hot[layer] = int(self.host.kfh_n_hot(self.h, int(layer)))

    def set_engine(self, on):
        """The persistent decode engine (kf_engine_*: all layers of a step in one launch) on / off; off = the five launches per layer.
        Same arithmetic either way, bit for bit, in the canonical order (the default); in the v_dot2c order the engine's fp32 attention sums are its own (tolerances)."""
        L.check(self.host.kfh_set_engine(self.h, int(bool(on))), "kfh_set_engine")

    def set_canonical(self, on):
        """1 (the library default): the decode kernels sum in the canonical order the CPU oracle shares (bit-exact logits, ids and KV rows); 0: the v_dot2c_f32_bf16 / fp32 forms"""
        L.check(self.host.kfh_set_canonical(self.h, int(bool(on))), "kfh_set_canonical")

    def engine_why(self):
        """why the persistent engine does not serve this model ("" when it does)"""
        self.host.kfh_engine_why.restype = C.c_char_p
        return self.host.kfh_engine_why(self.h).decode()

    def engine_tune(self, passes=2):
        """kf_engine_tune at the position the decode state holds: (mean launch us before, after)"""
        us = (C.c_float * 2)()
        L.check(self.host.kfh_engine_tune(self.h, int(passes), us), "kfh_engine_tune")
        return float(us[0]), float(us[1])

    def set_engine_autotune(self, passes):
        """> 0: the hand-off delays are measured once per position bucket, at the first multi-step launch inside it (passes of kf_engine_tune)"""
        L.check(self.host.kfh_set_engine_autotune(self.h, int(passes)), "kfh_set_engine_autotune")

    def weights_changed(self):
        """after an IN-PLACE update of weight data handed over as device pointers: drops the resident bf16 copies, the engine's tables and the captured graphs"""
        L.check(self.host.kfh_weights_changed(self.h), "kfh_weights_changed")

    def set_prefill_resident(self, on, max_bytes=0):
        """bf16 copies of the layers' quantised matrices kept in HBM for long prompts (kf_set_dequant_arena): takes effect at the next prefill.  OFF by default; turning it
        on is the caller's promise that weight data given as device pointers is not changed in place afterwards (or that weights_changed() is called when it is): the
        copies are keyed by the blobs' addresses.  max_bytes: budget (default 16 GiB; Qwen3-32B needs 62 GB)."""
        L.check(self.host.kfh_set_prefill_resident(self.h, int(bool(on)), int(max_bytes)), "kfh_set_prefill_resident")

    def resident_bytes(self):
        """bytes of resident dequantised copies the prefill has filled so far"""
        return int(self.host.kfh_resident_bytes(self.h))

    def engine_stats(self, pos):
        """kf_engine_stats: {'sweeps_per_poll': [6], 'polls', 'delay': [6], 'tuned'} for the hand-offs x, q|k|v, slice partials, ao, xB, act"""
        w = (C.c_int32 * 14)()
        L.check(self.host.kfh_engine_stats(self.h, int(pos), w), "kfh_engine_stats")
        polls = max(int(w[6]), 1)
        return {"sweeps_per_poll": [round(int(w[i]) / polls, 3) for i in range(6)], "polls": int(w[6]), "delay": [int(w[7 + i]) for i in range(6)], "tuned": int(w[13])}

    def engine_steps(self):
        """steps enqueued or captured through the engine so far (-1: the engine does not serve this model's shapes / storage)"""
        return int(self.host.kfh_engine_steps(self.h))

    def engine_only(self, n):
        """n launches of the engine kernel alone at the position the device state holds (timing); returns False when the engine does not serve the model"""
        rc = self.host.kfh_engine_only(self.h, int(n))
        if rc == 1:
            return False
        L.check(rc, "kfh_engine_only")
        return True

    def engine_check(self):
        """synchronises; raises when one of the engine's hand-off polls timed out (the launch was not fully resident)"""
        L.check(self.host.kfh_engine_check(self.h), "kfh_engine_check")

    def forward(self, token, pos, want_logits=True):
        logits = np.zeros(self.cfg["vocab"], dtype=np.uint16) if want_logits else None
        r = self.host.kfh_forward(self.h, int(token), int(pos), None if logits is None else logits.ctypes.data_as(C.c_void_p))
        if r < 0:
            L.check(r, "kfh_forward")
        return r, logits

    def generate(self, prompt, n_new, use_graph=True):
        p = np.ascontiguousarray(prompt, dtype=np.int32)
        out = np.zeros(n_new, dtype=np.int32)
        L.check(self.host.kfh_generate(self.h, p.ctypes.data_as(C.c_void_p), p.size, n_new, out.ctypes.data_as(C.c_void_p), int(use_graph)), "kfh_generate")
        return out.tolist()

    def set_sampler(self, temperature=0.0, top_p=0.95, top_k=50, seed=42, true_topk=False):
        """CHAT_SAMPLER: temperature 0 (or top_k 1) = greedy; otherwise GeneratOnPrompt::Sample on the device, rng reseeded here.
        true_topk: candidates = the k largest logits (kf_sample_topk) instead of the set the reference's heap keeps (kf_sample)."""
        L.check(self.host.kfh_set_sampler(self.h, float(temperature), float(top_p), int(top_k) | (0x10000 if true_topk else 0), int(seed)), "kfh_set_sampler")

    def set_prefill_mode(self, mode, chunk=0):
        """generate(): 0 = token-serial prefill through the decode path (like the reference), 1 = token batches on the MFMA kernels"""
        L.check(self.host.kfh_set_prefill_mode(self.h, int(mode), int(chunk)), "kfh_set_prefill_mode")

    def prefill(self, tokens, pos0=0, want_logits=True):
        """Batched prefill of `tokens` at positions pos0..; returns (greedy next id, logits of the last token as uint16 or None)."""
        t = np.ascontiguousarray(tokens, dtype=np.int32)
        L.check(self.host.kfh_prefill(self.h, t.ctypes.data_as(C.c_void_p), t.size, int(pos0)), "kfh_prefill")
        nxt = int(self.tokens_out(pos0 + t.size)[pos0 + t.size - 1])
        logits = None
        if want_logits:
            logits = np.zeros(self.cfg["vocab"], dtype=np.uint16)
            ctx = C.c_void_p(self.host.kfh_ctx(self.h))
            L.check(self.hip.kf_d2h(ctx, logits.ctypes.data_as(C.c_void_p), C.c_void_p(self.host.kfh_logits(self.h)), C.c_size_t(logits.size * 2)), "kf_d2h")
        return nxt, logits

    def logits(self):
        """the last step's logits (bf16 bit patterns as uint16 [vocab])"""
        out = np.zeros(self.cfg["vocab"], dtype=np.uint16)
        ctx = C.c_void_p(self.host.kfh_ctx(self.h))
        L.check(self.hip.kf_d2h(ctx, out.ctypes.data_as(C.c_void_p), C.c_void_p(self.host.kfh_logits(self.h)), C.c_size_t(out.size * 2)), "kf_d2h")
        return out

    def set_forced(self, ids):
        a = np.ascontiguousarray(ids, dtype=np.int32)
        L.check(self.host.kfh_set_forced(self.h, a.ctypes.data_as(C.c_void_p), a.size), "kfh_set_forced")

    def set_state(self, token, pos):
        L.check(self.host.kfh_set_state(self.h, int(token), int(pos)), "kfh_set_state")

    def run_steps(self, pos, n, use_graph=True):
        L.check(self.host.kfh_run_steps(self.h, int(pos), int(n), int(use_graph)), "kfh_run_steps")

    def sync(self):
        L.check(self.host.kfh_sync(self.h), "kfh_sync")

    def tokens_out(self, n):
        out = np.zeros(n, dtype=np.int32)
        L.check(self.host.kfh_get_tokens(self.h, out.ctypes.data_as(C.c_void_p), n), "kfh_get_tokens")
        return out

    def kv_to_host(self):
        """KV cache copied to host as uint16 arrays [n_layer, max_seq, kv_dim]."""
        c = self.cfg
        kvd = c["n_kv"] * c["head_dim"]
        n = c["n_layer"] * c["max_seq"] * kvd
        k = np.zeros(n, dtype=np.uint16)
        v = np.zeros(n, dtype=np.uint16)
        ctx = C.c_void_p(self.host.kfh_ctx(self.h))
        L.check(self.hip.kf_d2h(ctx, k.ctypes.data_as(C.c_void_p), C.c_void_p(self.host.kfh_kcache(self.h)), C.c_size_t(n * 2)), "kf_d2h")
        L.check(self.hip.kf_d2h(ctx, v.ctypes.data_as(C.c_void_p), C.c_void_p(self.host.kfh_vcache(self.h)), C.c_size_t(n * 2)), "kf_d2h")
        shp = (c["n_layer"], c["max_seq"], kvd)
        return k.reshape(shp), v.reshape(shp)

    def num_graphs(self):
        return self.host.kfh_num_graphs(self.h)

    def step_bytes(self, pos):
        """Algorithmic HBM bytes of one decode step at position `pos`: every weight's packed data +
        zero/step once, the norm vectors, and the KV rows 0..pos read once plus the new row written."""
        c = self.cfg
        kvd = c["n_kv"] * c["head_dim"]
        wb = 0
        hot = getattr(self, "_hot", {})
        for (layer, slot), w in self.weights.items():
            if layer == -1 and slot == 0:
                continue  # embedding: one row
            if layer in hot and slot in (4, 5):   # sparse forward: only the hot rows of gate / up are read
                wb += w.algorithmic_bytes() * hot[layer] // w.ne0
                continue
            wb += w.algorithmic_bytes()
        emb = self.weights[(-1, 0)]
        wb += emb.algorithmic_bytes() // emb.ne0
        norms = (c["n_layer"] * (2 * c["dim"] + 2 * c["head_dim"]) + c["dim"]) * 2
        kv = 2 * c["n_layer"] * (pos + 1) * kvd * 2 + 2 * c["n_layer"] * kvd * 2
        return wb + norms + kv


class LayeredDecoder(Qwen3):
    """A decoder described layer by layer (koifish::SeqFish, host/kf_seq.hpp): bf16 or true 32-bit.  The
    generation surface is the one every model has (generate, prefill, run_steps, set_sampler, ...); XcdReplicas(model, n) serves n requests at once."""

    def __init__(self, config, dtype="bfloat16", max_seq=0, device=0, shapes=None):
        """config: the dict of a config.json; the tensors are set one by one (set_tensor) before the first step.  shapes: {tensor name: shape} for the sizes that a design's
        config.json leaves to its tensors.  See from_dir for a checkpoint."""
        self._open(device)
        rc = C.c_int(0)
        doc = dict(config, tensor_shapes={k: list(v) for k, v in shapes.items()}) if shapes else config
        h = self.host.kfh_seq_create(json.dumps(doc).encode(), device, C.c_void_p(self._stream.cuda_stream), _storage(dtype), int(max_seq), C.byref(rc))
        self._made(h, rc, "kfh_seq_create", config, dtype)

    @classmethod
    def from_dir(cls, path, dtype="bfloat16", max_seq=0, device=0):
        """a directory with config.json and model.safetensors"""
        self = cls.__new__(cls)
        self._open(device)
        rc = C.c_int(0)
        st = _storage(dtype)
        h = self.host.kfh_load_hf(str(path).encode(), device, C.c_void_p(self._stream.cuda_stream), st, st, 0, int(max_seq), C.byref(rc))
        with open(os.path.join(str(path), "config.json")) as f:
            self._made(h, rc, "kfh_load_hf(%s)" % path, json.load(f), dtype)
        return self

    def _open(self, device):
        self.hip, self.host = L.load()
        if not torch.cuda.is_available():
            raise L.KFError("no GPU visible: koifish_amd runs on MI355X only (no CPU fallback)")
        torch.cuda.set_device(device)
        self.device, self._stream = torch.device("cuda", device), stream(device)

    def _made(self, h, rc, what, config, dtype):
        if not h:
            raise L.KFError("%s failed with %d: %s" % (what, rc.value, self.host.kfh_last_error().decode()))
        self.h = C.c_void_p(h)
        self._read_config()
        self.config, self.dtype = config, dtype

    def tensors(self):
        """{name: (rows, cols)} of the design; cols 1: a vector"""
        out, name, shape = {}, C.create_string_buffer(256), (C.c_int32 * 2)()
        for i in range(self.host.kfh_seq_tensor(self.h, -1, None, 0, None)):
            self.host.kfh_seq_tensor(self.h, i, name, 256, shape)
            out[name.value.decode()] = (shape[0], shape[1])
        return out

    def set_tensor(self, name, w):
        """w: torch.bfloat16, on the GPU or in host memory, [rows, cols] or [rows]"""
        w = w.contiguous()
        assert w.dtype == torch.bfloat16
        rows, cols = w.shape[0], (w.shape[1] if w.dim() > 1 else 1)
        L.check(self.host.kfh_seq_set_tensor(self.h, name.encode(), rows, cols, C.c_void_p(w.data_ptr()), int(w.is_cuda)), "kfh_seq_set_tensor(%s)" % name)
        if w.is_cuda:
            self.sync()   # the copy reads w on the stream

    def weights_bytes(self):
        """bytes of the design's tensors in this model's storage"""
        return sum(r * c for r, c in self.tensors().values()) * (4 if self.dtype == "float32" else 2)

    def tap(self, n_rows):
        """the residual stream after every layer of the prompt passes of exactly n_rows tokens: an array [layers, n_rows, width] that such a pass fills; tap(0) ends it"""
        if not n_rows:
            L.check(self.host.kfh_seq_tap(self.h, None, 0), "kfh_seq_tap")
            return None
        self._tap = np.zeros((self.cfg["n_layer"], n_rows, self.cfg["dim"]), dtype=np.float32)
        L.check(self.host.kfh_seq_tap(self.h, self._tap.ctypes.data_as(C.c_void_p), int(n_rows)), "kfh_seq_tap")
        return self._tap


class Tizusun(LayeredDecoder):
    """chunked gated attention, post-norm residual, dense or routed feed-forwards (host/kf_tizusun.cpp)"""


class Bolopel(LayeredDecoder):
    """gated delta rule layers and windowed attention beside a decayed sum, normed outputs added to the residual (host/kf_bolopel.cpp)"""


def _storage(dtype):
    try:
        return {"bfloat16": L.BF16, "float32": L.F32}[str(dtype)]
    except KeyError:
        raise L.KFError("dtype %r (bfloat16 or float32)" % (dtype,))


class XcdReplicas:
    """Up to eight independent decoders of ONE model on one GPU, one per XCD (koifish::XcdReplicas over kf_xengine_*): the sequences share the model's weights; each has its
    own KV cache, decode state, forced ids, ids out and logits.  Every sequence's results are bit for bit those of `model.run_steps` for it alone (canonical order)."""

    def __init__(self, model, n_seq=8):
        self.m, self.n_seq = model, int(n_seq)
        self.host, self.hip = model.host, model.hip
        rc = C.c_int(0)
        h = self.host.kfh_xr_create(model.h, self.n_seq, C.byref(rc))
        if not h:
            raise L.KFError("kfh_xr_create failed with %d: %s" % (rc.value, self.host.kfh_host_error().decode() or self.hip.kf_last_error().decode()))
        self.h = C.c_void_p(h)
        model._depends(self)

    def close(self):
        if getattr(self, "h", None):
            self.host.kfh_xr_destroy(self.h)
            self.h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    def set_forced(self, seq, ids):
        a = np.ascontiguousarray(ids, dtype=np.int32)
        L.check(self.host.kfh_xr_set_forced(self.h, int(seq), a.ctypes.data_as(C.c_void_p), a.size), "kfh_xr_set_forced")

    def set_state(self, seq, token, pos):
        L.check(self.host.kfh_xr_set_state(self.h, int(seq), int(token), int(pos)), "kfh_xr_set_state")

    def prefill(self, seq, tokens):
        """the sequence's prompt through the model's batched prefill; its K / V rows into the sequence's cache; the sequence then stands behind the prompt (state = {first generated id, len(tokens)})"""
        t = np.ascontiguousarray(tokens, dtype=np.int32)
        L.check(self.host.kfh_xr_prefill(self.h, int(seq), t.ctypes.data_as(C.c_void_p), t.size), "kfh_xr_prefill")

    def run_steps(self, n):
        """n greedy steps of EVERY sequence from wherever each stands; no host sync"""
        L.check(self.host.kfh_xr_run_steps(self.h, int(n)), "kfh_xr_run_steps")

    def set_steps_per_launch(self, n):
        L.check(self.host.kfh_xr_set_steps_per_launch(self.h, int(n)), "kfh_xr_set_steps_per_launch")

    def check(self):
        L.check(self.host.kfh_xr_check(self.h), "kfh_xr_check")

    @property
    def batch(self):
        """sequences per decoder of the form the engine launches: 1 (<= 8 sequences), 2 (<= 16) or 4 (<= 32): every unpacked block is multiplied against that many sequences' activations"""
        return 1 if self.n_seq <= 8 else (2 if self.n_seq <= 16 else 4)

    decoders_per_xcd = 1

    def park(self, seq, on=True):
        """a parked sequence is skipped by the launches; the others decode on"""
        L.check(self.host.kfh_xr_park(self.h, int(seq), int(bool(on))), "kfh_xr_park")

    def prefill_batch(self, slots, prompts):
        """several prompts at once (one token batch of len(prompts) x longest rows through the tile kernels; a prompt's rows attend to that prompt only): every prompt's
        K / V rows into its slot's cache, the slot stands behind its prompt, the last prompt token's logits in the slot's logits"""
        n = len(prompts)
        lens = np.array([len(p) for p in prompts], dtype=np.int32)
        stride = int(lens.max())
        flat = np.zeros((n, stride), dtype=np.int32)
        for i, p in enumerate(prompts):
            flat[i, :len(p)] = p
        sl = np.ascontiguousarray(slots, dtype=np.int32)
        L.check(self.host.kfh_xr_prefill_batch(self.h, sl.ctypes.data_as(C.c_void_p), flat.ctypes.data_as(C.c_void_p), lens.ctypes.data_as(C.c_void_p), n, stride), "kfh_xr_prefill_batch")

    def set_prefill_batch(self, n):
        """chat(): up to n waiting prompts are prefilled together when as many slots are free (1, the default: one by one -- the bits of the model's own prefill)"""
        L.check(self.host.kfh_xr_set_prefill_batch(self.h, int(n)), "kfh_xr_set_prefill_batch")

    def set_sampler(self, temperature=0.0, top_p=0.95, top_k=50, seed=42, true_topk=False):
        """chat()'s sampler (CHAT_SAMPLER; greedy by default).  Non-greedy: one launch per token leaves every slot's logits, kf_sample draws each slot's id with the slot's own
        rng, seeded with seed + the request's index at the request's start -- answer r == the model alone on prompt r under set_sampler(seed=seed + r)."""
        L.check(self.host.kfh_xr_set_sampler(self.h, float(temperature), float(top_p), int(top_k) | (0x10000 if true_topk else 0), int(seed)), "kfh_xr_set_sampler")

    def chat(self, prompts, max_new, eos=-1, max_new_each=None):
        """a queue of prompts answered through the sequences' slots (Fish::Chat's rounds over its prompt list, GoPT.cpp:1111-1180, n_seq rounds in flight): a free slot
        prefills the next prompt, the launches decode every occupied slot, an answer ends at `eos`, at max_new ids or at the last cache row.
        max_new_each: a limit of its own per request (each <= max_new).
        Returns (list of id lists in the prompts' order, {launches, steps, prefills, dropped})."""
        n = len(prompts)
        lens = np.array([len(p) for p in prompts], dtype=np.int32)
        stride = int(lens.max())
        flat = np.zeros((n, stride), dtype=np.int32)
        for i, p in enumerate(prompts):
            flat[i, :len(p)] = p
        out = np.zeros((n, int(max_new)), dtype=np.int32)
        out_len = np.zeros(n, dtype=np.int32)
        stats = np.zeros(4, dtype=np.int64)
        each = None if max_new_each is None else np.ascontiguousarray(max_new_each, dtype=np.int32)
        assert each is None or each.size == n
        L.check(self.host.kfh_xr_chat_each(self.h, flat.ctypes.data_as(C.c_void_p), lens.ctypes.data_as(C.c_void_p), n, stride, int(max_new), int(eos),
                                           out.ctypes.data_as(C.c_void_p), out_len.ctypes.data_as(C.c_void_p), stats.ctypes.data_as(C.c_void_p),
                                           None if each is None else each.ctypes.data_as(C.c_void_p)), "kfh_xr_chat_each")
        return [out[i, :out_len[i]].tolist() for i in range(n)], dict(zip(("launches", "steps", "prefills", "dropped"), (int(v) for v in stats)))

    # ---- models described layer by layer (LayeredDecoder): requests by slot, any mix of prompts and single tokens in one batch
    def acquire(self):
        """a slot for a new request"""
        s = self.host.kfh_xr_acquire(self.h)
        if s < 0:
            raise L.KFError("no free slot (%d requests live)" % self.n_seq)
        return s

    def release(self, seq):
        """the request in the slot is finished: its state is given back"""
        L.check(self.host.kfh_xr_release(self.h, int(seq)), "kfh_xr_release")

    def run(self, spans, want=()):
        """spans: [(slot, first position, tokens)], the next tokens of several requests as one batch; want: [(span, offset)].  Logits of the wanted rows, float32 [len(want), vocab]"""
        sp = np.array([(s, p, len(t)) for s, p, t in spans], dtype=np.int32).reshape(-1, 3)
        ids = np.concatenate([np.asarray(t, dtype=np.int32) for _, _, t in spans]).astype(np.int32)
        w = np.array(want, dtype=np.int32).reshape(-1, 2)
        out = np.zeros((len(w), self.m.cfg["vocab"]), dtype=np.float32)
        L.check(self.host.kfh_xr_run(self.h, len(sp), sp.ctypes.data_as(C.c_void_p), ids.ctypes.data_as(C.c_void_p), len(w), w.ctypes.data_as(C.c_void_p), out.ctypes.data_as(C.c_void_p)),
                "kfh_xr_run")
        return out

    def status(self, seq):
        """{token, pos, parked, status} of the sequence (status 64: the last launch would have left its cache rows and skipped it)"""
        out = np.zeros(4, dtype=np.int32)
        L.check(self.host.kfh_xr_status(self.h, int(seq), out.ctypes.data_as(C.c_void_p)), "kfh_xr_status")
        return [int(v) for v in out]

    def state(self, seq):
        out = np.zeros(2, dtype=np.int32)
        L.check(self.host.kfh_xr_get_state(self.h, int(seq), out.ctypes.data_as(C.c_void_p)), "kfh_xr_get_state")
        return int(out[0]), int(out[1])

    def tokens_out(self, seq, n):
        out = np.zeros(n, dtype=np.int32)
        L.check(self.host.kfh_xr_get_tokens(self.h, int(seq), out.ctypes.data_as(C.c_void_p), n), "kfh_xr_get_tokens")
        return out

    def _d2h(self, ptr, n_u16):
        out = np.zeros(n_u16, dtype=np.uint16)
        ctx = C.c_void_p(self.host.kfh_ctx(self.m.h))
        L.check(self.hip.kf_d2h(ctx, out.ctypes.data_as(C.c_void_p), C.c_void_p(ptr), C.c_size_t(out.size * 2)), "kf_d2h")
        return out

    def logits(self, seq):
        """the sequence's last logits (bf16 bit patterns as uint16 [vocab])"""
        return self._d2h(self.host.kfh_xr_logits(self.h, int(seq)), self.m.cfg["vocab"])

    def hidden(self, seq):
        return self._d2h(self.host.kfh_xr_hidden(self.h, int(seq)), self.m.cfg["dim"])

    def kv_to_host(self, seq):
        c = self.m.cfg
        kvd = c["n_kv"] * c["head_dim"]
        n = c["n_layer"] * c["max_seq"] * kvd
        shp = (c["n_layer"], c["max_seq"], kvd)
        return self._d2h(self.host.kfh_xr_kcache(self.h, int(seq)), n).reshape(shp), self._d2h(self.host.kfh_xr_vcache(self.h, int(seq)), n).reshape(shp)

    def variant(self, nwv, depth):
        """tuning runs: waves per workgroup x ring depth of the next launches (instantiated pairs only)"""
        self.host.kfh_xr_variant(self.h, int(nwv), int(depth))

    def stamps(self, seq, wg, steps, n_layer):
        """enable (steps > 0) / read the per-phase wall-clock stamps [step][layer][64] of one workgroup of one decoder (diagnostic instantiation)"""
        if steps > 0:
            L.check(self.host.kfh_xr_stamps_enable(self.h, int(seq), int(wg), int(steps)), "kfh_xr_stamps_enable")
            return None
        out = np.zeros((-steps) * n_layer * 64, dtype=np.uint64)
        self.host.kfh_xr_stamps(self.h, out.ctypes.data_as(C.c_void_p), out.size)
        return out.reshape(-steps, n_layer, 64)


class XcdTP:
    """ONE sequence of a model split over eight tensor-parallel ranks, the ranks as the eight XCDs of ONE launch (koifish::XcdTP over kf_xengine_create_tp).  `native_tp`: a
    koifish_amd.tp.NativeTP -- its ranks hold the shards (and stay usable: the per-launch rank step and this engine give the same bits).  K / V rows, state, forced ids, ids
    out and the full logits vector live in this object."""

    def __init__(self, native_tp):
        self.nt = native_tp
        r0 = native_tp.ranks[0]
        self.host, self.hip = r0.host, r0.hip
        self._hs = (C.c_void_p * len(native_tp.ranks))(*[m.h for m in native_tp.ranks])
        rc = C.c_int(0)
        h = self.host.kfh_xtp_create(self._hs, len(native_tp.ranks), C.byref(rc))
        if not h:
            raise L.KFError("kfh_xtp_create failed with %d: %s" % (rc.value, self.host.kfh_host_error().decode() or self.hip.kf_last_error().decode()))
        self.h = C.c_void_p(h)
        for m in native_tp.ranks:
            m._depends(self)

    def close(self):
        if getattr(self, "h", None):
            self.host.kfh_xtp_destroy(self.h)
            self.h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    def set_forced(self, ids):
        a = np.ascontiguousarray(ids, dtype=np.int32)
        L.check(self.host.kfh_xtp_set_forced(self.h, a.ctypes.data_as(C.c_void_p), a.size), "kfh_xtp_set_forced")

    def set_state(self, token, pos):
        L.check(self.host.kfh_xtp_set_state(self.h, int(token), int(pos)), "kfh_xtp_set_state")

    def run_steps(self, n):
        L.check(self.host.kfh_xtp_run_steps(self.h, int(n)), "kfh_xtp_run_steps")

    def set_steps_per_launch(self, n):
        L.check(self.host.kfh_xtp_set_steps_per_launch(self.h, int(n)), "kfh_xtp_set_steps_per_launch")

    def check(self):
        L.check(self.host.kfh_xtp_check(self.h), "kfh_xtp_check")

    def tokens_out(self, n):
        out = np.zeros(n, dtype=np.int32)
        L.check(self.host.kfh_xtp_get_tokens(self.h, out.ctypes.data_as(C.c_void_p), n), "kfh_xtp_get_tokens")
        return out

    def _d2h(self, ptr, n_u16):
        out = np.zeros(n_u16, dtype=np.uint16)
        ctx = C.c_void_p(self.host.kfh_ctx(self.nt.ranks[0].h))
        L.check(self.hip.kf_d2h(ctx, out.ctypes.data_as(C.c_void_p), C.c_void_p(ptr), C.c_size_t(out.size * 2)), "kf_d2h")
        return out

    def logits(self):
        """the last step's logits of the FULL vocabulary (the ranks' shards in rank order), bf16 bit patterns"""
        return self._d2h(self.host.kfh_xtp_logits(self.h), int(self.host.kfh_xtp_vocab(self.h)))

    def hidden(self):
        return self._d2h(self.host.kfh_xtp_hidden(self.h), self.nt.cfg["dim"])

    def kv_to_host(self):
        """[rank][layer][max_seq][head_dim]: rank r = kv-head r's rows"""
        c = self.nt.cfg
        kvd = (c["n_kv"] // len(self.nt.ranks)) * c["head_dim"]
        n = len(self.nt.ranks) * c["n_layer"] * c["max_seq"] * kvd
        shp = (len(self.nt.ranks), c["n_layer"], c["max_seq"], kvd)
        return self._d2h(self.host.kfh_xtp_kcache(self.h), n).reshape(shp), self._d2h(self.host.kfh_xtp_vcache(self.h), n).reshape(shp)

    def variant(self, nwv, depth):
        """tuning builds (-DXE_TP_VARIANTS): another instantiation for the next launches"""
        self.host.kfh_xtp_variant(self.h, int(nwv), int(depth))

    def stamps(self, rank, wg, steps, n_layer):
        """enable (steps > 0) / read the per-phase wall-clock stamps [step][layer][64] of one workgroup of one rank (diagnostic instantiation)"""
        if steps > 0:
            L.check(self.host.kfh_xtp_stamps_enable(self.h, int(rank), int(wg), int(steps)), "kfh_xtp_stamps_enable")
            return None
        n = -steps * n_layer * 64
        out = np.zeros(n, dtype=np.uint64)
        self.host.kfh_xtp_stamps(self.h, out.ctypes.data_as(C.c_void_p), n)
        return out.reshape(-steps, n_layer, 64)
