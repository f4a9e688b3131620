"""Layers whose sublayers run one after the other, for the dense decoder:

    x <- x + ls1 * mixer(norm1(x));   x <- x + ls2 * ff(norm2(x))

    mixers          LatentAttention   windowed softmax attention over a low-rank latent; the latent rows may be another layer's
                    MatrixMemory      mLSTM: matrix-valued recurrent state with exponential gates
    feed-forwards   DenseFF           two products around an activation
                    ExpertsFF         sigmoid-routed experts with clamped gates, and a gated shared expert

A sublayer stacks and pads its own tensors (zeros: padded rows and columns contribute nothing), owns its cache rows or state, and
runs on the decoder's residual in two ways: step() for one token, rows() for a portion.  Projections that read the normed row are one
product; the layer scale and the residual belong to the epilogue of the last one.
"""
import ctypes

import numpy as np
import torch

from . import capi
from .decoder import _dev_bytes

ACTIVATIONS = {"relu2": capi.ACT_RELU2, "silu": capi.ACT_SILU, "gelu_tanh": capi.ACT_GELU, "gelu_erf": capi.ACT_GELU_ERF,
               None: capi.ACT_NONE}
GEMV_MAX_K, GEMV_MAX_HEADS = 32768, 256


def _up(n, m):
    return (n + m - 1) // m * m


def bf16_to_f32(bits):
    return (np.ascontiguousarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


def place(shape, *parts):
    """Zeros of `shape` (of the first part's dtype) with every (index, array) written in."""
    out = np.zeros(shape, parts[0][1].dtype)
    for index, a in parts:
        out[index] = a
    return out


def pad_out(o, hidden, heads, size, padded, k):
    """Output projection [hidden, heads * size] -> [hidden, k] with heads `padded` columns apart."""
    spread = place((hidden, heads, padded), ((Ellipsis, slice(0, size)), np.asarray(o).reshape(hidden, heads, size)))
    return place((hidden, k), ((slice(None), slice(0, heads * padded)), spread.reshape(hidden, heads * padded)))


class Scratch:
    """Buffers all layers share, by name and row width (so that what lies behind a row's elements stays zero), grown to the most
    rows asked for."""

    def __init__(self):
        self.buffers = {}

    def rows(self, name, width, count, dtype):
        key = (name, width, dtype)
        if key not in self.buffers or self.buffers[key].numel() < width * count:
            self.buffers[key] = torch.zeros(width * count, dtype=dtype, device="cuda")
            torch.cuda.synchronize()
        return self.buffers[key].data_ptr()

    def space(self, name, nbytes):
        return self.rows(name, 1, _up(nbytes, 256), torch.uint8)


def rotary_tables(base, dims, positions):
    """cos and sin [positions][dims / 2] of the angles p base^(-2 i / dims), computed in double."""
    a = np.arange(positions)[:, None] * np.float64(base) ** (-2.0 * np.arange(dims // 2) / dims)
    return np.cos(a).astype(np.float32), np.sin(a).astype(np.float32)


class _Sublayer:
    """dec: the decoder (sizes, residual row, operand type, library); norm: the sublayer's norm weights; ls: layer scale or None."""

    def __init__(self, dec, norm, ls):
        self.dec, self.hidden, self.kx, self.eps = dec, dec.cfg["hidden"], dec.kx, dec.cfg["eps"]
        self.norm = _dev_bytes(place(self.kx, (slice(0, self.hidden), np.asarray(norm, np.float32))))
        self.ls = None if ls is None else _dev_bytes(np.ascontiguousarray(ls, np.float32))
        self.ls_ptr = None if ls is None else self.ls.data_ptr()

    def _check_row(self, k):
        if k > GEMV_MAX_K:
            raise ValueError("rows of %d elements are longer than the %d a decode step holds" % (k, GEMV_MAX_K))

    def _gemv(self, x, normed, w, n, k, bias=None, out=None, act_out=None, act=capi.ACT_NONE, residual=False):
        """One row x through w [n][k] into out, or through the activation into act_out."""
        x_out = self.dec.x.data_ptr() if residual else out
        capi.check(self.dec.L.dh_dense_gemv_scaled(x, self.norm.data_ptr() if normed else None, self.hidden, self.eps, w.data_ptr(), k, n,
                                                   k, 1.0, bias, self.ls_ptr if residual else None, x_out if residual else None, x_out,
                                                   n if act_out is None else 0, act_out, act))

    def _normed_rows(self, x, count):
        """Normed residual rows in the operand type."""
        d = self.dec
        out = d.scratch.rows("normed", self.kx, count, d.operand_torch)
        capi.check(d.L.dh_rmsnorm_rows(x, self.kx, None, self.norm.data_ptr(), out, d.operand, self.kx, count, self.hidden, self.eps))
        return out

    def _out_rows(self, a, k, w, x, count):
        """x += ls * W a over rows of k elements."""
        capi.check(self.dec.L.dh_dense_matmul_scaled(a, self.dec.operand, k, w.data_ptr(), k, count, self.hidden, k, 1.0, None, self.ls_ptr, x,
                                                     x, self.kx, self.hidden, None, 0, 0, capi.ACT_NONE))

    def state(self):
        """Recurrent buffers."""
        return []

    def step_bytes(self, ctx):
        """Bytes of weights, cache rows and state a step with ctx cached tokens has to move."""
        raise NotImplementedError


class LatentAttention(_Sublayer):
    """m: heads, dim, rot_dim, vdim, kv_rank, window (0: none), scale, rot_base; w: q, uk, uv, o and, unless `lender` (the layer
    whose rows are used) is given, dkv and latent_norm."""

    def __init__(self, dec, m, w, norm, ls, lender=None):
        super().__init__(dec, norm, ls)
        H, d, rot, e, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        D, R, VD, C = _up(d, 8), _up(rot, 32), _up(e, 8), _up(rank, 64)
        self.m, self.lender, self.width = m, lender, C + R
        q_rows = H * (D + R)
        self.n_in = q_rows + (0 if lender else C + R)
        self.ld = _up(max(self.n_in, H * VD), 8)
        self.k2 = _up(H * VD, 64)
        self._check_row(max(self.kx, self.k2))
        q = np.asarray(w["q"]).reshape(H, d + rot, self.hidden)
        w_in = np.zeros((self.n_in, self.kx), np.uint16)
        heads = w_in[:q_rows].reshape(H, D + R, self.kx)
        heads[:, :d, :self.hidden], heads[:, D:D + rot, :self.hidden] = q[:, :d], q[:, d:]
        if not lender:
            w_in[q_rows:q_rows + rank, :self.hidden] = w["dkv"][:rank]
            w_in[q_rows + C:q_rows + C + rot, :self.hidden] = w["dkv"][rank:]
        uk = place((H, D, C), ((slice(None), slice(0, d), slice(0, rank)), np.asarray(w["uk"]).reshape(H, d, rank)))
        uv = place((H, VD, C), ((slice(None), slice(0, e), slice(0, rank)), np.asarray(w["uv"]).reshape(H, e, rank)))
        half = dec.compute == "bf16"
        wide = (lambda a: bf16_to_f32(a).astype(np.float16)) if half else (lambda a: a)
        self.w_in = _dev_bytes(w_in)
        self.w_out = _dev_bytes(pad_out(w["o"], self.hidden, H, e, VD, self.k2))
        self.uk, self.uv = _dev_bytes(wide(uk)), _dev_bytes(wide(uv))
        self.uk_t, self.uv_rows = _dev_bytes(np.ascontiguousarray(uk.transpose(0, 2, 1))), _dev_bytes(uv) if half else self.uv
        if lender:
            self.cache = lender.cache
        else:
            self.latent_norm = _dev_bytes(np.ascontiguousarray(w["latent_norm"], np.float32))
            # the products read whole k tiles: what they touch behind the last row is zero too
            self.cache = torch.zeros((dec.max_seq + 1) * self.width, dtype=torch.float16 if half else torch.float32, device="cuda")
        cos, sin = dec.rotary(m["rot_base"], rot)
        self.spec = capi.Latent(H, D, R, VD, rank, C, rot, m["window"], dec.cache_code, -1 if lender else q_rows, self.ld, m["scale"],
                                self.eps, None if lender else self.latent_norm.data_ptr(), cos.data_ptr(), sin.data_ptr(),
                                self.uk.data_ptr(), self.uv.data_ptr(), self.uk_t.data_ptr(), self.uv_rows.data_ptr())
        self.ref = ctypes.byref(self.spec)
        dec.scratch.space("latent_decode", dec.L.dh_latent_decode_workspace_bytes(self.ref, dec.max_seq))
        dec.scratch.rows("row", self.ld, 1, torch.float32)
        dec.scratch.rows("mixed", self.k2, 1, torch.float32)

    def step(self, pos, kv_len):
        d = self.dec
        row, mixed = d.scratch.rows("row", self.ld, 1, torch.float32), d.scratch.rows("mixed", self.k2, 1, torch.float32)
        self._gemv(d.x.data_ptr(), True, self.w_in, self.n_in, self.kx, out=row)
        capi.check(d.L.dh_latent_decode(self.ref, row, self.cache.data_ptr(), mixed, pos, kv_len, d.max_seq, d.scratch.space("latent_decode", 1)))
        self._gemv(mixed, False, self.w_out, self.hidden, self.k2, residual=True)

    def rows(self, x, count, pos):
        d = self.dec
        normed = self._normed_rows(x, count)
        rows = d.scratch.rows("rows", self.ld, count, torch.float32)
        capi.check(d.L.dh_dense_matmul(normed, d.operand, self.kx, self.w_in.data_ptr(), self.kx, count, self.n_in, self.kx, 1.0, None, None, rows,
                                       self.ld, self.n_in, None, 0, 0, capi.ACT_NONE))
        capi.check(d.L.dh_latent_rows(self.ref, rows, self.cache.data_ptr(), count, pos))
        mixed = d.scratch.rows("mixed_rows", self.k2, count, d.operand_torch)
        ws = d.scratch.space("latent_prefill", d.L.dh_latent_prefill_workspace_bytes(self.ref, count, pos))
        capi.check(d.L.dh_latent_prefill(self.ref, rows, self.cache.data_ptr(), ws, mixed, d.operand, self.k2, count, pos))
        self._out_rows(mixed, self.k2, self.w_out, x, count)

    def step_bytes(self, ctx):
        m = self.m
        keys = min(ctx, m["window"]) if m["window"] else ctx
        return 2 * (self.n_in * self.hidden + self.hidden * m["heads"] * m["vdim"] + m["heads"] * m["kv_rank"] * (m["dim"] + m["vdim"])) + \
            keys * self.width * self.cache.element_size()


class MatrixMemory(_Sublayer):
    """m: heads, dim, vdim, gate_cap; w: q, k, v, g, i, f, o (bits), i_bias, f_bias, head_norm (f32)."""

    def __init__(self, dec, m, w, norm, ls):
        super().__init__(dec, norm, ls)
        H, d, e = m["heads"], m["dim"], m["vdim"]
        DP, VP = _up(d, 32), _up(e, 32)
        self.m, self.VP, self.o_width = m, VP, H * VP
        at = dict(q=0, k=H * DP, v=2 * H * DP, g=2 * H * DP + H * VP, i=2 * H * (DP + VP), f=2 * H * (DP + VP) + _up(H, 4))
        self.g_off, self.n_in = at["g"], at["f"] + _up(H, 4)
        self.k2 = _up(H * VP, 64)
        self._check_row(max(self.kx, self.k2))
        w_in, bias = np.zeros((self.n_in, self.kx), np.uint16), np.zeros(self.n_in, np.float32)
        for name, size, padded in (("q", d, DP), ("k", d, DP), ("v", e, VP), ("g", e, VP)):
            w_in[at[name]:at[name] + H * padded].reshape(H, padded, self.kx)[:, :size, :self.hidden] = np.asarray(w[name]).reshape(H, size, self.hidden)
        for name in ("i", "f"):
            w_in[at[name]:at[name] + H, :self.hidden] = w[name]
            bias[at[name]:at[name] + H] = w[name + "_bias"]
        self.w_in, self.bias = _dev_bytes(w_in), _dev_bytes(bias)
        self.w_out = _dev_bytes(pad_out(w["o"], self.hidden, H, e, VP, self.k2))
        self.head_norm = _dev_bytes(place((H, VP), ((slice(None), slice(0, e)), np.asarray(w["head_norm"], np.float32).reshape(H, e))))
        self.spec = capi.MLSTM(H, d, e, DP, VP, at["k"], at["v"], at["i"], at["f"], self.n_in, m["gate_cap"])
        self.ref = ctypes.byref(self.spec)
        self.memory = torch.zeros(int(dec.L.dh_mlstm_state_bytes(self.ref)), dtype=torch.uint8, device="cuda")
        dec.scratch.rows("row", self.n_in, 1, torch.float32)
        dec.scratch.rows("heads", self.o_width, 1, torch.float32)
        dec.scratch.rows("mixed", self.k2, 1, torch.float32)

    def state(self):
        return [self.memory]

    def _norm_gate(self, o, rows, out, dtype, count):
        m = self.m
        capi.check(self.dec.L.dh_head_norm_gate(o, self.o_width, rows + 4 * self.g_off, self.n_in, self.head_norm.data_ptr(), out, dtype, self.k2,
                                                count, m["heads"], self.VP, m["vdim"], self.eps))

    def step(self, pos, kv_len):
        d, f = self.dec, torch.float32
        row, o = d.scratch.rows("row", self.n_in, 1, f), d.scratch.rows("heads", self.o_width, 1, f)
        self._gemv(d.x.data_ptr(), True, self.w_in, self.n_in, self.kx, bias=self.bias.data_ptr(), out=row)
        capi.check(d.L.dh_mlstm_step(self.ref, row, self.memory.data_ptr(), o, pos, kv_len))
        self._out_step(o, row)

    def _out_step(self, o, row):
        d, m = self.dec, self.m
        if m["heads"] <= GEMV_MAX_HEADS:
            capi.check(d.L.dh_dense_gemv_heads(o, row + 4 * self.g_off, self.head_norm.data_ptr(), m["heads"], self.VP, m["vdim"], self.eps,
                                               self.w_out.data_ptr(), self.k2, self.hidden, self.k2, self.ls_ptr, d.x.data_ptr(), d.x.data_ptr()))
            return
        mixed = d.scratch.rows("mixed", self.k2, 1, torch.float32)
        self._norm_gate(o, row, mixed, capi.F32, 1)
        self._gemv(mixed, False, self.w_out, self.hidden, self.k2, residual=True)

    def rows(self, x, count, pos):
        d = self.dec
        normed = self._normed_rows(x, count)
        rows = d.scratch.rows("rows", self.n_in, count, torch.float32)
        capi.check(d.L.dh_dense_matmul(normed, d.operand, self.kx, self.w_in.data_ptr(), self.kx, count, self.n_in, self.kx, 1.0,
                                       self.bias.data_ptr(), None, rows, self.n_in, self.n_in, None, 0, 0, capi.ACT_NONE))
        o = d.scratch.rows("heads_rows", self.o_width, count, torch.float32)
        ws = d.scratch.space("mlstm_prefill", d.L.dh_mlstm_prefill_workspace_bytes(self.ref, count))
        capi.check(d.L.dh_mlstm_prefill(self.ref, rows, self.memory.data_ptr(), ws, o, self.o_width, count, pos))
        mixed = d.scratch.rows("mixed_rows", self.k2, count, d.operand_torch)
        self._norm_gate(o, rows, mixed, d.operand, count)
        self._out_rows(mixed, self.k2, self.w_out, x, count)

    def step_bytes(self, ctx):
        m = self.m
        H, d, e = m["heads"], m["dim"], m["vdim"]
        return 2 * self.hidden * H * (2 * d + 3 * e + 2) + 8 * H * d * (e + 1)


class DenseFF(_Sublayer):
    """m: ff, activation; w: up, down."""

    def __init__(self, dec, m, w, norm, ls):
        super().__init__(dec, norm, ls)
        self.ff, self.ffp, self.act = m["ff"], _up(m["ff"], 64), ACTIVATIONS[m["activation"]]
        self._check_row(max(self.kx, self.ffp))
        self.up = _dev_bytes(place((self.ff, self.kx), ((slice(None), slice(0, self.hidden)), np.asarray(w["up"]))))
        self.down = _dev_bytes(place((self.hidden, self.ffp), ((slice(None), slice(0, self.ff)), np.asarray(w["down"]))))
        dec.scratch.rows("act", self.ffp, 1, torch.float32)

    def step(self, pos, kv_len):
        d = self.dec
        act = d.scratch.rows("act", self.ffp, 1, torch.float32)
        self._gemv(d.x.data_ptr(), True, self.up, self.ff, self.kx, act_out=act, act=self.act)
        self._gemv(act, False, self.down, self.hidden, self.ffp, residual=True)

    def rows(self, x, count, pos):
        d = self.dec
        normed = self._normed_rows(x, count)
        act = d.scratch.rows("act_rows", self.ffp, count, d.operand_torch)
        capi.check(d.L.dh_dense_matmul(normed, d.operand, self.kx, self.up.data_ptr(), self.kx, count, self.ff, self.kx, 1.0, None, None, None, 0, 0,
                                       act, d.operand, self.ffp, self.act))
        self._out_rows(act, self.ffp, self.down, x, count)

    def step_bytes(self, ctx):
        return 4 * self.hidden * self.ff


def interleave_gate_up(gate, up, k):
    """[.., ff, n] gate and up rows -> [.., 2 ffp, k]: 32 gate rows, the same 32 up rows, the next 32 gate rows, ..; ff padded to 64."""
    lead, ff, n = gate.shape[:-2], gate.shape[-2], gate.shape[-1]
    ffp = _up(ff, 64)
    out = np.zeros(lead + (ffp // 32, 2, 32, k), gate.dtype)
    for i, a in enumerate((gate, up)):
        out[..., i, :, :n] = place(lead + (ffp, n), ((Ellipsis, slice(0, ff), slice(None)), a)).reshape(lead + (ffp // 32, 32, n))
    return out.reshape(lead + (2 * ffp, k))


class ExpertsFF(_Sublayer):
    """m: experts, top, ff, limit, shared (ff, limit) or None; w: router [E, hidden], gate, up [E, ff, hidden], down [E, hidden, ff] and
    shared_gate, shared_up, shared_down, shared_sg."""

    def __init__(self, dec, m, w, norm, ls):
        super().__init__(dec, norm, ls)
        E, ff, shared = m["experts"], m["ff"], m.get("shared")
        self.m, self.ffp, self.sfp = m, _up(ff, 64), _up(shared["ff"], 64) if shared else 0
        self._check_row(max(self.kx, m["top"] * self.ffp + self.sfp))
        router = np.zeros((E + (1 if shared else 0), self.kx), np.uint16)
        router[:E, :self.hidden] = w["router"]
        if shared:
            router[E, :self.hidden] = np.asarray(w["shared_sg"]).reshape(-1)
        self.router = _dev_bytes(router)
        pad_down = lambda a, ffp: place(a.shape[:-1] + (ffp,), ((Ellipsis, slice(0, a.shape[-1])), a))
        self.up, self.down = _dev_bytes(interleave_gate_up(w["gate"], w["up"], self.kx)), _dev_bytes(pad_down(w["down"], self.ffp))
        self.shared_up = _dev_bytes(interleave_gate_up(w["shared_gate"], w["shared_up"], self.kx)) if shared else None
        self.shared_down = _dev_bytes(pad_down(w["shared_down"], self.sfp)) if shared else None
        self.spec = capi.Experts(self.hidden, self.kx, E, m["top"], self.ffp, self.sfp, self.eps, m["limit"], shared["limit"] if shared else 0.0,
                                 self.norm.data_ptr(), self.ls_ptr, self.router.data_ptr(), self.up.data_ptr(), self.down.data_ptr(),
                                 self.shared_up.data_ptr() if shared else None, self.shared_down.data_ptr() if shared else None)
        self.ref = ctypes.byref(self.spec)
        self.ws_bytes = int(dec.L.dh_experts_step_workspace_bytes(self.ref))
        dec.scratch.space("experts_step", self.ws_bytes)

    def step(self, pos, kv_len):
        d = self.dec
        capi.check(d.L.dh_experts_step(self.ref, d.x.data_ptr(), d.scratch.space("experts_step", self.ws_bytes)))

    def rows(self, x, count, pos):
        d = self.dec
        normed = self._normed_rows(x, count)
        ws = d.scratch.space("experts_prefill", d.L.dh_experts_prefill_workspace_bytes(self.ref, d.operand, count))
        capi.check(d.L.dh_experts_prefill(self.ref, normed, d.operand, x, self.kx, ws, count))

    def step_bytes(self, ctx):
        m = self.m
        shared = m["shared"]["ff"] if m.get("shared") else 0
        return 2 * self.hidden * (m["experts"] + 3 * (m["top"] * m["ff"] + shared))


MIXERS = {"latent_attention": LatentAttention, "mlstm": MatrixMemory}
FEED_FORWARDS = {"dense": DenseFF, "experts": ExpertsFF}


class SequentialLayer:
    """spec: dict(mixer=dict(type, ..), mlp=dict(type, ..) or None); w: dict(norm1, ls1, mixer tensors, norm2, ls2, mlp tensors).
    earlier: the decoder's layers so far (one of them may lend its latent rows)."""

    def __init__(self, dec, spec, w, earlier):
        m, mlp = spec["mixer"], spec["mlp"]
        lend = {} if m.get("kv_from") is None else {"lender": earlier[m["kv_from"]].mixer}
        self.mixer = MIXERS[m["type"]](dec, m, w["mixer"], w["norm1"], w.get("ls1"), **lend)
        self.ff = FEED_FORWARDS[mlp["type"]](dec, mlp, w["mlp"], w["norm2"], w.get("ls2")) if mlp else None
        self.parts = [p for p in (self.mixer, self.ff) if p is not None]

    def step(self, pos, kv_len):
        for p in self.parts:
            p.step(pos, kv_len)

    def rows(self, x, count, pos):
        for p in self.parts:
            p.rows(x, count, pos)

    def state(self):
        return [t for p in self.parts for t in p.state()]

    def step_bytes(self, ctx):
        return sum(p.step_bytes(ctx) for p in self.parts)
