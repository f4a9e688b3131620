"""Decoder with dense bf16 weights, described layer by layer.  Layers are parallel (attention and feed-forward side by side, below) or
sequential (sublayers one after the other: sublayers.py); embedding, head, portions and state are the same for both.

A parallel layer is  x <- x + mixer(norm(x)) + ff(norm(x)).  Both sublayers read one normed row, and both results are added to
the residual, so a layer is two products:

    [ q | k | v | gate | up ] = W_in norm(x)         one stacked product; `up` leaves it through the activation
    x += W_out [ attention | act ]                   output and down projections side by side along k

    decode    norm + W_in (one GEMV) -> attention (appends the key and value itself) [-> merge of the key splits]
              -> W_out + residual (one GEMV): 3-4 launches per layer, f32 activations throughout
    prefill   norm into the operand type -> W_in (matrix cores) -> KV write -> attention -> W_out + residual

compute "bf16": matrix-core operands in bf16, f16 KV cache, everything else f32.  compute "f32": the same launches with
f32 operands (true 32-bit products) and an f32 KV cache.  The residual stream, norms, scores, softmax, biases and gates
are f32 in both.

Head sizes are padded to multiples of 8 (zero weight rows, zero weight columns behind them) and every k extent to a
multiple of 64, so the kernels see aligned rows whatever the model's sizes are.
"""
import ctypes

import numpy as np
import torch

from . import capi
from .decoder import DecoderBase, _dev_bytes
from .sublayers import ACTIVATIONS, GEMV_MAX_K, Scratch, SequentialLayer, _up, bf16_to_f32, rotary_tables

def f32_to_bf16(x):
    """Round to nearest even; returns uint16 bit patterns."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def _pad_heads(w, heads, size, padded):
    """[heads * size, ...] -> [heads * padded, ...] with zero rows behind every head."""
    if size == padded:
        return w
    out = np.zeros((heads, padded) + w.shape[1:], w.dtype)
    out[:, :size] = w.reshape((heads, size) + w.shape[1:])
    return out.reshape((heads * padded,) + w.shape[1:])


def stack_layer(mixer, mlp, w, hidden):
    """The two stacked matrices of a layer from its own tensors (bf16 bits) and the geometry the kernels are given:
    (W_in bits [N, kx], bias [n_first], W_out bits [hidden, k2], geometry dict)."""
    H, G, d, e = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    D, VD, ff = _up(d, 8), _up(e, 8), mlp["ff"] if mlp else 0
    gate_rows = _up(H, 8) if mixer["gate"] else 0
    kx, k2 = _up(hidden, 64), _up(H * VD + ff, 64)
    geo = dict(D=D, VD=VD, ff=ff, k_offset=H * D, v_offset=(H + G) * D, gate_offset=(H + G) * D + G * VD if mixer["gate"] else -1,
               n_first=(H + G) * D + G * VD + gate_rows, kx=kx, k2=k2, attn_cols=H * VD)
    geo["n"] = geo["n_first"] + ff
    w_in = np.zeros((geo["n"], kx), np.uint16)
    bias = np.zeros(geo["n_first"], np.float32)
    for name, heads, size, padded, at in (("q", H, d, D, 0), ("k", G, d, D, geo["k_offset"]), ("v", G, e, VD, geo["v_offset"])):
        rows = heads * padded
        w_in[at:at + rows, :hidden] = _pad_heads(w[name], heads, size, padded)
        if w.get(name + "_bias") is not None:
            bias[at:at + rows] = _pad_heads(w[name + "_bias"], heads, size, padded)
    if mixer["gate"]:
        w_in[geo["gate_offset"]:geo["gate_offset"] + H, :hidden] = w["gate"]
    w_out = np.zeros((hidden, k2), np.uint16)
    w_out[:, :H * VD] = _pad_heads(np.ascontiguousarray(w["o"].T), H, e, VD).T
    if mlp:
        w_in[geo["n_first"]:, :hidden] = w["up"]
        w_out[:, H * VD:H * VD + ff] = w["down"]
    return w_in, bias, w_out, geo


class DenseDecoder(DecoderBase):
    def __init__(self, cfg, weights, max_seq, compute="bf16", finiteness_guard=False, finiteness_abs_threshold=None):
        """cfg: dict(hidden, vocab, eps, logit_scale, max_positions (0: no position table),
        bigram=dict(buckets, mul_prev, mul_cur) or None,
        layers=[dict(mixer=dict(heads, kv_heads, dim, vdim, window (0: none), scale, log_bias, value_norm, gate),
                     mlp=dict(ff, activation) or None), or a sequential layer: dict(sequential=True, mixer=dict(type, ..),
                     mlp=dict(type, ..) or None)]);
        weights: dict(embed, bigram, pos, head: bf16 bits [rows, hidden]; final_norm f32;
        layers=[dict(norm, q_bias, k_bias, v_bias, bias_r1, bias_r2: f32; q, k, v, gate, o, up, down: bf16 bits [out, in]), or for a
        sequential layer what SequentialLayer takes])."""
        if compute not in ("bf16", "f32"):
            raise ValueError("compute must be 'bf16' or 'f32', got %r" % (compute,))
        if cfg["max_positions"] and max_seq > cfg["max_positions"]:
            raise ValueError("max_seq=%d exceeds the model's %d positions" % (max_seq, cfg["max_positions"]))
        self._init_base(cfg, max_seq, finiteness_guard, finiteness_abs_threshold)
        self.compute = compute
        self.operand = capi.BF16 if compute == "bf16" else capi.F32
        self.operand_torch = torch.bfloat16 if compute == "bf16" else torch.float32
        self.cache_code = capi.F16 if compute == "bf16" else capi.F32
        cache_torch = torch.float16 if compute == "bf16" else torch.float32
        Hd = self.cfg["hidden"]
        self.kx = _up(Hd, 64)
        f32 = lambda n: torch.zeros(n, dtype=torch.float32, device="cuda")

        def padded_f32(v):
            out = np.zeros(self.kx, np.float32)
            out[:Hd] = v
            return _dev_bytes(out)

        self.x = f32(self.kx)                 # residual stream of the step
        self.scratch = Scratch()
        self._rotary = {}
        self.layers = []
        ws = 256
        for spec, w in zip(self.cfg["layers"], weights["layers"]):
            if spec.get("sequential"):
                self.layers.append(SequentialLayer(self, spec, w, self.layers))
                continue
            m, mlp = spec["mixer"], spec["mlp"]
            w_in, bias, w_out, g = stack_layer(m, mlp, w, Hd)
            d = dict(geo=g, w_in=_dev_bytes(w_in), bias=_dev_bytes(bias), w_out=_dev_bytes(w_out), norm=padded_f32(w["norm"]),
                     act=ACTIVATIONS[mlp["activation"] if mlp else None],
                     cache_k=torch.zeros(max_seq * m["kv_heads"] * g["D"], dtype=cache_torch, device="cuda"),
                     cache_v=torch.zeros(max_seq * m["kv_heads"] * g["VD"], dtype=cache_torch, device="cuda"))
            if m["log_bias"]:
                d["r1"], d["r2"] = _dev_bytes(np.asarray(w["bias_r1"], np.float32)), _dev_bytes(np.asarray(w["bias_r2"], np.float32))
            d["spec"] = capi.AttnSpec(m["heads"], m["kv_heads"], g["D"], g["VD"], m["vdim"], m["window"], self.cache_code,
                                      int(bool(m["value_norm"])), g["k_offset"], g["v_offset"], g["gate_offset"], g["n_first"],
                                      m["scale"], self.cfg["eps"], d["r1"].data_ptr() if m["log_bias"] else None,
                                      d["r2"].data_ptr() if m["log_bias"] else None)
            ws = max(ws, int(self.L.dh_attn_spec_workspace_bytes(m["heads"], g["VD"], max_seq)))
            self.layers.append(d)
        self.attn_ws = torch.zeros(ws, dtype=torch.uint8, device="cuda")

        def table(bits):
            return _dev_bytes(bits) if bits is not None else None

        self.embed, self.bigram, self.pos = table(weights["embed"]), table(weights.get("bigram")), table(weights.get("pos"))
        head = np.zeros((self.cfg["vocab"], self.kx), np.uint16)
        head[:, :Hd] = weights["head"]
        self.head = _dev_bytes(head)
        self.final_norm = padded_f32(weights["final_norm"])
        self.recurrent = [t for d in self.layers if isinstance(d, SequentialLayer) for t in d.state()]
        self.qkv_n = max([d["geo"]["n_first"] for d in self._parallel()] + [1])
        self.qkv = f32(self.qkv_n)
        # [attention | act] rows: one buffer per layer shape, so that the padding behind the columns stays zero
        self.mixed = {s: f32(s[1]) for s in self._mixed_shapes()}
        self._pf_rows = 0
        torch.cuda.synchronize()

    def _parallel(self):
        return [d for d in self.layers if not isinstance(d, SequentialLayer)]

    def _recurrent_state(self):
        return self.recurrent

    def rotary(self, base, dims):
        """Device tables of the rotary angles of every position the cache holds, shared by layers with equal rotations."""
        if (base, dims) not in self._rotary:
            self._rotary[base, dims] = tuple(_dev_bytes(t) for t in rotary_tables(base, dims, self.max_seq))
        return self._rotary[base, dims]

    def capture_step(self, pos, want_logits=False, device_kv_len=True):
        if not device_kv_len:
            raise ValueError("captured steps of dense models read the key count on the device")
        return super().capture_step(pos, want_logits)

    def _mixed_shapes(self):
        return {self._mixed_key(d["geo"]) for d in self._parallel()}

    @staticmethod
    def _mixed_key(geo):
        return geo["attn_cols"] + geo["ff"], geo["k2"]

    def weight_bytes_per_token(self, ctx):
        """Algorithmic HBM bytes of one decode step with ctx tokens cached: weights, output head, visible KV rows."""
        elem = 2 if self.compute == "bf16" else 4
        total = self.cfg["vocab"] * self.cfg["hidden"] * 2
        for spec, d in zip(self.cfg["layers"], self.layers):
            if isinstance(d, SequentialLayer):
                total += d.step_bytes(ctx)
                continue
            m, g = spec["mixer"], d["geo"]
            rows = min(ctx, m["window"]) if m["window"] else ctx
            total += 2 * self.cfg["hidden"] * (g["n"] + g["attn_cols"] + g["ff"]) + rows * m["kv_heads"] * (g["D"] + g["VD"]) * elem
        return total

    # ------------------------------------------------------------------ decode step

    def _embed_args(self):
        b = self.cfg["bigram"] or dict(buckets=0, mul_prev=0, mul_cur=0)
        ptr = lambda t: None if t is None else t.data_ptr()
        return (self.embed.data_ptr(), self.cfg["vocab"], ptr(self.bigram), b["buckets"], b["mul_prev"], b["mul_cur"],
                ptr(self.pos), self.cfg["max_positions"])

    def _enqueue_embed(self, ids_ptr, prev_ptr, pos, device_kv_len):
        capi.check(self.L.dh_embed_sum(ids_ptr, 0, prev_ptr, *self._embed_args(), self.x.data_ptr(), self.kx, 1,
                                       self.cfg["hidden"], pos, self.ids.data_ptr() + 4 if device_kv_len else None))

    def _step_row(self):
        return self.x.data_ptr()

    def _enqueue_stack(self, pos, device_kv_len):
        L, c, ck = self.L, self.cfg, capi.check
        kv_len = self.ids.data_ptr() + 4 if device_kv_len else None
        for li, d in enumerate(self.layers):
            if isinstance(d, SequentialLayer):
                d.step(pos, kv_len)
            else:
                self._step_parallel(d, pos, kv_len)
            if self.finiteness_guard:
                ck(L.dh_check_finiteness(self.x.data_ptr(), capi.F32, c["hidden"], self.token.data_ptr() + 4 * self.TOKEN_RING,
                                         li, pos, self.finiteness_abs_threshold))

    def _step_parallel(self, d, pos, kv_len):
        L, c, ck, g = self.L, self.cfg, capi.check, d["geo"]
        mixed = self.mixed[self._mixed_key(g)]
        act = mixed.data_ptr() + 4 * g["attn_cols"] if g["ff"] else None
        if g["kx"] <= GEMV_MAX_K:
            ck(L.dh_dense_gemv(self.x.data_ptr(), d["norm"].data_ptr(), c["hidden"], c["eps"], d["w_in"].data_ptr(), g["kx"],
                               g["n"], g["kx"], 1.0, d["bias"].data_ptr(), None, self.qkv.data_ptr(), g["n_first"], act, d["act"]))
        else:
            self._enqueue_in(d, self.x.data_ptr(), self._wide_row().data_ptr(), capi.F32, self.qkv.data_ptr(), act, 1, g["k2"])
        ck(L.dh_attn_spec_decode(ctypes.byref(d["spec"]), self.qkv.data_ptr(), d["cache_k"].data_ptr(),
                                 d["cache_v"].data_ptr(), mixed.data_ptr(), pos, kv_len, self.max_seq,
                                 self.attn_ws.data_ptr()))
        if g["k2"] <= GEMV_MAX_K:
            ck(L.dh_dense_gemv(mixed.data_ptr(), None, 0, 0.0, d["w_out"].data_ptr(), g["k2"], c["hidden"], g["k2"], 1.0,
                               None, self.x.data_ptr(), self.x.data_ptr(), c["hidden"], None, capi.ACT_NONE))
        else:
            self._enqueue_out(d, mixed.data_ptr(), capi.F32, self.x.data_ptr(), 1)

    def _wide_row(self):
        if getattr(self, "_wide", None) is None:
            self._wide = torch.zeros(self.kx, dtype=torch.float32, device="cuda")
        return self._wide

    def _enqueue_head(self, row_ptr, out_index, logits_ptr):
        c, L = self.cfg, self.L
        if self.kx <= GEMV_MAX_K:
            capi.check(L.dh_dense_lmhead_argmax(row_ptr, self.final_norm.data_ptr(), c["hidden"], c["eps"], self.head.data_ptr(),
                                                self.kx, c["vocab"], self.kx, c["logit_scale"], self.lm_ws.data_ptr(),
                                                self.token.data_ptr(), out_index, logits_ptr))
            return
        logits_ptr = logits_ptr or self.logits.data_ptr()
        wide = self._wide_row().data_ptr()
        capi.check(L.dh_rmsnorm_rows(row_ptr, self.kx, None, self.final_norm.data_ptr(), wide, capi.F32, self.kx, 1, c["hidden"],
                                     c["eps"]))
        capi.check(L.dh_dense_matmul(wide, capi.F32, self.kx, self.head.data_ptr(), self.kx, 1, c["vocab"], self.kx,
                                     c["logit_scale"], None, None, logits_ptr, c["vocab"], c["vocab"], None, 0, 0, capi.ACT_NONE))
        capi.check(L.dh_argmax(logits_ptr, c["vocab"], -1, 0.0, self.lm_ws.data_ptr(), self.token.data_ptr(), out_index))

    # ------------------------------------------------------------------ several rows at once

    def _enqueue_in(self, d, x, normed, operand, qkv, act, rows, ld_act):
        """[q | k | v | gate] rows and activated `up` rows of the residual rows at x."""
        g, c = d["geo"], self.cfg
        capi.check(self.L.dh_rmsnorm_rows(x, self.kx, None, d["norm"].data_ptr(), normed, operand, self.kx, rows, c["hidden"], c["eps"]))
        capi.check(self.L.dh_dense_matmul(normed, operand, self.kx, d["w_in"].data_ptr(), g["kx"], rows, g["n"], g["kx"], 1.0,
                                          d["bias"].data_ptr(), None, qkv, g["n_first"], g["n_first"], act, operand, ld_act,
                                          d["act"]))

    def _enqueue_out(self, d, mixed, operand, x, rows):
        g, Hd = d["geo"], self.cfg["hidden"]
        capi.check(self.L.dh_dense_matmul(mixed, operand, g["k2"], d["w_out"].data_ptr(), g["k2"], rows, Hd, g["k2"], 1.0, None, x,
                                          x, self.kx, Hd, None, 0, 0, capi.ACT_NONE))

    def _prefill_chunk(self, ids, pos, rows):
        """A portion through the batched path.  rows: the most rows a portion of this prompt has."""
        L, c, ck = self.L, self.cfg, capi.check
        if self._pf_rows < rows:
            zeros = lambda n, t: torch.zeros(n, dtype=t, device="cuda")
            self._pf = dict(x=zeros(rows * self.kx, torch.float32), normed=zeros(rows * self.kx, self.operand_torch),
                            qkv=zeros(rows * self.qkv_n, torch.float32),
                            mixed={s: zeros(rows * s[1], self.operand_torch) for s in self._mixed_shapes()},
                            ids=zeros(rows + 1, torch.int32))
            self._pf_rows = rows
        b, T = self._pf, ids.size
        x = b["x"].data_ptr()
        up = np.concatenate([np.array([self._before(pos)], np.uint32), ids])      # the token before the portion, then its own
        ck(L.dh_upload(b["ids"].data_ptr(), 0, up.ctypes.data, up.nbytes))
        ck(L.dh_embed_sum(b["ids"].data_ptr(), 1, b["ids"].data_ptr(), *self._embed_args(), x, self.kx, T, c["hidden"], pos, None))
        elem = b["normed"].element_size()
        for d in self.layers:
            if isinstance(d, SequentialLayer):
                d.rows(x, T, pos)
                continue
            g = d["geo"]
            mixed = b["mixed"][self._mixed_key(g)].data_ptr()
            self._enqueue_in(d, x, b["normed"].data_ptr(), self.operand, b["qkv"].data_ptr(),
                             mixed + elem * g["attn_cols"] if g["ff"] else None, T, g["k2"])
            ck(L.dh_attn_spec_kv_write(ctypes.byref(d["spec"]), b["qkv"].data_ptr(), d["cache_k"].data_ptr(),
                                       d["cache_v"].data_ptr(), T, pos))
            ck(L.dh_attn_spec_prefill(ctypes.byref(d["spec"]), b["qkv"].data_ptr(), d["cache_k"].data_ptr(),
                                      d["cache_v"].data_ptr(), mixed, self.operand, g["k2"], T, pos))
            self._enqueue_out(d, mixed, self.operand, x, T)
        return x, self.kx

    def _logit_rows(self, base, stride, rows):
        c, L = self.cfg, self.L
        n = len(rows)
        idx = np.array(rows, np.uint32)
        d_idx = torch.zeros(n, dtype=torch.int32, device="cuda")
        normed = torch.zeros(n * self.kx, dtype=self.operand_torch, device="cuda")
        logits = torch.zeros(n * c["vocab"], dtype=torch.float32, device="cuda")
        capi.check(L.dh_upload(d_idx.data_ptr(), 0, idx.ctypes.data, idx.nbytes))
        capi.check(L.dh_rmsnorm_rows(base, stride, d_idx.data_ptr(), self.final_norm.data_ptr(), normed.data_ptr(), self.operand,
                                     self.kx, n, c["hidden"], c["eps"]))
        capi.check(L.dh_dense_matmul(normed.data_ptr(), self.operand, self.kx, self.head.data_ptr(), self.kx, n, c["vocab"],
                                     self.kx, c["logit_scale"], None, None, logits.data_ptr(), c["vocab"], c["vocab"], None, 0,
                                     0, capi.ACT_NONE))
        out = np.empty((n, c["vocab"]), np.float32)
        capi.check(L.dh_download(out.ctypes.data, logits.data_ptr(), 0, out.nbytes))
        return out

    def read_kv(self, layer, rows):
        """Cached keys and values of the first rows: f32 [rows, kv_heads, padded head size] each."""
        d, m = self.layers[layer], self.cfg["layers"][layer]["mixer"]
        out = []
        for name, size in (("cache_k", d["geo"]["D"]), ("cache_v", d["geo"]["VD"])):
            a = np.empty((rows, m["kv_heads"], size), np.float16 if self.compute == "bf16" else np.float32)
            capi.check(self.L.dh_download(a.ctypes.data, d[name].data_ptr(), 0, a.nbytes))
            out.append(a.astype(np.float32))
        return tuple(out)


def random_weights(cfg, seed=0, score_gain=1.0):
    """Random-init weights of a dense decoder: linears N(0, 1/in), norms N(1, 0.02), tables N(0, 1); keys and queries
    scaled by score_gain."""
    g = np.random.Generator(np.random.PCG64(seed))
    Hd = cfg["hidden"]

    def lin(n, k, gain=1.0):
        return f32_to_bf16(g.standard_normal((n, k), dtype=np.float32) * np.float32(gain / np.sqrt(k)))

    def vec(n, mean=0.0, std=0.02):
        return bf16_to_f32(f32_to_bf16(mean + std * g.standard_normal(n, dtype=np.float32)))

    layers = []
    for spec in cfg["layers"]:
        m, mlp = spec["mixer"], spec["mlp"]
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        w = dict(norm=vec(Hd, 1.0), q=lin(H * d, Hd, score_gain), k=lin(G * d, Hd, score_gain), v=lin(G * e, Hd),
                 q_bias=vec(H * d, 0.0, 0.2), k_bias=vec(G * d, 0.0, 0.2), v_bias=vec(G * e, 0.0, 0.2), o=lin(Hd, H * e))
        if m["gate"]:
            w["gate"] = lin(H, Hd)
        if m["log_bias"]:
            w["bias_r1"] = bf16_to_f32(f32_to_bf16(g.uniform(0.02, 1.2, H).astype(np.float32)))
            w["bias_r2"] = bf16_to_f32(f32_to_bf16(g.uniform(0.05, 0.6, H).astype(np.float32)))
        if mlp:
            w["up"], w["down"] = lin(mlp["ff"], Hd), lin(Hd, mlp["ff"])
        layers.append(w)
    b = cfg["bigram"]
    table = lambda n: f32_to_bf16(g.standard_normal((n, Hd), dtype=np.float32))
    return dict(embed=table(cfg["vocab"]), bigram=table(b["buckets"] + 1) if b else None,
                pos=table(cfg["max_positions"]) if cfg["max_positions"] else None, head=lin(cfg["vocab"], Hd),
                final_norm=vec(Hd, 1.0), layers=layers)
