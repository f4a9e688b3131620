"""Throughput of a design beside the closest decoder the package serves, at sizes that resemble a real model's layers.

Gusolorn (sequential layers: latent attention with a dense feed-forward, two of matrix memory with experts, and again) against
Zepavik with the same width, heads, layer count, window and active feed-forward width.  Zepavik (dense bf16, parallel layers, windowed
attention) against the Q4_K decoder with the same width, heads, feed-forward width and layer count.  Prefill and decode tokens/s, and
per kernel the share of its roofline (8 TB/s of HBM, 2.5 PFLOP/s on the matrix cores, 157 TFLOP/s for 32-bit products).  Random
weights; kernels cycle through more weights than the caches hold.
"""
import ctypes
import sys
import time

import numpy as np
import torch

HBM_GBPS, MFMA_TFLOPS, MFMA_F32_TFLOPS = 8000.0, 2500.0, 157.3
SIZES = {
    "1024": dict(hidden=1024, heads=16, kv_heads=8, head_dim=64, ff=3072, layers=24),
    "2048": dict(hidden=2048, heads=16, kv_heads=8, head_dim=128, ff=6144, layers=12),
    "4096": dict(hidden=4096, heads=32, kv_heads=8, head_dim=128, ff=12288, layers=6),
}
# what the second design's mixers add to a size: latent (dim, rotated, value, rank), memory (heads, dim, value), experts (count, top)
MIXED = {
    "1024": dict(latent=(64, 32, 64, 256), memory=(4, 128, 256), experts=(16, 4)),
    "2048": dict(latent=(128, 64, 128, 512), memory=(4, 256, 512), experts=(16, 4)),
    "4096": dict(latent=(128, 64, 128, 512), memory=(8, 256, 512), experts=(16, 4)),
}
VOCAB, WINDOW, PROMPT = 32000, 1024, 2048


def log(*a):
    print(*a, file=sys.stderr, flush=True)


def zepavik_config(s, max_seq):
    mixer = dict(heads=s["heads"], kv_heads=s["kv_heads"], dim=s["head_dim"], vdim=s["head_dim"], window=WINDOW,
                 scale=s["head_dim"] ** -0.5, log_bias=True, value_norm=True, gate=True)
    return dict(hidden=s["hidden"], vocab=VOCAB, eps=1e-5, logit_scale=1.0, max_positions=max_seq,
                bigram=dict(buckets=4096, mul_prev=31, mul_cur=7),
                layers=[dict(mixer=dict(mixer), mlp=dict(ff=s["ff"], activation="relu2")) for _ in range(s["layers"])])


def gusolorn_config(s, mixed):
    d, rot, e, rank = mixed["latent"]
    H, md, me = mixed["memory"]
    E, top = mixed["experts"]
    latent = dict(type="latent_attention", heads=s["heads"], dim=d, rot_dim=rot, vdim=e, kv_rank=rank, window=WINDOW, scale=(d + rot) ** -0.5,
                  rot_base=10000.0, kv_from=None)
    memory = dict(type="mlstm", heads=H, dim=md, vdim=me, gate_cap=15.0)
    experts = dict(type="experts", experts=E, top=top, ff=s["ff"] // 2 // top, limit=7.0, shared=dict(ff=s["ff"] // 2, limit=7.0))
    layers = []
    for i in range(s["layers"]):
        if i % 3 == 0:      # every second latent layer borrows the rows of the one before it
            layers.append(dict(sequential=True, mixer=dict(latent, kv_from=i - 3 if i % 6 == 3 else None),
                               mlp=dict(type="dense", ff=s["ff"], activation="gelu_erf")))
        else:
            layers.append(dict(sequential=True, mixer=dict(memory), mlp=dict(experts)))
    return dict(hidden=s["hidden"], vocab=VOCAB, eps=1e-6, logit_scale=1.0, max_positions=0, bigram=None, layers=layers)


def q4k_config(s, max_seq):
    return dict(layers=s["layers"], hidden=s["hidden"], inter=s["ff"], heads=s["heads"], kv_heads=s["kv_heads"],
                head_dim=s["head_dim"], vocab=VOCAB, eps=1e-6, qk_norm=1, theta=1e6, max_seq=max_seq)


class _Timer:
    def __init__(self, L):
        from . import capi
        self.L, self.ck = L, capi.check
        self.ev = [ctypes.c_void_p() for _ in range(2)]
        for e in self.ev:
            self.ck(L.dh_event_create(ctypes.byref(e)))

    def us(self, calls, reps=3):
        """Fastest sweep over the calls, per call."""
        for c in calls:
            c()
        self.ck(self.L.dh_sync())
        best = float("inf")
        for _ in range(reps):
            self.ck(self.L.dh_event_record(self.ev[0]))
            for c in calls:
                c()
            self.ck(self.L.dh_event_record(self.ev[1]))
            ms = ctypes.c_float()
            self.ck(self.L.dh_event_elapsed_ms(self.ev[0], self.ev[1], ctypes.byref(ms)))
            best = min(best, ms.value / len(calls))
        return best * 1e3

    def close(self):
        for e in self.ev:
            self.ck(self.L.dh_event_destroy(e))


def _throughput(dec, prompt, steps, warmup):
    """(prefill tokens/s, decode tokens/s) of a decoder through its own prefill and generation loop."""
    dec.prefill(prompt, chunk=PROMPT)
    dec.L.dh_sync()
    t0 = time.perf_counter()
    tok = dec.prefill(prompt, chunk=PROMPT)
    dec.L.dh_sync()
    prefill = len(prompt) / (time.perf_counter() - t0)
    out = dec.decode_greedy(tok, len(prompt), max(warmup, 1))
    dec.L.dh_sync()
    t0 = time.perf_counter()
    dec.decode_greedy(out[-1], len(prompt) + len(out), steps)
    dec.L.dh_sync()
    decode = steps / (time.perf_counter() - t0)
    dec.release_readback()
    return prefill, decode


def _replayed(dec, pos, steps):
    """Decode tokens/s of the captured step, one replay and one token readback per token."""
    tok = dec.step_graph(1, pos)
    dec.L.dh_sync()
    t0 = time.perf_counter()
    for k in range(steps):
        tok = dec.step_graph(tok, pos + 1 + k)
    rate = steps / (time.perf_counter() - t0)
    dec.release_graph()
    return rate


def _entry(name, us, nbytes=None, flops=None, peak=MFMA_TFLOPS):
    e = dict(kernel=name, us=round(us, 2))
    if nbytes is not None:
        e.update(gb_per_s=round(nbytes / us / 1e3, 1), hbm_frac=round(nbytes / us / 1e3 / HBM_GBPS, 4))
    else:
        e.update(tflop_per_s=round(flops / us / 1e6, 1), mfma_frac=round(flops / us / 1e6 / peak, 4))
    return e


def _attn_flops(T, heads, dim, window):
    pairs = sum(min(t + 1, window) if window else t + 1 for t in range(T))
    return 4.0 * pairs * heads * dim


def zepavik_kernels(dec, s, T):
    from . import capi
    L, ck, c = dec.L, capi.check, dec.cfg
    t, pos = _Timer(L), PROMPT + 8
    Hd, g = c["hidden"], dec.layers[0]["geo"]
    mixed = dec.mixed[dec._mixed_key(g)].data_ptr()
    act = mixed + 4 * g["attn_cols"]
    b = dec._pf
    pm, x, qkv = b["mixed"][dec._mixed_key(g)].data_ptr(), b["x"].data_ptr(), b["qkv"].data_ptr()
    elem = b["normed"].element_size()
    out = []
    sweep = lambda f: t.us([(lambda d=d: f(d)) for d in dec.layers])
    us = sweep(lambda d: ck(L.dh_dense_gemv(dec.x.data_ptr(), d["norm"].data_ptr(), Hd, c["eps"], d["w_in"].data_ptr(), g["kx"], g["n"],
                                            g["kx"], 1.0, d["bias"].data_ptr(), None, dec.qkv.data_ptr(), g["n_first"], act, d["act"])))
    out.append(_entry("decode: norm + q/k/v/gate/up", us, nbytes=2.0 * g["n"] * Hd))
    us = sweep(lambda d: ck(L.dh_dense_gemv(mixed, None, 0, 0.0, d["w_out"].data_ptr(), g["k2"], Hd, g["k2"], 1.0, None,
                                            dec.x.data_ptr(), dec.x.data_ptr(), Hd, None, capi.ACT_NONE)))
    out.append(_entry("decode: o/down + residual", us, nbytes=2.0 * Hd * (g["attn_cols"] + g["ff"])))
    us = sweep(lambda d: ck(L.dh_attn_spec_decode(ctypes.byref(d["spec"]), dec.qkv.data_ptr(), d["cache_k"].data_ptr(),
                                                  d["cache_v"].data_ptr(), mixed, pos, None, 0, dec.attn_ws.data_ptr())))
    out.append(_entry("decode: attention, %d keys" % WINDOW, us, nbytes=2.0 * WINDOW * s["kv_heads"] * (g["D"] + g["VD"])))
    us = sweep(lambda d: ck(L.dh_dense_lmhead_argmax(dec.x.data_ptr(), dec.final_norm.data_ptr(), Hd, c["eps"], dec.head.data_ptr(),
                                                     dec.kx, c["vocab"], dec.kx, 1.0, dec.lm_ws.data_ptr(), dec.token.data_ptr(), 0, None)))
    out.append(_entry("decode: norm + head + argmax (weights in cache where they fit)", us, nbytes=2.0 * c["vocab"] * Hd))
    us = t.us([lambda: dec._enqueue_embed(dec.ids.data_ptr(), dec.ids.data_ptr() + 8, pos, False)] * 20)
    out.append(_entry("decode: embedding sum", us, nbytes=10.0 * Hd))
    us = t.us([lambda: ck(L.dh_embed_sum(b["ids"].data_ptr(), 1, b["ids"].data_ptr(), *dec._embed_args(), x, dec.kx, T, Hd, 0, None))] * 10)
    out.append(_entry("prefill: embedding sum", us, nbytes=10.0 * T * Hd))
    us = sweep(lambda d: dec._enqueue_in(d, x, b["normed"].data_ptr(), dec.operand, qkv, pm + elem * g["attn_cols"], T, g["k2"]))
    out.append(_entry("prefill: norm, q/k/v/gate/up", us, flops=2.0 * T * g["n"] * Hd))
    us = sweep(lambda d: dec._enqueue_out(d, pm, dec.operand, x, T))
    out.append(_entry("prefill: o/down + residual", us, flops=2.0 * T * Hd * (g["attn_cols"] + g["ff"])))
    us = sweep(lambda d: ck(L.dh_attn_spec_prefill(ctypes.byref(d["spec"]), qkv, d["cache_k"].data_ptr(), d["cache_v"].data_ptr(), pm,
                                                   dec.operand, g["k2"], T, 0)))
    out.append(_entry("prefill: attention, window %d" % WINDOW, us, flops=_attn_flops(T, s["heads"], s["head_dim"], WINDOW)))
    us = sweep(lambda d: ck(L.dh_attn_spec_kv_write(ctypes.byref(d["spec"]), qkv, d["cache_k"].data_ptr(), d["cache_v"].data_ptr(), T, 0)))
    out.append(_entry("prefill: value norm + KV write", us, nbytes=6.0 * T * s["kv_heads"] * (g["D"] + g["VD"])))
    t.close()
    return out


def gusolorn_kernels(dec, s, T):
    from . import capi, sublayers as sl
    L, ck, c = dec.L, capi.check, dec.cfg
    t, pos, Hd = _Timer(L), PROMPT + 8, c["hidden"]
    kinds = lambda kind: [p for layer in dec.layers for p in layer.parts if isinstance(p, kind)]
    latent, memory, dense, experts = (kinds(k) for k in (sl.LatentAttention, sl.MatrixMemory, sl.DenseFF, sl.ExpertsFF))
    out, f32, x = [], torch.float32, dec.x.data_ptr()
    row = lambda p: dec.scratch.rows("row", p.ld if hasattr(p, "ld") else p.n_in, 1, f32)
    mixed = lambda p: dec.scratch.rows("mixed", p.k2, 1, f32)
    px = dec._pf["x"].data_ptr()

    def add(name, parts, f, nbytes=None, flops=None, peak=MFMA_TFLOPS):
        us = t.us([(lambda p=p: f(p)) for p in parts])
        out.append(_entry(name, us, nbytes=nbytes, flops=flops, peak=peak))
    own = [p for p in latent if p.lender is None]
    m = latent[0].m
    H, d, rot, e, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    n_in = H * (d + rot) + rank + rot
    add("decode: latent, norm + q/latent", own, lambda p: p._gemv(x, True, p.w_in, p.n_in, p.kx, out=row(p)), nbytes=2.0 * n_in * Hd)
    add("decode: latent attention, %d keys (with up projections)" % WINDOW, latent, lambda p: ck(L.dh_latent_decode(
        p.ref, row(p), p.cache.data_ptr(), mixed(p), pos, None, dec.max_seq, dec.scratch.space("latent_decode", 1))),
        nbytes=2.0 * (H * rank * (d + e) + WINDOW * (rank + rot)))
    add("decode: latent, o + residual", latent, lambda p: p._gemv(mixed(p), False, p.w_out, Hd, p.k2, residual=True), nbytes=2.0 * Hd * H * e)
    mm = memory[0].m
    MH, md, me = mm["heads"], mm["dim"], mm["vdim"]
    add("decode: memory, norm + q/k/v/gates", memory, lambda p: p._gemv(x, True, p.w_in, p.n_in, p.kx, bias=p.bias.data_ptr(), out=row(p)),
        nbytes=2.0 * MH * (2 * md + 2 * me + 2) * Hd)
    heads = lambda p: dec.scratch.rows("heads", p.o_width, 1, f32)
    add("decode: memory, state step", memory, lambda p: ck(L.dh_mlstm_step(p.ref, row(p), p.memory.data_ptr(), heads(p), pos, None)),
        nbytes=8.0 * MH * md * (me + 1))
    add("decode: memory, head norm, gate, o + residual", memory, lambda p: p._out_step(heads(p), row(p)), nbytes=2.0 * Hd * MH * me)
    ff = dense[0].ff
    act = dec.scratch.rows("act", dense[0].ffp, 1, f32)
    add("decode: dense ff, norm + up", dense, lambda p: p._gemv(x, True, p.up, p.ff, p.kx, act_out=act, act=p.act), nbytes=2.0 * ff * Hd)
    add("decode: dense ff, down + residual", dense, lambda p: p._gemv(act, False, p.down, Hd, p.ffp, residual=True), nbytes=2.0 * ff * Hd)
    add("decode: experts (router, up, down)", experts, lambda p: p.step(pos, None), nbytes=float(experts[0].step_bytes(0)))
    us = t.us([lambda: dec._enqueue_head(x, 0, None)] * 4)
    out.append(_entry("decode: norm + head + argmax (weights in cache where they fit)", us, nbytes=2.0 * c["vocab"] * Hd))

    def in_rows(p):
        normed = p._normed_rows(px, T)
        ld = p.ld if hasattr(p, "ld") else p.n_in
        ck(L.dh_dense_matmul(normed, dec.operand, p.kx, p.w_in.data_ptr(), p.kx, T, p.n_in, p.kx, 1.0, p.bias.data_ptr() if hasattr(p, "bias") else None,
                             None, dec.scratch.rows("rows", ld, T, f32), ld, p.n_in, None, 0, 0, capi.ACT_NONE))
    mixed_rows = lambda p: dec.scratch.rows("mixed_rows", p.k2, T, dec.operand_torch)
    rows = lambda p: dec.scratch.rows("rows", p.ld if hasattr(p, "ld") else p.n_in, T, f32)
    add("prefill: latent, norm, q/latent", own, in_rows, flops=2.0 * T * n_in * Hd)
    add("prefill: latent, rotation + cache rows", own, lambda p: ck(L.dh_latent_rows(p.ref, rows(p), p.cache.data_ptr(), T, 0)),
        nbytes=float(T * (8 * H * rot + 6 * (rank + rot))))
    ws = dec.scratch.space("latent_prefill", L.dh_latent_prefill_workspace_bytes(latent[0].ref, T, 0))
    pairs = _attn_flops(T, 1, 1, WINDOW) / 4
    add("prefill: latent attention, window %d (with up projections)" % WINDOW, latent, lambda p: ck(L.dh_latent_prefill(
        p.ref, rows(p), p.cache.data_ptr(), ws, mixed_rows(p), dec.operand, p.k2, T, 0)),
        flops=2.0 * H * (pairs * (d + rot + e) + T * rank * (d + e)))
    add("prefill: latent, o + residual", latent, lambda p: p._out_rows(mixed_rows(p), p.k2, p.w_out, px, T), flops=2.0 * T * Hd * H * e)
    add("prefill: memory, norm, q/k/v/gates", memory, in_rows, flops=2.0 * T * Hd * MH * (2 * md + 2 * me + 2))
    mws = dec.scratch.space("mlstm_prefill", L.dh_mlstm_prefill_workspace_bytes(memory[0].ref, T))
    head_rows = lambda p: dec.scratch.rows("heads_rows", p.o_width, T, f32)
    add("prefill: memory, chunks (32-bit products)", memory, lambda p: ck(L.dh_mlstm_prefill(p.ref, rows(p), p.memory.data_ptr(), mws, head_rows(p), p.o_width, T, 0)),
        flops=2.0 * T * MH * (2 * md * me + 32 * (md + me)), peak=MFMA_F32_TFLOPS)
    add("prefill: memory, head norm + gate", memory, lambda p: p._norm_gate(head_rows(p), rows(p), mixed_rows(p), dec.operand, T), nbytes=10.0 * T * MH * me)
    add("prefill: memory, o + residual", memory, lambda p: p._out_rows(mixed_rows(p), p.k2, p.w_out, px, T), flops=2.0 * T * Hd * MH * me)
    act_rows = dec.scratch.rows("act_rows", dense[0].ffp, T, dec.operand_torch)

    def up_rows(p):
        ck(L.dh_dense_matmul(p._normed_rows(px, T), dec.operand, p.kx, p.up.data_ptr(), p.kx, T, p.ff, p.kx, 1.0, None, None, None, 0, 0, act_rows, dec.operand,
                             p.ffp, p.act))
    add("prefill: dense ff, norm, up", dense, up_rows, flops=2.0 * T * Hd * ff)
    add("prefill: dense ff, down + residual", dense, lambda p: p._out_rows(act_rows, p.ffp, p.down, px, T), flops=2.0 * T * Hd * ff)
    me_ = experts[0].m
    add("prefill: experts (norm, router, sort, products, sum)", experts, lambda p: p.rows(px, T, 0),
        flops=6.0 * T * Hd * (me_["top"] * me_["ff"] + me_["shared"]["ff"]))
    t.close()
    return out


def q4k_kernels(dec, s, T):
    from . import capi, synth
    L, ck, c = dec.L, capi.check, dec.cfg
    t, pos = _Timer(L), PROMPT + 8
    Hd, I, H, Hkv, D = c["hidden"], c["inter"], c["heads"], c["kv_heads"], c["head_dim"]
    qkv_n, b = dec.qs + 2 * dec.ks, dec._pf
    out = []
    sweep = lambda f: t.us([(lambda d=d: f(d)) for d in dec.layers])
    for rows, x, normed, qkv, attn, act, y in ((1, dec.x, dec.normed, dec.qkv, dec.attn, dec.act, dec.x2),
                                               (T, b["x"], b["normed"], b["qkv"], b["attn"], b["act"], b["x2"])):
        def add(name, us, n, k, mats=1):
            phase = "decode: " if rows == 1 else "prefill: "
            out.append(_entry(phase + name, us, nbytes=float(mats * synth.q4k_nbytes(n, k))) if rows == 1 else
                       _entry(phase + name, us, flops=2.0 * rows * n * k * mats))
        add("norm + q/k/v", sweep(lambda d: ck(L.dh_q4k_matmul_rmsnorm(x.data_ptr(), d["input_norm"].data_ptr(), c["eps"], 0, d["wqkv"].data_ptr(),
                                                                       qkv.data_ptr(), capi.F32, rows, qkv_n, Hd, 1.0, None))), qkv_n, Hd)
        add("o + residual", sweep(lambda d: ck(L.dh_q4k_matmul(attn.data_ptr(), capi.F32, d["wo"].data_ptr(), y.data_ptr(), capi.F32, rows, Hd,
                                                               dec.qs, 1.0, x.data_ptr()))), Hd, dec.qs)
        add("norm + gate/up", sweep(lambda d: ck(L.dh_q4k_ffn_gate_up_rmsnorm(
            x.data_ptr(), d["post_attn_norm"].data_ptr(), c["eps"], 0, d["wgate"].data_ptr(), d["wup"].data_ptr(), act.data_ptr(), rows, Hd, I,
            capi.ACT_SILU, 1.0, 0.0))), I, Hd, 2)
        add("down + residual", sweep(lambda d: ck(L.dh_q4k_matmul(act.data_ptr(), capi.F32, d["wdown"].data_ptr(), y.data_ptr(), capi.F32, rows,
                                                                  Hd, I, 1.0, x.data_ptr()))), Hd, I)
    us = sweep(lambda d: ck(L.dh_attn_decode_qkv(dec.qkv.data_ptr(), d["q_norm"].data_ptr(), d["k_norm"].data_ptr(), dec.cos.data_ptr(),
                                                 dec.sin.data_ptr(), d["cache_k"].data_ptr(), d["cache_v"].data_ptr(), dec.attn.data_ptr(), H, Hkv,
                                                 D, pos, D, 0, c["eps"], 0, 1, dec.scale, 0.0, WINDOW, 0, capi.KV_CONTIGUOUS, dec.attn_ws.data_ptr())))
    out.append(_entry("decode: attention, %d keys" % WINDOW, us, nbytes=4.0 * WINDOW * Hkv * D))
    us = t.us([lambda: dec._enqueue_embed(dec.ids.data_ptr(), None, pos, False)] * 20)
    out.append(_entry("decode: embedding gather", us, nbytes=6.0 * Hd))
    us = t.us([lambda: ck(L.dh_gather_f16(b["ids"].data_ptr(), dec.embed.data_ptr(), b["x"].data_ptr(), T, Hd, c["vocab"], 0))] * 10)
    out.append(_entry("prefill: embedding gather", us, nbytes=6.0 * T * Hd))
    us = sweep(lambda d: dec._enqueue_head(dec.x.data_ptr(), 0, None))
    out.append(_entry("decode: norm + head + argmax (weights in cache where they fit)", us, nbytes=2.0 * c["vocab"] * Hd))
    us = sweep(lambda d: ck(L.dh_attn_prefill(b["q"].data_ptr(), d["cache_k"].data_ptr(), d["cache_v"].data_ptr(), b["attn"].data_ptr(), T, H, Hkv,
                                              D, T, dec.scale, 1, 0, 0.0, WINDOW)))
    out.append(_entry("prefill: attention, window %d" % WINDOW, us, flops=_attn_flops(T, H, D, WINDOW)))
    us = sweep(lambda d: ck(L.dh_qkv_norm_rope_kvwrite(b["qkv"].data_ptr(), d["q_norm"].data_ptr(), d["k_norm"].data_ptr(), dec.cos.data_ptr(),
                                                       dec.sin.data_ptr(), b["q"].data_ptr(), d["cache_k"].data_ptr(), d["cache_v"].data_ptr(), T, H,
                                                       Hkv, D, 0, D, 0, c["eps"], 0, 0, 1)))
    out.append(_entry("prefill: q/k norm + RoPE + KV write", us, nbytes=float(T * D * (8 * H + 6 * 2 * Hkv))))
    t.close()
    return out


def _measure(dec, prompt, steps, warmup, kernels, s):
    pre, step = _throughput(dec, prompt, steps, warmup)
    nbytes = dec.weight_bytes_per_token(PROMPT + steps // 2)
    r = dict(prefill_tokens_per_s=round(pre, 1), decode_tokens_per_s=round(step, 1), decode_hbm_frac=round(nbytes * step / 1e9 / HBM_GBPS, 4))
    if kernels in (zepavik_kernels, gusolorn_kernels):
        dec.prefill(prompt, chunk=PROMPT)
        r["replayed_tokens_per_s"] = round(_replayed(dec, PROMPT, steps), 1)
    r["kernels"] = kernels(dec, s, PROMPT)
    return r


def run(design, sizes, steps, warmup):
    from . import decoder, dense_decoder, gusolorn
    results = {}
    for name in sizes:
        s = SIZES[name]
        max_seq = PROMPT + warmup + steps + 80
        prompt = np.random.Generator(np.random.PCG64(1)).integers(0, VOCAB, PROMPT)
        r = dict(s, vocab=VOCAB, window=WINDOW, prompt=PROMPT)
        if design == "gusolorn":
            r.update(MIXED[name])

        def build(kind):
            log("[bench] %s %s" % (kind, name))
            if kind == "q4k":
                cfg = q4k_config(s, max_seq)
                layers, embed, final_norm, cos, sin = decoder.random_model(cfg, seed=3, max_seq=max_seq)
                return decoder.HipDecoder(cfg, layers, embed, final_norm, cos, sin, max_seq)
            if kind == "gusolorn":
                cfg = gusolorn_config(s, MIXED[name])
                return dense_decoder.DenseDecoder(cfg, gusolorn.random_weights(cfg, seed=4), max_seq)
            cfg = zepavik_config(s, max_seq)
            return dense_decoder.DenseDecoder(cfg, dense_decoder.random_weights(cfg, seed=2), max_seq)
        kernels = dict(zepavik=zepavik_kernels, q4k=q4k_kernels, gusolorn=gusolorn_kernels)
        for kind in (design, {"zepavik": "q4k", "gusolorn": "zepavik"}[design]):
            dec = build(kind)
            r[kind] = _measure(dec, prompt, steps, warmup, kernels[kind], s)
            log("[bench] %s %s: prefill %.0f tok/s, decode %.1f tok/s" % (kind, name, r[kind]["prefill_tokens_per_s"], r[kind]["decode_tokens_per_s"]))
            del dec
        results[name] = r
    return results
