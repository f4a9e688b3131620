"""Zepavik on the GPU: every mechanism alone against the plain restatement, then whole models through the framework's own
loading, step, cache, prefill and generation.

Tolerances: 32-bit paths must agree with the float64 restatement to ~1e-5; bf16 paths to what rounding operands to bf16
(products) and f16 (cached keys and values, queries) explains."""
import ctypes
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from doppler_amd import capi, decoder, dense_decoder, generate, models
from oracle import plain_zepavik as plain
from tests import zepavik_models as zm

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32_ROW, BF16_ROW = 3e-5, 0.03       # largest error of a row of logits (see zm.row_errors)


@pytest.fixture(scope="module")
def L():
    torch.cuda.init()
    return capi.init(torch.cuda.current_device())


def dev(a, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(a)).to(dtype).cuda()


def host(t):
    torch.cuda.synchronize()
    capi.check(capi.load().dh_sync())
    return t.float().cpu().numpy().astype(np.float64)


def rel(a, b):
    return float(np.linalg.norm(a - b) / max(np.linalg.norm(b), 1e-30))


def rng(seed):
    return np.random.Generator(np.random.PCG64(seed))


# ------------------------------------------------------------------ embedding, norms

@pytest.mark.parametrize("hidden,buckets,mp,mc", [(136, 61, 31, 13), (70, 1, 5, 9), (4104, 501, 2000003, 1999993), (2051, 77, 3, 2)])
def test_embedding_sum(L, hidden, buckets, mp, mc):
    """Portions of a sequence; products of ids and multipliers far above 32 bits."""
    V, P, n = 3001, 90, 40
    g = rng(1)
    E, B, T = (zm.bf16(g.standard_normal((r, hidden))) for r in (V, buckets + 1, P))
    toks = [int(t) for t in g.integers(0, V, n)]
    toks[3] = V - 1
    want = E[toks] + B[plain.bigram_rows(toks, buckets, mp, mc)] + T[np.arange(n)]
    dE, dB, dT = (dev(a, torch.bfloat16) for a in (E, B, T))
    ld = hidden + 24
    out = torch.full((n, ld), 7.0, device="cuda")
    ids = dev(np.array([0] + toks, np.int32), torch.int32)      # one unused word in front
    for a, b in ((0, 1), (1, 3), (3, 4), (4, 17), (17, n)):
        capi.check(L.dh_embed_sum(ids.data_ptr(), 1 + a, ids.data_ptr() + 4 * a, dE.data_ptr(), V, dB.data_ptr(), buckets, mp, mc,
                                  dT.data_ptr(), P, out.data_ptr() + 4 * ld * a, ld, b - a, hidden, a, None))
    got = host(out)
    assert np.abs(got[:, :hidden] - want).max() < 1e-5 and (got[:, hidden:] == 7.0).all()
    # the position from a key count on the device
    kv = dev(np.array([30], np.int32), torch.int32)
    row = torch.zeros(ld, device="cuda")
    capi.check(L.dh_embed_sum(ids.data_ptr(), 30, ids.data_ptr() + 4 * 29, dE.data_ptr(), V, dB.data_ptr(), buckets, mp, mc,
                              dT.data_ptr(), P, row.data_ptr(), ld, 1, hidden, 0, kv.data_ptr()))
    assert np.abs(host(row)[:hidden] - want[29]).max() < 1e-5
    assert L.dh_embed_sum(ids.data_ptr(), 0, None, dE.data_ptr(), V, dB.data_ptr(), buckets, mp, mc, dT.data_ptr(), P, out.data_ptr(),
                          ld, 1, hidden, 5, None) != 0
    assert L.dh_embed_sum(ids.data_ptr(), 0, ids.data_ptr(), dE.data_ptr(), V, dB.data_ptr(), buckets, mp, mc, dT.data_ptr(), P,
                          out.data_ptr(), ld, 1, hidden, P, None) != 0


@pytest.mark.parametrize("hidden,ld", [(136, 192), (70, 128), (4096, 4096), (9000, 9024)])
@pytest.mark.parametrize("eps", [1e-5, 0.3])
def test_row_norms(L, hidden, ld, eps):
    g = rng(2)
    x = g.standard_normal((5, ld)).astype(np.float32)
    x[1] *= 1e-3                                   # eps inside the root decides this row
    w = np.zeros(ld, np.float32)
    w[:hidden] = 1 + 0.3 * g.standard_normal(hidden)
    rows = np.array([4, 1, 1, 0], np.int32)
    dx, dw, dr = dev(x), dev(w), dev(rows, torch.int32)
    want = plain.rms_norm(x[rows][:, :hidden].astype(np.float64), eps, w[:hidden].astype(np.float64))
    out = torch.full((4, ld), 3.0, device="cuda")
    capi.check(L.dh_rmsnorm_rows(dx.data_ptr(), ld, dr.data_ptr(), dw.data_ptr(), out.data_ptr(), capi.F32, ld, 4, hidden, eps))
    got = host(out)
    assert rel(got[:, :hidden], want) < 1e-6 and not got[:, hidden:].any()
    out16 = torch.full((5, ld), 3.0, dtype=torch.bfloat16, device="cuda")
    capi.check(L.dh_rmsnorm_rows(dx.data_ptr(), ld, None, dw.data_ptr(), out16.data_ptr(), capi.BF16, ld, 5, hidden, eps))
    got = host(out16)
    want = plain.rms_norm(x[:, :hidden].astype(np.float64), eps, w[:hidden].astype(np.float64))
    assert np.abs(got[:, :hidden] - want).max() <= np.abs(want).max() * 2.0 ** -8 and not got[:, hidden:].any()


# ------------------------------------------------------------------ dense products

def act_of(name, z):
    return {"relu2": np.square(np.maximum(z, 0)), "silu": z / (1 + np.exp(-z)), None: z,
            "gelu_tanh": 0.5 * z * (1 + np.tanh(np.sqrt(2 / np.pi) * (z + 0.044715 * z ** 3)))}[name]


# both tiles, whole and in k slices, edges in both directions
@pytest.mark.parametrize("M,N,K,first", [(1, 5, 64, 5), (2, 130, 128, 40), (65, 200, 192, 72), (130, 2100, 320, 2100), (300, 1500, 256, 0),
                                         (1030, 4100, 128, 1000), (2048, 8200, 64, 8000),
                                         (3, 100, 4096, 60), (200, 1000, 8256, 904), (96, 70, 33088, 70)])
@pytest.mark.parametrize("operand", ["bf16", "f32"])
def test_dense_matmul(L, M, N, K, first, operand):
    g = torch.Generator().manual_seed(M + N)
    A = torch.randn(M, K, generator=g).to(torch.bfloat16 if operand == "bf16" else torch.float32)
    W = (torch.randn(N, K, generator=g) / K ** 0.5).to(torch.bfloat16)
    bias, res = torch.randn(max(first, 1), generator=g), torch.randn(M, max(first, 1) + 8, generator=g)
    acc = 0.75 * (A.double() @ W.double().T).numpy()
    dA, dW, db = A.cuda(), W.cuda(), bias.cuda()
    code = capi.BF16 if operand == "bf16" else capi.F32
    for name, act in (("relu2", capi.ACT_RELU2), ("silu", capi.ACT_SILU), ("gelu_tanh", capi.ACT_GELU)):
        C = res.cuda()
        ldc2 = N - first + 4
        C2 = torch.full((M, max(ldc2, 1)), 9.0, dtype=torch.bfloat16 if operand == "bf16" else torch.float32, device="cuda")
        capi.check(L.dh_dense_matmul(dA.data_ptr(), code, K, dW.data_ptr(), K, M, N, K, 0.75, db.data_ptr(), C.data_ptr(), C.data_ptr(),
                                     first + 8, first, C2.data_ptr(), code, ldc2, act))
        got, got2 = host(C), host(C2)
        if first:
            want = acc[:, :first] + bias.double().numpy()[:first] + res.double().numpy()[:, :first]
            assert np.abs(got[:, :first] - want).max() < 2e-5
            assert np.array_equal(got[:, first:], res.double().numpy()[:, first:])
        if first < N:
            want = act_of(name, acc[:, first:])
            tol = (2.0 ** -8 if operand == "bf16" else 1e-5) * max(1.0, np.abs(want).max())
            assert np.abs(got2[:, :N - first] - want).max() < tol
            assert (got2[:, N - first:] == 9.0).all()


def test_f32_products_are_not_reduced_precision(L):
    """Activations that differ from a constant in their last bits only: bf16- or TF32-like operands would lose them."""
    M, N, K = 40, 70, 256
    A = (1.0 + torch.randn(M, K, dtype=torch.float64) * 2.0 ** -20).float()
    W = torch.ones(N, K, dtype=torch.bfloat16)
    W[:, ::2] = -1.0
    dA, dW, C = A.cuda(), W.cuda(), torch.zeros(M, N, device="cuda")
    capi.check(L.dh_dense_matmul(dA.data_ptr(), capi.F32, K, dW.data_ptr(), K, M, N, K, 1.0, None, None, C.data_ptr(), N, N, None, 0, 0,
                                 capi.ACT_NONE))
    want = (A.double() @ W.double().T).numpy()
    assert rel(host(C), want) < 0.05 and np.abs(want).max() < 1e-4


@pytest.mark.parametrize("N,K,hidden,first", [(1, 64, 40, 1), (77, 192, 136, 77), (1003, 1024, 1000, 300), (33000, 512, 512, 20000), (130, 8256, 8200, 64),
                                              (700, 16448, 16400, 700), (65, 32768, 32768, 0)])
def test_dense_gemv(L, N, K, hidden, first):
    g = torch.Generator().manual_seed(N + K)
    x = torch.zeros(K)
    x[:hidden] = torch.randn(hidden, generator=g)
    w = torch.zeros(K)
    w[:hidden] = 1 + 0.3 * torch.randn(hidden, generator=g)
    W = (torch.randn(N, K, generator=g) / K ** 0.5).to(torch.bfloat16)
    bias, res = torch.randn(N, generator=g), torch.randn(N, generator=g)
    dx, dw, dW, db = x.cuda(), w.cuda(), W.cuda(), bias.cuda()
    for normed in (True, False):
        xn = plain.rms_norm(x[:hidden].double().numpy(), 1e-2, w[:hidden].double().numpy()) if normed else x[:hidden].double().numpy()
        acc = 1.25 * (W[:, :hidden].double().numpy() @ xn)
        C, C2 = res.cuda(), torch.full((N - first + 1,), 5.0, device="cuda")
        capi.check(L.dh_dense_gemv(dx.data_ptr(), dw.data_ptr() if normed else None, hidden, 1e-2, dW.data_ptr(), K, N, K, 1.25,
                                   db.data_ptr(), C.data_ptr(), C.data_ptr(), first, C2.data_ptr(), capi.ACT_RELU2))
        want = acc[:first] + bias.double().numpy()[:first] + res.double().numpy()[:first]
        got, got2 = host(C), host(C2)
        if first:
            assert np.abs(got[:first] - want).max() < 1e-5
        assert np.array_equal(got[first:], res.double().numpy()[first:])
        if first < N:
            assert np.abs(got2[:-1] - act_of("relu2", acc[first:])).max() < 2e-5
        assert got2[-1] == 5.0


@pytest.mark.parametrize("vocab,K,hidden", [(301, 192, 136), (70001, 512, 500), (900, 9024, 9000)])
def test_dense_head_argmax(L, vocab, K, hidden):
    g = torch.Generator().manual_seed(vocab)
    x, w = torch.zeros(K), torch.zeros(K)
    x[:hidden], w[:hidden] = torch.randn(hidden, generator=g), torch.rand(hidden, generator=g) + 0.5
    W = (torch.randn(vocab, K, generator=g) / K ** 0.5).to(torch.bfloat16)
    want = 0.3 * (W[:, :hidden].double().numpy() @ plain.rms_norm(x[:hidden].double().numpy(), 1e-5, w[:hidden].double().numpy()))
    best = int(want.argmax())
    W[min(best + 40, vocab - 1)] = W[best]             # a tie: the lower index wins
    logits, tok = torch.zeros(vocab, device="cuda"), torch.zeros(4, dtype=torch.int32, device="cuda")
    ws = torch.zeros(int(L.dh_lmhead_argmax_workspace_bytes(vocab)), dtype=torch.uint8, device="cuda")
    dx, dw, dW = x.cuda(), w.cuda(), W.cuda()
    capi.check(L.dh_dense_lmhead_argmax(dx.data_ptr(), dw.data_ptr(), hidden, 1e-5, dW.data_ptr(), K, vocab, K, 0.3, ws.data_ptr(),
                                        tok.data_ptr(), 2, logits.data_ptr()))
    got = host(logits)
    keep = np.arange(vocab) != min(best + 40, vocab - 1)
    assert np.abs(got - want)[keep].max() < 1e-5 and tok.cpu().tolist() == [0, 0, best, 0]


# ------------------------------------------------------------------ attention

class Attn:
    """One attention layer fed through the C ABI: projection rows in, gated outputs out."""

    def __init__(self, L, H, G, d, e, window, cache="f16", scale=None, seed=0, n=200, gain=1.0, bias=True, gate=True, norm=True, value_std=1.0):
        self.L, self.H, self.G, self.d, self.e, self.window = L, H, G, d, e, window
        self.D, self.VD = (d + 7) // 8 * 8, (e + 7) // 8 * 8
        self.scale, self.eps, self.n = scale or d ** -0.5, 2e-3, n
        g = rng(seed)
        self.q, self.k, self.v = (g.standard_normal((n, h, s)).astype(np.float32) for h, s in ((H, d), (G, d), (G, e)))
        self.q *= gain
        self.v *= value_std
        self.gate = g.standard_normal((n, H)).astype(np.float32)
        self.r1, self.r2 = (g.uniform(a, b, H).astype(np.float32) for a, b in ((0.02, 1.5), (0.05, 0.9)))
        self.bias, self.gated, self.norm = bias, gate, norm
        self.ko = H * self.D
        self.vo = self.ko + G * self.D
        self.go = self.vo + G * self.VD
        self.ld = (self.go + H + 7) // 8 * 8
        self.cache_t = torch.float16 if cache == "f16" else torch.float32
        self.kc = torch.full((n, G, self.D), 60.0, dtype=self.cache_t, device="cuda")     # rows of an earlier sequence
        self.vc = torch.full((n, G, self.VD), -60.0, dtype=self.cache_t, device="cuda")
        self.dr1, self.dr2 = dev(self.r1), dev(self.r2)
        self.spec = capi.AttnSpec(H, G, self.D, self.VD, e, window, capi.F16 if cache == "f16" else capi.F32, int(norm), self.ko, self.vo,
                                  self.go if gate else -1, self.ld, self.scale, self.eps, self.dr1.data_ptr() if bias else None,
                                  self.dr2.data_ptr() if bias else None)
        self.ws = torch.zeros(int(L.dh_attn_spec_workspace_bytes(H, self.VD, n)), dtype=torch.uint8, device="cuda")

    def rows(self):
        r = np.zeros((self.n, self.ld), np.float32)
        for a, at, heads, size in ((self.q, 0, self.H, self.D), (self.k, self.ko, self.G, self.D), (self.v, self.vo, self.G, self.VD)):
            block = np.zeros((self.n, heads, size), np.float32)
            block[:, :, :a.shape[2]] = a
            r[:, at:at + heads * size] = block.reshape(self.n, -1)
        r[:, self.go:self.go + self.H] = self.gate
        return dev(r)

    def want(self):
        z = np.zeros(self.H)
        f = lambda a: a.astype(np.float64)
        v = plain.rms_norm(f(self.v), self.eps) if self.norm else f(self.v)
        o = plain.attention(f(self.q), f(self.k), v, self.scale, f(self.r1) if self.bias else z, f(self.r2) if self.bias else z,
                            self.window or 10 ** 9)
        return o * (plain.sigmoid(f(self.gate))[:, :, None] if self.gated else 1.0)

    def run(self, portions, out="f32"):
        """portions: sizes; 1 goes through the decode op, more through KV write + prefill."""
        L, rows, at = self.L, self.rows(), 0
        o = torch.zeros((self.n, self.H * self.VD), dtype=torch.float32 if out == "f32" else torch.bfloat16, device="cuda")
        one = torch.zeros(self.H * self.VD, device="cuda")
        spec = ctypes.byref(self.spec)
        for t in portions:
            src = rows.data_ptr() + 4 * self.ld * at
            if t == 1:
                capi.check(L.dh_attn_spec_decode(spec, src, self.kc.data_ptr(), self.vc.data_ptr(), one.data_ptr(), at, None, 0, self.ws.data_ptr()))
                capi.check(L.dh_sync())
                o[at] = one.to(o.dtype)
                torch.cuda.synchronize()
            else:
                capi.check(L.dh_attn_spec_kv_write(spec, src, self.kc.data_ptr(), self.vc.data_ptr(), t, at))
                capi.check(L.dh_attn_spec_prefill(spec, src, self.kc.data_ptr(), self.vc.data_ptr(),
                                                  o.data_ptr() + o.element_size() * self.H * self.VD * at,
                                                  capi.F32 if out == "f32" else capi.BF16, self.H * self.VD, t, at))
            at += t
        return host(o)[:at].reshape(at, self.H, self.VD)


SHAPES = [(4, 4, 64, 64), (6, 2, 24, 40), (8, 2, 128, 128), (5, 1, 64, 104), (3, 3, 96, 20), (12, 1, 16, 8), (9, 1, 136, 24), (2, 1, 40, 264),
          (10, 2, 300, 500), (1, 1, 8, 8)]


@pytest.mark.parametrize("cache", ["f16", "f32"])
@pytest.mark.parametrize("H,G,d,e", SHAPES)
def test_attention_shapes_prefill_decode_and_portions(L, H, G, d, e, cache):
    n, window = 150, 70
    tol = 3e-3 if cache == "f16" else 3e-6
    for k, portions in enumerate(([n], [1] * n, [2, 3, 1, 1, 61, 2, 7, 1, 64, 5, 3])):
        a = Attn(L, H, G, d, e, window, cache, n=n, seed=H + d)
        got, want = a.run(portions), a.want()
        assert not got[:, :, e:].any()
        err = [rel(got[t, :, :e], want[t]) for t in range(n)]
        assert max(err) < tol, (k, int(np.argmax(err)), max(err))


@pytest.mark.parametrize("cache", ["f16", "f32"])
@pytest.mark.parametrize("window", [1, 2, 7, 63, 64, 65, 128, 129, 0])
def test_attention_window_edges(L, window, cache):
    """In every head one key stands out; the queries that just see it and just do not are far apart."""
    n, H, G, d, e = 300, 4, 2, 64, 48
    planted = 100
    tol = 4e-3 if cache == "f16" else 1e-5
    for portions in ([n], [1] * n, [64] * 4 + [44], [99, 2, 1, 60, 1, 1, 66, 70]):
        a = Attn(L, H, G, d, e, window, cache, n=n, seed=5, gain=0.1)
        a.q[:, :, 0] = 24.0
        a.k[:, :, 0] = 0.0
        a.k[planted, :, 0] = 9.0
        a.v[planted] = 5.0 * np.sign(a.v[planted])
        got, want = a.run(portions)[:, :, :e], a.want()
        err = np.abs(got - want).max(axis=(1, 2)) / np.abs(want).max(axis=(1, 2))
        assert err.max() < tol, (int(err.argmax()), err.max())
        if window:
            inside, outside = planted + window - 1, planted + window
            edge = n - 1 if inside >= n else inside
            probe = np.einsum("he,ge->hg", want[edge] / np.linalg.norm(want[edge], axis=1, keepdims=True),
                              np.sign(a.v[planted]) / np.sqrt(e))
            assert probe.max(axis=1).min() > 0.9                # the planted key decides the last query that sees it
            if outside < n:
                assert np.abs(want[outside] - want[edge]).max() > 0.1


@pytest.mark.parametrize("bias,gate,norm", [(False, True, True), (True, False, True), (True, True, False), (False, False, False)])
def test_attention_mechanisms_one_at_a_time(L, bias, gate, norm):
    for cache, tol in (("f16", 3e-3), ("f32", 3e-6)):
        for portions in ([90], [30] + [1] * 60):
            a = Attn(L, 6, 3, 32, 56, 40, cache, n=90, seed=9, bias=bias, gate=gate, norm=norm, scale=0.31)
            assert rel(a.run(portions)[:, :, :56], a.want()) < tol


def test_value_norm_with_small_values_keeps_eps_inside_the_root(L):
    for cache, tol in (("f16", 3e-3), ("f32", 1e-5)):
        a = Attn(L, 4, 2, 64, 20, 50, cache, n=80, seed=10, value_std=0.03)      # mean square 9e-4 against eps 2e-3
        assert rel(a.run([40] + [1] * 40)[:, :, :20], a.want()) < tol


def test_first_tokens_and_large_distances(L):
    """A window longer than the sequence over many key tiles and splits: the far keys' bias, and the first positions."""
    n = 1500
    for cache, tol in (("f16", 4e-3), ("f32", 3e-5)):
        a = Attn(L, 8, 2, 64, 64, 2000, cache, n=n, seed=11, gain=0.1)
        a.q[:, :, 3] = 30.0
        a.k[:, :, 3] = 0.0
        a.k[2, :, 3] = 6.0
        a.r1[0], a.r2[0] = 0.0, 0.0
        a.dr1.copy_(torch.from_numpy(a.r1))
        a.dr2.copy_(torch.from_numpy(a.r2))
        want = a.want()
        got = a.run([5, 1, 1, 1, 1492])
        assert max(rel(got[t], want[t]) for t in range(n)) < tol
        tail = a.run([1490] + [1] * 10)
        assert max(rel(tail[t], want[t]) for t in range(1490, n)) < tol


@pytest.mark.parametrize("window", [0, 40])
def test_decode_with_the_key_count_on_the_device(L, window):
    n = 200
    a, b = (Attn(L, 6, 2, 24, 40, window, "f16", n=n, seed=12) for _ in range(2))
    want = a.run([100] + [1] * 100)
    rows, one = b.rows(), torch.zeros(6 * 40, device="cuda")
    b.run([100])
    kv = torch.zeros(1, dtype=torch.int32, device="cuda")
    for p in range(100, n):
        kv.fill_(p + 1)
        torch.cuda.synchronize()
        capi.check(L.dh_attn_spec_decode(ctypes.byref(b.spec), rows.data_ptr() + 4 * b.ld * p, b.kc.data_ptr(), b.vc.data_ptr(),
                                         one.data_ptr(), 0, kv.data_ptr(), n, b.ws.data_ptr()))
        assert rel(host(one).reshape(6, 40), want[p]) < 1e-5, p
    assert torch.equal(a.kc, b.kc) and torch.equal(a.vc, b.vc)


def test_prefill_output_in_bf16(L):
    a = Attn(L, 6, 2, 24, 40, 30, "f16", n=70, seed=13)
    f = a.run([70])
    b = Attn(L, 6, 2, 24, 40, 30, "f16", n=70, seed=13)
    assert np.array_equal(b.run([70], out="bf16"), zm.bf16(f))


def test_bad_specs_are_refused(L):
    a = Attn(L, 4, 2, 64, 64, 10, n=20)
    rows = a.rows()
    for field, value, message in (("H", 5, "multiple"), ("D", 12, "multiples of 8"), ("VD", 520, "up to 512"), ("window", -1, "window"),
                                  ("cache_dtype", capi.BF16, "caches"), ("ld_qkv", 64, "does not hold"), ("value_dim", 65, "value_dim"),
                                  ("d_bias_r2", None, "both")):
        spec = capi.AttnSpec.from_buffer_copy(a.spec)
        setattr(spec, field, value)
        assert L.dh_attn_spec_kv_write(ctypes.byref(spec), rows.data_ptr(), a.kc.data_ptr(), a.vc.data_ptr(), 2, 0) != 0
        assert message in L.dh_last_error().decode(), (field, L.dh_last_error())
    assert L.dh_dense_matmul(rows.data_ptr(), 7, 64, rows.data_ptr(), 64, 1, 8, 64, 1.0, None, None, rows.data_ptr(), 8, 8, None, 0, 0, -1) != 0
    assert L.dh_dense_gemv(rows.data_ptr(), None, 0, 0.0, rows.data_ptr(), 100, 8, 100, 1.0, None, None, rows.data_ptr(), 8, None, -1) != 0


# ------------------------------------------------------------------ whole models

@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("zepavik")
    out = {}
    for name, cfg, seed in (("mixed", zm.MIXED, 21), ("wide-heads", zm.WIDE_HEADS, 22), ("even", zm.EVEN, 23), ("odd", zm.ODD, 24)):
        t = zm.tensors(cfg, seed)
        out[name] = (zm.write(base / name, cfg, t), cfg, t)
    return out


def feed_all(dec, tokens, portions):
    dec.reset()
    out, at = [], 0
    for n in portions:
        part = tokens[at:at + n]
        out.append(dec.feed(part, list(range(len(part)))))
        at += n
    assert at >= len(tokens)
    return np.concatenate(out)


@pytest.mark.parametrize("dtype,tol", [("float32", F32_ROW), ("bfloat16", BF16_ROW)])
@pytest.mark.parametrize("name", ["mixed", "wide-heads", "even", "odd"])
def test_logits_whole_decoded_and_in_portions(folders, name, dtype, tol):
    folder, cfg, t = folders[name]
    toks = zm.prompt(cfg, 180, 31)
    want = plain.forward(cfg, t, toks)
    dec = models.load(folder, 200, dtype)
    for portions in ([180], [1] * 180, [2] * 90, [3, 1, 62, 2, 1, 1, 64, 33, 13], [65, 115]):
        err = zm.row_errors(feed_all(dec, toks, portions), want)
        assert err.max() < tol, (portions[:4], int(err.argmax()), err.max())
    # one prompt in chunks of the batched path's own
    dec.reset()
    assert zm.row_errors(dec.prefill(toks, chunk=50, want=[0, 49, 50, 179]), want[[0, 49, 50, 179]]).max() < tol


def test_layers_of_the_residual_stream(folders, tmp_path):
    """Models cut after every layer: the stream itself, read from the step's residual row."""
    _, cfg, t = folders["mixed"]
    toks = zm.prompt(cfg, 40, 32)
    _, streams = plain.forward(cfg, t, toks, want_layers=True)
    for n in range(1, len(cfg["layers"]) + 1):
        dec = models.load(zm.write(tmp_path / str(n), dict(cfg, layers=cfg["layers"][:n]), t), 64, "float32")
        dec.prefill(toks[:-1])
        dec.step(toks[-1], 39)
        assert rel(host(dec.x)[:cfg["width"]], streams[n - 1, -1]) < 1e-5, n


@pytest.mark.parametrize("dtype,tol", [("float32", F32_ROW), ("bfloat16", BF16_ROW)])
def test_unequal_sequences_one_after_another_reuse_the_cache(folders, dtype, tol):
    """Long, short, long again: rows an earlier sequence left behind must not be seen, nor its last token."""
    folder, cfg, t = folders["mixed"]
    dec = models.load(folder, 160, dtype)
    for i, n in enumerate((150, 1, 2, 70, 9, 160)):
        toks = zm.prompt(cfg, n, 40 + i)
        want = plain.forward(cfg, t, toks)
        cut = n // 2
        assert zm.row_errors(feed_all(dec, toks, [cut, n - cut] if cut else [n]), want).max() < tol, n


def test_long_decoding_passes_every_window(folders):
    folder, cfg, t = folders["mixed"]
    toks = zm.prompt(cfg, 390, 51)
    want = plain.forward(cfg, t, toks)
    dec = models.load(folder, 400, "float32")
    got = feed_all(dec, toks, [20] + [1] * 370)
    assert zm.row_errors(got, want).max() < F32_ROW
    with pytest.raises(ValueError, match="max_seq"):
        feed_all(dec, toks + [1] * 11, [390, 11])


def test_the_caches_hold_what_the_equations_say(folders):
    folder, cfg, t = folders["wide-heads"]
    toks = zm.prompt(cfg, 30, 52)
    dec = models.load(folder, 40, "float32")
    feed_all(dec, toks, [20] + [1] * 10)
    m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    h = plain.rms_norm(plain.embed(cfg, t, toks), eps, t["l0.norm1"])
    k, v = dec.read_kv(0, 30)
    want_k = (h @ t["l0.mix.k"].T + t["l0.mix.k.b"]).reshape(30, m["kv_heads"], m["dim"])
    want_v = plain.rms_norm((h @ t["l0.mix.v"].T + t["l0.mix.v.b"]).reshape(30, m["kv_heads"], m["vdim"]), eps)
    assert rel(k[:, :, :m["dim"]], want_k) < 1e-5 and rel(v[:, :, :m["vdim"]], want_v) < 1e-5


def test_widths_beyond_the_single_row_kernel(tmp_path):
    """Rows longer than the decode GEMV holds take the matrix-core path for single tokens too."""
    cfg = zm.config(33000, 40, [zm.layer(2, 1, 8, 8, 3, ff=24)], max_positions=12, buckets=5)
    t = zm.tensors(cfg, 61)
    toks = zm.prompt(cfg, 10, 62)
    want = plain.forward(cfg, t, toks)
    dec = models.load(zm.write(tmp_path, cfg, t), 12, "float32")
    assert zm.row_errors(feed_all(dec, toks, [4, 1, 1, 2, 1, 1]), want).max() < 1e-4
    dec.prefill(toks[:6])
    assert dec.step(toks[6], 6) == int(want[6].argmax())


# ------------------------------------------------------------------ generation

def test_greedy_generation_every_way(folders):
    """The framework's own loops: generate, blocking steps, staged readback, batched submits, the captured step."""
    folder, cfg, t = folders["even"]
    prompt = zm.prompt(cfg, 30, 71)
    n = 40
    want = plain.greedy(cfg, t, prompt, n)
    dec = models.load(folder, 120, "float32")
    assert isinstance(dec, decoder.DecoderBase)
    assert dec.generate(prompt, n) == want
    assert dec.generate(prompt, n, chunk=7) == want
    first = dec.prefill(prompt)
    assert [first] + dec.decode_greedy(first, 30, n - 1) == want
    dec.release_readback()
    first = dec.prefill(prompt)
    assert [first] + dec.decode_batch(first, 30, 20) + dec.decode_batch(want[20], 50, n - 21) == want
    # token by token from nothing, then the captured step replayed with eager work between replays
    out = [dec.step(tok, p) for p, tok in enumerate(prompt)][-1:]
    graph = [dec.step_graph(out[0], 30)]
    for i in range(1, n - 1):
        if i % 7 == 0:
            assert dec.step(graph[-1], 30 + i) == want[i + 1]
        graph.append(dec.step_graph(graph[-1], 30 + i))
    assert out + graph == want
    # a replay for another sequence, from its first position on
    other = zm.prompt(cfg, 9, 72)
    for p, tok in enumerate(other):
        g = dec.step_graph(tok, p)
    assert g == plain.greedy(cfg, t, other, 1)[0]
    dec.release_graph()
    with pytest.raises(ValueError, match="does not fit"):
        dec.generate(prompt, 120)


def test_generation_in_the_served_precision_and_sampling(folders):
    folder, cfg, t = folders["mixed"]
    prompt = zm.prompt(cfg, 25, 73)
    dec = models.load(folder, 80)
    assert dec.compute == "bf16"
    a = dec.generate(prompt, 30)
    seq = prompt + a
    logits = plain.forward(cfg, t, seq)
    # every greedy token is the plain model's best or within the precision's reach of it
    for i, tok in enumerate(a):
        row = logits[len(prompt) + i - 1]
        assert row.max() - row[tok] < 0.1 * row.std()
    s = dict(temperature=0.9, topK=12, seed=5)
    b = dec.generate(prompt, 30, sampling=s)
    assert b == dec.generate(prompt, 30, sampling=s) and b != dec.generate(prompt, 30, sampling=dict(s, seed=6))
    logits = plain.forward(cfg, t, prompt + b)
    for i, tok in enumerate(b):
        row = logits[len(prompt) + i - 1]
        assert (row > row[tok] + 0.1 * row.std()).sum() < 12


def test_finiteness_guard(folders, tmp_path):
    _, cfg, t = folders["even"]
    dec = models.load(zm.write(tmp_path / "a", cfg, t), 40, finiteness_guard=True)
    tok = dec.prefill(zm.prompt(cfg, 5, 74))
    dec.step(tok, 5)
    bad = dict(t)
    bad["l1.mlp.down"] = zm.bf16(t["l1.mlp.down"] * 1e8)
    dec = models.load(zm.write(tmp_path / "b", cfg, bad), 40, finiteness_guard=True)
    tok = dec.prefill(zm.prompt(cfg, 5, 74))
    with pytest.raises(decoder.FinitenessError, match="layer 1"):
        dec.step(tok, 5)


def test_command_line_generates(folders, capsys):
    folder, cfg, t = folders["even"]
    prompt = zm.prompt(cfg, 12, 75)
    assert generate.main(["--model", folder, "--dtype", "float32", "--prompt", ",".join(map(str, prompt)), "--max-tokens", "15"]) == 0
    out = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert out["prompt"] == prompt and out["tokens"] == plain.greedy(cfg, t, prompt, 15)


@pytest.mark.parametrize("dtype,tol", [("float32", F32_ROW), ("bfloat16", BF16_ROW)])
def test_trace_replay(folders, tmp_path, dtype, tol):
    folder, cfg, t = folders["mixed"]
    a, b = zm.prompt(cfg, 90, 81), zm.prompt(cfg, 33, 82)
    steps = [("a", a[:50], [0, 49], []), ("a", a[50:52], [], []), ("a", a[52:53], [0], []), ("a", a[53:], [36, 3], ["a"]), ("b", b[:1], [0], []),
             ("b", b[1:], [31], ["b"])]
    lines = [json.dumps({"step": i, "entries": [{"id": r, "tokens": toks, "want": w}], "end": end}) for i, (r, toks, w, end) in enumerate(steps)]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "90"],
                       input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(6)]
    assert not os.path.exists(str(tmp_path / "1.f32"))
    la, lb = plain.forward(cfg, t, a), plain.forward(cfg, t, b)
    for step, want in ((0, la[[0, 49]]), (2, la[[52]]), (3, la[[89, 56]]), (4, lb[[0]]), (5, lb[[32]])):
        got = np.fromfile(str(tmp_path / ("%d.f32" % step)), "<f4").reshape(-1, cfg["vocab"])
        assert zm.row_errors(got, want).max() < tol, step


def test_the_quantised_decoder_feeds_the_same_way():
    """feed() belongs to every decoder: portions and single steps of the Q4_K model give the logits of its steps."""
    cfg = dict(layers=2, hidden=256, inter=512, heads=4, kv_heads=2, head_dim=64, vocab=300, eps=1e-6, qk_norm=1, max_seq=40, theta=1e6)
    layers, embed, final_norm, cos, sin = decoder.random_model(cfg, seed=11, max_seq=40)
    dec = decoder.HipDecoder(cfg, layers, embed, final_norm, cos, sin, 40)
    toks = [int(v) for v in rng(3).integers(0, 300, 30)]
    want = []
    for p, tok in enumerate(toks):
        dec.step(tok, p, want_logits=True)
        want.append(dec.read_logits())
    got = feed_all(dec, toks, [17, 1, 1, 11])
    assert zm.row_errors(got, np.array(want, np.float64)).max() < 2e-2


def test_random_weights_make_a_model():
    cfg = dict(hidden=128, vocab=90, eps=1e-5, logit_scale=1.0, max_positions=64, bigram=dict(buckets=7, mul_prev=3, mul_cur=5),
               layers=[dict(mixer=dict(heads=4, kv_heads=2, dim=32, vdim=32, window=16, scale=0.2, log_bias=True, value_norm=True, gate=True),
                            mlp=dict(ff=96, activation="relu2"))] * 2)
    w = dense_decoder.random_weights(cfg, seed=4)
    a = dense_decoder.DenseDecoder(cfg, w, 64, compute="f32").generate([1, 2, 3], 20)
    b = dense_decoder.DenseDecoder(cfg, w, 64, compute="f32").generate([1, 2, 3], 20, chunk=2)
    assert a == b and len(a) == 20
    with pytest.raises(ValueError, match="positions"):
        dense_decoder.DenseDecoder(cfg, w, 65)
