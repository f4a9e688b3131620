"""Gusolorn on the GPU: every mechanism alone against the plain restatement (models of one layer whose embedding rows are the layer's
inputs), then whole models through the framework's own loading, step, cache and state, prefill and generation.

Tolerances: 32-bit paths must agree with the float64 restatement to rounding; bf16 paths to what operands in bf16 (products) and f16
(latent rows, queries, expanded keys and values) explain."""
import copy
import ctypes
import json
import os
import subprocess

import numpy as np
import pytest
import torch

from doppler_amd import capi, decoder, dense_decoder, generate, gusolorn, models, sublayers
from oracle import plain_gusolorn as plain
from tests import gusolorn_models as gm

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]
ROW = {"float32": 3e-5, "bfloat16": 0.06}        # largest error of a row of logits (gm.row_errors)
PART = {"float32": 1e-4, "bfloat16": 0.04}       # of a sublayer's result, relative to its row


@pytest.fixture(scope="module")
def L():
    torch.cuda.init()
    return capi.init(torch.cuda.current_device())


def host(t):
    torch.cuda.synchronize()
    capi.check(capi.load().dh_sync())
    return t.float().cpu().numpy().astype(np.float64)


def rng(seed):
    return np.random.Generator(np.random.PCG64(seed))


def dev(a, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(a)).to(dtype).cuda()


def row_rel(got, want):
    """Per row: size of the difference over the size of the wanted row (rows near zero: over the mean size)."""
    size = np.linalg.norm(want, axis=-1)
    return np.linalg.norm(got - want, axis=-1) / np.maximum(size, 0.05 * size.mean() + 1e-30)


def streams(dec, tokens, portions):
    """Residual rows behind the last layer, the sequence fed in portions."""
    W = dec.cfg["hidden"]
    dec.reset()
    out, at = [], 0
    for n in portions:
        dec.feed(tokens[at:at + n])
        out.append(host(dec.x)[None, :W] if n == 1 else host(dec._pf["x"]).reshape(-1, dec.kx)[:n, :W])
        at += n
    assert at == len(tokens)
    return np.concatenate(out)


def one_layer(tmp_path, layer, x, edit, seed, dtype, eps=1e-5, max_seq=None):
    """A model of one layer whose embedding is x [n, W] (token t's row is x[t]); edit(t) changes its tensors."""
    n, W = x.shape
    cfg = gm.config(W, n, [layer], eps=eps)
    t = gm.tensors(cfg, seed)
    t["embed"] = gm.bf16(x)
    edit(t)
    t = {k: gm.bf16(v) for k, v in t.items()}
    folder = gm.write(tmp_path / ("m%d" % len(list(tmp_path.iterdir()))), cfg, t)
    want = plain.forward(cfg, t, list(range(n)), want_layers=True)[1][-1]
    return models.load(folder, max_seq or n, dtype), want - t["embed"], t


def parts_error(dec, want, t, portions, n):
    got = streams(dec, list(range(n)), portions) - t["embed"]
    return row_rel(got, want)


def close(err, dtype, every=True, slack=1.0):
    """Rows within their tolerance; not every: a few rows are ill-conditioned (a head's output divided by its own size where that is almost
    zero), so 16-bit operands may miss those."""
    return (err.max() if every or dtype == "float32" else np.quantile(err, 0.96)) < slack * PART[dtype]


PORTIONS = lambda n: ([n], [1] * n, [2, 3, 1, 1, 61, 2, 7, 1, 64, 5, n - 147])


# ------------------------------------------------------------------ matrix memory

def no_edit(t):
    pass


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,e,cap", [(3, 20, 44, 7.5), (1, 1, 1, 1.0), (2, 100, 260, 15.0), (5, 64, 32, 30.0), (4, 33, 129, 2.0)])
def test_memory_shapes_prefill_steps_and_portions(L, tmp_path, H, d, e, cap, dtype):
    n = 200
    x = rng(H + d).standard_normal((n, 72))
    dec, want, t = one_layer(tmp_path, gm.memory(H, d, e, cap), x, no_edit, 1, dtype)
    for portions in PORTIONS(n):
        err = parts_error(dec, want, t, portions, n)
        assert close(err, dtype, False), (portions[:3], int(err.argmax()), err.max())


def gates(i, f, icol=0, fcol=1, cap=15.0):
    """Edit: the gates are read from two columns of the (unnormed-scale) input, nothing else."""
    def edit(t):
        for name, col, gain, bias in (("i", icol, i[0], i[1]), ("f", fcol, f[0], f[1])):
            t["l0.mix." + name][:] = 0.0
            t["l0.mix." + name][:, col] = gain
            t["l0.mix." + name + ".b"][:] = bias
    return edit


@pytest.mark.parametrize("kind", ["forgets", "keeps", "spikes", "decays below its input", "small input gates"])
def test_memory_gates(L, tmp_path, kind):
    """Forget gates near 0 and near 1, input gates that overtake the maximum by far, a maximum that sinks with the forget gates until an
    input overtakes it, and a maximum that stays at its start (the e^-m branch of the denominator)."""
    n, W = 300, 72
    x = rng(7).standard_normal((n, W))
    x[:, 0] = 0.0
    edit = {"forgets": gates((0, 0.5), (0, -9.0)), "keeps": gates((0, -1.0), (0, 12.0)), "spikes": gates((3.0, -4.0), (0, 5.0)),
            "decays below its input": gates((0, -11.0), (0, 0.0)), "small input gates": gates((0, -14.0), (0, 14.0))}[kind]
    if kind == "spikes":
        x[[5, 64, 65, 127, 200], 0] = 5.0
    for dtype in DTYPES:
        dec, want, t = one_layer(tmp_path, gm.memory(2, 24, 40, 15.0), x, edit, 2, dtype)
        for portions in ([n], [1] * n, [63, 2, 1, 62, 72, 100], [64, 64, 172]):
            err = parts_error(dec, want, t, portions, n)
            assert close(err, dtype, False), (dtype, portions[:3], int(err.argmax()), err.max())


def test_memory_carries_a_far_token(L, tmp_path):
    """One token writes far more than all others; what it wrote decides the outputs hundreds of tokens later (and where a query is almost
    orthogonal to its key, the far smaller rest does)."""
    n, W = 700, 72
    x = rng(8).standard_normal((n, W))
    x[:, 0] = 0.0
    x[3, 0] = 6.0
    for dtype in DTYPES:
        dec, want, t = one_layer(tmp_path, gm.memory(2, 16, 24, 15.0), x, gates((3.0, -9.0), (0, 11.0)), 3, dtype)
        lost = copy.deepcopy(t)
        lost["l0.mix.i"][:] = 0.0
        without = plain.forward(gm.config(W, n, [gm.memory(2, 16, 24, 15.0)]), lost, list(range(n)), want_layers=True)[1][-1] - t["embed"]
        assert np.median(row_rel(without[400:], want[400:])) > 0.3
        for portions in ([n], [2] + [1] * 40 + [n - 42], [650] + [1] * 50):
            assert close(parts_error(dec, want, t, portions, n), dtype, False, slack=5.0), (dtype, portions[:3])


def test_memory_state_starts_at_zero_whatever_the_buffers_hold(L, tmp_path):
    x = rng(9).standard_normal((150, 72))
    dec, want, t = one_layer(tmp_path, gm.memory(3, 20, 44, 7.5), x, no_edit, 4, "float32")
    for portions in ([150], [1] * 150):
        for s in dec.recurrent:
            s.view(torch.float32).fill_(float("nan"))
        torch.cuda.synchronize()
        assert parts_error(dec, want, t, portions, 150).max() < PART["float32"]


def test_more_heads_than_the_fused_output_product_takes(L, tmp_path):
    x = rng(10).standard_normal((70, 40))
    for dtype in DTYPES:
        dec, want, t = one_layer(tmp_path, gm.memory(260, 3, 2, 5.0), x, no_edit, 5, dtype)
        for portions in ([70], [1] * 70):
            assert close(parts_error(dec, want, t, portions, 70), dtype, False)


@pytest.mark.parametrize("rows,H,size,padded", [(1, 3, 20, 32), (70, 5, 130, 160), (9, 1, 1, 32)])
def test_head_norm_and_gate(L, rows, H, size, padded):
    g = rng(11)
    x, gate, w = (np.zeros((r, H, padded), np.float32) for r in (rows, rows, 1))
    for a, std in ((x, 0.02), (gate, 2.0), (w, 1.0)):
        a[:, :, :size] = std * g.standard_normal(a[:, :, :size].shape)
    eps = 3e-4                                                         # about the mean square: eps belongs inside the root
    f = lambda a: a.astype(np.float64)
    want = plain.rms_norm(f(x)[:, :, :size], eps) * f(w)[:, :, :size] * plain.sigmoid(f(gate)[:, :, :size])
    ld = H * padded + 8
    rowed = lambda a: dev(np.pad(a.reshape(len(a), -1), ((0, 0), (0, 8))))
    dx, dg, dw = rowed(x), rowed(gate), dev(w.reshape(-1))
    for out, code, tol in ((torch.zeros(rows, ld, device="cuda"), capi.F32, 1e-6), (torch.zeros(rows, ld, device="cuda", dtype=torch.bfloat16), capi.BF16, 2.0 ** -8)):
        capi.check(L.dh_head_norm_gate(dx.data_ptr(), ld, dg.data_ptr(), ld, dw.data_ptr(), out.data_ptr(), code, ld, rows, H, padded, size, eps))
        got = host(out)[:, :H * padded].reshape(rows, H, padded)
        assert np.abs(got[:, :, :size] - want).max() < tol * max(1.0, np.abs(want).max()) and not got[:, :, size:].any()
    # the same in front of the output product of one row
    N, K = 50, (H * padded + 63) // 64 * 64
    W = torch.randn(N, K, generator=torch.Generator().manual_seed(1)).to(torch.bfloat16)
    scale, res = torch.randn(N), torch.randn(N)
    y, dW, ds, dr = torch.zeros(N, device="cuda"), W.cuda(), scale.cuda(), res.cuda()
    capi.check(L.dh_dense_gemv_heads(dx.data_ptr(), dg.data_ptr(), dw.data_ptr(), H, padded, size, eps, dW.data_ptr(), K, N, K, ds.data_ptr(), dr.data_ptr(),
                                     y.data_ptr()))
    full = np.zeros(K)
    full[:H * padded].reshape(H, padded)[:, :size] = want[0]
    assert np.abs(host(y) - (W.double().numpy() @ full * scale.double().numpy() + res.double().numpy())).max() < 1e-4


# ------------------------------------------------------------------ latent attention

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,rot,e,rank", [(5, 24, 12, 40, 72), (16, 64, 32, 64, 128), (17, 140, 40, 136, 576), (1, 7, 2, 9, 13), (33, 64, 64, 64, 300),
                                            (3, 8, 100, 264, 64), (2, 200, 6, 128, 1), (20, 96, 16, 24, 512)])
def test_latent_shapes_prefill_steps_and_portions(L, tmp_path, H, d, rot, e, rank, dtype):
    n = 200
    x = rng(H + d).standard_normal((n, 72))
    dec, want, t = one_layer(tmp_path, gm.latent(H, d, rot, e, rank, window=70, base=300.0), x, no_edit, 1, dtype)
    for portions in PORTIONS(n):
        err = parts_error(dec, want, t, portions, n)
        assert close(err, dtype, rank > 1), (portions[:3], int(err.argmax()), err.max())


def stand_out(planted, part, far=0):
    """Inputs and edit under which one token's key stands out for every later query, through its unrotated or its rotated part."""
    W = 72
    x = rng(12).standard_normal((300, W))
    x[:, 0], x[:, 1] = 0.0, 4.0
    x[planted] = 0.0
    x[planted, 0], x[planted, 1] = 20.0, 4.0
    x[planted, 8:] = 2.0 * rng(13).standard_normal(W - 8)

    def edit(t):
        m = "l0.mix."
        t["l0.norm1"][:] = 0.0
        t[m + "q"] *= 0.05
        t[m + "dkv"][:, :2] = 0.0
        rank = t[m + "dkv.norm"].shape[0]
        rot = t[m + "dkv"].shape[0] - rank
        d = t[m + "uk"].shape[0] // 4
        q = t[m + "q"].reshape(4, d + rot, W)
        if part == "latent":
            t[m + "dkv"][0] = 0.0
            t[m + "dkv"][0, 0] = 8.0
            t[m + "uk"].reshape(4, d, rank)[:, 0, :] = 0.0
            t[m + "uk"].reshape(4, d, rank)[:, 0, 0] = 6.0
            q[:, 0, 1] = 6.0
        else:                        # the slowest pair: its angle hardly moves over the sequence
            t[m + "dkv"][rank + rot - 2] = 0.0
            t[m + "dkv"][rank + rot - 2, 0] = 12.0
            q[:, d + rot - 2, 1] = 6.0
    return x, edit


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 2, 7, 63, 64, 65, 128, 129, None])
def test_latent_window_edges(L, tmp_path, window, dtype):
    """One key stands out: the queries that just see it and those that just do not are far apart."""
    n, planted = 300, 100
    for part in ("latent", "rotated"):
        x, edit = stand_out(planted, part)
        dec, want, t = one_layer(tmp_path, gm.latent(4, 24, 8, 40, 48, window=window, base=1e7, scale=0.3), x, edit, 6, dtype)
        if window and planted + window < n and window > 1:
            inside, outside = planted + window - 1, planted + window
            assert row_rel(want[None, outside], want[None, inside])[0] > 0.5 and row_rel(want[None, inside], want[None, planted])[0] < 0.3
        for portions in ([n], [1] * n, [64] * 4 + [44], [99, 2, 1, 60, 1, 1, 66, 70]):
            err = parts_error(dec, want, t, portions, n)
            assert close(err, dtype), (part, portions[:3], int(err.argmax()), err.max())


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_far_keys_and_first_tokens(L, tmp_path, dtype):
    """No window over many key tiles and splits: a key near the start decides queries more than a thousand tokens on."""
    n = 1500
    x0, edit = stand_out(2, "latent")
    x = np.concatenate([x0, rng(14).standard_normal((n - 300, 72))])
    x[300:, 0], x[300:, 1] = 0.0, 4.0
    dec, want, t = one_layer(tmp_path, gm.latent(4, 24, 8, 40, 48, base=1e7, scale=0.3), x, edit, 7, dtype)
    assert row_rel(want[-1:], want[2:3])[0] < 0.4
    for portions in ([n], [5, 1, 1, 1, 1492], [1490] + [1] * 10):
        assert close(parts_error(dec, want, t, portions, n), dtype), portions[:3]


def test_latent_norm_keeps_eps_inside_the_root_and_scale_is_a_parameter(L, tmp_path):
    x = rng(15).standard_normal((120, 72))

    def edit(t):
        t["l0.mix.dkv"][:48] *= 0.02                       # mean square of the raw latents about 4e-4
    for dtype in DTYPES:
        for scale in (0.05, 0.9):
            dec, want, t = one_layer(tmp_path, gm.latent(4, 24, 8, 40, 48, window=30, scale=scale), x, edit, 8, dtype, eps=1e-3)
            for portions in ([120], [1] * 120):
                assert close(parts_error(dec, want, t, portions, 120), dtype)


def test_lent_latent_rows_under_another_window(tmp_path, L):
    """The borrower sees further back than the lender and has heads of other sizes; it reads rows the lender wrote in the same step."""
    for dtype in DTYPES:
        cfg = gm.config(72, 90, [gm.latent(3, 16, 8, 24, 40, window=4, base=77.0), gm.memory(2, 16, 16, 5.0),
                                 gm.latent(6, 40, 8, 8, 40, window=90, base=77.0, scale=0.3, kv_from=0),
                                 gm.latent(2, 8, 8, 56, 40, base=77.0, kv_from=0)])
        t = gm.tensors(cfg, 9)
        toks = gm.prompt(cfg, 160, 10)
        want = plain.forward(cfg, t, toks)
        dec = models.load(gm.write(tmp_path / dtype, cfg, t), 160, dtype)
        for portions in ([160], [1] * 160, [2] * 80):
            assert gm.row_errors(feed_all(dec, toks, portions), want).max() < ROW[dtype]


def test_the_cache_holds_normed_latents_and_rotated_parts(L, tmp_path):
    x = rng(16).standard_normal((60, 72))
    layer = gm.latent(5, 24, 12, 40, 72, window=33, base=900.0)
    dec, _, t = one_layer(tmp_path, layer, x, no_edit, 10, "float32")
    streams(dec, list(range(60)), [30] + [1] * 30)
    h = plain.rms_norm(t["embed"], 1e-5, 1 + t["l0.norm1"])
    c, k = plain.latent_rows(layer["mixer"], {"l.dkv": t["l0.mix.dkv"], "l.dkv.norm": t["l0.mix.dkv.norm"]}, "l", h, 1e-5)
    rows = host(dec.layers[0].mixer.cache)[:60 * dec.layers[0].mixer.width].reshape(60, -1)
    assert np.abs(rows[:, :72] - c).max() < 2e-5 and np.abs(rows[:, 128:140] - k).max() < 2e-5
    assert not rows[:, 72:128].any() and not rows[:, 140:].any()


# ------------------------------------------------------------------ feed-forwards

def silent_mixer(t):
    t["l0.mix.o"][:] = 0.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [1, 88, 300])
def test_dense_feed_forward(L, tmp_path, ff, dtype):
    x = 2.0 * rng(17).standard_normal((160, 136))
    dec, want, t = one_layer(tmp_path, gm.memory(1, 8, 8, 5.0, mlp=gm.dense(ff)), x, silent_mixer, 11, dtype)
    for portions in ([160], [1] * 160):
        assert close(parts_error(dec, want, t, portions, 160), dtype, False)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,ff,limit,shared", [(5, 2, 36, 0.8, (52, 1.3)), (8, 1, 72, 1.2, (136, 1.7)), (3, 3, 130, 0.2, None), (8, 7, 20, 5.0, (7, 0.1)),
                                                   (1, 1, 1, 1.0, None)])
def test_experts(L, tmp_path, E, top, ff, limit, shared, dtype):
    n = 300
    x = rng(18).standard_normal((n, 136))
    x[:, :gm.LEVELS] = 1.5 * (np.argsort(rng(19).random((n, gm.LEVELS)), axis=1) - 3.5)
    dec, want, t = one_layer(tmp_path, gm.memory(1, 8, 8, 5.0, mlp=gm.moe(E, top, ff, limit, shared)), x, silent_mixer, 12, dtype)
    for portions in ([n], [1] * n, [2, 3, 295]):
        err = parts_error(dec, want, t, portions, n)
        assert close(err, dtype, False), (portions[:3], int(err.argmax()), err.max())


@pytest.mark.parametrize("E,top", [(65, 3), (300, 32), (1024, 2)])
def test_many_experts_are_chosen_exactly(L, tmp_path, E, top):
    """True 32-bit logits of many experts; a token whose expert nobody else uses, and one expert all tokens share."""
    n, W = 90, 64
    x = rng(20).standard_normal((n, W))

    def edit(t):
        silent_mixer(t)
        t["l0.norm2"][:] = 0.0
        for k in range(E):
            for name, shape in (("gate", (4, W)), ("up", (4, W)), ("down", (W, 4))):
                t["l0.mlp.e%d.%s" % (k, name)] = rng(1000 + k).standard_normal(shape)
        t["l0.mlp.router"] = rng(21).standard_normal((E, W)) * W ** -0.5
        t["l0.mlp.router"][E - 1, :] = 3.0 * np.sign(t["embed"][0]) / W                 # expert E - 1: the first token's, strongly
    layer = gm.memory(1, 8, 8, 5.0, mlp=gm.moe(8, 1, 4, 1.0))
    cfg = gm.config(W, n, [layer])
    t = gm.tensors(cfg, 13)
    t["embed"] = gm.bf16(x)
    layer["mlp"]["router"] = {"experts": E, "top": top}
    edit(t)
    t = {k: gm.bf16(v) for k, v in t.items()}
    # no call closer than rounding: the router's rows are moved until every token's is clear
    h = plain.rms_norm(t["embed"], 1e-5)
    z = np.sort(h @ t["l0.mlp.router"].T, axis=1)[:, ::-1]
    clear = (z[:, top - 1] - z[:, top]) > 1e-4
    assert clear.mean() > 0.8
    want = plain.forward(cfg, t, list(range(n)), want_layers=True)[1][-1] - t["embed"]
    dec = models.load(gm.write(tmp_path / "m", cfg, t), n, "float32")
    for portions in ([n], [1] * n):
        assert parts_error(dec, want, t, portions, n)[clear].max() < PART["float32"]


def test_equal_logits_go_to_the_lower_expert(L, tmp_path):
    x = rng(22).standard_normal((40, 64))

    def edit(t):
        silent_mixer(t)
        t["l0.mlp.router"][:] = 0.0
        t["l0.mlp.router"][1:4, 9] = 1.0
    for dtype in DTYPES:
        dec, want, t = one_layer(tmp_path, gm.memory(1, 8, 8, 5.0, mlp=gm.moe(6, 2, 8, 1.0)), x, edit, 14, dtype)
        for portions in ([40], [1] * 40):
            assert close(parts_error(dec, want, t, portions, 40), dtype)


def test_layer_scales_and_norms_around_zero(L, tmp_path):
    """Scales of either sign and zero, norm weights that are zero (factor 1) and -1 (factor 0)."""
    x = rng(23).standard_normal((90, 136))

    def edit(t):
        for k in ("1", "2"):
            t["l0.ls" + k] = rng(24).standard_normal(136)
            t["l0.ls" + k][10:20] = 0.0
        t["l0.norm1"][20:40] = 0.0
        t["l0.norm1"][40:50] = -1.0
    for dtype in DTYPES:
        dec, want, t = one_layer(tmp_path, gm.latent(3, 16, 8, 24, 40, window=20, mlp=gm.dense(60)), x, edit, 15, dtype)
        for portions in ([90], [1] * 90):
            assert close(parts_error(dec, want, t, portions, 90), dtype)
            assert not (streams(dec, list(range(90)), portions) - t["embed"])[:, 10:20].any()


def test_column_scales_and_exact_gelu_of_the_products(L):
    g = torch.Generator().manual_seed(3)
    for M, N, K in ((1, 70, 64), (70, 130, 192), (300, 1500, 256), (3, 100, 4096)):
        W = (torch.randn(N, K, generator=g) / K ** 0.5).to(torch.bfloat16)
        bias, scale = torch.randn(N, generator=g), torch.randn(N, generator=g)
        dW, db, ds = W.cuda(), bias.cuda(), scale.cuda()
        for code, dt in ((capi.F32, torch.float32), (capi.BF16, torch.bfloat16)):
            A = torch.randn(M, K, generator=g).to(dt)
            res = torch.randn(M, N, generator=g)
            acc = (A.double() @ W.double().T).numpy()
            dA, C, C2 = A.cuda(), res.cuda(), torch.zeros(M, N, dtype=dt, device="cuda")
            capi.check(L.dh_dense_matmul_scaled(dA.data_ptr(), code, K, dW.data_ptr(), K, M, N, K, 0.75, db.data_ptr(), ds.data_ptr(), C.data_ptr(), C.data_ptr(),
                                                N, N, None, 0, 0, capi.ACT_NONE))
            want = (0.75 * acc + bias.double().numpy()) * scale.double().numpy() + res.double().numpy()
            assert np.abs(host(C) - want).max() < 5e-5
            capi.check(L.dh_dense_matmul(dA.data_ptr(), code, K, dW.data_ptr(), K, M, N, K, 1.0, None, None, None, 0, 0, C2.data_ptr(), code, N, capi.ACT_GELU_ERF))
            want = plain.gelu_erf(acc)
            assert np.abs(host(C2) - want).max() < (2.0 ** -8 if code == capi.BF16 else 1e-5) * max(1.0, np.abs(want).max())
            if M == 1 and code == capi.F32:
                y, y2 = res.cuda(), torch.zeros(N, device="cuda")
                capi.check(L.dh_dense_gemv_scaled(dA.data_ptr(), None, 0, 0.0, dW.data_ptr(), K, N, K, 0.75, db.data_ptr(), ds.data_ptr(), y.data_ptr(), y.data_ptr(),
                                                  N, None, capi.ACT_NONE))
                assert np.abs(host(y) - host(C)[0]).max() < 1e-5
                capi.check(L.dh_dense_gemv(dA.data_ptr(), None, 0, 0.0, dW.data_ptr(), K, N, K, 1.0, None, None, None, 0, y2.data_ptr(), capi.ACT_GELU_ERF))
                assert np.abs(host(y2) - plain.gelu_erf(acc)[0]).max() < 1e-5


def test_half_precision_products(L):
    """f16 activations stand for f16 weights (rows an f16 cache holds)."""
    g = torch.Generator().manual_seed(4)
    for M, N, K, lda in ((1, 40, 64, 96), (200, 300, 128, 160), (130, 2100, 512, 544)):
        A, W = torch.randn(M, lda, generator=g).to(torch.float16), (torch.randn(N, K, generator=g) / K ** 0.5).to(torch.float16)
        dA, dW, out = A.cuda(), W.cuda(), torch.zeros(M, N, dtype=torch.float16, device="cuda")
        capi.check(L.dh_dense_matmul(dA.data_ptr(), capi.F16, lda, dW.data_ptr(), K, M, N, K, 1.0, None, None, None, 0, 0, out.data_ptr(), capi.F16, N, capi.ACT_NONE))
        want = (A[:, :K].double() @ W.double().T).numpy()
        assert np.abs(host(out) - want).max() < 2.0 ** -10 * np.abs(want).max()


def test_bad_specs_are_refused(L, tmp_path):
    x = rng(25).standard_normal((20, 72))
    dec, _, _ = one_layer(tmp_path, gm.latent(3, 16, 8, 24, 40, window=5, mlp=gm.moe(4, 2, 8, 1.0)), x, no_edit, 16, "float32")
    lat, ex = dec.layers[0].mixer, dec.layers[0].ff
    some = dec.x.data_ptr()
    for field, value, message in (("D", 12, "multiples of 8"), ("R", 16, "of 32"), ("C", 40, "latent"), ("rot_dim", 7, "rot_dim"), ("window", -1, "window"),
                                  ("cache_dtype", capi.BF16, "caches"), ("ld_row", 8, "does not hold"), ("d_cos", None, "null")):
        s = capi.Latent.from_buffer_copy(lat.spec)
        setattr(s, field, value)
        assert L.dh_latent_rows(ctypes.byref(s), some, lat.cache.data_ptr(), 2, 0) != 0
        assert message in L.dh_last_error().decode(), (field, L.dh_last_error())
    for field, value, message in (("top", 5, "experts"), ("ff", 40, "multiples of 64"), ("K", 65, "multiple of 64"), ("d_router", None, "null"), ("experts", 2000, "experts")):
        s = capi.Experts.from_buffer_copy(ex.spec)
        setattr(s, field, value)
        assert L.dh_experts_step(ctypes.byref(s), some, some) != 0
        assert message in L.dh_last_error().decode(), (field, L.dh_last_error())
    good = dict(H=2, dim=8, vdim=8, DP=32, VP=32, k_offset=64, v_offset=128, i_offset=192, f_offset=194, ld_row=196, gate_cap=1.0)
    for field, value, message in (("DP", 8, "multiples of 32"), ("gate_cap", 0.0, "cap"), ("ld_row", 192, "does not hold"), ("k_offset", 32, "does not hold")):
        s = capi.MLSTM(*[dict(good, **{field: value})[k] for k, _ in capi.MLSTM._fields_])
        assert L.dh_mlstm_step(ctypes.byref(s), some, some, some, 0, None) != 0
        assert message in L.dh_last_error().decode(), (field, L.dh_last_error())
    with pytest.raises(ValueError, match="longer"):
        sublayers.DenseFF(dec, dict(ff=40000, activation="gelu_erf"), {}, np.zeros(72), None)


# ------------------------------------------------------------------ whole models

@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("gusolorn")
    out = {}
    for name, cfg, seed in (("mixed", gm.MIXED, 21), ("wide", gm.WIDE, 22), ("even", gm.EVEN, 23), ("odd", gm.ODD, 24)):
        t = gm.tensors(cfg, seed)
        out[name] = (gm.write(base / name, cfg, t), cfg, t)
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


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide", "even", "odd"])
def test_logits_whole_decoded_and_in_portions(folders, name, dtype):
    folder, cfg, t = folders[name]
    toks = gm.prompt(cfg, 180, 31)
    want = plain.forward(cfg, t, toks)
    dec = models.load(folder, 200, dtype)
    for portions in ([180], [1] * 180, [2] * 90, [3, 1, 62, 2, 1, 1, 64, 33, 13], [65, 115]):
        err = gm.row_errors(feed_all(dec, toks, portions), want)
        assert err.max() < ROW[dtype], (portions[:4], int(err.argmax()), err.max())
    # one prompt in chunks of the batched path's own
    dec.reset()
    assert gm.row_errors(dec.prefill(toks, chunk=50, want=[0, 49, 50, 179]), want[[0, 49, 50, 179]]).max() < ROW[dtype]


def test_layers_of_the_residual_stream(folders, tmp_path):
    """Models cut after every layer: the stream itself, of a portion and of a step."""
    _, cfg, t = folders["mixed"]
    toks = gm.prompt(cfg, 40, 32)
    _, want = plain.forward(cfg, t, toks, want_layers=True)
    for n in range(1, len(cfg["layers"]) + 1):
        dec = models.load(gm.write(tmp_path / str(n), dict(cfg, layers=cfg["layers"][:n]), t), 64, "float32")
        for portions in ([40], [39, 1]):
            assert row_rel(streams(dec, toks, portions), want[n - 1]).max() < 1e-5, n


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_sequences_one_after_another_reuse_cache_and_state(folders, dtype):
    """Long, short, long again: rows and states an earlier sequence left behind must not be seen."""
    folder, cfg, t = folders["mixed"]
    dec = models.load(folder, 160, dtype)
    for i, n in enumerate((150, 1, 2, 70, 9, 160)):
        toks = gm.prompt(cfg, n, 40 + i)
        want = plain.forward(cfg, t, toks)
        cut = n // 2
        for portions in ([cut, n - cut] if cut else [n], [1] * n):
            assert gm.row_errors(feed_all(dec, toks, portions), want).max() < ROW[dtype], n


def test_a_sequence_does_not_depend_on_what_ran_before_it(folders):
    """The same portions after different predecessors give the same bits."""
    folder, cfg, _ = folders["mixed"]
    toks = gm.prompt(cfg, 100, 50)
    for dtype in DTYPES:
        dec = models.load(folder, 160, dtype)
        first = feed_all(dec, toks, [70, 1, 1, 28])
        feed_all(dec, gm.prompt(cfg, 160, 51), [160])
        assert np.array_equal(feed_all(dec, toks, [70, 1, 1, 28]), first)


def test_long_decoding_passes_every_window(folders):
    folder, cfg, t = folders["mixed"]
    toks = gm.prompt(cfg, 390, 51)
    want = plain.forward(cfg, t, toks)
    dec = models.load(folder, 400, "float32")
    assert gm.row_errors(feed_all(dec, toks, [20] + [1] * 370), want).max() < ROW["float32"]
    with pytest.raises(ValueError, match="max_seq"):
        feed_all(dec, toks + [1] * 11, [390, 11])


def test_a_long_prompt_in_chunks(folders):
    """More tokens than a portion of the batched path takes, over many memory chunks."""
    folder, cfg, t = folders["even"]
    toks = gm.prompt(cfg, 1100, 53)
    want = plain.forward(cfg, t, toks)
    for dtype in DTYPES:
        dec = models.load(folder, 1100, dtype)
        at = list(range(0, 1100, 37)) + [1099]
        for chunk in (512, 2048):
            dec.reset()
            assert gm.row_errors(dec.prefill(toks, chunk=chunk, want=at), want[at]).max() < ROW[dtype], (dtype, chunk)


def test_positions_that_do_not_follow_are_refused(folders):
    folder, cfg, _ = folders["even"]
    dec = models.load(folder, 60, "float32")
    dec.prefill(gm.prompt(cfg, 10, 54))
    with pytest.raises(ValueError, match="stands at position 10"):
        dec.step(3, 12)
    with pytest.raises(ValueError, match="stands at position 10"):
        dec.prefill([1, 2, 3], start_pos=9)
    dec.step(3, 10)


# ------------------------------------------------------------------ generation

def test_greedy_generation_every_way(folders):
    """The framework's own loops: generate, blocking steps, staged readback, batched submits, the captured step."""
    folder, cfg, t = folders["even"]
    prompt = gm.prompt(cfg, 30, 71)
    n = 40
    want = plain.greedy(cfg, t, prompt, n)
    dec = models.load(folder, 120, "float32")
    assert isinstance(dec, decoder.DecoderBase) and isinstance(dec, dense_decoder.DenseDecoder)
    assert dec.generate(prompt, n) == want
    assert dec.generate(prompt, n, chunk=7) == want
    first = dec.prefill(prompt)
    assert [first] + dec.decode_greedy(first, 30, n - 1) == want
    dec.release_readback()
    first = dec.prefill(prompt)
    assert [first] + dec.decode_batch(first, 30, 20) + dec.decode_batch(want[20], 50, n - 21) == want
    # token by token from nothing, then the captured step replayed, capture in the middle of the sequence
    out = [dec.step(tok, p) for p, tok in enumerate(prompt)][-1:]
    graph = [dec.step_graph(out[0], 30)]
    for i in range(1, n - 1):
        if i % 7 == 0:
            graph.append(dec.step(graph[-1], 30 + i))
        else:
            graph.append(dec.step_graph(graph[-1], 30 + i))
    assert out + graph == want
    # a replay for another sequence, from its first position on
    other = gm.prompt(cfg, 9, 72)
    for p, tok in enumerate(other):
        g = dec.step_graph(tok, p)
    assert g == plain.greedy(cfg, t, other, 1)[0]
    dec.release_graph()
    with pytest.raises(ValueError, match="on the device"):
        dec.capture_step(5, device_kv_len=False)
    with pytest.raises(ValueError, match="does not fit"):
        dec.generate(prompt, 120)


def test_generation_in_the_served_precision_and_sampling(folders):
    folder, cfg, t = folders["mixed"]
    prompt = gm.prompt(cfg, 25, 73)
    dec = models.load(folder, 80)
    assert dec.compute == "bf16"
    a = dec.generate(prompt, 30)
    logits = plain.forward(cfg, t, prompt + a)
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
    dec = models.load(gm.write(tmp_path / "a", cfg, t), 40, finiteness_guard=True)
    tok = dec.prefill(gm.prompt(cfg, 5, 74))
    dec.step(tok, 5)
    bad = dict(t)
    bad["l1.mlp.down"] = gm.bf16(t["l1.mlp.down"] * 1e8)
    dec = models.load(gm.write(tmp_path / "b", cfg, bad), 40, finiteness_guard=True)
    tok = dec.prefill(gm.prompt(cfg, 5, 74))
    with pytest.raises(decoder.FinitenessError, match="layer 1"):
        dec.step(tok, 5)


def test_command_line_generates(folders, capsys):
    folder, cfg, t = folders["even"]
    prompt = gm.prompt(cfg, 12, 75)
    assert generate.main(["--model", folder, "--dtype", "float32", "--prompt", ",".join(map(str, prompt)), "--max-tokens", "15"]) == 0
    out = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert out["prompt"] == prompt and out["tokens"] == plain.greedy(cfg, t, prompt, 15)


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(folders, tmp_path, dtype):
    folder, cfg, t = folders["mixed"]
    a, b = gm.prompt(cfg, 90, 81), gm.prompt(cfg, 33, 82)
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
        assert gm.row_errors(got, want).max() < ROW[dtype], step


def test_random_weights_make_a_model():
    cfg = gusolorn.decoder_config(gm.EVEN)
    w = gusolorn.random_weights(cfg, seed=4)
    a = dense_decoder.DenseDecoder(cfg, w, 64, compute="f32").generate([1, 2, 3], 20)
    b = dense_decoder.DenseDecoder(cfg, w, 64, compute="f32").generate([1, 2, 3], 20, chunk=2)
    assert a == b and len(a) == 20
