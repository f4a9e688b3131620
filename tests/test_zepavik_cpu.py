"""Zepavik without a GPU: configuration and tensor reading, the stacked and padded weights, the registry, and the plain
restatement itself (its mechanisms against hand-made cases, so that the GPU tests compare with something checked)."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from doppler_amd import build, capi, dense_decoder, models, safetensors_file, zepavik
from oracle import plain_zepavik as plain
from tests import zepavik_models as zm

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ------------------------------------------------------------------ plain restatement

def test_plain_window_is_exact_at_both_edges():
    m = plain.window_mask(12, 4)
    assert [list(np.flatnonzero(r)) for r in m[:6]] == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [1, 2, 3, 4], [2, 3, 4, 5]]
    assert np.array_equal(plain.window_mask(5, 1), np.eye(5, dtype=bool))


def test_plain_attention_of_equal_scores_follows_the_distance_bias():
    """Zero queries: the weights are (1 + r2 x)^-r1, normalised over the window."""
    n, w = 9, 5
    v = np.random.default_rng(1).standard_normal((n, 1, 3))
    r1, r2 = np.array([0.8, 0.0]), np.array([0.4, 7.0])
    out = plain.attention(np.zeros((n, 2, 4)), np.ones((n, 1, 4)), v, 0.3, r1, r2, w)
    for h in range(2):
        x = np.arange(w)
        p = (1 + r2[h] * x) ** -r1[h]
        want = sum(p[k] * v[n - 1 - k, 0] for k in range(w)) / p.sum()
        assert np.allclose(out[n - 1, h], want)
    assert np.allclose(out[0, 0], v[0, 0])


def test_plain_bigram_rows_and_norm():
    assert list(plain.bigram_rows([3, 5, 2], 7, 10, 3)) == [7, (30 + 15) % 7, (50 + 6) % 7]
    x = np.array([[3.0, 4.0]])
    assert np.allclose(plain.rms_norm(x, 0.5), x / np.sqrt(12.5 + 0.5))
    assert np.allclose(plain.rms_norm(np.zeros((1, 4)), 1e-5), 0.0)


def test_plain_model_is_causal_and_reads_the_previous_token():
    cfg, t = zm.EVEN, zm.tensors(zm.EVEN, 3)
    a = zm.prompt(cfg, 20, 4)
    b = list(a)
    b[12] = (b[12] + 1) % cfg["vocab"]
    la, lb = plain.forward(cfg, t, a), plain.forward(cfg, t, b)
    assert np.allclose(la[:12], lb[:12]) and not np.allclose(la[12], lb[12]) and not np.allclose(la[13], lb[13])


# ------------------------------------------------------------------ configuration, weights, registry

def test_configuration_round_trip_and_unknown_keys_fail_closed():
    for c in (zm.MIXED, zm.WIDE_HEADS, zm.EVEN, zm.ODD):
        assert zepavik.config_json(zepavik.decoder_config(c)) == c

    def broken(edit):
        c = copy.deepcopy(zm.MIXED)
        edit(c)
        return c
    for edit, message in (
            (lambda c: c.update(rope={}), "rope"),
            (lambda c: c["layers"][0]["mixer"].update(softcap=3), "softcap"),
            (lambda c: c["layers"][1]["mixer"]["mask"].update(first=2), "first"),
            (lambda c: c["layers"][0]["mixer"].pop("vdim"), "vdim"),
            (lambda c: c["layers"][0].update(type="recurrent"), "recurrent"),
            (lambda c: c["layers"][0]["mlp"].update(kind="experts"), "experts"),
            (lambda c: c["layers"][0]["mixer"].update(heads=7), "multiple"),
            (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
            (lambda c: c.update(architecture="Other"), "Other")):
        with pytest.raises(zepavik.ConfigError, match=message):
            zepavik.decoder_config(broken(edit))


def test_model_folder_is_read_back_exactly(tmp_path):
    cfg, t = zm.MIXED, zm.tensors(zm.MIXED, 5)
    got_cfg, w = zepavik.load_arrays(zm.write(tmp_path / "a", cfg, t))
    assert np.array_equal(dense_decoder.bf16_to_f32(w["embed"]).astype(np.float64), t["embed"])
    assert np.array_equal(w["layers"][2]["k_bias"].astype(np.float64), t["l2.mix.k.b"])
    assert "up" not in w["layers"][1] and w["layers"][3]["down"].shape == (136, 56)
    # written by the package's own writer, read by both readers
    zepavik.write_model(str(tmp_path / "b"), got_cfg, w)
    cfg2, w2 = zepavik.load_arrays(str(tmp_path / "b"))
    assert cfg2 == got_cfg and all(np.array_equal(w[k], w2[k]) for k in ("embed", "bigram", "pos", "head", "final_norm"))
    from safetensors.torch import load_file
    assert np.array_equal(load_file(str(tmp_path / "b" / "model.safetensors"))["l0.mix.g"].double().numpy(), t["l0.mix.g"])
    # a tensor of another shape is named
    bad = dict(t, **{"l1.mix.o": t["l1.mix.o"][:, :-1]})
    with pytest.raises(safetensors_file.SafetensorsError, match="l1.mix.o"):
        zepavik.load_arrays(zm.write(tmp_path / "c", cfg, bad))
    del bad["l1.mix.o"]
    with pytest.raises(safetensors_file.SafetensorsError, match="l1.mix.o"):
        zepavik.load_arrays(zm.write(tmp_path / "d", cfg, bad))


def test_truncated_files_are_refused(tmp_path):
    d = zm.write(tmp_path, zm.EVEN, zm.tensors(zm.EVEN, 6))
    path = os.path.join(d, "model.safetensors")
    data = open(path, "rb").read()
    open(path, "wb").write(data[:-64])
    st = safetensors_file.SafetensorsFile(path)
    with pytest.raises(safetensors_file.SafetensorsError, match="data range"):
        for name in st.names():
            st.tensor(name)
    open(path, "wb").write(data[:6])
    with pytest.raises(safetensors_file.SafetensorsError, match="too short"):
        safetensors_file.SafetensorsFile(path)


@pytest.mark.parametrize("cfg", [zm.MIXED, zm.WIDE_HEADS, zm.ODD], ids=["mixed", "wide-heads", "odd"])
def test_stacked_and_padded_weights_are_the_separate_products(tmp_path, cfg):
    t = zm.tensors(cfg, 7)
    c, w = zepavik.load_arrays(zm.write(tmp_path, cfg, t))
    x = np.random.default_rng(8).standard_normal(c["hidden"])
    for i, spec in enumerate(c["layers"]):
        m, p = spec["mixer"], "l%d." % i
        w_in, bias, w_out, g = dense_decoder.stack_layer(m, spec["mlp"], w["layers"][i], c["hidden"])
        assert w_in.shape[1] % 64 == 0 and w_out.shape[1] % 64 == 0 and g["D"] % 8 == 0 and g["VD"] % 8 == 0
        y = dense_decoder.bf16_to_f32(w_in).astype(np.float64) @ np.pad(x, (0, w_in.shape[1] - x.size))
        y[:g["n_first"]] += bias
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for name, heads, size, padded, at in (("q", H, d, g["D"], 0), ("k", G, d, g["D"], g["k_offset"]), ("v", G, e, g["VD"], g["v_offset"])):
            got = y[at:at + heads * padded].reshape(heads, padded)
            want = (t[p + "mix." + name] @ x + t[p + "mix." + name + ".b"]).reshape(heads, size)
            assert np.allclose(got[:, :size], want) and not got[:, size:].any()
        assert np.allclose(y[g["gate_offset"]:g["gate_offset"] + H], t[p + "mix.g"] @ x)
        attn = np.random.default_rng(9).standard_normal((H, e))
        row = np.zeros(w_out.shape[1])
        row[:H * g["VD"]].reshape(H, g["VD"])[:, :e] = attn
        want = t[p + "mix.o"] @ attn.reshape(-1)
        if spec["mlp"]:
            act = np.random.default_rng(10).standard_normal(g["ff"])
            assert np.allclose(y[g["n_first"]:], t[p + "mlp.up"] @ x)
            row[g["attn_cols"]:g["attn_cols"] + g["ff"]] = act
            want = want + t[p + "mlp.down"] @ act
        else:
            assert y.size == g["n_first"]
        assert np.allclose(dense_decoder.bf16_to_f32(w_out).astype(np.float64) @ row, want)


def test_bf16_rounding_helpers():
    x = np.array([1.0, 1.00390625, 1.01171875, -3.3e38, 1e-40, 0.1], np.float32)
    import torch
    want = torch.from_numpy(x).to(torch.bfloat16).view(torch.int16).numpy().view(np.uint16)
    assert np.array_equal(dense_decoder.f32_to_bf16(x), want)
    assert np.array_equal(dense_decoder.f32_to_bf16(dense_decoder.bf16_to_f32(want)), want)


def test_registry_chooses_by_the_folder(tmp_path):
    d = zm.write(tmp_path / "z", zm.EVEN, zm.tensors(zm.EVEN, 11))
    assert models.find(d).name == "Zepavik" and models.find(d).library == "dense"
    with pytest.raises(models.UnsupportedDtype):
        models.RDRR.load(d, 16, "float32")
    os.makedirs(str(tmp_path / "r"))
    open(str(tmp_path / "r" / "manifest.json"), "w").write("{}")
    assert models.find(str(tmp_path / "r")) is models.RDRR
    os.makedirs(str(tmp_path / "u"))
    json.dump({"architecture": "Nobody"}, open(str(tmp_path / "u" / "config.json"), "w"))
    with pytest.raises(models.UnknownModel, match="Nobody"):
        models.find(str(tmp_path / "u"))
    os.makedirs(str(tmp_path / "e"))
    with pytest.raises(models.UnknownModel, match="neither"):
        models.find(str(tmp_path / "e"))


def test_dense_sources_are_a_closed_set():
    """Every dh:: function the dense families call is defined among them (the library linked from them alone would
    otherwise fail to load where only it is built)."""
    import re
    text = {s: open(os.path.join(build.CSRC, s)).read() for s in os.listdir(build.CSRC) if s.endswith(".hip")}
    common = open(os.path.join(build.CSRC, "dh_common.h")).read()
    for name in ("q4k_gemm", "q4k_gemv_i8", "q4k_gemv_rows", "q4k_gemm_gate_up"):
        assert re.search(r"\b%s\(" % name, common)
        for s in build.DENSE_SOURCES:
            assert not re.search(r"\b%s\(" % name, text[s]), (s, name)
    wanted = {"dh_dense_matmul", "dh_dense_gemv", "dh_dense_lmhead_argmax", "dh_embed_sum", "dh_rmsnorm_rows", "dh_attn_spec_decode",
              "dh_attn_spec_prefill", "dh_attn_spec_kv_write", "dh_sample_topk", "dh_argmax", "dh_check_finiteness", "dh_graph_begin"}
    joined = "\n".join(text[s] for s in build.DENSE_SOURCES)
    for name in wanted:
        assert name in capi.SIGNATURES and re.search(r"\b%s\(" % name, joined), name


def test_command_lines_explain_themselves():
    for cmd in ([sys.executable, "-m", "doppler_amd.generate", "--help"], [os.path.join(ROOT, "bin", "trace_run"), "--help"]):
        r = subprocess.run(cmd, cwd=ROOT, capture_output=True, text=True, timeout=120)
        assert r.returncode == 0 and "--model" in r.stdout


def test_argument_errors_need_no_device():
    """Shapes are refused on the host (here already for want of a device, on a GPU by the same calls' own checks)."""
    L = capi.load()
    assert L.dh_dense_matmul(None, capi.BF16, 64, None, 64, 1, 1, 64, 1.0, None, None, None, 1, 1, None, 0, 0, capi.ACT_NONE) != 0
    assert L.dh_attn_spec_workspace_bytes(4, 64, 1000) == 4 * 16 * 66 * 4
