"""Gusolorn without a GPU: configuration and tensor reading, padding and stacking, the registry, and the plain restatement itself
(its mechanisms against hand-made cases, so that the GPU tests compare with something checked)."""
import copy
import math
import os
from types import SimpleNamespace

import numpy as np
import pytest

from doppler_amd import build, capi, decoder, gusolorn, models, safetensors_file, sublayers
from doppler_amd.config_fields import ConfigError
from oracle import plain_gusolorn as plain
from tests import gusolorn_models as gm

MODELS = {"mixed": gm.MIXED, "wide": gm.WIDE, "odd": gm.ODD, "even": gm.EVEN}


def rng(seed):
    return np.random.Generator(np.random.PCG64(seed))


# ------------------------------------------------------------------ plain restatement

def test_plain_window_is_exact_at_both_edges():
    m = plain.window_mask(12, 4)
    assert [list(np.flatnonzero(r)) for r in m[:6]] == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [1, 2, 3, 4], [2, 3, 4, 5]]
    assert np.array_equal(plain.window_mask(5, 1), np.eye(5, dtype=bool))


def test_plain_rotation_depends_on_the_distance_and_pairs_neighbours():
    g = rng(1)
    q, k = g.standard_normal((2, 1, 6))
    dot = lambda p, r: float((plain.rotate(q, 50.0, [p]) * plain.rotate(k, 50.0, [r])).sum())
    assert np.isclose(dot(9, 4), dot(105, 100)) and not np.isclose(dot(9, 4), dot(9, 5))
    # the second pair of four: angle p base^(-1/2), elements 2 and 3
    x = np.array([[0.0, 0.0, 1.0, 0.0]])
    a = 3 * 100.0 ** -0.5
    assert np.allclose(plain.rotate(x, 100.0, [3]), [[0.0, 0.0, math.cos(a), math.sin(a)]])
    assert np.allclose(plain.rotate(np.array([[0.0, 1.0]]), 7.0, [2]), [[-math.sin(2), math.cos(2)]])


def test_plain_memory_is_the_direct_sum_over_earlier_tokens():
    """o_t = sum_s w_ts (q_t . k_s) v_s / (max(|sum_s w_ts q_t . k_s|, e^-m) + 1e-6), w_ts = e^(F_t - F_s + i_s - m_t)."""
    g = rng(2)
    n, H, d, e = 30, 2, 3, 4
    q, k, v = g.standard_normal((n, H, d)), g.standard_normal((n, H, d)), g.standard_normal((n, H, e))
    i, f = 2.0 * g.standard_normal((n, H)), plain.log_sigmoid(2.0 * g.standard_normal((n, H)))
    got, (S, N, m_end) = plain.matrix_memory(q, k, v, i, f)
    F = np.cumsum(f, axis=0)
    for h in range(H):
        for t in range(n):
            m = max(F[t, h], max(F[t, h] - F[s, h] + i[s, h] for s in range(t + 1)))      # the maximum starts at 0
            w = np.exp(F[t, h] - F[:t + 1, h] + i[:t + 1, h] - m) * (k[:t + 1, h] @ q[t, h])
            assert np.allclose(got[t, h], w @ v[:t + 1, h] / (max(abs(w.sum()), math.exp(-m)) + 1e-6))
        assert np.isclose(m_end[h], m)
    # carried state: the second half from the first half's
    a, state = plain.matrix_memory(q[:13], k[:13], v[:13], i[:13], f[:13])
    b, _ = plain.matrix_memory(q[13:], k[13:], v[13:], i[13:], f[13:], state)
    assert np.allclose(np.concatenate([a, b]), got)


def test_plain_gates_and_activations():
    assert np.isclose(plain.soft_cap(1e3, 15.0), 15.0) and np.isclose(plain.soft_cap(0.01, 15.0), 0.01, atol=1e-6)
    assert np.isclose(plain.log_sigmoid(0.3), math.log(1 / (1 + math.exp(-0.3)))) and np.isclose(plain.log_sigmoid(-800.0), -800.0)
    assert np.isclose(plain.gelu_erf(np.array([1.0]))[0], 0.8413447460685429)
    # the gate is clamped from above only, the up value on both sides
    s = lambda z: 1 / (1 + math.exp(-1.702 * z))
    assert np.isclose(plain.clamped_glu(9.0, 9.0, 2.0), 2 * s(2) * 3) and np.isclose(plain.clamped_glu(-9.0, -9.0, 2.0), -9 * s(-9) * -1)


def test_plain_experts_weigh_their_inputs_and_choose_the_largest():
    g = rng(3)
    W, E, ff = 6, 4, 5
    w = {"x.router": g.standard_normal((E, W)), "x.shared.sg": g.standard_normal((1, W))}
    for name in ["x.e%d" % j for j in range(E)] + ["x.shared"]:
        w.update({name + ".gate": g.standard_normal((ff, W)), name + ".up": g.standard_normal((ff, W)), name + ".down": g.standard_normal((W, ff))})
    h = g.standard_normal((1, W))
    s = 1 / (1 + np.exp(-(h @ w["x.router"].T)))[0]
    a, b = sorted(range(E), key=lambda j: -s[j])[:2]
    mlp = {"router": {"experts": E, "top": 2}, "expert": {"limit": 0.5}, "shared": {"limit": 0.7}}
    want = sum(plain.expert(w, "x.e%d" % j, s[j] * h, 0.5) for j in (a, b)) + plain.sigmoid(h @ w["x.shared.sg"].T) * plain.expert(w, "x.shared", h, 0.7)
    assert np.allclose(plain.experts_ff(mlp, w, "x", h), want)
    assert not np.allclose(want, sum(s[j] * plain.expert(w, "x.e%d" % j, h, 0.5) for j in (a, b)) +
                           plain.sigmoid(h @ w["x.shared.sg"].T) * plain.expert(w, "x.shared", h, 0.7))
    assert plain.route(np.array([[0.2, 0.9, 0.9, 0.1]]), 3).tolist() == [[1, 2, 0]]


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_plain_model_is_causal(name):
    cfg = MODELS[name]
    t = gm.tensors(cfg, 3)
    a = gm.prompt(cfg, 20, 4)
    b = list(a)
    b[12] = (b[12] + 1) % cfg["vocab"]
    la, lb = plain.forward(cfg, t, a), plain.forward(cfg, t, b)
    assert np.allclose(la[:12], lb[:12]) and not np.allclose(la[12], lb[12]) and not np.allclose(la[13], lb[13])


def test_the_test_weights_exercise_every_branch():
    """Clamps on either side, gates that overtake the running maximum and gates that do not, scores far enough apart."""
    cfg = gm.MIXED
    t = gm.tensors(cfg, 21)
    seen = dict(clamped=0, free=0, overtakes=0, keeps=0)
    route, glu, mem = plain.route, plain.clamped_glu, plain.matrix_memory
    gaps = []

    def spy_route(scores, top):
        z = np.sort(np.log(scores / (1 - scores)), axis=1)[:, ::-1]
        if top < z.shape[1]:
            gaps.append((z[:, top - 1] - z[:, top]).min())
        return route(scores, top)

    def spy_glu(gate, u, limit):
        over = (gate > limit) | (np.abs(u) > limit)
        seen["clamped"] += int(over.sum())
        seen["free"] += int((~over).sum())
        return glu(gate, u, limit)

    def spy_memory(q, k, v, i, f, state=None):
        m = 0.0
        for t_ in range(len(q)):
            seen["overtakes"] += int((i[t_] > f[t_] + m).sum())
            seen["keeps"] += int((i[t_] <= f[t_] + m).sum())
            m = np.maximum(f[t_] + m, i[t_])
        return mem(q, k, v, i, f, state)
    plain.route, plain.clamped_glu, plain.matrix_memory = spy_route, spy_glu, spy_memory
    try:
        plain.forward(cfg, t, gm.prompt(cfg, 120, 31))
    finally:
        plain.route, plain.clamped_glu, plain.matrix_memory = route, glu, mem
    assert min(seen.values()) > 30 and min(gaps) > 0.1, (seen, min(gaps))


# ------------------------------------------------------------------ configuration, weights, registry

def test_configuration_round_trip_and_unknown_keys_fail_closed():
    for c in MODELS.values():
        assert gusolorn.config_json(gusolorn.decoder_config(c)) == c

    def broken(edit):
        c = copy.deepcopy(gm.MIXED)
        edit(c)
        return c
    mixer = lambda c, i: c["layers"][i]["mixer"]
    for edit, message in (
            (lambda c: c.update(rope={}), "rope"),
            (lambda c: mixer(c, 0).update(softcap=3), "softcap"),
            (lambda c: mixer(c, 0)["mask"].update(first=2), "first"),
            (lambda c: mixer(c, 0)["rot"].update(dims=10), "rotated"),
            (lambda c: mixer(c, 0).update(rot_dim=11), "rotated"),
            (lambda c: mixer(c, 1).pop("vdim"), "vdim"),
            (lambda c: mixer(c, 1).update(gate_cap=0), "gate_cap"),
            (lambda c: mixer(c, 1).update(conv=4), "conv"),
            (lambda c: mixer(c, 2).update(kv_from=1), "kv_from"),
            (lambda c: mixer(c, 2).update(kv_from=4), "kv_from"),
            (lambda c: mixer(c, 4).update(kv_from=2, kv_rank=72, rot_dim=12, rot=mixer(c, 0)["rot"]), "kv_from"),
            (lambda c: mixer(c, 2).update(kv_rank=71), "kv_rank"),
            (lambda c: mixer(c, 2)["rot"].update(base=901.0), "rot"),
            (lambda c: c["layers"][1].update(type="recurrent"), "recurrent"),
            (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "gated"),
            (lambda c: c["layers"][1]["mlp"]["router"].update(top=6), "top"),
            (lambda c: c["layers"][1]["mlp"]["router"].update(norm=True), "norm"),
            (lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"), "limit"),
            (lambda c: mixer(c, 0)["mask"].update(size=0), "size"),
            (lambda c: c.update(architecture="Other"), "Other")):
        with pytest.raises(ConfigError, match=message):
            gusolorn.decoder_config(broken(edit))


def test_model_folder_is_read_back_exactly(tmp_path):
    cfg, t = gm.MIXED, gm.tensors(gm.MIXED, 5)
    got_cfg, w = gusolorn.load_arrays(gm.write(tmp_path / "a", cfg, t))
    wide = lambda bits: sublayers.bf16_to_f32(bits).astype(np.float64)
    assert np.array_equal(wide(w["embed"]), t["embed"])
    assert np.allclose(w["layers"][0]["norm1"], 1 + t["l0.norm1"]) and np.allclose(w["final_norm"], 1 + t["final.norm"])
    assert np.array_equal(w["layers"][1]["mixer"]["head_norm"], t["l1.mix.norm"].astype(np.float32))
    assert np.array_equal(wide(w["layers"][1]["mlp"]["gate"][4]), t["l1.mlp.e4.gate"]) and w["layers"][3]["mlp"] == {}
    assert "dkv" not in w["layers"][2]["mixer"]
    # written by the package's own writer, read by both readers
    gusolorn.write_model(str(tmp_path / "b"), got_cfg, w)
    cfg2, w2 = gusolorn.load_arrays(str(tmp_path / "b"))
    assert cfg2 == got_cfg and all(np.array_equal(w[k], w2[k]) for k in ("embed", "head"))
    from safetensors.torch import load_file
    back = load_file(str(tmp_path / "b" / "model.safetensors"))
    assert sorted(back) == sorted(t) and np.array_equal(back["l2.mlp.e6.down"].double().numpy(), t["l2.mlp.e6.down"])
    for name in ("l1.mlp.e3.up", "l0.mix.dkv.norm", "l4.mlp.shared.sg"):
        bad = dict(t, **{name: t[name][:-1] if t[name].shape[0] > 1 else np.zeros((2, 3))})
        with pytest.raises(safetensors_file.SafetensorsError, match=name):
            gusolorn.load_arrays(gm.write(tmp_path / "c", cfg, bad))
        del bad[name]
        with pytest.raises(safetensors_file.SafetensorsError, match=name):
            gusolorn.load_arrays(gm.write(tmp_path / "d", cfg, bad))


def test_gate_and_up_rows_alternate_in_blocks():
    g = rng(4)
    gate, up = (g.integers(1, 60000, (3, 70, 10)).astype(np.uint16) for _ in range(2))
    w = sublayers.interleave_gate_up(gate, up, 64)
    assert w.shape == (3, 256, 64) and not w[:, :, 10:].any()
    for c in range(128):
        row = 64 * (c // 32) + c % 32
        if c < 70:
            assert np.array_equal(w[:, row, :10], gate[:, c]) and np.array_equal(w[:, row + 32, :10], up[:, c])
        else:
            assert not w[:, row].any() and not w[:, row + 32].any()


def test_output_projections_skip_the_padding_between_heads():
    o = np.arange(1, 4 * 15 + 1, dtype=np.uint16).reshape(4, 15)
    w = sublayers.pad_out(o, 4, 3, 5, 8, 64)
    assert w.shape == (4, 64)
    for h in range(3):
        assert np.array_equal(w[:, 8 * h:8 * h + 5], o[:, 5 * h:5 * h + 5])
    assert (w != 0).sum() == 60


def test_rotary_tables_are_computed_in_double():
    cos, sin = sublayers.rotary_tables(50.0, 6, 100000)
    a = 99999 * 50.0 ** (-2 / 6)
    assert abs(cos[99999, 1] - math.cos(a)) < 1e-6 and abs(sin[99999, 1] - math.sin(a)) < 1e-6 and cos.shape == (100000, 3)


def test_random_weights_fit_the_configuration(tmp_path):
    cfg = gusolorn.decoder_config(gm.MIXED)
    w = gusolorn.random_weights(cfg, seed=9)
    gusolorn.write_model(str(tmp_path), cfg, w)
    cfg2, w2 = gusolorn.load_arrays(str(tmp_path))
    assert cfg2 == cfg and np.array_equal(w["layers"][1]["mlp"]["down"], w2["layers"][1]["mlp"]["down"])
    assert np.array_equal(w["layers"][0]["mixer"]["latent_norm"], w2["layers"][0]["mixer"]["latent_norm"])


def test_registry_and_library():
    m = models.ARCHITECTURES["Gusolorn"]
    assert m.dtypes == ("bfloat16", "float32") and m.library == "dense"
    text = "\n".join(open(os.path.join(build.CSRC, s)).read() for s in build.DENSE_SOURCES)
    for name in ("dh_latent_rows", "dh_latent_prefill", "dh_latent_decode", "dh_mlstm_step", "dh_mlstm_prefill", "dh_head_norm_gate", "dh_experts_step",
                 "dh_experts_prefill", "dh_dense_gemv_heads", "dh_dense_gemv_scaled", "dh_dense_matmul_scaled"):
        assert name in capi.SIGNATURES and ("%s(" % name) in text, name


def test_recurrent_state_follows_the_positions():
    """Positions that do not follow one another are refused where a model carries state, and only there."""
    stand = SimpleNamespace(_state_pos=0, _recurrent_state=lambda: ["state"])
    step = lambda pos, n: decoder.DecoderBase._advance(stand, pos, n)
    step(0, 5)
    step(5, 1)
    with pytest.raises(ValueError, match="position 6, not at 5"):
        step(5, 1)
    step(0, 3)                       # a new sequence
    stand._recurrent_state = list
    step(50, 1)


def test_spec_sizes_without_a_device():
    L = capi.load()
    import ctypes
    spec = capi.MLSTM(3, 20, 44, 32, 64, 96, 192, 600, 604, 608, 2.0)
    assert L.dh_mlstm_state_bytes(ctypes.byref(spec)) == -(-(3 * 32 * 64 + 2 * 3 * 32 + 2 * 3) * 4 // 256) * 256
    assert L.dh_mlstm_step(ctypes.byref(spec), None, None, None, 0, None) != 0
    assert L.dh_experts_prefill(None, None, capi.BF16, None, 0, None, 1) != 0
