"""Gusolorn through the JavaScript host: the same kernels, so the tokens of the Python host and of the plain restatement."""
import json
import os
import shutil
import subprocess

import numpy as np
import pytest

from doppler_amd import models
from oracle import plain_gusolorn as plain
from tests import gusolorn_models as gm

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
NODE = shutil.which("node")


def run_node(code):
    r = subprocess.run([NODE, "--input-type=module", "-e", code], cwd=ROOT, capture_output=True, text=True, timeout=60)
    assert r.returncode == 0, r.stderr[-2000:]
    return r.stdout.strip().splitlines()[-1]


def test_js_loader_reads_the_folder_and_refuses_unknown_keys(tmp_path):
    if NODE is None:
        pytest.skip("node not installed")
    cfg, t = gm.MIXED, gm.tensors(gm.MIXED, 5)
    d = gm.write(tmp_path / "m", cfg, t)
    out = json.loads(run_node("""
      import { loadGusolorn } from './doppler_amd/js/loader/gusolorn-loader.js';
      const { config, weights } = loadGusolorn(%r, 100);
      const sum = (a) => a.reduce((x, y) => x + y, 0);
      console.log(JSON.stringify({ maxSeq: config.maxSeq, layers: config.layers, down: sum(weights.layers[1].mlp.down[3]),
        norm: Array.from(weights.layers[0].norm1), bias: Array.from(weights.layers[3].mixer.fBias) }));""" % d))
    assert out["maxSeq"] == 100 and out["layers"][3]["mlp"] is None and out["layers"][2]["mixer"]["kvFrom"] == 0
    assert out["layers"][1] == {"sequential": True, "mixer": {"type": "mlstm", "heads": 3, "dim": 20, "vdim": 44, "gateCap": 7.5},
                                "mlp": {"type": "experts", "experts": 5, "top": 2, "ff": 36, "limit": 0.8, "shared": {"ff": 52, "limit": 1.3}}}
    from doppler_amd import dense_decoder
    assert out["down"] == int(dense_decoder.f32_to_bf16(t["l1.mlp.e3.down"]).astype(np.int64).sum())
    assert np.allclose(out["norm"], 1 + t["l0.norm1"]) and np.allclose(out["bias"], t["l3.mix.f.b"])
    for edit, message in ((lambda c: c["layers"][0]["mixer"].update(softcap=1), "softcap"), (lambda c: c["layers"][2]["mixer"].update(kv_rank=71), "kv_from"),
                          (lambda c: c["layers"][4]["mixer"].update(kv_from=1), "kv_from"), (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "top")):
        bad = json.loads(json.dumps(cfg))
        edit(bad)
        e = gm.write(tmp_path / message, bad, t)
        assert message in run_node("""
          import { loadGusolorn } from './doppler_amd/js/loader/gusolorn-loader.js';
          try { loadGusolorn(%r); console.log('accepted'); } catch (e) { console.log(e.message); }""" % e)


def test_js_half_precision_bits_are_numpys():
    if NODE is None:
        pytest.skip("node not installed")
    got = json.loads(run_node("""
      import { bf16ToF16 } from './doppler_amd/js/pipeline/sublayers.js';
      console.log(JSON.stringify(Array.from(bf16ToF16(Uint16Array.from({ length: 65536 }, (_, i) => i)))));"""))
    wide = (np.arange(65536, dtype=np.uint32) << 16).view(np.float32)
    number = ~np.isnan(wide)
    with np.errstate(over="ignore"):
        want = wide.astype(np.float16).view(np.uint16)
    assert np.array_equal(np.array(got)[number], want[number])


@pytest.mark.gpu
def test_js_host_generates_what_the_python_host_does(tmp_path):
    if NODE is None:
        pytest.skip("node not installed")
    jobs, want = [], {}
    for name, cfg, seed in (("mixed", gm.MIXED, 21), ("even", gm.EVEN, 23), ("wide", gm.WIDE, 22)):
        t = gm.tensors(cfg, seed)
        d = gm.write(tmp_path / name, cfg, t)
        prompt = gm.prompt(cfg, 40, seed)
        for dtype in ("float32", "bfloat16"):
            dec = models.load(d, 120, dtype)
            tokens = dec.generate(prompt, 40)
            if dtype == "float32":
                assert tokens == plain.greedy(cfg, t, prompt, 40)
            base = dict(dir=d, maxSeq=120, dtype=dtype, prompt=prompt, count=40)
            for mode in ("generate", "greedy", "graph"):
                key = "%s-%s-%s" % (name, dtype, mode)
                jobs.append(dict(base, name=key, mode=mode))
                want[key] = tokens
            sampling = dict(temperature=0.8, topK=9, seed=3)
            key = "%s-%s-sampled" % (name, dtype)
            jobs.append(dict(base, name=key, mode="generate", sampling=sampling))
            want[key] = dec.generate(prompt, 40, sampling=sampling)
        key = name + "-portions"
        jobs.append(dict(dir=d, maxSeq=120, dtype="float32", prompt=prompt, count=40, name=key, mode="portions", sizes=[3, 1, 2, 20, 1, 13], chunk=8))
        want[key] = plain.greedy(cfg, t, prompt, 40)
        key = name + "-order"
        jobs.append(dict(dir=d, maxSeq=120, dtype="float32", prompt=prompt, count=1, name=key, mode="order"))
        stands = "the sequence's recurrent state stands at position 40, not at %d"
        want[key] = [stands % 42, stands % 39, "ran"]
        big = dict(t)
        big["l1.mix.o"] = gm.bf16(t["l1.mix.o"] * 1e8)
        key = name + "-guard"
        jobs.append(dict(dir=gm.write(tmp_path / (name + "-big"), cfg, big), maxSeq=50, dtype="bfloat16", prompt=prompt, count=2, name=key, mode="guard",
                         config=dict(finitenessGuard=True)))
        want[key] = ["FinitenessError: F16 bounds exceeded during generation (layer 1, step 40)"]
    path = str(tmp_path / "jobs.json")
    json.dump(jobs, open(path, "w"))
    r = subprocess.run([NODE, os.path.join(ROOT, "tests", "js", "run_models.mjs"), path], cwd=ROOT, capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-3000:]
    got = json.loads(r.stdout.strip().splitlines()[-1])
    for key in want:
        assert got[key] == want[key], key
