"""Zepavik through the JavaScript host: the same kernels, so the tokens of the Python host and of the plain restatement."""
import json
import os
import shutil
import subprocess

import numpy as np
import pytest

from doppler_amd import models
from oracle import plain_zepavik as plain
from tests import zepavik_models as zm

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
NODE = shutil.which("node")


def run_node(code):
    r = subprocess.run([NODE, "--input-type=module", "-e", code], cwd=ROOT, capture_output=True, text=True, timeout=60)
    assert r.returncode == 0, r.stderr[-2000:]
    return r.stdout.strip().splitlines()[-1]


def test_js_loader_reads_the_folder_and_refuses_unknown_keys(tmp_path):
    if NODE is None:
        pytest.skip("node not installed")
    cfg, t = zm.MIXED, zm.tensors(zm.MIXED, 5)
    d = zm.write(tmp_path / "m", cfg, t)
    out = json.loads(run_node("""
      import { loadZepavik } from './doppler_amd/js/loader/zepavik-loader.js';
      const { config, weights } = loadZepavik(%r, 100);
      const sum = (a) => a.reduce((x, y) => x + y, 0);
      console.log(JSON.stringify({ maxSeq: config.maxSeq, hidden: config.hidden, mlp: config.layers.map((l) => l.mlp), window: config.layers[1].mixer.window,
        bits: sum(weights.layers[2].q), bias: Array.from(weights.layers[0].kBias), r1: Array.from(weights.layers[3].biasR1) }));""" % d))
    assert out["maxSeq"] == 100 and out["hidden"] == 136 and out["window"] == 65
    assert out["mlp"] == [{"ff": 88, "activation": "relu2"}, None, {"ff": 300, "activation": "relu2"}, {"ff": 56, "activation": "relu2"}]
    from doppler_amd import dense_decoder
    assert out["bits"] == int(dense_decoder.f32_to_bf16(t["l2.mix.q"]).astype(np.int64).sum())
    assert np.allclose(out["bias"], t["l0.mix.k.b"]) and np.allclose(out["r1"], t["l3.mix.r1"])
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["mixer"]["softcap"] = 1
    e = zm.write(tmp_path / "b", bad, t)
    assert "softcap" in run_node("""
      import { loadZepavik } from './doppler_amd/js/loader/zepavik-loader.js';
      try { loadZepavik(%r); console.log('accepted'); } catch (e) { console.log(e.message); }""" % e)


@pytest.mark.gpu
def test_js_host_generates_what_the_python_host_does(tmp_path):
    if NODE is None:
        pytest.skip("node not installed")
    jobs, want = [], {}
    for name, cfg, seed in (("mixed", zm.MIXED, 21), ("even", zm.EVEN, 23)):
        t = zm.tensors(cfg, seed)
        d = zm.write(tmp_path / name, cfg, t)
        prompt = zm.prompt(cfg, 40, seed)
        for dtype in ("float32", "bfloat16"):
            dec = models.load(d, 120, dtype)
            tokens = dec.generate(prompt, 40)
            if dtype == "float32":
                assert tokens == plain.greedy(cfg, t, prompt, 40)
            base = dict(dir=d, maxSeq=120, dtype=dtype, prompt=prompt, count=40)
            for mode, extra in (("generate", {}), ("greedy", {}), ("graph", {})):
                key = "%s-%s-%s" % (name, dtype, mode)
                jobs.append(dict(base, name=key, mode=mode, **extra))
                want[key] = tokens
            sampling = dict(temperature=0.8, topK=9, seed=3)
            key = "%s-%s-sampled" % (name, dtype)
            jobs.append(dict(base, name=key, mode="generate", sampling=sampling))
            want[key] = dec.generate(prompt, 40, sampling=sampling)
        key = name + "-portions"
        jobs.append(dict(dir=d, maxSeq=120, dtype="float32", prompt=prompt, count=40, name=key, mode="portions", sizes=[3, 1, 2, 20, 1, 13], chunk=8))
        want[key] = plain.greedy(cfg, t, prompt, 40)
        big = dict(t)
        big["l1.mix.o"] = zm.bf16(t["l1.mix.o"] * 1e8)
        key = name + "-guard"
        jobs.append(dict(dir=zm.write(tmp_path / (name + "-big"), cfg, big), maxSeq=50, dtype="bfloat16", prompt=prompt, count=2, name=key, mode="guard",
                         config=dict(finitenessGuard=True)))
        want[key] = ["FinitenessError: F16 bounds exceeded during generation (layer 1, step 40)"]
    path = str(tmp_path / "jobs.json")
    json.dump(jobs, open(path, "w"))
    r = subprocess.run([NODE, os.path.join(ROOT, "tests", "js", "run_models.mjs"), path], cwd=ROOT, capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-3000:]
    got = json.loads(r.stdout.strip().splitlines()[-1])
    for key in want:
        assert got[key] == want[key], key
