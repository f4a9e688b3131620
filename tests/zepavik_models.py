"""Small Zepavik models for the tests: a configuration, seeded weights (already representable in bf16), a model folder.

The weights are made so that attention is peaked (queries and keys scaled up): with flat scores a missing window edge or
a wrong key among many would hardly move the logits."""
import json
import os

import numpy as np
import torch
from safetensors.torch import save_file


def bf16(a):
    """float64 values a bf16 tensor of `a` holds."""
    return torch.from_numpy(np.ascontiguousarray(a, np.float32)).to(torch.bfloat16).to(torch.float64).numpy()


def layer(heads, kv_heads, dim, vdim, window, scale=None, ff=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
                      "mask": {"size": window}},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, max_positions=400, buckets=61, mul_prev=31, mul_cur=13, eps=1e-5, logit_scale=0.7):
    return {"architecture": "Zepavik", "width": width, "vocab": vocab, "max_positions": max_positions,
            "norm": {"eps": eps}, "logit_scale": logit_scale,
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}, "layers": layers}


# sizes that agree in nothing, heads that need padding, a layer without feed-forward, windows on either side of a key tile
MIXED = config(136, 211, [layer(6, 2, 24, 40, 9, ff=88), layer(4, 4, 64, 32, 65, scale=0.2), layer(5, 1, 20, 12, 33, ff=300),
                          layer(2, 1, 72, 104, 64, ff=56)], eps=3e-4, logit_scale=1.3)
# many query heads per key/value head, heads wider than the matrix-core kernel's
WIDE_HEADS = config(96, 130, [layer(12, 1, 16, 8, 40, ff=64), layer(3, 1, 136, 24, 70, ff=40), layer(2, 2, 40, 264, 21, ff=24)])
# sizes that are multiples of nothing
ODD = config(90, 131, [layer(3, 1, 7, 9, 5, ff=33), layer(2, 2, 33, 65, 17, scale=0.11, ff=1), layer(7, 7, 3, 5, 66)], buckets=1, eps=0.02)
# even sizes, one kind of layer
EVEN = config(192, 301, [layer(4, 2, 64, 64, 50, ff=256)] * 3)


def tensors(cfg, seed, gain=2.5):
    g = np.random.Generator(np.random.PCG64(seed))
    n = lambda *s, std=1.0, mean=0.0: bf16(mean + std * g.standard_normal(s))
    W, V = cfg["width"], cfg["vocab"]
    t = {"embed": n(V, W), "bigram": n(cfg["embedding"]["bigram"]["buckets"] + 1, W), "pos": n(cfg["max_positions"], W, std=0.5),
         "final.norm": n(W, std=0.3, mean=1.0), "head": n(V, W, std=W ** -0.5)}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        t[p + "norm1"] = n(W, std=0.3, mean=1.0)
        for name, rows, k in (("q", H * d, gain), ("k", G * d, gain), ("v", G * e, 1.0)):
            t[p + "mix." + name] = n(rows, W, std=k * W ** -0.5)
            t[p + "mix." + name + ".b"] = n(rows, std=0.4)
        t[p + "mix.r1"] = bf16(g.uniform(0.02, 1.5, H))
        t[p + "mix.r2"] = bf16(g.uniform(0.05, 0.9, H))
        t[p + "mix.g"] = n(H, W, std=1.5 * W ** -0.5)
        t[p + "mix.o"] = n(W, H * e, std=(H * e) ** -0.5)
        if l["mlp"]:
            ff = l["mlp"]["ff"]
            t[p + "mlp.up"] = n(ff, W, std=W ** -0.5)
            t[p + "mlp.down"] = n(W, ff, std=ff ** -0.5)
    return t


def write(directory, cfg, t):
    os.makedirs(str(directory), exist_ok=True)
    with open(os.path.join(str(directory), "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: torch.from_numpy(np.ascontiguousarray(v)).to(torch.bfloat16) for k, v in t.items()},
              os.path.join(str(directory), "model.safetensors"))
    return str(directory)


def prompt(cfg, n, seed):
    return [int(v) for v in np.random.Generator(np.random.PCG64(seed)).integers(0, cfg["vocab"], n)]


def row_errors(got, want):
    """Per row: root mean square of the difference (mean taken off) over the root mean square of the wanted row."""
    d = np.asarray(got, np.float64) - want
    d = d - d.mean(axis=-1, keepdims=True)
    w = want - want.mean(axis=-1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=-1) / (w ** 2).mean(axis=-1))
