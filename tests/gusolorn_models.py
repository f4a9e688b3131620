"""Small Gusolorn models for the tests: configurations, seeded weights (already representable in bf16), model folders.

The weights are made so that faults show: attention is peaked, the memories' input gates now and then overtake their running maximum,
the experts' clamps bite, and the experts are chosen by columns of the residual that only the embedding writes, far enough apart that
rounding cannot change a choice."""
import numpy as np

from tests.zepavik_models import bf16, prompt, row_errors, write  # noqa: F401  (re-exported)

LEVELS = 8          # columns behind which experts are chosen


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, shared=None):
    m = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def latent(heads, dim, rot, vdim, rank, window=None, scale=None, base=10000.0, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": (dim + rot) ** -0.5 if scale is None else scale,
         "rot": {"base": base, "dims": rot}}
    if window is not None:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def memory(heads, dim, vdim, cap, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Gusolorn", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


# sizes that agree in nothing; lent latent rows under another window, head count and head size; layers without feed-forward
MIXED = config(136, 211, [latent(5, 24, 12, 40, 72, window=33, base=900.0, mlp=dense(88)),
                          memory(3, 20, 44, 7.5, mlp=moe(5, 2, 36, 0.8, shared=(52, 1.3))),
                          latent(3, 40, 12, 20, 72, window=65, scale=0.21, base=900.0, kv_from=0, mlp=moe(7, 3, 24, 1.1)),
                          memory(2, 33, 17, 2.0),
                          latent(4, 16, 32, 8, 24, window=9, mlp=moe(3, 1, 40, 0.5, shared=(20, 0.9))),
                          memory(1, 64, 96, 15.0, mlp=dense(300))], eps=3e-4)
# more heads than a matrix-core tile holds, latents beyond its reach, wide heads, no window; a memory of several column groups
WIDE = config(96, 130, [latent(17, 140, 40, 136, 576, mlp=dense(40)), memory(2, 100, 260, 4.0, mlp=moe(8, 5, 70, 1.0, shared=(130, 2.0))),
                        latent(18, 8, 40, 264, 576, window=70, kv_from=0), latent(33, 64, 64, 64, 300, window=40, mlp=moe(2, 1, 200, 3.0))])
# sizes that are multiples of nothing, ones, every expert chosen
ODD = config(90, 131, [memory(1, 1, 1, 1.0, mlp=moe(1, 1, 1, 1.0, shared=(1, 0.3))), latent(1, 7, 2, 9, 13, window=5, base=3.0, mlp=dense(1)),
                       memory(7, 3, 5, 30.0, mlp=moe(4, 4, 33, 0.7)), latent(7, 3, 6, 5, 1, window=1, scale=1.7),
                       latent(2, 33, 6, 65, 1, window=2, scale=0.4, kv_from=3)], eps=0.02)
# even sizes for generation
EVEN = config(128, 301, [memory(2, 32, 64, 10.0, mlp=moe(6, 2, 64, 1.5, shared=(64, 1.0))), latent(4, 32, 16, 32, 64, window=50, mlp=dense(192)),
                         latent(4, 32, 16, 32, 64, window=20, kv_from=1, mlp=moe(6, 2, 64, 1.5, shared=(64, 1.0)))])


def tensors(cfg, seed, gain=2.0):
    g = np.random.Generator(np.random.PCG64(seed))
    n = lambda *s, std=1.0, mean=0.0: bf16(mean + std * g.standard_normal(s))
    W, V = cfg["width"], cfg["vocab"]

    def out(rows, k, std=1.0):
        w = n(rows, k, std=std * k ** -0.5)
        w[:LEVELS] = 0.0                            # the columns the experts are chosen by stay the embedding's
        return w
    t = {"embed": n(V, W), "final.norm": n(W, std=0.3), "head": n(V, W, std=W ** -0.5)}
    t["embed"][:, :LEVELS] = bf16(1.5 * (np.argsort(g.random((V, LEVELS)), axis=1) - (LEVELS - 1) / 2))
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        H, d, e = m["heads"], m["dim"], m["vdim"]
        t.update({p + "norm1": n(W, std=0.3), p + "ls1": n(W, std=0.3, mean=0.8)})
        if l["type"] == "mlstm":
            for name, rows, std in (("q", H * d, 1.0), ("k", H * d, 1.0), ("v", H * e, 1.0), ("g", H * e, 1.0), ("i", H, 2.0), ("f", H, 2.0)):
                t[p + "mix." + name] = n(rows, W, std=std * W ** -0.5)
            t.update({p + "mix.i.b": n(H, std=1.0), p + "mix.f.b": n(H, std=1.0, mean=2.5), p + "mix.norm": n(H * e, std=0.3, mean=1.0)})
        else:
            r, rot = m["kv_rank"], m["rot_dim"]
            t[p + "mix.q"] = n(H * (d + rot), W, std=gain * W ** -0.5)
            t[p + "mix.uk"], t[p + "mix.uv"] = n(H * d, r, std=gain * r ** -0.5), n(H * e, r, std=r ** -0.5)
            if m.get("kv_from") is None:
                t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = n(r + rot, W, std=W ** -0.5), n(r, std=0.3, mean=1.0)
                t[p + "mix.dkv"][r:] = bf16(gain * t[p + "mix.dkv"][r:])
        t[p + "mix.o"] = out(W, H * e)
        mlp = l["mlp"]
        if mlp is None:
            continue
        t.update({p + "norm2": n(W, std=0.3), p + "ls2": n(W, std=0.3, mean=0.8)})
        if mlp["kind"] == "dense":
            t[p + "mlp.up"], t[p + "mlp.down"] = n(mlp["ff"], W, std=W ** -0.5), out(W, mlp["ff"])
            continue
        E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        t[p + "norm2"][:LEVELS] = 0.0
        t[p + "mlp.router"] = n(E, W, std=0.005)
        t[p + "mlp.router"][np.arange(E), np.arange(E)] = 0.703125
        parts = [("e%d" % k, ff) for k in range(E)]
        if mlp.get("shared"):
            parts.append(("shared", mlp["shared"]["ff"]))
            t[p + "mlp.shared.sg"] = n(1, W, std=W ** -0.5)
        for name, f in parts:
            q = p + "mlp." + name
            t.update({q + ".gate": n(f, W, std=1.5 * W ** -0.5), q + ".up": n(f, W, std=1.5 * W ** -0.5), q + ".down": out(W, f)})
    return t
