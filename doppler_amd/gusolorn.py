"""Gusolorn models (config.json + model.safetensors) -> the dense decoder.

Sequential layers with layer scales and norm weights stored around zero; mixers are a matrix memory (mlstm) or windowed attention over a
low-rank latent, whose rows a later layer may borrow; feed-forwards are dense with the exact gelu, or sigmoid-routed experts with clamped
gates and a gated shared expert, or none.  The configuration gives every size layer by layer; a key this reader does not know fails
closed with its name.
"""
import json
import os

import numpy as np

from .config_fields import ConfigError, count, number, take
from .dense_decoder import DenseDecoder, bf16_to_f32, f32_to_bf16
from .safetensors_file import SafetensorsFile, write_safetensors

ARCHITECTURE = "Gusolorn"
DEFAULT_POSITIONS = 4096


def _latent(m, at, i, entries):
    take(m, at, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot"), ("mask", "kv_from"))
    rot = take(m["rot"], at + ".rot", ("base", "dims"))
    out = {k: count(m, k, at) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank")}
    if out["rot_dim"] % 2 or rot["dims"] != out["rot_dim"]:
        raise ConfigError("%s: the rotated part of %d elements must be even and rotated whole (rot.dims %r)" % (at, out["rot_dim"], rot["dims"]))
    mask = m.get("mask")
    window = count(take(mask, at + ".mask", ("size",)), "size", at + ".mask") if mask is not None else 0
    src = m.get("kv_from")
    if src is not None:
        ok = isinstance(src, int) and not isinstance(src, bool) and 0 <= src < i and entries[src]["type"] == "latent_attention" and \
            entries[src]["mixer"].get("kv_from") is None
        if not ok:
            raise ConfigError("%s.kv_from %r is not an earlier layer with latent rows of its own" % (at, src))
        other = entries[src]["mixer"]
        for k in ("kv_rank", "rot_dim", "rot"):
            if other[k] != m[k]:
                raise ConfigError("%s.kv_from: %s is %r here and %r in layer %d" % (at, k, m[k], other[k], src))
    return dict(out, type="latent_attention", window=window, scale=number(m, "scale", at), rot_base=number(rot, "base", at + ".rot", True), kv_from=src)


def _mlstm(m, at, i, entries):
    take(m, at, ("heads", "dim", "vdim", "gate_cap"))
    return dict({k: count(m, k, at) for k in ("heads", "dim", "vdim")}, type="mlstm", gate_cap=number(m, "gate_cap", at, True))


def _feed_forward(mlp, at):
    if mlp is None:
        return None
    kind = mlp.get("kind") if isinstance(mlp, dict) else None
    if kind == "dense":
        return dict(type="dense", ff=count(take(mlp, at, ("kind", "ff")), "ff", at), activation="gelu_erf")
    if kind != "moe":
        raise ConfigError("%s.kind %r is not a feed-forward of this design" % (at, kind))
    take(mlp, at, ("kind", "router", "expert"), ("shared",))
    router = take(mlp["router"], at + ".router", ("experts", "top"))
    width = lambda e, w: dict(ff=count(take(e, w, ("ff", "limit")), "ff", w), limit=number(e, "limit", w))
    experts, top = count(router, "experts", at + ".router"), count(router, "top", at + ".router")
    if top > experts:
        raise ConfigError("%s.router.top %d exceeds %d experts" % (at, top, experts))
    shared = mlp.get("shared")
    return dict(width(mlp["expert"], at + ".expert"), type="experts", experts=experts, top=top,
                shared=None if shared is None else width(shared, at + ".shared"))


MIXERS = {"latent_attention": _latent, "mlstm": _mlstm}


def decoder_config(config):
    """cfg dict of DenseDecoder from a parsed config.json."""
    c = take(config, "config", ("architecture", "layers", "norm", "vocab", "width"))
    if c["architecture"] != ARCHITECTURE:
        raise ConfigError("architecture is %r, not %s" % (c["architecture"], ARCHITECTURE))
    layers = []
    for i, entry in enumerate(c["layers"]):
        where = "layers[%d]" % i
        take(entry, where, ("type", "mixer"), ("mlp",))
        if entry["type"] not in MIXERS:
            raise ConfigError("%s.type %r is not a mixer of this design" % (where, entry["type"]))
        layers.append(dict(sequential=True, mixer=MIXERS[entry["type"]](entry["mixer"], where + ".mixer", i, c["layers"]),
                           mlp=_feed_forward(entry.get("mlp"), where + ".mlp")))
    return dict(hidden=count(c, "width", "config"), vocab=count(c, "vocab", "config"),
                eps=number(take(c["norm"], "norm", ("eps",)), "eps", "norm"), logit_scale=1.0, max_positions=0, bigram=None, layers=layers)


def layer_tensors(i, spec, W):
    """Part of a layer ("", "mixer", "mlp") -> key -> (tensor name, shape, how it is kept) of layer i: "bits" as they are, "f32"
    widened, "around 0" widened with 1 added."""
    m, mlp, p = spec["mixer"], spec["mlp"], "l%d." % i
    mix = p + "mix."
    H, d, e = m["heads"], m["dim"], m["vdim"]
    own = {"norm1": (p + "norm1", [W], "around 0"), "ls1": (p + "ls1", [W], "f32")}
    if mlp:
        own.update(norm2=(p + "norm2", [W], "around 0"), ls2=(p + "ls2", [W], "f32"))
    if m["type"] == "mlstm":
        t = {n: (mix + n, [H * size, W], "bits") for n, size in (("q", d), ("k", d), ("v", e), ("g", e), ("i", 1), ("f", 1))}
        t.update(o=(mix + "o", [W, H * e], "bits"), head_norm=(mix + "norm", [H * e], "f32"), i_bias=(mix + "i.b", [H], "f32"),
                 f_bias=(mix + "f.b", [H], "f32"))
    else:
        rank, rot = m["kv_rank"], m["rot_dim"]
        t = {"q": (mix + "q", [H * (d + rot), W], "bits"), "uk": (mix + "uk", [H * d, rank], "bits"), "uv": (mix + "uv", [H * e, rank], "bits"),
             "o": (mix + "o", [W, H * e], "bits")}
        if m["kv_from"] is None:
            t.update(dkv=(mix + "dkv", [rank + rot, W], "bits"), latent_norm=(mix + "dkv.norm", [rank], "f32"))
    ff = {}
    if mlp and mlp["type"] == "dense":
        ff = {"up": (p + "mlp.up", [mlp["ff"], W], "bits"), "down": (p + "mlp.down", [W, mlp["ff"]], "bits")}
    elif mlp:
        ff = {"router": (p + "mlp.router", [mlp["experts"], W], "bits")}
        for n, shape in (("gate", [mlp["ff"], W]), ("up", [mlp["ff"], W]), ("down", [W, mlp["ff"]])):
            ff[n] = [("%smlp.e%d.%s" % (p, k, n), shape, "bits") for k in range(mlp["experts"])]
        if mlp["shared"]:
            s = mlp["shared"]["ff"]
            for n, shape in (("gate", [s, W]), ("up", [s, W]), ("down", [W, s]), ("sg", [1, W])):
                ff["shared_" + n] = (p + "mlp.shared." + n, shape, "bits")
    return {"": own, "mixer": t, "mlp": ff}


def model_tensors(cfg):
    W, V = cfg["hidden"], cfg["vocab"]
    return {"embed": ("embed", [V, W], "bits"), "final_norm": ("final.norm", [W], "around 0"), "head": ("head", [V, W], "bits")}


def load_arrays(directory):
    """(cfg, weights) in the form DenseDecoder takes."""
    with open(os.path.join(directory, "config.json")) as f:
        cfg = decoder_config(json.load(f))
    st = SafetensorsFile(os.path.join(directory, "model.safetensors"))

    def one(entry):
        if isinstance(entry, list):
            return np.stack([one(e) for e in entry])
        name, shape, kept = entry
        a = st.tensor(name, "BF16", shape)
        return a if kept == "bits" else bf16_to_f32(a) + np.float32(1.0 if kept == "around 0" else 0.0)

    read = lambda entries: {key: one(e) for key, e in entries.items()}
    weights = dict(read(model_tensors(cfg)), layers=[])
    for i, spec in enumerate(cfg["layers"]):
        parts = layer_tensors(i, spec, cfg["hidden"])
        weights["layers"].append(dict(read(parts[""]), mixer=read(parts["mixer"]), mlp=read(parts["mlp"])))
    return cfg, weights


def load_decoder(directory, max_seq=None, dtype="bfloat16", **decoder_kwargs):
    """A ready DenseDecoder; positions are bounded by the cache alone."""
    cfg, weights = load_arrays(directory)
    return DenseDecoder(cfg, weights, max_seq or DEFAULT_POSITIONS, compute={"bfloat16": "bf16", "float32": "f32"}[dtype], **decoder_kwargs)


def config_json(cfg):
    """The config.json of a DenseDecoder cfg of this design (inverse of decoder_config)."""
    layers = []
    for s in cfg["layers"]:
        m, mlp = s["mixer"], s["mlp"]
        if m["type"] == "mlstm":
            mixer = {k: m[k] for k in ("heads", "dim", "vdim", "gate_cap")}
        else:
            mixer = {k: m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale")}
            mixer["rot"] = {"base": m["rot_base"], "dims": m["rot_dim"]}
            if m["window"]:
                mixer["mask"] = {"size": m["window"]}
            if m["kv_from"] is not None:
                mixer["kv_from"] = m["kv_from"]
        if mlp is None:
            ff = None
        elif mlp["type"] == "dense":
            ff = {"kind": "dense", "ff": mlp["ff"]}
        else:
            ff = {"kind": "moe", "router": {"experts": mlp["experts"], "top": mlp["top"]}, "expert": {"ff": mlp["ff"], "limit": mlp["limit"]}}
            if mlp["shared"]:
                ff["shared"] = dict(mlp["shared"])
        layers.append({"type": m["type"], "mixer": mixer, "mlp": ff})
    return {"architecture": ARCHITECTURE, "layers": layers, "norm": {"eps": cfg["eps"]}, "vocab": cfg["vocab"], "width": cfg["hidden"]}


def write_model(directory, cfg, weights):
    """Writes a model folder from a DenseDecoder cfg and weights."""
    os.makedirs(directory, exist_ok=True)
    with open(os.path.join(directory, "config.json"), "w") as f:
        json.dump(config_json(cfg), f, indent=1)
    tensors = {}

    def put(entry, a):
        if isinstance(entry, list):
            for e, part in zip(entry, a):
                put(e, part)
            return
        name, shape, kept = entry
        bits = a if kept == "bits" else f32_to_bf16(np.asarray(a, np.float32) - np.float32(1.0 if kept == "around 0" else 0.0))
        tensors[name] = ("BF16", np.asarray(bits).reshape(shape))

    for key, e in model_tensors(cfg).items():
        put(e, weights[key])
    for i, (spec, w) in enumerate(zip(cfg["layers"], weights["layers"])):
        parts = layer_tensors(i, spec, cfg["hidden"])
        for part, values in (("", w), ("mixer", w["mixer"]), ("mlp", w["mlp"])):
            for key, e in parts[part].items():
                put(e, values[key])
    write_safetensors(os.path.join(directory, "model.safetensors"), tensors)


def random_weights(cfg, seed=0):
    """Random-init weights: linears N(0, 1/in), norms N(1, 0.02), layer scales N(1, 0.1), the table N(0, 1), forget gates that mostly keep."""
    g = np.random.Generator(np.random.PCG64(seed))

    def one(key, entry):
        if isinstance(entry, list):
            return np.stack([one(key, e) for e in entry])
        _, shape, kept = entry
        if kept == "bits" and int(np.prod(shape)) >= 1 << 20:
            # large matrices from random bits: sign and mantissa of +-[1, 2) times the power of two that gives about the same spread
            r = g.integers(0, 256, shape, dtype=np.uint8).astype(np.uint16)
            e = 127 if key == "embed" else 127 + int(np.round(np.log2(shape[-1] ** -0.5 / 1.53)))
            return ((r & 0x80) << 8) | np.uint16(e << 7) | (r & 0x7F)
        z = g.standard_normal(shape, dtype=np.float32)
        if kept == "bits":
            return f32_to_bf16(z if key == "embed" else z * np.float32(shape[-1] ** -0.5))
        mean, std = {"i_bias": (-2.0, 0.5), "f_bias": (4.0, 0.5), "ls1": (1.0, 0.1), "ls2": (1.0, 0.1)}.get(key, (1.0, 0.02))
        return bf16_to_f32(f32_to_bf16(z * np.float32(std) + np.float32(mean)))

    make = lambda entries: {key: one(key, e) for key, e in entries.items()}
    weights = dict(make(model_tensors(cfg)), layers=[])
    for i, spec in enumerate(cfg["layers"]):
        parts = layer_tensors(i, spec, cfg["hidden"])
        weights["layers"].append(dict(make(parts[""]), mixer=make(parts["mixer"]), mlp=make(parts["mlp"])))
    return weights
