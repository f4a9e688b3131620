"""Zepavik models (config.json + model.safetensors) -> the dense decoder.

Token, bigram and position tables are summed into the residual stream; every layer runs windowed attention (logarithmic
distance bias, normed values, one gate per head) and an optional squared-relu feed-forward side by side; the head is
untied and scaled.  The configuration gives every size layer by layer; a key this reader does not know fails
closed with its name.
"""
import json
import os

from .config_fields import ConfigError, count as _count, take as _take
from .dense_decoder import DenseDecoder, bf16_to_f32, f32_to_bf16
from .safetensors_file import SafetensorsFile, write_safetensors

ARCHITECTURE = "Zepavik"


def decoder_config(config):
    """cfg dict of DenseDecoder from a parsed config.json."""
    c = _take(config, "config", ("architecture", "embedding", "layers", "logit_scale", "max_positions", "norm", "vocab", "width"))
    if c["architecture"] != ARCHITECTURE:
        raise ConfigError("architecture is %r, not %s" % (c["architecture"], ARCHITECTURE))
    bigram = _take(_take(c["embedding"], "embedding", ("bigram",))["bigram"], "embedding.bigram", ("buckets", "mul_prev", "mul_cur"))
    layers = []
    for i, entry in enumerate(c["layers"]):
        where = "layers[%d]" % i
        _take(entry, where, ("type", "mixer"), ("mlp",))
        if entry["type"] != "attention":
            raise ConfigError("%s.type %r is not a mixer of this design" % (where, entry["type"]))
        m = _take(entry["mixer"], where + ".mixer", ("heads", "kv_heads", "dim", "vdim", "scale", "mask"))
        at = where + ".mixer"
        mask = _take(m["mask"], at + ".mask", ("size",))
        heads, kv_heads = _count(m, "heads", at), _count(m, "kv_heads", at)
        if heads % kv_heads:
            raise ConfigError("%s: %d heads are not a multiple of %d key/value heads" % (at, heads, kv_heads))
        mlp = entry.get("mlp")
        if mlp is not None:
            _take(mlp, where + ".mlp", ("kind", "ff"))
            if mlp["kind"] != "dense":
                raise ConfigError("%s.mlp.kind %r is not a feed-forward of this design" % (where, mlp["kind"]))
            mlp = dict(ff=_count(mlp, "ff", where + ".mlp"), activation="relu2")
        layers.append(dict(mixer=dict(heads=heads, kv_heads=kv_heads, dim=_count(m, "dim", at), vdim=_count(m, "vdim", at),
                                      window=_count(mask, "size", at + ".mask"), scale=float(m["scale"]), log_bias=True,
                                      value_norm=True, gate=True), mlp=mlp))
    return dict(hidden=_count(c, "width", "config"), vocab=_count(c, "vocab", "config"),
                eps=float(_take(c["norm"], "norm", ("eps",))["eps"]), logit_scale=float(c["logit_scale"]),
                max_positions=_count(c, "max_positions", "config"),
                bigram=dict(buckets=_count(bigram, "buckets", "embedding.bigram"), mul_prev=int(bigram["mul_prev"]),
                            mul_cur=int(bigram["mul_cur"])), layers=layers)


def _layer_tensors(i, m, mlp, Hd):
    """DenseDecoder key -> (tensor name, shape, matrix?) of layer i."""
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    mix = "l%d.mix." % i
    t = {"norm": ("l%d.norm1" % i, [Hd], False),
         "q": (mix + "q", [H * d, Hd], True), "q_bias": (mix + "q.b", [H * d], False),
         "k": (mix + "k", [G * d, Hd], True), "k_bias": (mix + "k.b", [G * d], False),
         "v": (mix + "v", [G * e, Hd], True), "v_bias": (mix + "v.b", [G * e], False),
         "bias_r1": (mix + "r1", [H], False), "bias_r2": (mix + "r2", [H], False),
         "gate": (mix + "g", [H, Hd], True), "o": (mix + "o", [Hd, H * e], True)}
    if mlp:
        t["up"] = ("l%d.mlp.up" % i, [mlp["ff"], Hd], True)
        t["down"] = ("l%d.mlp.down" % i, [Hd, mlp["ff"]], True)
    return t


def _model_tensors(cfg):
    Hd, V = cfg["hidden"], cfg["vocab"]
    return {"embed": ("embed", [V, Hd], True), "bigram": ("bigram", [cfg["bigram"]["buckets"] + 1, Hd], True),
            "pos": ("pos", [cfg["max_positions"], Hd], True), "final_norm": ("final.norm", [Hd], False),
            "head": ("head", [V, Hd], True)}


def load_arrays(directory):
    """(cfg, weights) in the form DenseDecoder takes: matrices and tables as bf16 bits, vectors widened to f32."""
    with open(os.path.join(directory, "config.json")) as f:
        cfg = decoder_config(json.load(f))
    st = SafetensorsFile(os.path.join(directory, "model.safetensors"))

    def read(entries):
        out = {}
        for key, (name, shape, matrix) in entries.items():
            a = st.tensor(name, "BF16", shape)
            out[key] = a if matrix else bf16_to_f32(a)
        return out

    weights = read(_model_tensors(cfg))
    weights["layers"] = [read(_layer_tensors(i, s["mixer"], s["mlp"], cfg["hidden"])) for i, s in enumerate(cfg["layers"])]
    return cfg, weights


def load_decoder(directory, max_seq=None, dtype="bfloat16", **decoder_kwargs):
    """A ready DenseDecoder; max_seq None: as many positions as the model has."""
    cfg, weights = load_arrays(directory)
    max_seq = cfg["max_positions"] if max_seq is None else min(max_seq, cfg["max_positions"])
    return DenseDecoder(cfg, weights, max_seq, compute={"bfloat16": "bf16", "float32": "f32"}[dtype], **decoder_kwargs)


def config_json(cfg):
    """The config.json of a DenseDecoder cfg of this design (inverse of decoder_config)."""
    layers = []
    for s in cfg["layers"]:
        m = s["mixer"]
        layers.append({"type": "attention",
                       "mixer": {"heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"], "vdim": m["vdim"],
                                 "scale": m["scale"], "mask": {"size": m["window"]}},
                       "mlp": {"kind": "dense", "ff": s["mlp"]["ff"]} if s["mlp"] else None})
    return {"architecture": ARCHITECTURE, "embedding": {"bigram": dict(cfg["bigram"])}, "layers": layers,
            "logit_scale": cfg["logit_scale"], "max_positions": cfg["max_positions"], "norm": {"eps": cfg["eps"]},
            "vocab": cfg["vocab"], "width": cfg["hidden"]}


def write_model(directory, cfg, weights):
    """Writes a model folder from a DenseDecoder cfg and weights."""
    os.makedirs(directory, exist_ok=True)
    with open(os.path.join(directory, "config.json"), "w") as f:
        json.dump(config_json(cfg), f, indent=1)
    tensors = {}

    def put(entries, values):
        for key, (name, shape, matrix) in entries.items():
            a = values[key] if matrix else f32_to_bf16(values[key])
            tensors[name] = ("BF16", a.reshape(shape))

    put(_model_tensors(cfg), weights)
    for i, (s, w) in enumerate(zip(cfg["layers"], weights["layers"])):
        put(_layer_tensors(i, s["mixer"], s["mlp"], cfg["hidden"]), w)
    write_safetensors(os.path.join(directory, "model.safetensors"), tensors)
