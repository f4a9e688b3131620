"""Model registry: which loader and kernel families serve a model folder.

A folder holds either an RDRR artifact (manifest.json: the Q4_K decoder) or config.json + model.safetensors, whose
`architecture` names a design.  Every entry loads a ready decoder (doppler_amd.decoder.DecoderBase).
"""
import json
import os


class UnknownModel(ValueError):
    pass


class UnsupportedDtype(ValueError):
    pass


class Model:
    """name; dtypes it runs in (the first is what it is served in); load(directory, max_seq, dtype, **kwargs);
    library: None for the whole library, or the build target that holds all its kernels."""

    def __init__(self, name, dtypes, load, library=None):
        self.name, self.dtypes, self._load, self.library = name, tuple(dtypes), load, library

    def load(self, directory, max_seq=None, dtype=None, **kwargs):
        dtype = dtype or self.dtypes[0]
        if dtype not in self.dtypes:
            raise UnsupportedDtype("%s models run in %s, not %s" % (self.name, ", ".join(self.dtypes), dtype))
        return self._load(directory, max_seq, dtype, **kwargs)


def _load_rdrr(directory, max_seq, dtype, **kwargs):
    from . import rdrr
    return rdrr.load_decoder(directory, max_seq or 4096, **kwargs)


def _load_zepavik(directory, max_seq, dtype, **kwargs):
    from . import zepavik
    return zepavik.load_decoder(directory, max_seq, dtype, **kwargs)


def _load_gusolorn(directory, max_seq, dtype, **kwargs):
    from . import gusolorn
    return gusolorn.load_decoder(directory, max_seq, dtype, **kwargs)


RDRR = Model("RDRR Q4_K", ["bfloat16"], _load_rdrr)
ARCHITECTURES = {
    "Zepavik": Model("Zepavik", ["bfloat16", "float32"], _load_zepavik, library="dense"),
    "Gusolorn": Model("Gusolorn", ["bfloat16", "float32"], _load_gusolorn, library="dense"),
}


def find(directory):
    """The registry entry of a model folder."""
    if os.path.exists(os.path.join(directory, "manifest.json")):
        return RDRR
    path = os.path.join(directory, "config.json")
    if not os.path.exists(path):
        raise UnknownModel("%s holds neither manifest.json nor config.json" % directory)
    with open(path) as f:
        name = json.load(f).get("architecture")
    if name not in ARCHITECTURES:
        raise UnknownModel("architecture %r is not one of %s" % (name, ", ".join(sorted(ARCHITECTURES))))
    return ARCHITECTURES[name]


def ensure_library(model):
    """Binds the native library, compiling it first where this checkout has none: the families the model needs and
    no more."""
    import torch  # noqa: F401  (first: the native library must bind the HIP runtime that torch brings)
    from . import build, capi
    if os.path.exists(capi.LIB_PATH):
        capi.load()
    elif model.library == "dense":
        if not os.path.exists(capi.DENSE_LIB_PATH):
            build.build_dense()
        capi.load(capi.DENSE_LIB_PATH)
    else:
        build.build_hip()
        capi.load()


def load(directory, max_seq=None, dtype=None, **kwargs):
    """A ready decoder for a model folder."""
    model = find(directory)
    ensure_library(model)
    return model.load(directory, max_seq, dtype, **kwargs)
