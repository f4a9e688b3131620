"""Reader and writer of .safetensors files: an 8-byte little-endian length, that many bytes of JSON (tensor name ->
dtype, shape, data_offsets), then the data.  Tensors come back as views of the mapped file; BF16 as uint16 bit patterns."""
import json
import mmap
import os
import struct

import numpy as np

DTYPES = {"BF16": np.uint16, "F16": np.float16, "F32": np.float32, "I32": np.int32, "I64": np.int64, "U8": np.uint8}


class SafetensorsError(ValueError):
    pass


class SafetensorsFile:
    def __init__(self, path):
        size = os.path.getsize(path)
        with open(path, "rb") as f:
            head = f.read(8)
            if len(head) != 8:
                raise SafetensorsError("%s: too short for a safetensors header" % path)
            n = struct.unpack("<Q", head)[0]
            if n > size - 8:
                raise SafetensorsError("%s: header of %d bytes does not fit the file" % (path, n))
            try:
                self.header = json.loads(f.read(n))
            except ValueError as e:
                raise SafetensorsError("%s: header is not JSON (%s)" % (path, e))
            self.header.pop("__metadata__", None)
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        self.path, self._base, self._size = path, 8 + n, size

    def names(self):
        return list(self.header)

    def __contains__(self, name):
        return name in self.header

    def tensor(self, name, dtype=None, shape=None):
        """The tensor as an array; dtype and shape, when given, must be what the file holds."""
        info = self.header.get(name)
        if info is None:
            raise SafetensorsError("Tensor '%s' is not in %s" % (name, os.path.basename(self.path)))
        if info["dtype"] not in DTYPES or (dtype is not None and info["dtype"] != dtype):
            raise SafetensorsError("Tensor '%s' has dtype %s%s" % (name, info["dtype"], " where %s is expected" % dtype if dtype else ""))
        if shape is not None and list(info["shape"]) != list(shape):
            raise SafetensorsError("Tensor '%s' has shape %r, the configuration implies %r" % (name, info["shape"], list(shape)))
        t = np.dtype(DTYPES[info["dtype"]])
        a, b = info["data_offsets"]
        count = int(np.prod(info["shape"], dtype=np.int64))
        if b - a != count * t.itemsize or a < 0 or self._base + b > self._size:
            raise SafetensorsError("Tensor '%s' does not fit its data range" % name)
        return np.frombuffer(self._map, t, count, self._base + a).reshape(info["shape"])


def write_safetensors(path, tensors):
    """tensors: name -> (dtype code, array of that dtype's storage type)."""
    header, at, blobs = {}, 0, []
    for name, (code, a) in tensors.items():
        a = np.ascontiguousarray(a, DTYPES[code])
        header[name] = {"dtype": code, "shape": list(a.shape), "data_offsets": [at, at + a.nbytes]}
        at += a.nbytes
        blobs.append(a)
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)))
        f.write(text)
        for a in blobs:
            f.write(a.tobytes())
