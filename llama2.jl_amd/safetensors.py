"""Reader and writer of the safetensors container: an 8-byte little-endian length, that many bytes of JSON
(name -> dtype, shape, data_offsets), then the data.  Tensors are memory-mapped; bf16 ones are uint16 arrays."""
import json
import os
import struct

import numpy as np

_DTYPES = {"F32": np.dtype("<f4"), "BF16": np.dtype("<u2"), "I32": np.dtype("<i4")}


class SafetensorsError(ValueError):
    pass


def read_safetensors(path):
    """name -> (dtype name, array)"""
    size = os.path.getsize(path)
    with open(path, "rb") as f:
        head = f.read(8)
        n = struct.unpack("<Q", head)[0] if len(head) == 8 else -1
        if n < 2 or 8 + n > size:
            raise SafetensorsError("%s: header length %d does not fit the file" % (path, n))
        header = json.loads(f.read(n))
    data = np.memmap(path, dtype=np.uint8, mode="r") if size > 8 + n else np.zeros(0, np.uint8)
    base, out = 8 + n, {}
    for name, t in header.items():
        if name == "__metadata__":
            continue
        if t["dtype"] not in _DTYPES:
            raise SafetensorsError("%s: tensor %s has type %s" % (path, name, t["dtype"]))
        dt = _DTYPES[t["dtype"]]
        lo, hi = t["data_offsets"]
        if lo < 0 or hi < lo or base + hi > size or hi - lo != dt.itemsize * int(np.prod(t["shape"], dtype=np.int64)):
            raise SafetensorsError("%s: tensor %s: offsets %d..%d do not fit its shape or the file" % (path, name, lo, hi))
        raw = data[base + lo:base + hi]
        if (base + lo) % dt.itemsize:
            raw = np.array(raw)
        out[name] = (t["dtype"], raw.view(dt).reshape(t["shape"]))
    return out


def write_safetensors(path, tensors):
    """tensors: name -> array; uint16 arrays are bf16 bit patterns"""
    names = {np.dtype("<f4"): "F32", np.dtype("<u2"): "BF16", np.dtype("<i4"): "I32"}
    header, at = {}, 0
    for name, a in tensors.items():
        header[name] = {"dtype": names[a.dtype], "shape": list(a.shape), "data_offsets": [at, at + a.nbytes]}
        at += a.nbytes
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for a in tensors.values():
            f.write(np.ascontiguousarray(a).tobytes())
