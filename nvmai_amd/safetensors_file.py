"""Reader and writer of the safetensors container: eight bytes of little-endian header length, a JSON header
(name -> dtype, shape, data_offsets), the data."""
import json
import os
import struct

import numpy as np
import torch

_DTYPES = {"BF16": (torch.bfloat16, 2), "F16": (torch.float16, 2), "F32": (torch.float32, 4), "F64": (torch.float64, 8),
           "I8": (torch.int8, 1), "U8": (torch.uint8, 1), "I16": (torch.int16, 2), "I32": (torch.int32, 4), "I64": (torch.int64, 8)}
_NAMES = {v[0]: k for k, v in _DTYPES.items()}
HEADER_MAX = 100 << 20


class SafetensorsError(ValueError):
    pass


class SafetensorsFile:
    """The tensors of one file, mapped and copied out one at a time."""

    def __init__(self, path):
        size = os.path.getsize(path)
        with open(path, "rb") as f:
            head = f.read(8)
            if len(head) < 8:
                raise SafetensorsError("%s: truncated" % path)
            n = struct.unpack("<Q", head)[0]
            if n > HEADER_MAX or 8 + n > size:
                raise SafetensorsError("%s: header of %d bytes in a file of %d" % (path, n, size))
            header = json.loads(f.read(n))
        header.pop("__metadata__", None)
        self.path, self.entries = path, {}
        for name, e in header.items():
            if e["dtype"] not in _DTYPES:
                raise SafetensorsError("%s: %s has unsupported dtype %s" % (path, name, e["dtype"]))
            dtype, width = _DTYPES[e["dtype"]]
            a, b = e["data_offsets"]
            shape = tuple(int(v) for v in e["shape"])
            count = int(np.prod(shape, dtype=np.int64))
            if not (0 <= a <= b <= size - 8 - n) or b - a != count * width:
                raise SafetensorsError("%s: %s does not fit its place in the file" % (path, name))
            self.entries[name] = (dtype, shape, a, b)
        self._data = np.memmap(path, dtype=np.uint8, mode="r", offset=8 + n) if size > 8 + n else np.zeros(0, np.uint8)

    def __contains__(self, name):
        return name in self.entries

    def shape(self, name):
        return self.entries[name][1]

    def tensor(self, name):
        """A host tensor of its own (the file may be closed or replaced afterwards)."""
        dtype, shape, a, b = self.entries[name]
        raw = torch.from_numpy(np.array(self._data[a:b]))
        return raw.view(dtype).reshape(shape) if b > a else torch.empty(shape, dtype=dtype)


def write_safetensors(path, tensors):
    """tensors: name -> host tensor."""
    header, at, parts = {}, 0, []
    for name, t in tensors.items():
        raw = t.contiguous().reshape(-1).view(torch.uint8).numpy().tobytes() if t.numel() else b""
        header[name] = {"dtype": _NAMES[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        at += len(raw)
        parts.append(raw)
    head = json.dumps(header).encode()
    head += b" " * (-len(head) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head)
        for raw in parts:
            f.write(raw)
