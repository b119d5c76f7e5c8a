"""safetensors files: an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets) and
the tensors' bytes.  Mapped, not read: a tensor's bytes go from the file to the device."""
from __future__ import annotations

import json
import os
from typing import Dict, Tuple

import numpy as np

# dtype -> (bytes per element, kind of the state dict)
_KINDS = {"F32": (4, "f32"), "F16": (2, "f16"), "BF16": (2, "bf16"), "I32": (4, "i32")}


def read(path: str) -> Dict[str, Tuple[str, tuple, np.ndarray]]:
    """name -> (kind, shape, raw bytes)"""
    size = os.path.getsize(path)
    if size < 8:
        raise ValueError(f"{path}: not a safetensors file")
    data = np.memmap(path, np.uint8, "r")
    n = int.from_bytes(data[:8].tobytes(), "little")
    if n > size - 8:
        raise ValueError(f"{path}: the header's {n} bytes exceed the file")
    header = json.loads(data[8:8 + n].tobytes())
    out = {}
    for name, t in header.items():
        if name == "__metadata__":
            continue
        if t["dtype"] not in _KINDS:
            raise ValueError(f"{path}: tensor {name} has dtype {t['dtype']} (supported: {', '.join(_KINDS)})")
        width, kind = _KINDS[t["dtype"]]
        shape = tuple(int(d) for d in t["shape"])
        lo, hi = t["data_offsets"]
        want = width * int(np.prod(shape, dtype=np.int64))
        if not 0 <= lo <= hi <= size - 8 - n or hi - lo != want:
            raise ValueError(f"{path}: tensor {name} {shape} has bytes {lo}..{hi}, expected {want} of them")
        out[name] = (kind, shape, data[8 + n + lo:8 + n + hi])
    return out


def write(path: str, tensors: Dict[str, Tuple[str, tuple, np.ndarray]]) -> None:
    names = {kind: dtype for dtype, (_, kind) in _KINDS.items()}
    header, off = {}, 0
    for name, (kind, shape, raw) in tensors.items():
        n = np.asarray(raw).view(np.uint8).size
        header[name] = {"dtype": names[kind], "shape": list(shape), "data_offsets": [off, off + n]}
        off += n
    h = json.dumps(header).encode()
    h += b" " * (-len(h) % 8)
    with open(path, "wb") as f:
        f.write(len(h).to_bytes(8, "little"))
        f.write(h)
        for _, _, raw in tensors.values():
            f.write(np.ascontiguousarray(raw).view(np.uint8).tobytes())
