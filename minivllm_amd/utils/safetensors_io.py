"""Reader of .safetensors files: an 8-byte little-endian header length, a JSON header (name -> dtype, shape,
data_offsets), the data.  Tensors are views of a private memory map of the file."""
from __future__ import annotations

import json
import mmap

import torch

_DTYPES = {"F64": torch.float64, "F32": torch.float32, "F16": torch.float16, "BF16": torch.bfloat16, "I64": torch.int64,
           "I32": torch.int32, "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8, "BOOL": torch.bool}


def read_safetensors(path: str) -> dict[str, torch.Tensor]:
    with open(path, "rb") as f:
        size = int.from_bytes(f.read(8), "little")
        header = json.loads(f.read(size))
        data = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)
    out = {}
    for name, entry in header.items():
        if name == "__metadata__":
            continue
        dtype, shape = _DTYPES[entry["dtype"]], entry["shape"]
        begin, end = entry["data_offsets"]
        count = 1
        for n in shape:
            count *= n
        if count * dtype.itemsize != end - begin:
            raise ValueError(f"{path}: {name} has {end - begin} bytes, {dtype} {shape} needs {count * dtype.itemsize}")
        at = 8 + size + begin
        if count == 0:
            out[name] = torch.empty(shape, dtype=dtype)
        elif at % dtype.itemsize:
            out[name] = torch.frombuffer(bytearray(data[at:at + end - begin]), dtype=dtype).view(shape)
        else:
            out[name] = torch.frombuffer(data, dtype=dtype, count=count, offset=at).view(shape)
    return out
