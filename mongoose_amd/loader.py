"""Model folders: config.json (which model class, its sizes and constants) and model.safetensors (its weights)."""
import json
import os

import numpy as np

from . import configs


class SafeTensors:
    """A safetensors file: 8 bytes of little-endian header length, a JSON header, the data.  Mapped, not read."""

    DTYPES = {"BF16": np.uint16, "I32": np.int32, "F32": np.float32}

    def __init__(self, path):
        self._map = np.memmap(path, dtype=np.uint8, mode="r")
        n = int.from_bytes(self._map[:8].tobytes(), "little")
        if 8 + n > self._map.size:
            raise ValueError(f"{path}: header length past the end of the file")
        self.header = json.loads(self._map[8:8 + n].tobytes())
        self.header.pop("__metadata__", None)
        self._data = 8 + n

    def names(self):
        return list(self.header)

    def shape(self, name):
        return tuple(self.header[name]["shape"])

    def array(self, name):
        """The tensor; bf16 as its 16 bits (uint16)."""
        h = self.header[name]
        if h["dtype"] not in self.DTYPES:
            raise ValueError(f"{name}: dtype {h['dtype']} is not supported")
        lo, hi = h["data_offsets"]
        dt = np.dtype(self.DTYPES[h["dtype"]])
        count = int(np.prod(h["shape"], dtype=np.int64))
        if hi - lo != count * dt.itemsize or self._data + hi > self._map.size:
            raise ValueError(f"{name}: data offsets do not fit its shape")
        return np.frombuffer(self._map[self._data + lo:self._data + hi].tobytes(), dt).reshape(h["shape"])


def read_model(folder):
    """(model description, weights) of a model folder, by config.json's "architecture"."""
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    arch = cfg.get("architecture")
    if arch not in configs.ARCHITECTURES:
        raise ValueError(f"architecture {arch!r} is not one of {sorted(configs.ARCHITECTURES)}")
    weights = SafeTensors(os.path.join(folder, "model.safetensors"))
    return configs.ARCHITECTURES[arch](cfg, weights.shape), weights


def set_weights(model, weights):
    """Every tensor of the model from `weights` (names(), shape(name), array(name)); a missing, unknown or misshapen one
    is an error."""
    from .lib import last_error
    want, have = set(model.TensorNames()), set(weights.names())
    if want != have:
        raise ValueError(f"tensors missing: {sorted(want - have)}; unknown: {sorted(have - want)}")
    for name in sorted(want):
        if tuple(weights.shape(name)) != model.TensorShape(name):
            raise ValueError(f"{name}: shape {weights.shape(name)}, expected {model.TensorShape(name)}")
        bits = weights.array(name)
        if bits.dtype != np.uint16:
            raise ValueError(f"{name}: expected bf16 weights")
        if model.SetTensor(name, bits) != 0:
            raise RuntimeError(f"{name}: {last_error()}")


def load_model(folder, maxSeq, dtype="bfloat16", device=0):
    """The model of a folder, on the GPU, ready to generate."""
    from . import engine
    from .lib import last_error
    spec, weights = read_model(folder)
    eng = engine.NewHIP(device)
    if eng is None:
        raise RuntimeError("no HIP device")
    model = engine.NewHIPLayeredInference(eng, spec, maxSeq, dtype)
    if model is None:
        raise RuntimeError(last_error())
    set_weights(model, weights)
    return model
