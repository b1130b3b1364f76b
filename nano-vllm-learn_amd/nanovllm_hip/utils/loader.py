"""Checkpoint reading: config.json and *.safetensors of a model folder."""
import glob
import json
import os

from safetensors import safe_open


def read_config(path):
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


class Checkpoint:
    """Tensors of a folder by name; every tensor is read when asked for, and unread names can be listed."""

    def __init__(self, path):
        files = sorted(glob.glob(os.path.join(path, "*.safetensors")))
        if not files:
            raise FileNotFoundError(f"no .safetensors file in {path}")
        self._files = [safe_open(f, framework="pt", device="cpu") for f in files]
        self._where = {name: f for f in self._files for name in f.keys()}
        self._unread = set(self._where)

    def __contains__(self, name):
        return name in self._where

    def __call__(self, name):
        if name not in self._where:
            raise KeyError(f"checkpoint holds no tensor {name!r}")
        self._unread.discard(name)
        return self._where[name].get_tensor(name)

    def unread(self):
        return sorted(self._unread)
