"""Reading a checkpoint folder's tensors, checked against the shapes its configuration gives."""
from __future__ import annotations

from pathlib import Path


def open_tensors(ckpt_dir) -> dict:
    """name -> open safetensors file of a checkpoint folder."""
    from safetensors import safe_open

    files = sorted(Path(ckpt_dir).glob("*.safetensors"))
    if not files:
        raise FileNotFoundError(f"no *.safetensors in {ckpt_dir}")
    where = {}
    for f in files:
        fh = safe_open(str(f), framework="pt", device="cpu")
        where |= {k: fh for k in fh.keys()}
    return where


def tensor_reader(ckpt_dir, shapes: dict):
    """get(name) -> tensor; every name of ``shapes`` must be there and have its shape."""
    where = open_tensors(ckpt_dir)
    missing = sorted(set(shapes) - set(where))
    if missing:
        raise KeyError(f"{ckpt_dir}: tensors missing: {', '.join(missing[:8])}")

    def get(name):
        t = where[name].get_tensor(name)
        if tuple(t.shape) != shapes[name]:
            raise ValueError(f"{name}: shape {tuple(t.shape)}, config.json gives {shapes[name]}")
        return t
    return get
