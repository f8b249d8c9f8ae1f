"""What the designs' readers share: strict config keys, and tensors by name."""
from __future__ import annotations

import torch


def only(d: dict, keys: str, where: str) -> dict:
    """`d`, which must have exactly the given keys."""
    unknown, missing = set(d) - set(keys.split()), set(keys.split()) - set(d)
    if unknown or missing:
        raise ValueError(f"config, {where}: unknown keys {sorted(unknown)}, missing keys {sorted(missing)}")
    return d


def put(dst: torch.Tensor, src: torch.Tensor, name: str) -> None:
    """Copy a checkpoint's tensor (vectors kept per head and channel may be stored in either shape)."""
    if dst.numel() != src.numel() or (dst.dim() > 1 and tuple(dst.shape) != tuple(src.shape)):
        raise ValueError(f"tensor {name} has shape {tuple(src.shape)}, expected {tuple(dst.shape)}")
    dst.copy_(src.reshape(dst.shape))


class Checkpoint:
    """Tensors of a safetensors file, read one at a time; `finish` complains about unread ones."""

    def __init__(self, path: str):
        from safetensors import safe_open
        self._file = safe_open(path, framework="pt", device="cpu")
        self._left = set(self._file.keys())
        self.shapes = {n: tuple(self._file.get_slice(n).get_shape()) for n in self._left}

    def take(self, name: str) -> torch.Tensor:
        if name not in self.shapes:
            raise ValueError(f"the checkpoint has no tensor {name}")
        self._left.discard(name)
        return self._file.get_tensor(name)

    def ignore(self, name: str) -> None:
        """`name` may be in the file and is not needed."""
        self._left.discard(name)

    def finish(self) -> None:
        if self._left:
            raise ValueError(f"the checkpoint has tensors the model does not know: {sorted(self._left)[:8]}")
