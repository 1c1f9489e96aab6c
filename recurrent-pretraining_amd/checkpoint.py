"""Local checkpoint directories: `config.json` plus `model.safetensors`, sharded `model-XXXXX-of-YYYYY.safetensors` with
`model.safetensors.index.json`, or `pytorch_model.bin` (read with weights_only=True).  Nothing is downloaded; at most one shard
is held in host memory."""

from __future__ import annotations

import json
import os
import struct
from typing import Dict, Iterator, Tuple

import torch


def read_config(path: str) -> dict:
    path = str(path)
    if not os.path.isdir(path):
        raise FileNotFoundError(f"{path} is not a local directory (nothing is downloaded)")
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


def files(path: str) -> list:
    path = str(path)
    index = os.path.join(path, "model.safetensors.index.json")
    if os.path.exists(index):
        with open(index) as f:
            return [os.path.join(path, s) for s in sorted(set(json.load(f)["weight_map"].values()))]
    for name in ("model.safetensors", "pytorch_model.bin"):
        if os.path.exists(os.path.join(path, name)):
            return [os.path.join(path, name)]
    raise FileNotFoundError(f"no model.safetensors(.index.json) or pytorch_model.bin under {path}")


def tensors(path: str) -> Iterator[Tuple[str, torch.Tensor]]:
    """(name, CPU tensor) of every tensor, shard by shard."""
    for file in files(path):
        if file.endswith(".safetensors"):
            from safetensors.torch import load_file
            part = load_file(file, device="cpu")
        else:
            part = torch.load(file, map_location="cpu", weights_only=True)
        yield from part.items()
        del part


def shapes(path: str) -> Dict[str, tuple]:
    """name -> shape, from the headers alone where the files are safetensors."""
    out: Dict[str, tuple] = {}
    for file in files(path):
        if file.endswith(".safetensors"):
            with open(file, "rb") as f:
                header = json.loads(f.read(struct.unpack("<Q", f.read(8))[0]))
            out.update({k: tuple(v["shape"]) for k, v in header.items() if k != "__metadata__"})
        else:
            out.update({k: tuple(v.shape) for k, v in torch.load(file, map_location="cpu", weights_only=True).items()})
    return out


def write(path: str, config: dict, state: Dict[str, torch.Tensor], max_shard_bytes: int) -> None:
    """`config.json` and safetensors shards, with an index when there are several."""
    from safetensors.torch import save_file
    path = str(path)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f, indent=1, sort_keys=True)
    shards, cur, size = [], {}, 0
    for name, t in state.items():
        t = t.detach().to("cpu").contiguous()
        nbytes = t.numel() * t.element_size()
        if cur and size + nbytes > max_shard_bytes:
            shards.append(cur)
            cur, size = {}, 0
        cur[name] = t
        size += nbytes
    shards.append(cur)
    if len(shards) == 1:
        save_file(shards[0], os.path.join(path, "model.safetensors"), metadata={"format": "pt"})
        return
    weight_map = {}
    for i, part in enumerate(shards):
        fname = f"model-{i + 1:05d}-of-{len(shards):05d}.safetensors"
        save_file(part, os.path.join(path, fname), metadata={"format": "pt"})
        weight_map.update({k: fname for k in part})
    total = sum(t.numel() * t.element_size() for part in shards for t in part.values())
    with open(os.path.join(path, "model.safetensors.index.json"), "w") as f:
        json.dump({"metadata": {"total_size": total}, "weight_map": weight_map}, f, indent=1)
