"""Configuration of the Banitar family (``"architecture": "Banitar"`` in ``config.json``).

The file is nested: ``layers`` lists the decoder layers in order, each with the ``type`` of its mixer (``"attention"`` or
``"latent_attention"``), the mixer's sizes and constants (``mixer``) and its feed-forward (``mlp``: ``{"kind": "dense", ...}``
or ``null``); ``loop`` names a run of layers (``start`` .. ``stop - 1``) that is repeated ``times`` times in a row with the same
weights, every pass with caches of its own.  Everything that can differ between two checkpoints of the family is read from
the file; this class only names and checks the fields.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from .configuration_geponex import RotarySpec


@dataclass
class ChunkedAttentionSpec:
    """Softmax attention within chunks of ``chunk`` positions, counted from the sequence's first token (None: over all)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: Optional[int]
    rot: RotarySpec


@dataclass
class WindowedLatentSpec:
    """Latent attention over a token and the ``window - 1`` before it (None: all)."""
    heads: int
    dim: int              # unrotated query / key size per head
    rot_dim: int          # rotated size per head (the key's rotated part is shared by the heads)
    vdim: int
    kv_rank: int
    scale: float
    window: Optional[int]
    rot: RotarySpec


@dataclass
class DenseMlpSpec:
    ff: int


@dataclass
class BanitarLayerSpec:
    type: str
    mixer: Any
    mlp: Optional[DenseMlpSpec]


class BanitarConfig:
    model_type = "banitar"
    architectures = ["BanitarForCausalLM"]

    def __init__(self, raw: Dict[str, Any]):
        self.raw = raw
        self.vocab_size = int(raw["vocab"])
        self.hidden_size = int(raw["width"])
        self.norm_eps = float(raw["norm"]["eps"])
        self.embed_scale = float((raw.get("embedding") or {}).get("scale", 1.0))
        self.layers: List[BanitarLayerSpec] = []
        for i, entry in enumerate(raw["layers"]):
            kind, mx = entry["type"], entry["mixer"]
            heads, dim, size = int(mx["heads"]), int(mx["dim"]), (mx.get("mask") or {}).get("size")
            vdim, scale, size = int(mx.get("vdim", dim)), float(mx["scale"]), None if size is None else int(size)
            if size is not None and size < 1:
                raise ValueError(f"layer {i}: mask.size counts tokens")
            rot = mx.get("rot") or {}
            if kind == "attention":
                kv = int(mx.get("kv_heads", heads))
                if kv < 1 or heads % kv:
                    raise ValueError(f"layer {i}: {heads} heads do not split over {kv} key/value heads")
                turning = self._rotation(i, rot, dim)
                mixer = ChunkedAttentionSpec(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale, chunk=size, rot=turning)
            elif kind == "latent_attention":
                rot_dim = int(mx["rot_dim"])
                turning = self._rotation(i, rot, rot_dim)
                mixer = WindowedLatentSpec(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=int(mx["kv_rank"]), scale=scale, window=size, rot=turning)
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            mlp = entry.get("mlp")
            if mlp is not None:
                if mlp.get("kind", "dense") != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
                mlp = DenseMlpSpec(ff=int(mlp["ff"]))
            self.layers.append(BanitarLayerSpec(kind, mixer, mlp))
        self.num_hidden_layers = len(self.layers)
        loop = raw.get("loop") or None
        self.has_loop = loop is not None
        self.loop_start, self.loop_stop, self.loop_times = (int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else (0, 0, 1)
        if self.has_loop and not (0 <= self.loop_start < self.loop_stop <= self.num_hidden_layers and self.loop_times >= 1):
            raise ValueError(f"loop {loop} does not name a run of the {self.num_hidden_layers} layers")

    @staticmethod
    def _rotation(i: int, rot: Dict[str, Any], size: int) -> RotarySpec:
        spec = RotarySpec(dims=int(rot.get("dims", size)), base=float(rot.get("base", 10000.0)), scaling=rot.get("scaling"))
        if spec.dims % 2 or not 0 <= spec.dims <= size:
            raise ValueError(f"layer {i}: {spec.dims} rotated dimensions do not fit {size}")
        return spec

    def layer_runs(self) -> List[Tuple[int, int]]:
        """``(layer, pass)`` in the order of execution; layers outside the loop run as pass 0."""
        runs: List[Tuple[int, int]] = []
        i = 0
        while i < self.num_hidden_layers:
            if self.has_loop and i == self.loop_start:
                runs += [(j, t) for t in range(self.loop_times) for j in range(self.loop_start, self.loop_stop)]
                i = self.loop_stop
            else:
                runs.append((i, 0))
                i += 1
        return runs

    def enters_pass(self, run: Tuple[int, int]) -> bool:
        return self.has_loop and run[0] == self.loop_start

    @classmethod
    def from_pretrained(cls, model_dir: str) -> "BanitarConfig":
        with open(os.path.join(model_dir, "config.json")) as f:
            return cls(json.load(f))
