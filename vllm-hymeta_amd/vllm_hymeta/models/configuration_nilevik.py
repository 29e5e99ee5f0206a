"""Configuration of the Nilevik family (``"architecture": "Nilevik"`` in ``config.json``).

The file is nested: ``layers`` lists the decoder layers in order, each with the ``type`` of its mixer (``"attention"`` or
``"delta"``), the mixer's sizes and constants (``mixer``) and its feed-forward (``mlp``: ``{"kind": "dense", ...}`` or
``null``).  Everything that can differ between two checkpoints of the family is read from the file; this class only names
and checks the fields.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Any, Dict, List, Optional


@dataclass
class KeyValueAttentionSpec:
    """Softmax attention whose values are its projected keys.  ``window``: a query sees itself and the ``window - 1`` keys
    before it (None: all); queries are multiplied by ``1 + temp_coef ln(floor((p + 1) / temp_every) + 1)``."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: Optional[int]
    temp_coef: float
    temp_every: float

    def slopes(self) -> List[float]:
        """The distance penalty of every head: the geometric sequence that ends at ``2^-8``."""
        return [2.0 ** (-8.0 * (h + 1) / self.heads) for h in range(self.heads)]


@dataclass
class DeltaSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    @property
    def conv_channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


@dataclass
class GatedMlpSpec:
    ff: int


@dataclass
class NilevikLayerSpec:
    type: str
    mixer: Any
    mlp: Optional[GatedMlpSpec]


class NilevikConfig:
    model_type = "nilevik"
    architectures = ["NilevikForCausalLM"]
    position_base = 10000.0

    def __init__(self, raw: Dict[str, Any]):
        self.raw = raw
        self.vocab_size = int(raw["vocab"])
        self.hidden_size = int(raw["width"])
        self.norm_eps = float(raw["norm"]["eps"])
        self.side_dim = int((raw.get("token_side") or {}).get("dim", 0))
        self.layers: List[NilevikLayerSpec] = []
        for i, entry in enumerate(raw["layers"]):
            kind, mx = entry["type"], entry["mixer"]
            heads = int(mx["heads"])
            kv = int(mx.get("kv_heads", heads))
            if kv < 1 or heads % kv:
                raise ValueError(f"layer {i}: {heads} heads do not split over {kv} key/value heads")
            if kind == "attention":
                mask, temp = mx.get("mask") or {}, mx.get("q_temp") or {}
                mixer = KeyValueAttentionSpec(heads=heads, kv_heads=kv, dim=int(mx["dim"]), scale=float(mx["scale"]),
                                              window=int(mask["size"]) if mask.get("size") is not None else None,
                                              temp_coef=float(temp.get("coef", 0.0)), temp_every=float(temp.get("every", 1.0)))
                if int(mx.get("vdim", mixer.dim)) != mixer.dim:
                    raise ValueError(f"layer {i}: the values are the keys, so vdim must be dim")
                if mixer.window is not None and mixer.window < 1:
                    raise ValueError(f"layer {i}: the window counts tokens")
                if not mixer.temp_every > 0:
                    raise ValueError(f"layer {i}: q_temp.every counts tokens")
            elif kind == "delta":
                mixer = DeltaSpec(heads=heads, kv_heads=kv, dim=int(mx["dim"]), vdim=int(mx.get("vdim", mx["dim"])), conv=int(mx["conv"]))
                if mixer.conv < 1:
                    raise ValueError(f"layer {i}: conv counts taps")
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            mlp = entry.get("mlp")
            if mlp is not None:
                if mlp.get("kind", "dense") != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
                mlp = GatedMlpSpec(ff=int(mlp["ff"]))
            self.layers.append(NilevikLayerSpec(kind, mixer, mlp))
        self.num_hidden_layers = len(self.layers)

    def position_frequencies(self) -> List[float]:
        """Of the sinusoidal position vector, one per pair of columns."""
        return [self.position_base ** (-2.0 * i / self.hidden_size) for i in range((self.hidden_size + 1) // 2)]

    @classmethod
    def from_pretrained(cls, model_dir: str) -> "NilevikConfig":
        with open(os.path.join(model_dir, "config.json")) as f:
            return cls(json.load(f))
