"""Decoder block that reads the fp32 residual stream as it is and norms what it adds:

    x <- x + norm(mixer(x)),   x <- x + norm(ff(x)),   x <- x + norm(token input(x))

``norm`` is an RMS norm with a weight.  The stream stays fp32 whatever the activation type; a sublayer reads its rounded
copy, which the launch that adds the previous sublayer's output writes beside it.  Beside ``StreamBlock``
(``stream_block.py``: norms on both sides of a sublayer) and ``PostNormBlock`` (``post_norm_block.py``: the norm after the sum).
"""

from __future__ import annotations

from typing import Optional

import torch

from .. import hip_ops
from ..linear import HymetaLinear
from .stream_block import StepLayout


class AddNormed(torch.nn.Module):
    """``x += rms(y) w`` in place on the stream; returns what the next sublayer reads: the stream itself where activations
    are fp32, else its copy in y's type."""

    def __init__(self, weight: torch.Tensor, eps: float):
        super().__init__()
        self.register_buffer("weight", weight.float().contiguous())
        self.eps = float(eps)

    def forward(self, x: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
        return hip_ops.norm_residual_(x, y, self.weight, self.eps, copy=y.dtype != torch.float32)


class TokenInput(torch.nn.Module):
    """A layer's own input from the token: ``W_proj (gelu(W_gate h) * table[token])``, ``table`` the layer's columns of a table
    that all layers share."""

    def __init__(self, gate: HymetaLinear, proj: HymetaLinear, table: torch.Tensor):
        """``table [vocab, dim]``: a view with any row stride."""
        super().__init__()
        self.gate, self.proj = gate, proj
        self._table = (table,)        # a view of the model's table

    def forward(self, h: torch.Tensor, token_ids: torch.Tensor) -> torch.Tensor:
        return self.proj(hip_ops.gelu_mul_rows(self.gate(h), self._table[0], token_ids))


class AddedNormBlock(torch.nn.Module):
    """One decoder layer.  ``mixer(h, layout, state)`` and ``mlp(h)`` take and return activations; ``mlp`` and ``side`` may be
    absent, each comes with its norm."""

    def __init__(self, mixer: torch.nn.Module, mixer_add: AddNormed, mlp: Optional[torch.nn.Module] = None, mlp_add: Optional[AddNormed] = None,
                 side: Optional[TokenInput] = None, side_add: Optional[AddNormed] = None):
        super().__init__()
        self.mixer, self.mixer_add, self.mlp, self.mlp_add, self.side, self.side_add = mixer, mixer_add, mlp, mlp_add, side, side_add

    def forward(self, x: torch.Tensor, h: torch.Tensor, layout: StepLayout, mixer_state) -> torch.Tensor:
        """``h``: the stream as the mixer reads it (``x`` itself or its copy).  Returns the same for the next layer."""
        h = self.mixer_add(x, self.mixer(h, layout, mixer_state))
        if self.mlp is not None:
            h = self.mlp_add(x, self.mlp(h))
        if self.side is not None:
            h = self.side_add(x, self.side(h, layout.token_ids))
        return h
