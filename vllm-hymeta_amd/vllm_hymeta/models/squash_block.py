"""Decoder block on an fp32 residual stream with a squashing norm on both sides of every sublayer, and the entry of a pass
through a repeated run of such blocks:

    x <- x + norm_out(mixer(norm_in(x))),   x <- x + norm_out'(ff(norm_in'(x))),   norm(v) = tanh(alpha v) w + b

(element by element, no statistic over a row; "Transformers without Normalization", Zhu et al. 2025).  So what follows a
sublayer -- its output's norm, the sum onto the stream, the next sublayer's norm -- is ONE elementwise launch
(``hip_ops.tanh_stream_``), and a block is handed the way in which whoever comes after it reads the stream.

    pass entry:  x <- W_in [x; x0] + step_t,   x0 the embedding output

with ``W_in``'s two halves apart: ``W_in'' x0`` is the same in every pass and computed once per model step; the products leave
in fp32, since they become the stream.

The stream stays fp32 whatever the activation type; a sublayer reads and returns activations (bf16 or fp32).  Beside
``StreamBlock`` (``stream_block.py``: RMS norms on both sides of a sublayer), ``AddedNormBlock`` and ``PostNormBlock``.
"""

from __future__ import annotations

from typing import Optional

import torch

from .. import hip_ops
from ..linear import linear_fp32
from .stream_block import StepLayout


class TanhNorm(torch.nn.Module):
    def __init__(self, alpha: float, weight: torch.Tensor, bias: torch.Tensor):
        super().__init__()
        self.alpha = float(alpha)
        self.register_buffer("weight", weight.float().contiguous())
        self.register_buffer("bias", bias.float().contiguous())

    @property
    def constants(self) -> hip_ops.SquashNorm:
        return hip_ops.SquashNorm(self.alpha, self.weight, self.bias)

    def forward(self, x: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
        """The norm of the stream alone (nothing is added to it)."""
        return hip_ops.tanh_stream_(x, read=self.constants, out_dtype=out_dtype)


def add_and_read(x: torch.Tensor, y, out_norm: TanhNorm, read: Optional[TanhNorm], act_dtype: torch.dtype) -> torch.Tensor:
    """``x += out_norm(y)``, ``y`` a sublayer's output or the partial sums of its last projection; returns what the next sublayer
    reads: ``read(x)``, or (None) the stream itself."""
    if read is None and act_dtype == torch.float32:
        hip_ops.tanh_stream_(x, y, out_norm.constants)
        return x
    return hip_ops.tanh_stream_(x, y, out_norm.constants, read=None if read is None else read.constants, out_dtype=act_dtype)


class SquashBlock(torch.nn.Module):
    """One decoder layer.  ``mixer(h, layout, state, defer=True)`` and ``mlp(h, defer=True)`` take activations and return them,
    or the partial sums of their last projection; ``mlp`` may be absent."""

    def __init__(self, mixer_in: TanhNorm, mixer: torch.nn.Module, mixer_out: TanhNorm, mlp_in: Optional[TanhNorm] = None,
                 mlp: Optional[torch.nn.Module] = None, mlp_out: Optional[TanhNorm] = None):
        super().__init__()
        self.mixer_in, self.mixer, self.mixer_out = mixer_in, mixer, mixer_out
        self.mlp_in, self.mlp, self.mlp_out = mlp_in, mlp, mlp_out

    def forward(self, x: torch.Tensor, h: torch.Tensor, layout: StepLayout, mixer_state, read: Optional[TanhNorm]) -> torch.Tensor:
        """``h``: ``mixer_in`` of the stream.  Returns ``read`` of the stream after the layer (None: its copy)."""
        act = h.dtype
        y = self.mixer(h, layout, mixer_state, defer=True)
        if self.mlp is None:
            return add_and_read(x, y, self.mixer_out, read, act)
        h = add_and_read(x, y, self.mixer_out, self.mlp_in, act)
        return add_and_read(x, self.mlp(h, defer=True), self.mlp_out, read, act)


class PassEntry(torch.nn.Module):
    """``x <- W_stream x + W_start x0 + step_t`` in front of a pass."""

    def __init__(self, stream_weight: torch.Tensor, start_weight: torch.Tensor, steps: torch.Tensor):
        """``stream_weight``, ``start_weight [W, W]``; ``steps [times, W]``."""
        super().__init__()
        self.register_buffer("stream_weight", stream_weight.contiguous())
        self.register_buffer("start_weight", start_weight.contiguous())
        self.register_buffer("steps", steps.float().contiguous())

    def start_part(self, h0: torch.Tensor) -> torch.Tensor:
        """The embedding output's part, fp32: the same in every pass.  ``h0``: activations."""
        return linear_fp32(h0, self.start_weight)

    def forward(self, x: torch.Tensor, h: torch.Tensor, start: torch.Tensor, t: int, read: TanhNorm, out_dtype: torch.dtype) -> torch.Tensor:
        """``h``: the stream as activations; ``start``: ``start_part``.  Renews ``x`` and returns ``read`` of it."""
        return hip_ops.tanh_stream_(x, base=linear_fp32(h, self.stream_weight), base2=start, add=self.steps[t], read=read.constants, out_dtype=out_dtype)
