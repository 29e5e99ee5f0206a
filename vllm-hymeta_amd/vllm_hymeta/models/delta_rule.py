"""Gated delta-rule mixer ("Gated Delta Networks: Improving Mamba2 with Delta Rule", Yang, Kautz and Hatamizadeh): linear
attention whose state forgets by a scalar per head and token and is corrected towards every token's value before it is read:

    q, k, v = silu(causal conv over time per channel (W_q h, W_k h, W_v h));   q, k to unit length per head, q times D^-1/2
    beta = sigmoid(W_b h);   log a = -exp(A_log) softplus(W_a h + dt_bias)
    S <- a S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
    out = W_o (rms(o) w silu(W_g h))              (the norm per head, one weight for all heads)

The six input projections are one linear layer; the convolution with the decays is ``hip_ops.causal_conv_silu`` (its last
taps - 1 input rows are part of a sequence's state), the recurrence ``hip_ops.delta_rule`` with the state fp32 ``[slots, H, D,
Dv]``, the norm and gate ``hip_ops.gated_rms_norm``, which a step of single rows runs inside the recurrence's launch.  Beside
``StateSpaceMixer`` (``state_space.py``) and ``RetentionMixer`` (``retention.py``), whose states only add.
"""

from __future__ import annotations

import torch

from .. import hip_ops
from ..linear import HymetaLinear

UNIT_EPS = 1e-6       # under the root of a query's or key's length


class DeltaRuleMixer(torch.nn.Module):
    def __init__(self, in_proj: HymetaLinear, o_proj: HymetaLinear, heads: int, kv_heads: int, dim: int, vdim: int, conv_weight: torch.Tensor,
                 a_log: torch.Tensor, dt_bias: torch.Tensor, norm_weight: torch.Tensor, eps: float):
        """``in_proj``: rows = queries, keys (``kv_heads dim`` each), values, output gate (``heads vdim`` each), write strengths and
        decays (``heads`` each); ``conv_weight [channels of q, k, v, taps]``."""
        super().__init__()
        self.in_proj, self.o_proj = in_proj, o_proj
        self.H, self.G, self.D, self.Dv, self.eps = heads, kv_heads, dim, vdim, float(eps)
        for name, t in (("conv_weight", conv_weight), ("a_log", a_log), ("dt_bias", dt_bias), ("norm_weight", norm_weight)):
            self.register_buffer(name, t.float().contiguous())
        self.register_buffer("row_norm_weight", self.norm_weight.repeat(heads))

    def forward(self, h: torch.Tensor, layout, state) -> torch.Tensor:
        """``state``: ``(S fp32 [slots, H, D, Dv], conv inputs [slots, taps - 1, channels] in the activations' type)``, updated in
        place for the step's sequences."""
        S, conv_state = state
        H, G, D, Dv = self.H, self.G, self.D, self.Dv
        ch = 2 * G * D + H * Dv
        proj = self.in_proj(h)
        gate = proj[:, ch:ch + H * Dv]
        beta, a = proj[:, ch + H * Dv:ch + H * Dv + H], proj[:, ch + H * Dv + H:ch + H * Dv + 2 * H]
        qkv, _, log2_decay = hip_ops.causal_conv_silu(proj[:, :ch], self.conv_weight, None, conv_state, layout.query_start_loc,
                                                      layout.context_lens, layout.slot_idx, dt_in=a, dt_bias=self.dt_bias, a_log=self.a_log,
                                                      max_query_len=layout.max_query_len)
        q, k = qkv[:, :G * D].view(-1, G, D), qkv[:, G * D:2 * G * D].view(-1, G, D)
        args = (q, k, qkv[:, 2 * G * D:].view(-1, H, Dv), beta, log2_decay, S, layout.query_start_loc, layout.context_lens, layout.slot_idx,
                layout.max_query_len, D ** -0.5, UNIT_EPS)
        single = layout.max_query_len == 1 and h.shape[0] == layout.slot_idx.numel()
        if single and hip_ops.delta_rule_step_supported(D, Dv):
            y = hip_ops.delta_rule(*args, norm_weight=self.norm_weight, gate=gate, norm_eps=self.eps)
        else:
            y = hip_ops.gated_rms_norm(hip_ops.delta_rule(*args), gate, self.row_norm_weight, self.eps, groups=H, gate_act="silu")
        return self.o_proj(y)
