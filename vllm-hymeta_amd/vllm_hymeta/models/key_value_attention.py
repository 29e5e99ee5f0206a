"""Causal softmax attention over a paged cache whose values are its keys: the projection ``k = W_k h`` is the value as it
stands and, after an RMS norm, the key.  No rotation; a penalty linear in the distance, a sink, a sliding window, a
temperature on the queries that grows with their position, an elementwise output gate:

    q_i = rms(W_q h_i) w_q (1 + coef ln(floor((i + 1) / every) + 1));   k_j = W_k h_j;   n_j = rms(k_j) w_k
    s_ij = scale q_i . n_j - slope_h (i - j),   0 <= i - j < window
    p_ij = exp(s_ij) / (exp(sink_h) + sum_j exp(s_ij));   out = W_o (concat_h(sum_j p_ij k_j) * sigmoid(W_g h))

``q . n_j = (q w_k) . k_j / rms(k_j)``: a cache row holds the projected key once per key/value head and its inverse root
mean square as an fp32 factor of the score (``hip_ops.KV_SCALED_KEY`` rows, half of what keys and values apart would take),
and ``w_k`` rides in the queries.  The queries' norm and the cache write are ``hip_ops.scaled_key_cache_``, the attention
with the gate in its epilogue ``hip_ops.sink_attention``.  ``PagedKeyValueAttention`` is the cache-owning object an engine
finds by name and binds a cache to (as ``PagedBiasAttention``, ``PagedWindowAttention``); ``KeyValueAttentionMixer`` is the
sublayer around it.
"""

from __future__ import annotations

from typing import List, Optional, Tuple

import torch

from .. import hip_ops
from ..linear import HymetaLinear
from . import attention as _registry


class PagedKeyValueAttention(torch.nn.Module):
    def __init__(self, num_heads: int, num_kv_heads: int, head_dim: int, scale: float, prefix: str, slopes: Optional[torch.Tensor] = None,
                 sink_logits: Optional[torch.Tensor] = None, sliding_window: Optional[int] = None, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.num_heads, self.num_kv_heads, self.head_size, self.v_size = num_heads, num_kv_heads, head_dim, head_dim
        self.scale, self.dtype = float(scale), dtype
        self.window_left = -1 if sliding_window is None else sliding_window - 1
        self.register_buffer("slopes", None if slopes is None else slopes.float().contiguous())
        self.register_buffer("sink_logits", None if sink_logits is None else sink_logits.float().contiguous())
        if prefix in _registry._LAYERS:
            raise ValueError(f"Duplicate layer name: {prefix}")
        _registry._LAYERS[prefix] = self
        self.layer_name = prefix
        self.kv_cache: List[torch.Tensor] = [torch.tensor([])]

    def kv_cache_shape(self, num_blocks: int, block_size: int) -> Tuple[int, ...]:
        return (num_blocks, block_size, 1, hip_ops.scaled_key_row(self.num_kv_heads, self.head_size, self.dtype))

    def cache(self) -> torch.Tensor:
        kv = self.kv_cache[0]
        if kv.numel() == 0:
            raise RuntimeError(f"{self.layer_name}: no KV cache bound")
        return kv

    def forward(self, q: torch.Tensor, layout, gate: Optional[torch.Tensor] = None) -> torch.Tensor:
        """``q [T, H, D]`` against the cached rows (this step's are stored already) -> ``[T, H, D]``; ``gate [T, H D]``."""
        return hip_ops.sink_attention(q, self.cache(), layout.block_tables, layout.query_start_loc, layout.seq_lens, self.num_kv_heads,
                                      self.head_size, self.head_size, self.scale, layout.max_query_len, layout.max_seq_len,
                                      sink=self.sink_logits is not None, sink_logits=self.sink_logits, window_left=self.window_left,
                                      scaled_key=True, slopes=self.slopes, elem_gate=gate)


class KeyValueAttentionMixer(torch.nn.Module):
    def __init__(self, in_proj: HymetaLinear, o_proj: HymetaLinear, attn: PagedKeyValueAttention, q_norm_weight: torch.Tensor,
                 k_norm_weight: torch.Tensor, eps: float, temp_coef: float = 0.0, temp_every: float = 1.0, gated: bool = True):
        """``in_proj``: rows = queries, keys and (``gated``) the output gate (``H D``)."""
        super().__init__()
        self.in_proj, self.o_proj, self.eps, self.gated = in_proj, o_proj, float(eps), bool(gated)
        self.temp_coef, self.temp_every = float(temp_coef), float(temp_every)
        self.register_buffer("q_norm_weight", q_norm_weight.float().contiguous())
        self.register_buffer("k_norm_weight", k_norm_weight.float().contiguous())
        self._attn = (attn,)          # owned (and registered as a module) by the model

    def forward(self, h: torch.Tensor, layout, attn: Optional[PagedKeyValueAttention] = None) -> torch.Tensor:
        attn = attn or self._attn[0]
        H, G, D = attn.num_heads, attn.num_kv_heads, attn.head_size
        proj = self.in_proj(h)
        hip_ops.scaled_key_cache_(proj, H, G, D, self.q_norm_weight, self.k_norm_weight, self.eps, attn.cache(), layout.slot_mapping,
                                  self.temp_coef, self.temp_every, layout.positions)
        gate = proj[:, (H + G) * D:(2 * H + G) * D] if self.gated else None
        o = attn(proj[:, :H * D].view(-1, H, D), layout, gate)
        return self.o_proj(o.view(-1, H * D))
