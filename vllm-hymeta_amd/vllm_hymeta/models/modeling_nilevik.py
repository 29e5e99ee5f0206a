"""The Nilevik decoder: a token embedding plus a sinusoidal vector of the position on an fp32 residual stream; layers that
read the stream itself and norm what they add (``AddedNormBlock``): a mixer, a tanh-gelu gated feed-forward or none, and an
input of the layer's own from the token (a gated row of a second table).  Mixers: a windowed softmax attention whose values
are its unnormed keys (``key_value_attention.py``) or a gated delta rule (``delta_rule.py``).  The embedding table is the
output projection.

The class has the surface of the package's other model classes (``GLAswaForCausalLM``, ``SonuzenForCausalLM``,
``GeponexForCausalLM``, ``LidizenForCausalLM``, ``DapuzenForCausalLM``): ``forward(input_ids, positions, attn_metadata=...,
request_ids_to_seq_ids=..., finished_requests_ids=...)`` returns the final hidden states of the step's rows,
``compute_logits`` the fp32 logits of the rows asked for, ``load_weights`` takes the checkpoint as a stream of named
tensors; the attention layers are found by name and bound to paged caches by whoever drives the model, the recurrent and
convolution states live in a slot-indexed cache that follows the requests' ids.
"""

from __future__ import annotations

from typing import Dict, Iterable, List, Optional, Set, Tuple

import torch

from .. import hip_ops
from .._compat import HasInnerState, IsHybrid
from ..linear import HymetaLinear
from ..lm_head import lm_head_logits
from ..state_cache import ConstantSizeStateCache
from .added_norm_block import AddedNormBlock, AddNormed, TokenInput
from .attention import bind_kv_cache, current_attn_metadata, standalone_prefix
from .configuration_nilevik import DeltaSpec, KeyValueAttentionSpec, NilevikConfig
from .delta_rule import DeltaRuleMixer
from .feed_forward import GeluGluMLP
from .key_value_attention import KeyValueAttentionMixer, PagedKeyValueAttention
from .stream_block import NormConvIn, StepLayout


class NilevikStateCache(ConstantSizeStateCache):
    """Per delta layer the fp32 state ``[1, slots, heads, D, Dv]`` and its convolution's last inputs ``[1, slots, taps - 1,
    channels]`` in the activations' type.  A slot needs no clearing when it changes hands: a sequence's first step does not
    read it."""

    def __init__(self, specs: List[DeltaSpec], act_dtype: torch.dtype, max_batch_size: int, device):
        super().__init__(max_batch_size, device)
        self.recurrent = [torch.zeros(1, max_batch_size, m.heads, m.dim, m.vdim, dtype=torch.float32, device=self.device) for m in specs]
        self.conv = [torch.zeros(1, max_batch_size, max(m.conv - 1, 1), m.conv_channels, dtype=act_dtype, device=self.device) for m in specs]

    @property
    def cache(self):
        return (self.recurrent, self.conv)

    def _slot_tensors(self):
        return tuple(self.recurrent) + tuple(self.conv)


class NilevikModel(torch.nn.Module):
    def __init__(self, config: NilevikConfig, max_num_seqs: int = 256, dtype: torch.dtype = torch.bfloat16, device="cuda",
                 prefix: Optional[str] = None):
        super().__init__()
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Nilevik runs in bfloat16 or float32")
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.prefix = standalone_prefix("model") if prefix is None else prefix
        # the cache-owning attention layers exist from construction on (an engine sizes its pages from them)
        self.attn_layers = torch.nn.ModuleDict()
        self._state_index: Dict[int, int] = {}
        for i, spec in enumerate(config.layers):
            m = spec.mixer
            if isinstance(m, KeyValueAttentionSpec):
                self.attn_layers[str(i)] = PagedKeyValueAttention(m.heads, m.kv_heads, m.dim, m.scale, f"{self.prefix}.layers.{i}.attn",
                                                                  slopes=torch.tensor(m.slopes(), dtype=torch.float32, device=self.device),
                                                                  sliding_window=m.window, dtype=dtype)
            else:
                self._state_index[i] = len(self._state_index)
        self.state_cache = NilevikStateCache([config.layers[i].mixer for i in self._state_index], dtype, max_num_seqs, self.device)
        self.register_buffer("pos_freqs", torch.tensor(config.position_frequencies(), dtype=torch.float64, device=self.device))
        self.embed: Optional[torch.Tensor] = None
        self.side_embed: Optional[torch.Tensor] = None
        self.final_norm: Optional[NormConvIn] = None
        self.layers = torch.nn.ModuleList()

    def layout_of(self, attn_metadata, slot_idx: torch.Tensor, token_ids: torch.Tensor, positions: Optional[torch.Tensor]) -> StepLayout:
        md = attn_metadata
        max_seq = max(md.seq_lens) if md.seq_lens else max(md.max_prefill_seq_len, md.max_decode_seq_len)
        if positions is None:                  # every row's place in its sequence
            starts = md.query_start_loc.to(torch.int64)
            lens = starts[1:] - starts[:-1]
            first = md.context_lens_tensor.to(torch.int64) - starts[:-1]
            positions = torch.arange(token_ids.numel(), device=token_ids.device) + torch.repeat_interleave(first, lens, output_size=token_ids.numel())
        return StepLayout(query_start_loc=md.query_start_loc, context_lens=md.context_lens_tensor, seq_lens=md.seq_lens_tensor,
                          slot_idx=slot_idx, block_tables=md.block_tables, slot_mapping=md.slot_mapping,
                          max_query_len=int(md.max_query_len or 1), max_seq_len=int(max_seq), token_ids=token_ids, positions=positions)

    def forward(self, input_ids: torch.Tensor, positions: Optional[torch.Tensor] = None, attn_metadata=None,
                kv_caches: Optional[List[torch.Tensor]] = None, residual_out: Optional[List[torch.Tensor]] = None,
                **kwargs) -> torch.Tensor:
        """``positions``: int64, one per row (None: the rows' places in their sequences).  ``kv_caches``: one page tensor per
        attention layer, in layer order, bound before the step (callers without an engine).  ``residual_out``: a list that
        receives a copy of the stream after every layer (debugging)."""
        if kv_caches is not None:
            for layer, kv in zip(self.attn_layers.values(), kv_caches):
                bind_kv_cache(layer, kv)
        md = attn_metadata if attn_metadata is not None else current_attn_metadata()
        if md is None:
            raise RuntimeError("NilevikModel.forward needs the step's attention metadata")
        kwargs.setdefault("request_ids_to_seq_ids", {})
        kwargs.setdefault("finished_requests_ids", [])
        (recurrent, conv), slot_idx = self.state_cache.current_run_tensors(**kwargs)
        input_ids = input_ids.to(torch.int64).contiguous()
        if positions is not None:
            positions = positions.to(torch.int64).contiguous()
        layout = self.layout_of(md, slot_idx, input_ids, positions)
        copy = self.dtype != torch.float32            # sublayers read the stream itself, or its copy in the activations' type
        rows = hip_ops.embed_rows(input_ids, self.embed, positions=layout.positions, pos_freqs=self.pos_freqs, copy=copy)
        x, h = rows if copy else (rows, rows)
        for i, block in enumerate(self.layers):
            if i in self._state_index:
                k = self._state_index[i]
                state = (recurrent[k][0], conv[k][0])
            else:
                state = self.attn_layers[str(i)]
            h = block(x, h, layout, state)
            if residual_out is not None:
                residual_out.append(x.clone())
        return self.final_norm(x, self.dtype)


class NilevikForCausalLM(torch.nn.Module, HasInnerState, IsHybrid):
    # csrc/*.hip sources whose kernels this class calls (a first run in a fresh checkout builds these, see _C.build_library)
    kernel_sources = ("api_misc", "norm_conv", "parallel_ops", "lightning", "sink_attn", "delta_rule", "gated_ops", "glue",
                      "dense_gemm", "stream_gemm", "tall_gemm")

    def __init__(self, config: Optional[NilevikConfig] = None, max_num_seqs: int = 256, dtype: torch.dtype = torch.bfloat16,
                 device="cuda", *, vllm_config=None, prefix: Optional[str] = None):
        super().__init__()
        if vllm_config is not None:
            mc = vllm_config.model_config
            config = mc.hf_config if isinstance(mc.hf_config, NilevikConfig) else NilevikConfig(mc.hf_config.to_dict())
            max_num_seqs = int(vllm_config.scheduler_config.max_num_seqs)
            dtype = getattr(mc, "dtype", dtype)
            device = getattr(getattr(vllm_config, "device_config", None), "device", None) or device
            prefix = f"{prefix}.model" if prefix else "model"
        if config is None:
            raise TypeError("NilevikForCausalLM needs vllm_config= or a NilevikConfig")
        self.config = config
        self.model = NilevikModel(config, max_num_seqs=max_num_seqs, dtype=dtype, device=device, prefix=prefix)

    # what an engine asks a model with states of its own (the package's other model classes answer the same calls)
    def copy_inputs_before_cuda_graphs(self, input_buffers, **kwargs):
        return self.model.state_cache.copy_inputs_before_cuda_graphs(input_buffers, **kwargs)

    def get_seqlen_agnostic_capture_inputs(self, batch_size: int):
        return self.model.state_cache.get_seqlen_agnostic_capture_inputs(batch_size)

    def forward(self, input_ids, positions=None, intermediate_tensors=None, inputs_embeds=None, **kwargs):
        return self.model(input_ids, positions, **kwargs)

    def compute_logits(self, hidden_states: torch.Tensor, sampling_metadata=None) -> torch.Tensor:
        idx = getattr(sampling_metadata, "selected_token_indices", None)
        if idx is not None:
            hidden_states = hidden_states.index_select(0, idx)
        return lm_head_logits(hidden_states, self.model.embed)

    # ------------------------------------------------------------------ weights
    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> Set[str]:
        """Checkpoint names: ``embed``, ``side.embed``, ``final.norm``, and per layer ``l<i>.norm1`` (``norm2`` with a
        feed-forward); ``l<i>.mix.<q|k|g|o|q.norm|k.norm|sink>`` (attention) or ``l<i>.mix.<q|k|v>`` with ``.conv``,
        ``l<i>.mix.<b|a|g|o|A_log|dt_bias|norm>`` (delta); ``l<i>.mlp.<gate|up|down>``; ``l<i>.side.<gate|proj|norm>``.
        Linear weights ``[out, in]``."""
        cfg, m = self.config, self.model
        dev, dt = m.device, m.dtype
        got: Dict[str, torch.Tensor] = dict(weights)
        loaded: Set[str] = set()

        def take(name: str, shape: Tuple[int, ...]) -> torch.Tensor:
            if name not in got:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            loaded.add(name)
            if tuple(got[name].shape) != tuple(shape):
                raise ValueError(f"{name} is {tuple(got[name].shape)}, the configuration says {tuple(shape)}")
            return got[name]

        def act(name: str, shape) -> torch.Tensor:
            return take(name, shape).to(device=dev, dtype=dt).contiguous()

        def f32(name: str, shape) -> torch.Tensor:
            return take(name, shape).to(device=dev, dtype=torch.float32).contiguous()

        def linear(*parts: torch.Tensor, pad: bool = False) -> HymetaLinear:
            rows = list(parts)
            # zero rows keep the projection's row a whole number of 16 bytes, which the kernels that read slices of it in
            # 16-byte pieces ask of its stride
            short = -sum(r.shape[0] for r in rows) % 8
            if pad and short:
                rows.append(torch.zeros(short, rows[0].shape[1], dtype=dt, device=dev))
            return HymetaLinear.from_weight(rows[0] if len(rows) == 1 else torch.cat(rows, 0).contiguous())

        W, eps = cfg.hidden_size, cfg.norm_eps
        m.embed = act("embed", (cfg.vocab_size, W))
        if cfg.side_dim:
            m.side_embed = act("side.embed", (cfg.vocab_size, cfg.num_hidden_layers * cfg.side_dim))
        m.final_norm = NormConvIn(f32("final.norm", (W,)), eps, weight_offset=0.0)
        m.layers = torch.nn.ModuleList()
        for i, spec in enumerate(cfg.layers):
            p, a = f"l{i}.", spec.mixer
            H, G, D = a.heads, a.kv_heads, a.dim
            if isinstance(a, KeyValueAttentionSpec):
                attn = m.attn_layers[str(i)]
                attn.sink_logits = f32(p + "mix.sink", (H,))
                in_proj = linear(act(p + "mix.q", (H * D, W)), act(p + "mix.k", (G * D, W)), act(p + "mix.g", (H * D, W)), pad=True)
                mixer = KeyValueAttentionMixer(in_proj, linear(act(p + "mix.o", (W, H * D))), attn, f32(p + "mix.q.norm", (D,)),
                                               f32(p + "mix.k.norm", (D,)), eps, a.temp_coef, a.temp_every)
            else:
                assert isinstance(a, DeltaSpec)
                Dv, qk = a.vdim, G * D
                in_proj = linear(act(p + "mix.q", (qk, W)), act(p + "mix.k", (qk, W)), act(p + "mix.v", (H * Dv, W)), act(p + "mix.g", (H * Dv, W)),
                                 act(p + "mix.b", (H, W)), act(p + "mix.a", (H, W)), pad=True)
                conv = torch.cat([f32(p + "mix.q.conv", (qk, a.conv)), f32(p + "mix.k.conv", (qk, a.conv)), f32(p + "mix.v.conv", (H * Dv, a.conv))], 0)
                mixer = DeltaRuleMixer(in_proj, linear(act(p + "mix.o", (W, H * Dv))), H, G, D, Dv, conv, f32(p + "mix.A_log", (H,)),
                                       f32(p + "mix.dt_bias", (H,)), f32(p + "mix.norm", (Dv,)), eps)
            mlp = mlp_add = side = side_add = None
            if spec.mlp is not None:
                ff = spec.mlp.ff
                mlp = GeluGluMLP(linear(act(p + "mlp.gate", (ff, W)), act(p + "mlp.up", (ff, W))), linear(act(p + "mlp.down", (W, ff))))
                mlp_add = AddNormed(f32(p + "norm2", (W,)), eps)
            if cfg.side_dim:
                d = cfg.side_dim
                side = TokenInput(linear(act(p + "side.gate", (d, W))), linear(act(p + "side.proj", (W, d))), m.side_embed[:, i * d:(i + 1) * d])
                side_add = AddNormed(f32(p + "side.norm", (W,)), eps)
            m.layers.append(AddedNormBlock(mixer, AddNormed(f32(p + "norm1", (W,)), eps), mlp, mlp_add, side, side_add))
        return loaded
