"""The Banitar decoder: a scaled token embedding on an fp32 residual stream; layers with a squashing norm on both sides of
every sublayer (``SquashBlock``): a mixer and a silu-gated feed-forward or none.  Mixers: an attention within chunks of the
sequence (biased projections, interleaved rotation with YaRN frequencies, queries and keys of unit root mean square, a gate
per head: ``rotary_window_attention.py``) or a windowed latent attention with a sink (``latent_attention.py``).  A run of layers
is repeated with the same weights; every pass is entered through a linear map of the stream beside the embedding output and
has caches of its own.  The output projection is a tensor of its own.

The class has the surface of the package's other model classes (``GLAswaForCausalLM``, ``SonuzenForCausalLM``,
``GeponexForCausalLM``, ``LidizenForCausalLM``, ``DapuzenForCausalLM``, ``NilevikForCausalLM``): ``forward(input_ids, positions,
attn_metadata=...)`` returns the final hidden states of the step's rows, ``compute_logits`` the fp32 logits of the rows asked
for, ``load_weights`` takes the checkpoint as a stream of named tensors; the attention layers are found by name and bound to
paged caches by whoever drives the model.  All of a sequence's past lies in those pages: there is no state cache, and the
request ids that an engine passes for one are not read.
"""

from __future__ import annotations

from typing import Dict, Iterable, List, Optional, Set, Tuple

import torch

from .. import hip_ops
from ..linear import HymetaLinear
from ..lm_head import lm_head_logits
from .attention import bind_kv_cache, current_attn_metadata, standalone_prefix
from .configuration_banitar import BanitarConfig, ChunkedAttentionSpec, WindowedLatentSpec
from .feed_forward import SiluGluMLP
from .latent_attention import LatentAttentionMixer, PagedLatentAttention
from .rotary_window_attention import PagedWindowAttention, WindowAttentionMixer
from .squash_block import PassEntry, SquashBlock, TanhNorm
from .stream_block import StepLayout


class BanitarModel(torch.nn.Module):
    def __init__(self, config: BanitarConfig, dtype: torch.dtype = torch.bfloat16, device="cuda", prefix: Optional[str] = None):
        super().__init__()
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Banitar runs in bfloat16 or float32")
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.prefix = standalone_prefix("model") if prefix is None else prefix
        self.runs: List[Tuple[int, int]] = config.layer_runs()
        # the cache-owning attention layers exist from construction on (an engine sizes its pages from them); a layer inside
        # the loop has one per pass
        self.attn_layers = torch.nn.ModuleDict()
        for (i, t) in self.runs:
            m, name = config.layers[i].mixer, f"{self.prefix}.layers.{i}.pass{t}.attn"
            if isinstance(m, ChunkedAttentionSpec):
                attn = PagedWindowAttention(m.heads, m.kv_heads, m.dim, m.vdim, m.scale, name, dtype=dtype, chunk=m.chunk)
            else:
                attn = PagedLatentAttention(m.heads, m.kv_rank, m.rot_dim, m.scale, name, dtype=dtype, sliding_window=m.window)
            self.attn_layers[f"{i}_{t}"] = attn
        self.embed: Optional[torch.Tensor] = None
        self.layers = torch.nn.ModuleList()
        self.entry: Optional[PassEntry] = None
        self.final_norm: Optional[TanhNorm] = None

    def layout_of(self, attn_metadata, token_ids: torch.Tensor, positions: Optional[torch.Tensor]) -> StepLayout:
        md = attn_metadata
        max_seq = max(md.seq_lens) if md.seq_lens else max(md.max_prefill_seq_len, md.max_decode_seq_len)
        return StepLayout(query_start_loc=md.query_start_loc, context_lens=md.context_lens_tensor, seq_lens=md.seq_lens_tensor,
                          slot_idx=None, block_tables=md.block_tables, slot_mapping=md.slot_mapping,
                          max_query_len=int(md.max_query_len or 1), max_seq_len=int(max_seq), token_ids=token_ids, positions=positions)

    def _read_after(self, n: int) -> Optional[TanhNorm]:
        """How the stream is read after run ``n``: by the next layer's norm, by the last norm, or (None) as it is, where the next
        run enters a pass."""
        if n + 1 >= len(self.runs):
            return self.final_norm
        run = self.runs[n + 1]
        return None if self.config.enters_pass(run) else self.layers[run[0]].mixer_in

    def forward(self, input_ids: torch.Tensor, positions: Optional[torch.Tensor] = None, attn_metadata=None,
                kv_caches: Optional[List[torch.Tensor]] = None, residual_out: Optional[List[torch.Tensor]] = None,
                **kwargs) -> torch.Tensor:
        """``positions``: int64, one per row (None: the rows' places in their sequences).  ``kv_caches``: one page tensor per
        attention layer and pass, in execution order, bound before the step (callers without an engine).  ``residual_out``: a
        list that receives a copy of the stream after every layer run (debugging)."""
        if kv_caches is not None:
            for layer, kv in zip(self.attn_layers.values(), kv_caches):
                bind_kv_cache(layer, kv)
        md = attn_metadata if attn_metadata is not None else current_attn_metadata()
        if md is None:
            raise RuntimeError("BanitarModel.forward needs the step's attention metadata")
        input_ids = input_ids.to(torch.int64).contiguous()
        if positions is not None:
            positions = positions.to(torch.int64).contiguous()
        layout = self.layout_of(md, input_ids, positions)
        cfg, act = self.config, self.dtype
        copy = cfg.has_loop and act != torch.float32        # the embedding output as activations: the pass entry reads it
        rows = hip_ops.embed_rows(input_ids, self.embed, scale=cfg.embed_scale, copy=copy)
        x, h0 = rows if copy else (rows, rows)
        start = self.entry.start_part(h0) if cfg.has_loop else None
        h = h0 if cfg.enters_pass(self.runs[0]) else self.layers[self.runs[0][0]].mixer_in(x, act)
        for n, (i, t) in enumerate(self.runs):
            block = self.layers[i]
            if cfg.enters_pass((i, t)):
                h = self.entry(x, h, start, t, block.mixer_in, act)
            h = block(x, h, layout, self.attn_layers[f"{i}_{t}"], self._read_after(n))
            if residual_out is not None:
                residual_out.append(x.clone())
        return h


class BanitarForCausalLM(torch.nn.Module):
    # csrc/*.hip sources whose kernels this class calls (a first run in a fresh checkout builds these, see _C.build_library)
    kernel_sources = ("api_misc", "norm_conv", "tanh_norm", "parallel_ops", "latent_attn", "sink_attn", "gated_ops", "glue",
                      "dense_gemm", "stream_gemm", "tall_gemm")

    def __init__(self, config: Optional[BanitarConfig] = None, max_num_seqs: int = 256, dtype: torch.dtype = torch.bfloat16,
                 device="cuda", *, vllm_config=None, prefix: Optional[str] = None):
        """``max_num_seqs``: not read (the family carries no state per sequence beside its pages)."""
        super().__init__()
        if vllm_config is not None:
            mc = vllm_config.model_config
            config = mc.hf_config if isinstance(mc.hf_config, BanitarConfig) else BanitarConfig(mc.hf_config.to_dict())
            dtype = getattr(mc, "dtype", dtype)
            device = getattr(getattr(vllm_config, "device_config", None), "device", None) or device
            prefix = f"{prefix}.model" if prefix else "model"
        if config is None:
            raise TypeError("BanitarForCausalLM needs vllm_config= or a BanitarConfig")
        self.config = config
        self.model = BanitarModel(config, dtype=dtype, device=device, prefix=prefix)
        self.lm_head: Optional[torch.Tensor] = None

    def forward(self, input_ids, positions=None, intermediate_tensors=None, inputs_embeds=None, **kwargs):
        return self.model(input_ids, positions, **kwargs)

    def compute_logits(self, hidden_states: torch.Tensor, sampling_metadata=None) -> torch.Tensor:
        idx = getattr(sampling_metadata, "selected_token_indices", None)
        if idx is not None:
            hidden_states = hidden_states.index_select(0, idx)
        return lm_head_logits(hidden_states, self.lm_head)

    # ------------------------------------------------------------------ weights
    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> Set[str]:
        """Checkpoint names: ``embed``, ``head``, ``final.norm``, with a loop ``loop.in`` and ``loop.step``, and per layer ``l<i>.norm1``
        and ``norm1b`` (``norm2`` and ``norm2b`` with a feed-forward), every norm with ``.b`` and ``.alpha``; ``l<i>.mix.<q|k|v>`` with
        ``.b``, ``l<i>.mix.<g|o>`` (attention) or ``l<i>.mix.<q|dkv|dkv.norm|uk|uv|sink|o>`` (latent attention);
        ``l<i>.mlp.<gate|up|down>``.  Linear weights ``[out, in]``."""
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

        def act(name: str, *shape: int) -> torch.Tensor:
            return take(name, shape).to(device=dev, dtype=dt).contiguous()

        def f32(name: str, *shape: int) -> torch.Tensor:
            return take(name, shape).to(device=dev, dtype=torch.float32).contiguous()

        def linear(*parts: torch.Tensor, bias: Tuple[torch.Tensor, ...] = (), pad: bool = False) -> HymetaLinear:
            """``bias``: of the leading parts (the rest have none).  ``pad``: zero rows behind, up to whole 64s -- what the
            weight-streaming kernels of decode-sized batches take, and rows of whole 16 bytes for whoever reads slices."""
            rows = list(parts)
            short = -sum(r.shape[0] for r in rows) % 64
            if pad and short:
                rows.append(torch.zeros(short, rows[0].shape[1], dtype=dt, device=dev))
            b = None
            if bias:
                left = sum(r.shape[0] for r in rows) - sum(v.numel() for v in bias)
                b = torch.cat([*bias, torch.zeros(left, dtype=dt, device=dev)]).contiguous()
            return HymetaLinear.from_weight(rows[0] if len(rows) == 1 else torch.cat(rows, 0).contiguous(), b)

        W, eps = cfg.hidden_size, cfg.norm_eps

        def norm(name: str) -> TanhNorm:
            return TanhNorm(float(take(name + ".alpha", ())), f32(name, W), f32(name + ".b", W))

        m.embed = act("embed", cfg.vocab_size, W)
        self.lm_head = act("head", cfg.vocab_size, W)
        m.final_norm = norm("final.norm")
        if cfg.has_loop:
            w_in = act("loop.in", W, 2 * W)
            m.entry = PassEntry(w_in[:, :W], w_in[:, W:], f32("loop.step", cfg.loop_times, W))
        m.layers = torch.nn.ModuleList()
        for i, spec in enumerate(cfg.layers):
            p, a = f"l{i}.", spec.mixer
            H, D, Dv = a.heads, a.dim, a.vdim
            passes = [m.attn_layers[f"{j}_{t}"] for (j, t) in m.runs if j == i]
            freqs, mag = a.rot.frequencies()
            freqs = torch.tensor(freqs, dtype=torch.float64, device=dev)
            if isinstance(a, ChunkedAttentionSpec):
                G = a.kv_heads
                in_proj = linear(act(p + "mix.q", H * D, W), act(p + "mix.k", G * D, W), act(p + "mix.v", G * Dv, W), act(p + "mix.g", H, W), pad=True,
                                 bias=(act(p + "mix.q.b", H * D), act(p + "mix.k.b", G * D), act(p + "mix.v.b", G * Dv)))
                mixer = WindowAttentionMixer(in_proj, linear(act(p + "mix.o", W, H * Dv)), passes[0], a.rot.dims, freqs, True, interleaved=True,
                                             rot_mag=mag, unit_eps=eps)
            else:
                assert isinstance(a, WindowedLatentSpec)
                C, R = a.kv_rank, a.rot_dim
                sink = f32(p + "mix.sink", H)
                for attn in passes:               # every pass's cache owner gets the heads' constants
                    attn.sink_logits = sink
                mixer = LatentAttentionMixer(
                    linear(act(p + "mix.q", H * (D + R), W), act(p + "mix.dkv", C + R, W), pad=True), None, act(p + "mix.uk", H * D, C).view(H, D, C),
                    act(p + "mix.uv", H * Dv, C).view(H, Dv, C).transpose(1, 2).contiguous(), linear(act(p + "mix.o", W, H * Dv)), passes[0],
                    H, D, R, Dv, C, 0, None, f32(p + "mix.dkv.norm", C), eps, a.rot.dims, freqs, mag, gate=False, rot_half=True)
            mlp = mlp_in = mlp_out = None
            if spec.mlp is not None:
                ff = spec.mlp.ff
                mlp = SiluGluMLP(linear(act(p + "mlp.gate", ff, W), act(p + "mlp.up", ff, W)), linear(act(p + "mlp.down", W, ff)))
                mlp_in, mlp_out = norm(p + "norm2"), norm(p + "norm2b")
            m.layers.append(SquashBlock(norm(p + "norm1"), mixer, norm(p + "norm1b"), mlp_in, mlp, mlp_out))
        return loaded
