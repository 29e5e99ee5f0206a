"""Host side of the Nilevik family: configuration, registry, kernel sources, checkpoint names, and the oracle's own
consistency (no GPU)."""
import json
import math
import os

import pytest
import torch

from oracle.nilevik import (attention_config, delta_config, delta_rule_ref, nilevik_config, nilevik_random_weights, nilevik_ref,
                            penalised_sink_attention_ref, query_temperature_ref, short_conv_ref, sinusoid_ref, slope_ref)


def test_config_reads_every_size_and_constant():
    from vllm_hymeta.models.configuration_nilevik import DeltaSpec, GatedMlpSpec, KeyValueAttentionSpec, NilevikConfig
    raw = nilevik_config(vocab=90, width=60, eps=3e-6, side=10, layers=[
        ("attention", attention_config(heads=6, kv_heads=3, dim=10, window=21, coef=0.25, every=37, scale=0.3), None),
        ("delta", delta_config(heads=8, kv_heads=2, dim=12, vdim=20, conv=5), 44)])
    cfg = NilevikConfig(raw)
    assert (cfg.vocab_size, cfg.hidden_size, cfg.norm_eps, cfg.side_dim, cfg.num_hidden_layers) == (90, 60, 3e-6, 10, 2)
    a, d = cfg.layers[0].mixer, cfg.layers[1].mixer
    assert isinstance(a, KeyValueAttentionSpec) and (a.heads, a.kv_heads, a.dim, a.scale, a.window, a.temp_coef, a.temp_every) == (6, 3, 10, 0.3, 21, 0.25, 37)
    assert a.slopes() == [2.0 ** (-8 * (h + 1) / 6) for h in range(6)] and cfg.layers[0].mlp is None
    assert isinstance(d, DeltaSpec) and (d.heads, d.kv_heads, d.dim, d.vdim, d.conv, d.conv_channels) == (8, 2, 12, 20, 5, 2 * 2 * 12 + 8 * 20)
    assert isinstance(cfg.layers[1].mlp, GatedMlpSpec) and cfg.layers[1].mlp.ff == 44
    assert cfg.position_frequencies()[7] == 10000.0 ** (-14.0 / 60) and len(cfg.position_frequencies()) == 30
    # what a file may leave out
    bare = nilevik_config()
    del bare["layers"][1]["mixer"]["mask"], bare["layers"][1]["mixer"]["q_temp"], bare["layers"][1]["mixer"]["vdim"]
    m = NilevikConfig(bare).layers[1].mixer
    assert m.window is None and m.temp_coef == 0.0
    for breaker in (lambda c: c["layers"][0].update(type="lstm"), lambda c: c["layers"][1]["mixer"].update(kv_heads=4), lambda c: c["layers"][1]["mixer"].update(vdim=5),
                    lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0),
                    lambda c: c["layers"][0]["mlp"].update(kind="moe"), lambda c: c["layers"][0]["mixer"].update(conv=0)):
        bad = json.loads(json.dumps(nilevik_config()))
        breaker(bad)
        with pytest.raises(ValueError):
            NilevikConfig(bad)


def test_registry_serves_the_family(tmp_path):
    from vllm_hymeta import registry
    from vllm_hymeta.models.configuration_nilevik import NilevikConfig
    (tmp_path / "config.json").write_text(json.dumps(nilevik_config()))
    assert registry.architecture_of(str(tmp_path)) == "Nilevik" and "Nilevik" in registry.known_architectures()
    cls, cfg = registry.resolve(str(tmp_path))
    assert cls.__name__ == "NilevikForCausalLM" and isinstance(cfg, NilevikConfig)
    sources = registry.kernel_sources(str(tmp_path))
    assert tuple(sources) == tuple(cls.kernel_sources) and {"delta_rule", "sink_attn", "norm_conv"} <= set(sources)
    csrc = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "vllm-hymeta_amd", "csrc")
    assert all(os.path.exists(os.path.join(csrc, s + ".hip")) for s in sources)


def test_checkpoint_names_load_into_the_model_on_the_cpu():
    """Every tensor of the oracle's checkpoint is taken by name and shape; a missing or misshapen one is refused."""
    from vllm_hymeta.models.configuration_nilevik import NilevikConfig
    from vllm_hymeta.models.modeling_nilevik import NilevikForCausalLM
    cfg = nilevik_config()
    w = nilevik_random_weights(cfg, seed=2)

    def model():
        return NilevikForCausalLM(NilevikConfig(cfg), max_num_seqs=2, dtype=torch.float32, device="cpu")

    m = model()
    assert m.load_weights(w.items()) == set(w)
    assert sorted(m.model.attn_layers) == ["1", "2"] and m.model.attn_layers["1"].kv_cache_shape(7, 16)[:3] == (7, 16, 1)
    rec, conv = m.model.state_cache.cache
    assert [tuple(t.shape) for t in rec] == [(1, 2, 4, 16, 24), (1, 2, 3, 24, 16)] and [tuple(t.shape) for t in conv] == [(1, 2, 3, 160), (1, 2, 1, 192)]
    assert m.model.layers[2].mlp is None and m.model.layers[1].mlp is not None
    assert m.model.layers[3].side._table[0].data_ptr() == m.model.side_embed[:, 36:].data_ptr()
    for name in ("l1.mix.sink", "l0.mix.k.conv", "side.embed", "l3.side.norm"):
        short = {k: v for k, v in w.items() if k != name}
        with pytest.raises(KeyError):
            model().load_weights(short.items())
        with pytest.raises(ValueError):
            model().load_weights(dict(w, **{name: torch.zeros(7, 9)}).items())


def test_a_cache_row_holds_one_vector_and_one_factor_per_head():
    from vllm_hymeta import hip_ops
    assert hip_ops.scaled_key_row(4, 128, torch.bfloat16) * 2 == 4 * 128 * 2 + 16
    assert hip_ops.scaled_key_row(3, 5, torch.bfloat16) * 2 == 48        # 30 bytes of keys, the factors from byte 32 on
    assert hip_ops.scaled_key_row(1, 40, torch.float32) * 4 == 176


def test_sinusoid_temperature_slopes_and_sink_of_the_oracle():
    s = sinusoid_ref(4, 6)
    assert torch.equal(s[0], torch.tensor([0.0, 1.0, 0.0, 1.0, 0.0, 1.0], dtype=torch.float64))
    assert math.isclose(float(s[3, 2]), math.sin(3 * 10000 ** (-2 / 6))) and math.isclose(float(s[3, 3]), math.cos(3 * 10000 ** (-2 / 6)))
    t = query_temperature_ref(10, 0.5, 4)
    assert t[:3].tolist() == [1.0, 1.0, 1.0] and math.isclose(float(t[3]), 1 + 0.5 * math.log(2)) and math.isclose(float(t[7]), 1 + 0.5 * math.log(3))
    assert [slope_ref(h, 4) for h in range(4)] == [0.25, 0.0625, 0.015625, 0.00390625]
    # zero queries: the output counts the visible keys against the sink, which has no penalty
    T = 6
    q, k = torch.zeros(T, 1, 2, dtype=torch.float64), torch.zeros(T, 1, 2, dtype=torch.float64)
    v = torch.ones(T, 1, 1, dtype=torch.float64)
    o = penalised_sink_attention_ref(q, k, v, 1.0, 3, [0.0], torch.tensor([math.log(2.0)], dtype=torch.float64))
    assert torch.allclose(o[:, 0, 0], torch.tensor([1 / 3, 2 / 4, 3 / 5, 3 / 5, 3 / 5, 3 / 5], dtype=torch.float64))
    o = penalised_sink_attention_ref(q, k, v, 1.0, None, [math.log(2.0)], torch.tensor([0.0], dtype=torch.float64))
    assert torch.allclose(o[2, 0, 0], torch.tensor(1.75 / 2.75, dtype=torch.float64))
    # the last tap weighs the current token
    y = short_conv_ref(torch.tensor([[1.0], [10.0]], dtype=torch.float64), torch.tensor([[3.0, 2.0]], dtype=torch.float64))
    assert torch.allclose(y[:, 0], torch.nn.functional.silu(torch.tensor([2.0, 23.0], dtype=torch.float64)))
    # a full write replaces what the key held; the read-out sees it
    e = torch.eye(2, dtype=torch.float64)
    k2 = e[[0, 1, 0]].view(3, 1, 2)
    vals = torch.tensor([5.0, 7.0, 9.0], dtype=torch.float64).view(3, 1, 1)
    ones = torch.ones(3, 1, dtype=torch.float64)
    assert delta_rule_ref(k2, k2, vals, ones, ones)[:, 0, 0].tolist() == [5.0, 7.0, 9.0]
    q2 = e[[0, 0, 0]].view(3, 1, 2)
    assert delta_rule_ref(q2, k2, vals, ones, 0.5 * ones)[:, 0, 0].tolist() == [5.0, 2.5, 9.0]


def test_every_mechanism_shows_in_the_oracles_logits():
    cfg = nilevik_config()
    w = nilevik_random_weights(cfg, seed=1)
    toks = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(0)).tolist()
    ref = nilevik_ref(cfg, w, toks)

    def moved(cfg2=None, w2=None):
        out = nilevik_ref(cfg2 or cfg, w2 or w, toks)
        return float((out - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt())

    def changed(path, value):
        c = json.loads(json.dumps(cfg))
        node = c
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = value
        return c

    assert moved() == 0.0
    for path, value in ((("layers", 1, "mixer", "mask", "size"), 12), (("layers", 1, "mixer", "q_temp", "every"), 8), (("layers", 1, "mixer", "q_temp", "coef"), 0.2),
                        (("layers", 1, "mixer", "scale"), 0.5), (("norm", "eps"), 0.5)):
        assert moved(changed(path, value)) > 1e-4, path
    for name in ("l0.mix.A_log", "l0.mix.dt_bias", "l0.mix.b", "l0.mix.q.conv", "l0.mix.norm", "l0.mix.g", "l1.mix.sink", "l1.mix.k.norm", "l1.mix.q.norm", "l1.mix.g",
                 "l1.norm2", "l2.norm1", "l2.side.norm", "side.embed", "l1.mlp.up", "final.norm", "embed"):
        w2 = dict(w)
        w2[name] = w[name] + 0.5
        assert moved(w2=w2) > 1e-4, name
