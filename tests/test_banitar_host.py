"""Host side of the Banitar family: configuration, registry, kernel sources, checkpoint names, and the oracle's own
consistency (no GPU)."""
import json
import math
import os

import pytest
import torch

from oracle.banitar import (attend_ref, banitar_config, banitar_random_weights, banitar_ref, chunked_config, in_chunk, in_window, latent_config,
                            layer_runs_ref, rotate_ref, rotation_frequencies_ref, tanh_norm_ref)


def test_config_reads_every_size_and_constant():
    from vllm_hymeta.models.configuration_banitar import BanitarConfig, ChunkedAttentionSpec, WindowedLatentSpec
    raw = banitar_config(vocab=90, width=60, eps=3e-6, embed_scale=7.5, loop=(1, 2, 5), layers=[
        ("attention", chunked_config(heads=6, kv_heads=3, dim=10, vdim=14, chunk=21, rot_dims=6, base=300.0, scale=0.3), None),
        ("latent_attention", latent_config(heads=8, dim=12, rot_dim=6, vdim=20, kv_rank=34, window=9, base=77.0, scale=0.2), 44)])
    cfg = BanitarConfig(raw)
    assert (cfg.vocab_size, cfg.hidden_size, cfg.norm_eps, cfg.embed_scale, cfg.num_hidden_layers) == (90, 60, 3e-6, 7.5, 2)
    a, m = cfg.layers[0].mixer, cfg.layers[1].mixer
    assert isinstance(a, ChunkedAttentionSpec) and (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.chunk, a.rot.dims, a.rot.base) == (6, 3, 10, 14, 0.3, 21, 6, 300.0)
    assert isinstance(m, WindowedLatentSpec) and (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale, m.window, m.rot.dims, m.rot.base) == (8, 12, 6, 20, 34, 0.2, 9, 6, 77.0)
    assert cfg.layers[0].mlp is None and cfg.layers[1].mlp.ff == 44
    assert cfg.layer_runs() == [(0, 0)] + [(1, t) for t in range(5)] and [cfg.enters_pass(r) for r in cfg.layer_runs()] == [False] + [True] * 5
    for breaker in (lambda c: c["layers"][0].update(type="lstm"), lambda c: c["layers"][0]["mixer"].update(kv_heads=4), lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
                    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), lambda c: c["layers"][1]["mixer"]["rot"].update(dims=14), lambda c: c["layers"][0]["mlp"].update(kind="moe"),
                    lambda c: c["loop"].update(stop=9), lambda c: c["loop"].update(stop=1), lambda c: c["loop"].update(times=0)):
        bad = json.loads(json.dumps(banitar_config()))
        breaker(bad)
        with pytest.raises(ValueError):
            BanitarConfig(bad)


@pytest.mark.parametrize("loop", [None, (0, 4, 2), (0, 1, 3), (3, 4, 2), (1, 3, 1), (1, 3, 4)])
def test_order_of_layer_runs(loop):
    from vllm_hymeta.models.configuration_banitar import BanitarConfig
    raw = banitar_config(loop=loop)
    cfg = BanitarConfig(raw)
    assert [(i, t, cfg.enters_pass((i, t))) for i, t in cfg.layer_runs()] == layer_runs_ref(raw)


def test_rotation_frequencies_plain_and_scaled_match_the_oracle():
    from vllm_hymeta.models.configuration_banitar import BanitarConfig
    for dims, base, scaling in ((16, 900.0, None), (16, 900.0, {"factor": 5.0, "original": 64, "fast": 4.0, "slow": 1.0}), (2, 10.0, {"factor": 3.0, "original": 9, "fast": 1.0, "slow": 1.0}),
                                (64, 1e6, {"factor": 32.0, "original": 4096, "fast": 32.0, "slow": 1.0})):
        cfg = BanitarConfig(banitar_config(loop=None, layers=[("attention", chunked_config(dim=80, rot_dims=dims, base=base, scaling=scaling), None)]))
        got, mag = cfg.layers[0].mixer.rot.frequencies()
        want, want_mag = rotation_frequencies_ref(dims, base, scaling)
        assert len(got) == dims // 2 and all(math.isclose(a, b, rel_tol=1e-12) for a, b in zip(got, want)) and math.isclose(mag, want_mag)


def test_registry_serves_the_family(tmp_path):
    from vllm_hymeta import registry
    from vllm_hymeta.models.configuration_banitar import BanitarConfig
    (tmp_path / "config.json").write_text(json.dumps(banitar_config()))
    assert registry.architecture_of(str(tmp_path)) == "Banitar" and "Banitar" in registry.known_architectures()
    cls, cfg = registry.resolve(str(tmp_path))
    assert cls.__name__ == "BanitarForCausalLM" and isinstance(cfg, BanitarConfig)
    sources = registry.kernel_sources(str(tmp_path))
    assert tuple(sources) == tuple(cls.kernel_sources) and {"tanh_norm", "sink_attn", "latent_attn", "parallel_ops"} <= set(sources)
    csrc = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "vllm-hymeta_amd", "csrc")
    assert all(os.path.exists(os.path.join(csrc, s + ".hip")) for s in sources)


def test_checkpoint_names_load_into_the_model_on_the_cpu():
    """Every tensor of the oracle's checkpoint is taken by name and shape; a missing or misshapen one is refused."""
    from vllm_hymeta.models.configuration_banitar import BanitarConfig
    from vllm_hymeta.models.modeling_banitar import BanitarForCausalLM
    cfg = banitar_config()
    w = banitar_random_weights(cfg, seed=2)

    def model():
        return BanitarForCausalLM(BanitarConfig(cfg), dtype=torch.float32, device="cpu")

    m = model()
    assert m.load_weights(w.items()) == set(w)
    assert list(m.model.attn_layers) == ["0_0", "1_0", "2_0", "1_1", "2_1", "1_2", "2_2", "3_0"]
    assert m.model.attn_layers["0_0"].kv_cache_shape(7, 16) == (7, 16, 2, 40) and m.model.attn_layers["1_2"].kv_cache_shape(7, 16) == (7, 16, 1, 48)
    assert m.model.attn_layers["1_0"].sink_logits is m.model.attn_layers["1_2"].sink_logits and torch.equal(m.model.attn_layers["1_1"].sink_logits, w["l1.mix.sink"])
    assert (m.model.attn_layers["0_0"].chunk, m.model.attn_layers["1_1"].window_left) == (29, 12)
    in_proj = m.model.layers[0].mixer.in_proj
    rows = 6 * 24 + 2 * 24 + 2 * 16
    assert in_proj.weight.shape[0] % 64 == 0 and torch.equal(in_proj.weight[rows:rows + 6], w["l0.mix.g"]) and not in_proj.weight[rows + 6:].any()
    assert torch.equal(in_proj.bias[:rows], torch.cat([w[f"l0.mix.{n}.b"] for n in "qkv"])) and not in_proj.bias[rows:].any()
    assert m.model.layers[2].mlp is None and m.model.layers[1].mlp is not None
    assert m.model.layers[0].mixer_in.alpha == float(w["l0.norm1.alpha"])
    for name in ("l1.mix.sink", "l0.mix.k.b", "loop.in", "loop.step", "l3.norm2b.alpha", "head"):
        short = {k: v for k, v in w.items() if k != name}
        with pytest.raises(KeyError):
            model().load_weights(short.items())
        with pytest.raises(ValueError):
            model().load_weights(dict(w, **{name: torch.zeros(7, 9)}).items())


def test_norm_masks_sink_and_rotation_of_the_oracle():
    x = torch.tensor([0.0, 1.0, -50.0], dtype=torch.float64)
    one = torch.ones(3, dtype=torch.float64)
    assert torch.allclose(tanh_norm_ref(x, torch.tensor(2.0, dtype=torch.float64), 3 * one, one), torch.tensor([1.0, 1 + 3 * math.tanh(2), -2.0], dtype=torch.float64))
    assert [in_chunk(4)(i) for i in (0, 3, 4, 7, 8)] == [0, 0, 4, 4, 8] and [in_window(4)(i) for i in (0, 3, 4, 8)] == [0, 0, 1, 5]
    # zero queries: the output counts the visible keys against the sink
    T = 6
    q, v = torch.zeros(T, 1, 2, dtype=torch.float64), torch.ones(T, 1, 1, dtype=torch.float64)
    o = attend_ref(q, q, v, 1.0, in_window(3), torch.tensor([math.log(2.0)], dtype=torch.float64))
    assert torch.allclose(o[:, 0, 0], torch.tensor([1 / 3, 2 / 4, 3 / 5, 3 / 5, 3 / 5, 3 / 5], dtype=torch.float64))
    ramp = torch.arange(T, dtype=torch.float64).view(T, 1, 1)
    assert torch.allclose(attend_ref(q, q, ramp, 1.0, in_chunk(4))[:, 0, 0], torch.tensor([0, 0.5, 1.0, 1.5, 4.0, 4.5], dtype=torch.float64))
    # a quarter turn at position 1: neighbours against halves
    x = torch.tensor([[1.0, 2.0, 3.0, 4.0, 9.0]] * 2, dtype=torch.float64).view(2, 1, 5)
    quarter = [math.pi / 2, 0.0]
    assert torch.allclose(rotate_ref(x, 4, quarter, 1.0, False)[1, 0], torch.tensor([-2.0, 1.0, 3.0, 4.0, 9.0], dtype=torch.float64))
    assert torch.allclose(rotate_ref(x, 4, quarter, 2.0, True)[1, 0], torch.tensor([-6.0, 4.0, 2.0, 8.0, 9.0], dtype=torch.float64))


def test_every_mechanism_shows_in_the_oracles_logits():
    cfg = banitar_config()
    w = banitar_random_weights(cfg, seed=1)
    toks = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(0)).tolist()
    ref = banitar_ref(cfg, w, toks)

    def moved(cfg2=None, w2=None):
        out = banitar_ref(cfg2 or cfg, w2 or w, toks)
        return float((out - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt())

    def changed(path, value):
        c = json.loads(json.dumps(cfg))
        node = c
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = value
        return c

    assert moved() == 0.0
    mixer = lambda i, *p: ("layers", i, "mixer") + p      # noqa: E731
    for path, value in ((mixer(0, "mask", "size"), 28), (mixer(1, "mask", "size"), 12), (mixer(1, "scale"), 0.5), (mixer(0, "scale"), 0.5), (mixer(0, "rot", "base"), 800.0),
                        (mixer(0, "rot", "dims"), 14), (mixer(0, "rot", "scaling", "factor"), 4.0), (mixer(0, "rot", "scaling", "fast"), 9.0), (mixer(0, "rot", "scaling", "slow"), 0.3),
                        (mixer(0, "rot", "scaling", "original"), 200), (mixer(1, "rot", "base"), 400.0), (("norm", "eps"), 0.5), (("embedding", "scale"), 2.5), (("loop", "times"), 2)):
        assert moved(changed(path, value)) > 1e-4, path
    for name in ("l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b", "l0.mix.g", "l1.mix.sink", "l1.mix.dkv.norm", "l1.mix.uk", "l1.mix.uv", "l1.norm1", "l1.norm1.b", "l1.norm1.alpha", "l1.norm1b.alpha",
                 "l1.norm2b", "l0.norm2.b", "loop.in", "loop.step", "l1.mlp.up", "final.norm", "final.norm.alpha", "embed", "head"):
        w2 = dict(w)
        w2[name] = w[name] + 0.5 * torch.randn(w[name].shape, generator=torch.Generator().manual_seed(3))
        assert moved(w2=w2) > 1e-4, name
