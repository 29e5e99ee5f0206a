"""Side benchmark of the Banitar design (``bench.py --design banitar``): prefill and decode throughput of a Banitar stack at
layer sizes that resemble a real model's (random weights), beside the package's closest existing models at equal sizes:
Geponex with latent attention in every layer and Dapuzen with its windowed, head-gated rotary attention in every layer (fp32
streams, the same paged attention kernels) -- same width, heads, latent and head sizes, layer runs, and dense feed-forwards of
the same number of weights -- and, kernel by kernel, how far each new kernel is from its roofline next to the like kernel of
those models.

Not the headline benchmark: ``bench.py`` without ``--design`` is unchanged.  Prints one JSON line.
"""
from __future__ import annotations

import json

import torch

from bench_geponex import geponex_checkpoint
from bench_nilevik import dapuzen_dense_checkpoint, dapuzen_dense_config
from bench_sonuzen import BLOCK, HBM_GBS, MFMA_TFLOPS, SonuzenRunner, _events_ms


def banitar_config(width, heads, kv_heads, layers, ff, vocab, window, chunk, kv_rank=128, rot_dim=64, dim=128, latent_dim=64, loop=(1, 3, 2)):
    attn = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5, mask=dict(size=chunk),
                rot=dict(base=500000.0, dims=dim, scaling=dict(factor=8.0, original=4096, fast=32.0, slow=1.0)))
    latent = dict(heads=heads, dim=latent_dim, rot_dim=rot_dim, vdim=dim, kv_rank=kv_rank, scale=(latent_dim + rot_dim) ** -0.5, mask=dict(size=window),
                  rot=dict(base=10000.0, dims=rot_dim))
    cfg = dict(architecture="Banitar", vocab=vocab, width=width, norm=dict(eps=1e-6), embedding=dict(scale=8.0),
               layers=[dict(type=k, mixer=attn if k == "attention" else latent, mlp=dict(kind="dense", ff=ff)) for k in layers])
    if loop:
        cfg["loop"] = dict(start=loop[0], stop=loop[1], times=loop[2])
    return cfg


def banitar_checkpoint(cfg, dev, seed=0):
    g = torch.Generator(device=dev)
    g.manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, std=1.0):
        return (torch.randn(shape, device=dev, generator=g, dtype=torch.float32) * std).to(torch.bfloat16)

    def lin(o, i):
        return rnd(o, i, std=i ** -0.5)

    def norm(name, alpha):
        yield name, 1 + rnd(W, std=0.05)
        yield name + ".b", rnd(W, std=0.05)
        yield name + ".alpha", torch.tensor(alpha, device=dev).to(torch.bfloat16)

    yield "embed", rnd(V, W, std=0.1)
    yield "head", lin(V, W)
    yield from norm("final.norm", 0.5)
    if cfg.get("loop"):
        yield "loop.in", lin(W, 2 * W)
        yield "loop.step", rnd(cfg["loop"]["times"], W, std=0.1)
    for i, spec in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", spec["mixer"], spec["mlp"]["ff"]
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b", "norm2", "norm2b"):
            yield from norm(p + n, 0.5)
        if spec["type"] == "attention":
            G = m["kv_heads"]
            for n, o in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                yield p + "mix." + n, lin(o, W)
                yield p + f"mix.{n}.b", rnd(o, std=0.1)
            yield p + "mix.g", lin(H, W)
        else:
            R, C = m["rot_dim"], m["kv_rank"]
            yield p + "mix.q", lin(H * (D + R), W)
            yield p + "mix.dkv", lin(C + R, W)
            yield p + "mix.dkv.norm", 1 + rnd(C, std=0.05)
            yield p + "mix.uk", lin(H * D, C)
            yield p + "mix.uv", lin(H * Dv, C)
            yield p + "mix.sink", rnd(H)
        yield p + "mix.o", lin(W, H * Dv)
        yield p + "mlp.gate", lin(ff, W)
        yield p + "mlp.up", lin(ff, W)
        yield p + "mlp.down", lin(W, ff)


def geponex_dense_config(width, heads, runs, ff, vocab, kv_rank=128, rot_dim=64, dim=64, vdim=128):
    """``runs`` layers of latent attention, plain and with sink and gate in turn; ``ff``: of the gated feed-forward with as many
    weights (two matrices here, three there)."""
    mixer = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=width // 4, scale=(dim + rot_dim) ** -0.5,
                 rot=dict(base=10000.0, dims=rot_dim))
    return dict(architecture="Geponex", vocab=vocab, width=width, norm=dict(eps=1e-6, groups=2), postln_alpha=2.0,
                layers=[dict(type="latent_attention_2" if i % 2 else "latent_attention", mixer=mixer, mlp=dict(kind="dense", ff=ff * 3 // 2)) for i in range(runs)])


def geponex_dense_checkpoint(cfg, dev):
    """The neighbour's checkpoint, whose generator makes mixtures: the feed-forward's tensors are made here."""
    W = cfg["width"]
    moe = dict(kind="moe", expert=dict(ff=1), shared=dict(ff=1), router=dict(experts=0, top=0))
    bare = dict(cfg, layers=[dict(l, mlp=moe) for l in cfg["layers"]])
    for name, t in geponex_checkpoint(bare, dev):
        if ".mlp." not in name:
            yield name, t
    g = torch.Generator(device=dev)
    g.manual_seed(7)
    for i, l in enumerate(cfg["layers"]):
        ff = l["mlp"]["ff"]
        yield f"l{i}.mlp.up", (torch.randn(ff, W, device=dev, generator=g) * W ** -0.5).to(torch.bfloat16)
        yield f"l{i}.mlp.up.b", torch.zeros(ff, device=dev)
        yield f"l{i}.mlp.down", (torch.randn(W, ff, device=dev, generator=g) * ff ** -0.5).to(torch.bfloat16)
        yield f"l{i}.mlp.down.b", torch.zeros(W, device=dev)
        yield f"l{i}.mlp.act", torch.tensor([0.5, 0.5], device=dev)


def kernel_table(dev, W, H, G, D, B, ctx, L, ff, window, chunk, R=64):
    """(name, ms, fraction of the roofline that bounds it) for each new kernel and the like kernel of the neighbours."""
    from vllm_hymeta import hip_ops
    from vllm_hymeta.linear import linear_fp32
    rows = []
    bf = torch.bfloat16

    def rnd(*shape, std=1.0, dtype=bf):
        return (torch.randn(*shape, device=dev, dtype=torch.float32) * std).to(dtype)

    def i32(v):
        return torch.tensor(v, dtype=torch.int32, device=dev)

    def add(name, fn, nbytes=0, flops=0, iters=20):
        ms = _events_ms(fn, iters=iters)
        t_mem, t_mma = nbytes / (HBM_GBS * 1e9) * 1e3, flops / (MFMA_TFLOPS * 1e12) * 1e3
        rows.append(dict(kernel=name, ms=round(ms, 4), roofline_ms=round(max(t_mem, t_mma), 4), bound="hbm" if t_mem >= t_mma else "mfma",
                         fraction_of_roofline=round(max(t_mem, t_mma) / ms, 3)))

    # ---- attention over one prompt of L tokens
    nblk = (L + BLOCK - 1) // BLOCK
    bt = torch.arange(nblk, dtype=torch.int32, device=dev).view(1, nblk)
    q0, s0 = i32([0, L]), i32([L])
    qs, kvs, gate = rnd(L, H, D), rnd(nblk, BLOCK, G, 2 * D), rnd(L, H)
    in_window = lambda w: sum(min(i + 1, w) for i in range(L))              # noqa: E731
    in_chunk = lambda c: sum(i % c + 1 for i in range(L))                    # noqa: E731
    add(f"chunked attention prefill, gated L={L}, chunks of {chunk} (H={H}, {G} kv heads of {D})",
        lambda: hip_ops.sink_attention(qs, kvs, bt, q0, s0, G, D, D, D ** -0.5, L, L, sink=False, chunk=chunk, head_gate=gate), flops=4 * H * D * in_chunk(chunk), iters=5)
    add(f"window attention prefill, gated (Dapuzen) L={L}, window {window}",
        lambda: hip_ops.sink_attention(qs, kvs, bt, q0, s0, G, D, D, D ** -0.5, L, L, sink=False, window_left=window - 1, head_gate=gate), flops=4 * H * D * in_window(window), iters=5)
    bps = (ctx + 1 + BLOCK - 1) // BLOCK
    btd = torch.randperm(B * bps).to(torch.int32).view(B, bps).to(dev)
    sl = torch.full((B,), ctx, dtype=torch.int32, device=dev)               # the last position of a chunk: all of it is seen
    qsl = torch.arange(B + 1, dtype=torch.int32, device=dev)
    qd, kvd, gd = rnd(B, H, D), rnd(B * bps, BLOCK, G, 2 * D), rnd(B, H)
    add(f"chunked attention decode B={B} ctx={ctx}, chunk {chunk}",
        lambda: hip_ops.sink_attention(qd, kvd, btd, qsl, sl, G, D, D, D ** -0.5, 1, ctx, sink=False, chunk=chunk, head_gate=gd), nbytes=B * G * min(chunk, ctx) * 2 * D * 2)
    add(f"window attention decode, gated (Dapuzen) B={B} ctx={ctx}, window {chunk}",
        lambda: hip_ops.sink_attention(qd, kvd, btd, qsl, sl, G, D, D, D ** -0.5, 1, ctx, sink=False, window_left=chunk - 1, head_gate=gd), nbytes=B * G * min(chunk, ctx) * 2 * D * 2)
    for C, h in ((128, H), (512, 16)):
        ql, kvl, sinks = rnd(L, h, C + R), rnd(nblk, BLOCK, 1, C + R), rnd(h, dtype=torch.float32)
        for win in (window, None):
            wl, tag = (-1 if win is None else win - 1), ("no window (Geponex)" if win is None else f"window {win}")
            add(f"latent attention prefill L={L} (H={h}, {C}+{R}), {tag}",
                lambda: hip_ops.sink_attention(ql, kvl, bt, q0, s0, 1, C + R, C, 0.1, L, L, sink=True, sink_logits=sinks, value_in_key=True, window_left=wl),
                flops=h * in_window(win or L) * 2 * (2 * C + R), iters=5)
        qld, kvld = rnd(B, h, C + R), rnd(B * bps, BLOCK, 1, C + R)
        for win in (window, None):
            wl, tag = (-1 if win is None else win - 1), ("no window (Geponex)" if win is None else f"window {win}")
            add(f"latent attention decode B={B} ctx={ctx} (H={h}, {C}+{R}), {tag}",
                lambda: hip_ops.sink_attention(qld, kvld, btd, qsl, sl, 1, C + R, C, 0.1, 1, ctx, sink=True, sink_logits=sinks, value_in_key=True, window_left=wl),
                nbytes=B * min(win or ctx, ctx) * (C + R) * 2)
    # ---- between the projections and the attention
    freqs, lf = (torch.tensor([10000.0 ** (-2.0 * i / n) for i in range(n // 2)], dtype=torch.float64, device=dev) for n in (D, R))
    C, Dn, Q = 128, 64, W // 4
    wq, wk = torch.ones(Q, device=dev), torch.ones(C, device=dev)
    for T in (B, L):
        lay = (qsl, sl) if T == B else (q0, s0)
        sm = torch.arange(T, dtype=torch.int64, device=dev)
        qkv, ck, kl = rnd(T, (H + 2 * G) * D + 64), kvd if T == B else kvs, rnd(max(T // BLOCK, 1), BLOCK, 1, C + R)
        moved = T * ((H + 2 * G) * D * 2 + (H + G) * D * 2 + 2 * G * D * 2)
        add(f"rotary_cache, interleaved pairs, unit heads T={T}",
            lambda: hip_ops.rotary_cache_(qkv, H, G, D, D, D, freqs, 1.0, ck, sm, positions=sm, interleaved=True, rot_mag=1.2, unit_eps=1e-6), nbytes=moved)
        add(f"rotary_cache (Dapuzen) T={T}", lambda: hip_ops.rotary_cache_(qkv, H, G, D, D, D, freqs, 1.0, ck, sm, positions=sm), nbytes=moved)
        pa, pb = rnd(T, H * (Dn + R) + C + R), rnd(T, Q + C + R)
        add(f"latent_kv_prep without a query latent T={T}",
            lambda: hip_ops.latent_kv_prep_(pa, 0, 0, H * (Dn + R), C, R, R, None, wk, 1e-6, lf, 1.0, kl, sm, *lay, True), nbytes=T * 2 * (C + R) * 2)
        add(f"latent_kv_prep (Geponex) T={T}",
            lambda: hip_ops.latent_kv_prep_(pb, 0, Q, Q, C, R, R, wq, wk, 1e-6, lf, 1.0, kl, sm, *lay), nbytes=T * 2 * (C + R + Q) * 2)
        qv, qf = pa[:, :H * (Dn + R)].view(T, H, Dn + R), rnd(T, H, C + R)
        for half, tag in ((True, "rotate half"), (False, "neighbouring pairs (Geponex)")):
            add(f"latent_q_rotate, {tag} T={T}", lambda: hip_ops.latent_q_rotate_(qf, qv, Dn, R, R, lf, 1.0, *lay, half), nbytes=T * H * R * 2 * 2)
    # ---- the stream
    etab, win_w = rnd(32768, W), rnd(W, W, std=W ** -0.5)
    for T in (B, L):
        x, y, base, base2 = rnd(T, W, dtype=torch.float32), rnd(T, W), rnd(T, W, dtype=torch.float32), rnd(T, W, dtype=torch.float32)
        vec = [1 + rnd(W, std=0.1, dtype=torch.float32) for _ in range(5)]
        n1, n2 = hip_ops.SquashNorm(0.5, vec[0], vec[1]), hip_ops.SquashNorm(0.7, vec[2], vec[3])
        add(f"tanh_stream: output norm, sum, next norm T={T}", lambda: hip_ops.tanh_stream_(x, y, n1, read=n2, out_dtype=bf), nbytes=T * W * (8 + 2 + 2))
        add(f"tanh_stream: pass entry T={T}", lambda: hip_ops.tanh_stream_(x, base=base, base2=base2, add=vec[4], read=n2, out_dtype=bf), nbytes=T * W * (8 + 4 + 2))
        add(f"add_group_norm with its copy (Geponex) T={T}", lambda: hip_ops.add_group_norm(x, y, vec[0], 2, 1e-6, 1.0, None, True, bf), nbytes=T * W * (8 + 2 + 2))
        add(f"stream_add_norm, 1 term (Dapuzen) T={T}", lambda: hip_ops.stream_add_norm_(x, [(y, 1.0, None)], 1.1, 1e-6, bf), nbytes=T * W * (8 + 2 + 2))
        ids = torch.randint(0, 32768, (T,), device=dev)
        add(f"embed_rows, scaled, with copy T={T}", lambda: hip_ops.embed_rows(ids, etab, scale=8.0, copy=True), nbytes=T * W * (2 + 4 + 2))
        add(f"embed_rows (Dapuzen) T={T}", lambda: hip_ops.embed_rows(ids, etab), nbytes=T * W * (2 + 4))
        flops, moved = 2 * T * W * W, 2 * W * W + T * W * 6
        add(f"pass entry's product, fp32 result T={T}", lambda: linear_fp32(y, win_w), nbytes=moved, flops=flops)
        add(f"the same product, bf16 result (every model's linears) T={T}", lambda: torch.nn.functional.linear(y, win_w), nbytes=moved - 2 * T * W, flops=flops)
        gu, up = rnd(T, 2 * ff), rnd(T, ff * 3 // 2)
        add(f"silu_mul T={T}, ff {ff}", lambda: hip_ops.silu_mul(gu), nbytes=T * ff * 6)
        add(f"xielu (Geponex, Dapuzen) T={T}, ff {ff * 3 // 2}", lambda: hip_ops.xielu(up, 0.7, 1.2), nbytes=T * (ff * 3 // 2) * 4)
    return rows


def main(args):
    from vllm_hymeta.models.configuration_banitar import BanitarConfig
    from vllm_hymeta.models.configuration_dapuzen import DapuzenConfig
    from vllm_hymeta.models.configuration_geponex import GeponexConfig
    from vllm_hymeta.models.modeling_banitar import BanitarForCausalLM
    from vllm_hymeta.models.modeling_dapuzen import DapuzenForCausalLM
    from vllm_hymeta.models.modeling_geponex import GeponexForCausalLM

    torch.cuda.set_device(0)
    dev = torch.device("cuda", 0)
    B, ctx, L = args.batch, args.ctx if args.ctx_given else 4096, min(args.prefill_ctx, 8192)
    vocab, window, chunk = 32768, 1024, 2048
    layers = ("attention", "latent_attention", "attention", "latent_attention")       # with the middle two run twice: six layer runs
    runs = 6
    out = {"metric": "banitar_vs_geponex_dapuzen_tokens_per_s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
           "sizes": []}
    for (W, H, ff) in ((2048, 16, 8192), (3584, 28, 18944)):
        res = {}
        for name in ("geponex", "dapuzen", "banitar"):
            kw = dict(max_num_seqs=max(B, 4), dtype=torch.bfloat16, device=dev)
            if name == "geponex":
                cfg = geponex_dense_config(W, H, runs, ff, vocab)
                model, weights = GeponexForCausalLM(GeponexConfig(cfg), **kw), geponex_dense_checkpoint(cfg, dev)
            elif name == "dapuzen":
                cfg = dapuzen_dense_config(W, H, 4, ["attention"] * runs, ff, vocab, window)
                model, weights = DapuzenForCausalLM(DapuzenConfig(cfg), **kw), dapuzen_dense_checkpoint(cfg, dev)
            else:
                cfg = banitar_config(W, H, 4, layers, ff, vocab, window, chunk)
                model, weights = BanitarForCausalLM(BanitarConfig(cfg), **kw), banitar_checkpoint(cfg, dev)
            model.load_weights(weights)
            run = SonuzenRunner(model, dev)
            dec = run.decode(B, ctx, args.steps, args.warmup)
            pre = run.prefill(L)
            res[name] = {"decode_ms_per_step": round(dec, 3), "decode_tokens_per_s": round(B / dec * 1e3, 1), "prefill_ms": round(pre, 2),
                         "prefill_tokens_per_s": round(L / pre * 1e3, 1)}
            del run, model, weights
            torch.cuda.empty_cache()
        out["sizes"].append({"width": W, "heads": H, "kv_heads": 4, "head_dim": 128, "latent": "128+64", "layer_runs": runs, "ff": ff, "batch": B, "ctx": ctx,
                             "prompt": L, "window": window, "chunk": chunk, **res})
        print(json.dumps(out["sizes"][-1]), flush=True)
    out["kernels"] = kernel_table(dev, 3584, 28, 4, 128, B, ctx, L, 18944, window, chunk)
    s = out["sizes"][-1]
    out["value"], out["unit"] = s["banitar"]["decode_tokens_per_s"], "tokens/s"
    out["config"] = {"model": "Banitar 4 layers, the middle two run twice (chunked attention, windowed latent attention; dense silu-gated feed-forward)",
                     "global_batch": B, "seq_len": ctx, "parallelism": "tp1"}
    print(json.dumps(out))
