"""Side benchmark of the Nilevik design (``bench.py --design nilevik``): prefill and decode throughput of a Nilevik stack at
layer sizes that resemble a real model's (random weights), beside the package's closest existing model, Dapuzen (fp32 stream,
windowed attention in the same paged kernels, a linear recurrence with a carried matrix state), at equal sizes -- same width,
heads, layers, window, dense feed-forwards of the same number of weights, recurrent heads of 128 x 128 -- and, kernel by
kernel, how far each new kernel is from its roofline next to the like kernel of that model.

Not the headline benchmark: ``bench.py`` without ``--design`` is unchanged.  Prints one JSON line.
"""
from __future__ import annotations

import json

import torch

from bench_dapuzen import dapuzen_checkpoint
from bench_sonuzen import BLOCK, HBM_GBS, MFMA_TFLOPS, SonuzenRunner, _events_ms


def nilevik_config(width, heads, kv_heads, layers, ff, vocab, window, dim=128, side=256, conv=4):
    attn = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5, mask=dict(size=window), q_temp=dict(coef=0.1, every=8192))
    delta = dict(heads=heads, kv_heads=heads // 2, dim=dim, vdim=dim, conv=conv)
    return dict(architecture="Nilevik", vocab=vocab, width=width, norm=dict(eps=1e-6), token_side=dict(dim=side),
                layers=[dict(type=k, mixer=attn if k == "attention" else delta, mlp=dict(kind="dense", ff=ff)) for k in layers])


def nilevik_checkpoint(cfg, dev, seed=0):
    g = torch.Generator(device=dev)
    g.manual_seed(seed)
    W, V, side = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"]

    def rnd(*shape, std=1.0):
        return (torch.randn(shape, device=dev, generator=g, dtype=torch.float32) * std).to(torch.bfloat16)

    def lin(o, i):
        return rnd(o, i, std=i ** -0.5)

    yield "embed", rnd(V, W, std=0.5)
    yield "side.embed", rnd(V, len(cfg["layers"]) * side)
    yield "final.norm", 1 + rnd(W, std=0.05)
    for i, spec in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", spec["mixer"], spec["mlp"]["ff"]
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm2", "side.norm"):
            yield p + n, 1 + rnd(W, std=0.05)
        if spec["type"] == "attention":
            for n, o in (("q", H * D), ("k", G * D), ("g", H * D)):
                yield p + "mix." + n, lin(o, W)
            yield p + "mix.q.norm", 1 + rnd(D, std=0.05)
            yield p + "mix.k.norm", 1 + rnd(D, std=0.05)
            yield p + "mix.sink", rnd(H)
        else:
            for n, o in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                yield p + "mix." + n, lin(o, W)
                yield p + f"mix.{n}.conv", rnd(o, m["conv"], std=0.5)
            yield p + "mix.g", lin(H * Dv, W)
            yield p + "mix.b", lin(H, W)
            yield p + "mix.a", lin(H, W)
            yield p + "mix.A_log", rnd(H, std=0.5) - 2.0
            yield p + "mix.dt_bias", rnd(H, std=0.5)
            yield p + "mix.norm", 1 + rnd(Dv, std=0.05)
        yield p + "mix.o", lin(W, H * Dv)
        yield p + "mlp.gate", lin(ff, W)
        yield p + "mlp.up", lin(ff, W)
        yield p + "mlp.down", lin(W, ff)
        yield p + "side.gate", lin(side, W)
        yield p + "side.proj", lin(W, side)


def dapuzen_dense_config(width, heads, kv_heads, layers, ff, vocab, window, dim=128):
    """``ff``: of the gated feed-forward with as many weights (two matrices here, three there)."""
    attn = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5, mask=dict(size=window), rot=dict(base=10000.0, dims=dim))
    ret = dict(heads=heads, dim=dim, vdim=dim, rot=dict(base=10000.0, dims=dim), decay=[1.0 - 2.0 ** (-5 - 3 * h / max(heads - 1, 1)) for h in range(heads)])
    return dict(architecture="Dapuzen", vocab=vocab, width=width, norm=dict(eps=1e-6), embedding=dict(scale=1.0),
                layers=[dict(type=k, mixer=attn if k == "attention" else ret, mlp=dict(kind="dense", ff=ff * 3 // 2)) for k in layers])


def dapuzen_dense_checkpoint(cfg, dev):
    """The neighbour's checkpoint, whose generator makes mixtures: the feed-forward's tensors are made here."""
    W = cfg["width"]
    moe = dict(kind="moe", expert=dict(ff=1), shared=dict(ff=1), router=dict(experts=0, identity=1, top=1))
    bare = dict(cfg, layers=[dict(l, mlp=moe) for l in cfg["layers"]])
    for name, t in dapuzen_checkpoint(bare, dev):
        if ".mlp." not in name:
            yield name, t
    g = torch.Generator(device=dev)
    g.manual_seed(7)
    for i, l in enumerate(cfg["layers"]):
        ff = l["mlp"]["ff"]
        yield f"l{i}.mlp.up", (torch.randn(ff, W, device=dev, generator=g) * W ** -0.5).to(torch.bfloat16)
        yield f"l{i}.mlp.down", (torch.randn(W, ff, device=dev, generator=g) * ff ** -0.5).to(torch.bfloat16)
        yield f"l{i}.mlp.act", torch.tensor([0.5, 0.5], device=dev)


def kernel_table(dev, W, H, G, D, B, ctx, L, ff, window, side=256):
    """(name, ms, fraction of the roofline that bounds it) for each new kernel and the like kernel of the neighbours."""
    from vllm_hymeta import hip_ops
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

    # ---- attention over one prompt of L tokens in a window: keys that are values (sink, linear penalty, elementwise gate),
    # beside the neighbour's (gate per head) and Sonuzen's (log penalty, sink) on rows of keys and values
    nblk = (L + BLOCK - 1) // BLOCK
    bt = torch.arange(nblk, dtype=torch.int32, device=dev).view(1, nblk)
    qs, kvs, gate, eg = rnd(L, H, D), rnd(nblk, BLOCK, G, 2 * D), rnd(L, H), rnd(L, H * D)
    row = hip_ops.scaled_key_row(G, D, bf)
    sks = rnd(nblk, BLOCK, 1, row)
    slopes = torch.tensor([2.0 ** (-8 * (h + 1) / H) for h in range(H)], device=dev)
    sinks = torch.zeros(H, device=dev)
    r1, r2 = torch.full((H,), 0.5, device=dev), torch.full((H,), 0.1, device=dev)
    q0, s0 = i32([0, L]), i32([L])
    for win in (window, None):
        seen = sum(min(i + 1, win or L) for i in range(L))
        wl = -1 if win is None else win - 1
        tag = f"L={L}, " + (f"window {win}" if win else "no window")
        add(f"scaled-key attention prefill {tag} (H={H}, {G} kv heads of {D})",
            lambda: hip_ops.sink_attention(qs, sks, bt, q0, s0, G, D, D, D ** -0.5, L, L, sink=True, sink_logits=sinks, window_left=wl, scaled_key=True,
                                           slopes=slopes, elem_gate=eg), flops=4 * H * D * seen, iters=5)
        add(f"window attention prefill, gated (Dapuzen) {tag}",
            lambda: hip_ops.sink_attention(qs, kvs, bt, q0, s0, G, D, D, D ** -0.5, L, L, sink=False, window_left=wl, head_gate=gate), flops=4 * H * D * seen, iters=5)
        add(f"sink_attention prefill (Sonuzen) {tag}",
            lambda: hip_ops.sink_attention(qs, kvs, bt, q0, s0, G, D, D, D ** -0.5, L, L, r1, r2, True, wl), flops=4 * H * D * seen, iters=5)
    bps = (ctx + 1 + BLOCK - 1) // BLOCK
    btd = torch.randperm(B * bps).to(torch.int32).view(B, bps).to(dev)
    sl = torch.full((B,), ctx + 1, dtype=torch.int32, device=dev)
    qsl = torch.arange(B + 1, dtype=torch.int32, device=dev)
    qd, kvd, skd, gd, egd = rnd(B, H, D), rnd(B * bps, BLOCK, G, 2 * D), rnd(B * bps, BLOCK, 1, row), rnd(B, H), rnd(B, H * D)
    for win in (window, None):
        keys, wl = min(ctx + 1, win or ctx + 1), -1 if win is None else win - 1
        tag = f"B={B} ctx={ctx}, " + (f"window {win}" if win else "no window")
        add(f"scaled-key attention decode {tag}",
            lambda: hip_ops.sink_attention(qd, skd, btd, qsl, sl, G, D, D, D ** -0.5, 1, ctx + 1, sink=True, sink_logits=sinks, window_left=wl, scaled_key=True,
                                           slopes=slopes, elem_gate=egd), nbytes=B * keys * row * 2)
        add(f"window attention decode, gated (Dapuzen) {tag}",
            lambda: hip_ops.sink_attention(qd, kvd, btd, qsl, sl, G, D, D, D ** -0.5, 1, ctx + 1, sink=False, window_left=wl, head_gate=gd), nbytes=B * G * keys * 2 * D * 2)
    # ---- between the projection and the attention
    freqs = torch.tensor([10000.0 ** (-2.0 * i / D) for i in range(D // 2)], dtype=torch.float64, device=dev)
    w1 = torch.ones(D, device=dev)
    for T in (B, L):
        qkg, qkv = rnd(T, (2 * H + G) * D), rnd(T, (H + 2 * G) * D)
        sm = torch.arange(T, dtype=torch.int64, device=dev)
        cs, ck = (skd, kvd) if T == B else (sks, kvs)
        add(f"scaled_key_cache T={T}", lambda: hip_ops.scaled_key_cache_(qkg, H, G, D, w1, w1, 1e-6, cs, sm, 0.1, 8192, sm),
            nbytes=T * ((H + G) * D * 2 + H * D * 2 + row * 2))
        add(f"rotary_cache (Dapuzen) T={T}", lambda: hip_ops.rotary_cache_(qkv, H, G, D, D, D, freqs, 1.0, ck, sm, positions=sm),
            nbytes=T * ((H + 2 * G) * D * 2 + (H + G) * D * 2 + 2 * G * D * 2))
    # ---- recurrences
    Hk = H // 2
    ones = torch.ones(B, dtype=torch.int32, device=dev)
    sidx = torch.arange(B, dtype=torch.int32, device=dev)
    decay = torch.full((H,), 0.99, device=dev)

    def split(T):
        p = rnd(T, (2 * Hk + H) * D)
        return p[:, :Hk * D].view(T, Hk, D), p[:, Hk * D:2 * Hk * D].view(T, Hk, D), p[:, 2 * Hk * D:].view(T, H, D), rnd(T, H), -torch.rand(T, H, device=dev) * 0.1

    q_, k_, v_, b_, ld = split(L)
    st = torch.zeros(2, H, D, D, device=dev)
    one, ctx0 = i32([1]), i32([0])
    add(f"delta_rule prefill L={L} (H={H}, {Hk} query / key heads, {D}x{D})",
        lambda: hip_ops.delta_rule(q_, k_, v_, b_, ld, st, q0, ctx0, one, L, D ** -0.5, 1e-6),
        nbytes=L * (2 * Hk * D * 2 + H * (D * 2 + D * 4)), flops=L * H * (6 * D * D + 8 * 64 * D), iters=5)
    proj = rnd(L, 3 * H * D)
    q2, k2, v2 = (proj[:, j * H * D:(j + 1) * H * D].view(L, H, D) for j in range(3))
    add(f"decay_scan prefill, retention (Dapuzen) L={L} (H={H}, {D}x{D})",
        lambda: hip_ops.decay_scan(q2, k2, v2, st, q0, ctx0, one, L, decay=decay),
        nbytes=L * H * (3 * D * 2 + D * 4), flops=L * H * (4 * D * D + 4 * 64 * D), iters=5)
    qd_, kd_, vd_, bd_, ldd = split(B)
    std_ = torch.zeros(B, H, D, D, device=dev)
    wn_, gg = torch.ones(D, device=dev), rnd(B, H * D)
    add(f"delta_rule decode with norm and gate B={B}",
        lambda: hip_ops.delta_rule(qd_, kd_, vd_, bd_, ldd, std_, qsl, ones, sidx, 1, D ** -0.5, 1e-6, norm_weight=wn_, gate=gg, norm_eps=1e-6),
        nbytes=B * H * (2 * D * D * 4 + 4 * D * 2) + B * 2 * Hk * D * 2)
    projd = rnd(B, 3 * H * D)
    q3, k3, v3 = (projd[:, j * H * D:(j + 1) * H * D].view(B, H, D) for j in range(3))
    add(f"decay_scan decode, retention (Dapuzen) B={B}", lambda: hip_ops.decay_scan(q3, k3, v3, std_, qsl, ones, sidx, 1, decay=decay),
        nbytes=B * H * (2 * D * D * 4 + 3 * D * 2 + D * 4))
    # ---- the convolution, the stream, the units
    table, etab = rnd(32768, 4 * side), rnd(32768, W)
    pf = torch.tensor([10000.0 ** (-2.0 * i / W) for i in range(W // 2)], dtype=torch.float64, device=dev)
    for T in (B, L):
        lay = (qsl, ones, sidx) if T == B else (q0, ctx0, one)
        C = (2 * Hk + H) * D
        pin = rnd(T, C + H)
        cw = rnd(C, 4, std=0.5, dtype=torch.float32).contiguous()
        cstate = torch.zeros(max(B, 4), 3, C, dtype=bf, device=dev)
        dtb, alog = torch.zeros(H, device=dev), torch.zeros(H, device=dev)
        add(f"causal_conv_silu (+ decays; Dapuzen's kernel) T={T}, {C} channels",
            lambda: hip_ops.causal_conv_silu(pin[:, :C], cw, None, cstate, *lay, dt_in=pin[:, C:], dt_bias=dtb, a_log=alog, max_query_len=1 if T == B else T),
            nbytes=T * C * 4)
        x, y = rnd(T, W, dtype=torch.float32), rnd(T, W)
        wn = 1 + rnd(W, std=0.1, dtype=torch.float32)
        add(f"norm_residual with the stream's copy T={T}", lambda: hip_ops.norm_residual_(x, y, wn, 1e-6, copy=True), nbytes=T * W * (8 + 2 + 2))
        add(f"stream_add_norm, 1 term (Dapuzen) T={T}", lambda: hip_ops.stream_add_norm_(x, [(y, 1.0, None)], 1.1, 1e-6, bf), nbytes=T * W * (8 + 2 + 2))
        ids = torch.randint(0, 32768, (T,), device=dev)
        pos = torch.arange(T, dtype=torch.int64, device=dev)
        add(f"embed_rows with the position's sinusoid and copy T={T}", lambda: hip_ops.embed_rows(ids, etab, positions=pos, pos_freqs=pf, copy=True), nbytes=T * W * (2 + 4 + 2))
        add(f"embed_rows (Dapuzen) T={T}", lambda: hip_ops.embed_rows(ids, etab), nbytes=T * W * (2 + 4))
        gu, sg, up = rnd(T, 2 * ff), rnd(T, side), rnd(T, ff * 3 // 2)
        add(f"gelu_mul T={T}, ff {ff}", lambda: hip_ops.gelu_mul(gu), nbytes=T * ff * 6)
        add(f"xielu (Dapuzen) T={T}, ff {ff * 3 // 2}", lambda: hip_ops.xielu(up, 0.7, 1.2), nbytes=T * (ff * 3 // 2) * 4)
        add(f"gelu_mul_rows T={T}, {side} columns", lambda: hip_ops.gelu_mul_rows(sg, table[:, side:2 * side], ids), nbytes=T * side * 6)
        o, gt = rnd(T, H * D, dtype=torch.float32), rnd(T, H * D)
        wg = torch.ones(H * D, device=dev)
        add(f"gated_rms_norm per head, silu gate (Dapuzen's kernel) T={T}", lambda: hip_ops.gated_rms_norm(o, gt, wg, 1e-6, groups=H, gate_act="silu"),
            nbytes=T * H * D * (4 + 2 + 2))
    return rows


def main(args):
    from vllm_hymeta.models.configuration_dapuzen import DapuzenConfig
    from vllm_hymeta.models.configuration_nilevik import NilevikConfig
    from vllm_hymeta.models.modeling_dapuzen import DapuzenForCausalLM
    from vllm_hymeta.models.modeling_nilevik import NilevikForCausalLM

    torch.cuda.set_device(0)
    dev = torch.device("cuda", 0)
    B, ctx, L = args.batch, args.ctx if args.ctx_given else 4096, min(args.prefill_ctx, 8192)
    vocab, window = 32768, 1024
    layers = ("attention", "delta", "attention", "delta")
    out = {"metric": "nilevik_vs_dapuzen_tokens_per_s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
           "sizes": []}
    for (W, H, ff) in ((2048, 16, 8192), (3584, 28, 18944)):
        res = {}
        for name in ("dapuzen", "nilevik"):
            if name == "dapuzen":
                cfg = dapuzen_dense_config(W, H, 4, ["retention" if k == "delta" else k for k in layers], ff, vocab, window)
                model = DapuzenForCausalLM(DapuzenConfig(cfg), max_num_seqs=max(B, 4), dtype=torch.bfloat16, device=dev)
                model.load_weights(dapuzen_dense_checkpoint(cfg, dev))
            else:
                cfg = nilevik_config(W, H, 4, layers, ff, vocab, window)
                model = NilevikForCausalLM(NilevikConfig(cfg), max_num_seqs=max(B, 4), dtype=torch.bfloat16, device=dev)
                model.load_weights(nilevik_checkpoint(cfg, dev))
            run = SonuzenRunner(model, dev)
            dec = run.decode(B, ctx, args.steps, args.warmup)
            pre = run.prefill(L)
            res[name] = {"decode_ms_per_step": round(dec, 3), "decode_tokens_per_s": round(B / dec * 1e3, 1), "prefill_ms": round(pre, 2),
                         "prefill_tokens_per_s": round(L / pre * 1e3, 1)}
            del run, model
            torch.cuda.empty_cache()
        out["sizes"].append({"width": W, "heads": H, "kv_heads": 4, "head_dim": 128, "layers": 4, "ff": ff, "token_side": 256, "batch": B, "ctx": ctx,
                             "prompt": L, "window": window, "recurrent": {"heads": H, "dim": 128, "vdim": 128}, **res})
        print(json.dumps(out["sizes"][-1]), flush=True)
    out["kernels"] = kernel_table(dev, 3584, 28, 4, 128, B, ctx, L, 18944, window)
    s = out["sizes"][-1]
    out["value"], out["unit"] = s["nilevik"]["decode_tokens_per_s"], "tokens/s"
    out["config"] = {"model": "Nilevik 4 layers (windowed attention whose values are its keys, gated delta rule; dense gelu-gated feed-forward, per-layer token input)",
                     "global_batch": B, "seq_len": ctx, "parallelism": "tp1"}
    print(json.dumps(out))
