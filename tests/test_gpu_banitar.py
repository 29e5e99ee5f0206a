"""The Banitar building blocks and the model under the engine, against the plain CPU statement in ``oracle/banitar.py``.

Mechanisms alone first (the squashing norm's launch in every form, the partial sums it reads, rotation in both layouts with
unit heads and the paged write, the latent rows, attention in chunks and latent attention in a window with keys just inside
and just outside, the entry of a pass), then whole models of several shapes: a prompt in one step against the oracle, and the
same tokens cut into steps in every way the engine allows (token by token, portions down to two tokens, unequal requests in
one batch, pages used again) against the one-step result.
"""
import math

import pytest
import torch

pytestmark = pytest.mark.gpu

from oracle.banitar import (attend_ref, banitar_config, banitar_random_weights, banitar_ref, chunked_attention_ref, chunked_config,  # noqa: E402
                            in_chunk, in_window, latent_attention_ref, latent_config, rms_ref, rotate_ref, rotation_frequencies_ref, silu_glu_ref, tanh_norm_ref)

DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


def rel_err(got: torch.Tensor, ref: torch.Tensor) -> float:
    got, ref = got.double().cpu(), ref.double().cpu()
    assert torch.isfinite(got).all()
    return float((got - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def layout_of(portions, contexts, block_tables, block_size=16):
    """A step's layout from (rows, tokens before them) per sequence."""
    from itertools import accumulate
    from vllm_hymeta.models.stream_block import StepLayout
    qsl = list(accumulate(portions, initial=0))
    bt = torch.zeros(len(block_tables), max(len(t) for t in block_tables), dtype=torch.int32)
    sm = []
    for s, (n, ctx) in enumerate(zip(portions, contexts)):
        bt[s, :len(block_tables[s])] = torch.tensor(block_tables[s], dtype=torch.int32)
        sm += [block_tables[s][p // block_size] * block_size + p % block_size for p in range(ctx, ctx + n)]
    positions = torch.tensor(sum((list(range(c, c + n)) for n, c in zip(portions, contexts)), []), dtype=torch.int64, device=DEV)
    return StepLayout(query_start_loc=i32(qsl), context_lens=i32(contexts), seq_lens=i32([c + n for c, n in zip(contexts, portions)]),
                      slot_idx=None, block_tables=bt.to(DEV), slot_mapping=torch.tensor(sm, dtype=torch.int64, device=DEV), max_query_len=max(portions),
                      max_seq_len=max(c + n for c, n in zip(contexts, portions)), positions=positions)


def scattered(num_seqs, pages_each, seed=0):
    order = torch.randperm(num_seqs * pages_each, generator=torch.Generator().manual_seed(seed)).tolist()
    return [order[s * pages_each:(s + 1) * pages_each] for s in range(num_seqs)]


# --------------------------------------------------------------------------- the stream between sublayers
def _norm(g, W, alpha):
    return alpha, 1 + 0.3 * torch.randn(W, generator=g), 0.2 * torch.randn(W, generator=g)


def _on_device(n):
    from vllm_hymeta import hip_ops
    return hip_ops.SquashNorm(n[0], n[1].to(DEV), n[2].to(DEV))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,width,pad", [(7, 56, 0), (5, 33, 0), (3, 64, 3), (1, 1, 0), (9, 1024, 8), (1027, 72, 0), (1100, 33, 0), (2, 5000, 0)])
def test_stream_in_every_form(dtype, T, width, pad):
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(width)
    wide = torch.randn(T, width + pad, generator=g)
    y = (2 * torch.randn(T, width + pad, generator=g)).to(dtype)[:, :width]
    base, base2, add = torch.randn(T, width, generator=g), torch.randn(T, width, generator=g), torch.randn(width, generator=g)
    n1, n2 = _norm(g, width, 0.7), _norm(g, width, -1.3)
    ref = lambda v, n: tanh_norm_ref(v.double(), torch.tensor(n[0], dtype=torch.float64), n[1].double(), n[2].double())      # noqa: E731
    f32, act = 2e-6, 2e-6 if dtype == torch.float32 else 4e-3
    x0 = wide[:, :width]
    ydev = torch.zeros(T, width + pad, dtype=dtype, device=DEV)
    ydev[:, :width] = y.to(DEV)

    def stream():
        return wide.to(DEV)[:, :width]

    x = stream()                                                         # output norm, sum, next norm
    h = hip_ops.tanh_stream_(x, ydev[:, :width], _on_device(n1), read=_on_device(n2), out_dtype=dtype)
    want = x0.double() + ref(y, n1)
    assert rel_err(x, want) < f32 and rel_err(h, ref(want, n2)) < act and h.dtype == dtype
    x = stream()                                                         # sum, copy
    h = hip_ops.tanh_stream_(x, ydev[:, :width], _on_device(n1), out_dtype=dtype)
    assert rel_err(x, want) < f32 and torch.equal(h, x.to(dtype))
    x = stream()                                                         # sum alone
    assert hip_ops.tanh_stream_(x, ydev[:, :width], _on_device(n1)) is None and rel_err(x, want) < f32
    x = stream()                                                         # next norm alone: the stream stays
    h = hip_ops.tanh_stream_(x, read=_on_device(n2), out_dtype=dtype)
    assert torch.equal(x.cpu(), x0) and rel_err(h, ref(x0, n2)) < act
    for b2, ad in ((base2, add), (None, add), (base2, None), (None, None)):      # the stream anew
        x = stream()
        h = hip_ops.tanh_stream_(x, base=base.to(DEV), base2=None if b2 is None else b2.to(DEV), add=None if ad is None else ad.to(DEV), read=_on_device(n2), out_dtype=dtype)
        want = base.double() + (0 if b2 is None else b2.double()) + (0 if ad is None else ad.double())
        assert rel_err(x, want) < f32 and rel_err(h, ref(want, n2)) < act


@pytest.mark.parametrize("dtype", DTYPES)
def test_squash_is_accurate_from_tiny_to_saturated(dtype):
    """Relative accuracy of the squashed value itself (no weight, no bias), elementwise, over the whole range."""
    from vllm_hymeta import hip_ops
    v = torch.cat([torch.logspace(-20, 2, 4000, base=10.0), torch.linspace(0.2, 0.3, 97)])
    v = torch.cat([v, -v, torch.zeros(2)]).view(1, -1)
    W = v.shape[1]
    x = v.to(DEV)
    one, nil = torch.ones(W, device=DEV), torch.zeros(W, device=DEV)
    y = v.to(dtype).to(DEV)
    zero = torch.zeros(1, W, device=DEV)
    hip_ops.tanh_stream_(zero, y, hip_ops.SquashNorm(1.0, one, nil))
    want = torch.tanh(v.to(dtype).double())
    assert float(((zero.double().cpu() - want).abs() / want.abs().clamp_min(1e-30)).max()) < (1e-6 if dtype == torch.bfloat16 else 4e-7)
    h = hip_ops.tanh_stream_(x, read=hip_ops.SquashNorm(3.0, one, nil), out_dtype=torch.float32)
    assert float((h.double().cpu() - torch.tanh(3 * v.double())).abs().max()) < 3e-7


@pytest.mark.parametrize("rows,N,K", [(1, 256, 2048), (17, 192, 4096), (64, 512, 4096), (128, 256, 2048)])
def test_partial_sums_of_a_projection_give_the_projections_bits(rows, N, K):
    from vllm_hymeta import hip_ops
    from vllm_hymeta.linear import HymetaLinear
    g = torch.Generator().manual_seed(rows)
    h = torch.randn(rows, K, generator=g).to(torch.bfloat16).to(DEV)
    lin = HymetaLinear.from_weight((torch.randn(N, K, generator=g) * K ** -0.5).to(torch.bfloat16).to(DEV), torch.randn(N, generator=g).to(torch.bfloat16).to(DEV))
    n1, n2 = _on_device(_norm(g, N, 0.8)), _on_device(_norm(g, N, 0.5))
    x0 = torch.randn(rows, N, generator=g).to(DEV)
    xa, xb = x0.clone(), x0.clone()
    ha = hip_ops.tanh_stream_(xa, lin(h), n1, read=n2, out_dtype=torch.bfloat16)
    y = lin(h, defer=True)
    assert isinstance(y, hip_ops.PartialSums)
    hb = hip_ops.tanh_stream_(xb, y, n1, read=n2, out_dtype=torch.bfloat16)
    assert torch.equal(xa, xb) and torch.equal(ha, hb)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,width", [(5, 56), (3, 256), (300, 128)])
def test_entry_of_a_pass(dtype, T, width):
    """Both halves of the map, the vector of the pass, the norm behind them; the stream is not rounded to bf16."""
    from vllm_hymeta.models.squash_block import PassEntry, TanhNorm
    g = torch.Generator().manual_seed(width)
    w = (torch.randn(width, 2 * width, generator=g) * (2 * width) ** -0.5).to(dtype)
    steps = torch.randn(3, width, generator=g)
    n = _norm(g, width, 0.6)
    x, x0 = torch.randn(T, width, generator=g).to(dtype).float(), torch.randn(T, width, generator=g).to(dtype).float()
    entry, read = PassEntry(w[:, :width].to(DEV), w[:, width:].to(DEV), steps.to(DEV)), TanhNorm(n[0], n[1].to(DEV), n[2].to(DEV))
    start = entry.start_part(x0.to(dtype).to(DEV))
    for t in range(3):
        xd = x.to(DEV)
        h = entry(xd, xd.to(dtype), start, t, read, dtype)
        want = torch.cat([x, x0], -1).double() @ w.double().T + steps[t].double()
        assert rel_err(xd, want) < 2e-6
        assert rel_err(h, tanh_norm_ref(want, torch.tensor(n[0]).double(), n[1].double(), n[2].double())) < (2e-6 if dtype == torch.float32 else 4e-3)


# --------------------------------------------------------------------------- rotation, unit heads, cache rows
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("interleaved,unit,mag,k_scale", [(True, True, 1.3, 1.0), (True, False, 1.0, 1.0), (False, True, 0.8, 1.0), (True, True, 1.0, 0.25), (False, False, 1.5, 1.0)])
@pytest.mark.parametrize("H,G,D,Dv,rot", [(6, 2, 24, 16, 16), (3, 3, 10, 7, 6), (1, 1, 8, 8, 8), (8, 2, 128, 64, 128), (5, 1, 64, 12, 24), (2, 1, 40, 20, 0), (2, 2, 600, 8, 64)])
def test_rotation_with_unit_heads_and_the_paged_write(dtype, interleaved, unit, mag, k_scale, H, G, D, Dv, rot):
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(D)
    T, eps, page, pos = 9, 1e-3, 16, [0, 1, 2, 63, 64, 1000, 99991, 5, 17]
    cols = (H + G) * D + G * Dv + 5
    cols += -cols % 8 if D % 8 == 0 else 0                # rows of whole 16 bytes, or any
    qkv = torch.randn(T, cols, generator=g).to(dtype)
    qkv[4] *= 1e-3                                        # where eps counts
    freqs = torch.tensor([100.0 ** (-2 * i / max(rot, 1)) for i in range(rot // 2)], dtype=torch.float64)
    slots = [5, 40, -1, 0, 47, 17, 33, 1, 2]
    cache = torch.zeros(3, page, G, D + Dv, dtype=dtype, device=DEV)
    dev = qkv.to(DEV)
    hip_ops.rotary_cache_(dev, H, G, D, Dv, rot, freqs.to(DEV) if rot else None, k_scale, cache, torch.tensor(slots, device=DEV),
                          positions=torch.tensor(pos, device=DEV), interleaved=interleaved, rot_mag=mag, unit_eps=eps if unit else None)
    tol = 3e-6 if dtype == torch.float32 else 5e-3
    heads = qkv[:, :(H + G) * D].double().view(T, H + G, D)
    want = torch.empty_like(heads)
    for t in range(T):
        x = heads[t].clone()
        for i in range(rot // 2):
            p, r = (2 * i, 2 * i + 1) if interleaved else (i, i + rot // 2)
            c, s = math.cos(pos[t] * float(freqs[i])) * mag, math.sin(pos[t] * float(freqs[i])) * mag
            x[:, p], x[:, r] = heads[t, :, p] * c - heads[t, :, r] * s, heads[t, :, r] * c + heads[t, :, p] * s
        want[t] = rms_ref(x, eps) if unit else x
    want[:, H:] *= k_scale
    for t in range(T):
        assert rel_err(dev[t, :(H + G) * D].view(H + G, D), want[t]) < tol, t
    assert torch.equal(dev[:, (H + G) * D:].cpu(), qkv[:, (H + G) * D:])
    flat = cache.view(3 * page, G, D + Dv).cpu()
    for t, slot in enumerate(slots):
        if slot >= 0:
            assert torch.equal(flat[slot, :, :D], dev[t, H * D:(H + G) * D].view(G, D).cpu())
            assert torch.equal(flat[slot, :, D:], qkv[t, (H + G) * D:(H + G) * D + G * Dv].view(G, Dv))
    untouched = [s for s in range(3 * page) if s not in slots]
    assert not flat[untouched].any()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("half", [True, False])
@pytest.mark.parametrize("H,D,R,rot,C", [(6, 24, 12, 12, 36), (1, 5, 2, 2, 3), (4, 64, 64, 64, 128), (3, 16, 12, 8, 40), (2, 8, 0, 0, 24)])
def test_latent_rows_and_queries_without_a_query_latent(dtype, half, H, D, R, rot, C):
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(C)
    portions, contexts, eps, mag = [4, 1, 3], [0, 70, 29999], 1e-4, 1.0
    T, cols = sum(portions), H * (D + R)
    proj = torch.randn(T, cols + C + R + 3, generator=g).to(dtype)
    w = 1 + 0.3 * torch.randn(C, generator=g)
    freqs = torch.tensor([500.0 ** (-2 * i / max(rot, 1)) for i in range(rot // 2)], dtype=torch.float64, device=DEV)
    qsl, seq = i32([0, 4, 5, 8]), i32([4, 71, 30002])
    slots = [3, 0, 17, 31, 5, -1, 30, 8]
    cache = torch.zeros(2, 16, 1, C + R, dtype=dtype, device=DEV)
    dev = proj.to(DEV)
    hip_ops.latent_kv_prep_(dev, 0, 0, cols, C, R, rot, None, w.to(DEV), eps, freqs, mag, cache, torch.tensor(slots, device=DEV), qsl, seq, half)
    out = torch.full((T, H, C + R), 7.0, dtype=dtype, device=DEV)
    hip_ops.latent_q_rotate_(out, dev[:, :cols].view(T, H, D + R), D, R, rot, freqs, mag, qsl, seq, half)
    assert torch.equal(dev.cpu(), proj) and bool((out[:, :, :C] == 7.0).all())
    tol = 3e-6 if dtype == torch.float32 else 5e-3
    pos = [p for n, c in zip(portions, contexts) for p in range(c, c + n)]

    def turned(x, p):                                     # x [heads, R] at position p
        y = x.clone()
        for i in range(rot // 2):
            a, b = (i, i + rot // 2) if half else (2 * i, 2 * i + 1)
            c, s = math.cos(p * float(freqs[i])), math.sin(p * float(freqs[i]))
            y[:, a], y[:, b] = x[:, a] * c - x[:, b] * s, x[:, b] * c + x[:, a] * s
        return y

    for t, slot in enumerate(slots):
        row = proj[t].double()
        if R:
            assert rel_err(out[t, :, C:], turned(row[:cols].view(H, D + R)[:, D:], pos[t])) < tol
        if slot >= 0:
            want = torch.cat([rms_ref(row[cols:cols + C], eps) * w.double(), turned(row[None, cols + C:cols + C + R], pos[t])[0]])
            assert rel_err(cache.view(32, C + R)[slot], want) < tol


# --------------------------------------------------------------------------- attention in chunks, latent attention in a window
def _paged(rows, tables, page):
    """Rows per sequence (lists of [tokens, ...]) laid into their pages."""
    pages = sum(len(t) for t in tables)
    cache = torch.zeros(pages, page, *rows[0].shape[1:], dtype=rows[0].dtype)
    for r, t in zip(rows, tables):
        for j in range(r.shape[0]):
            cache[t[j // page], j % page] = r[j]
    return cache.to(DEV)


SHAPES = [(6, 2, 24, 16), (2, 2, 64, 64), (8, 2, 128, 128), (4, 1, 64, 128), (3, 3, 128, 64), (40, 1, 64, 64), (1, 1, 10, 7)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [1, 2, 29, 63, 64, 65, 100, 128, 1000])
@pytest.mark.parametrize("H,G,D,Dv", SHAPES)
def test_chunked_attention_of_portions_and_single_rows(dtype, chunk, H, G, D, Dv):
    """Portions and single rows of unequal sequences in one step, their keys on scattered pages."""
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(chunk + D)
    page = 16 if chunk % 2 else 64
    portions, contexts = [70, 1, 2, 1, 12, 1], [0, 0, 63, 130, 95, 99]
    totals = [n + c for n, c in zip(portions, contexts)]
    tables = scattered(len(portions), (max(totals) + page - 1) // page, chunk)
    q = [torch.randn(n, H, D, generator=g).to(dtype) for n in portions]
    kv = [torch.randn(n, G, D + Dv, generator=g).to(dtype) for n in totals]
    gate = torch.randn(sum(portions), H, generator=g).to(dtype)
    lay = layout_of(portions, contexts, tables, page)
    out = hip_ops.sink_attention(torch.cat(q).to(DEV), _paged(kv, tables, page), lay.block_tables, lay.query_start_loc, lay.seq_lens, G, D, Dv, D ** -0.5,
                                 lay.max_query_len, lay.max_seq_len, sink=False, chunk=chunk, head_gate=gate.to(DEV))
    tol, r = (2e-5 if dtype == torch.float32 else 6e-3), 0
    for n, ctx, qs, rows in zip(portions, contexts, q, kv):
        full = torch.cat([torch.zeros(ctx, H, D, dtype=torch.float64), qs.double()])
        ref = attend_ref(full, rows[:, :, :D].double(), rows[:, :, D:].double(), D ** -0.5, in_chunk(chunk))[ctx:]
        ref = ref * torch.sigmoid(gate[r:r + n].double())[:, :, None]
        assert rel_err(out[r:r + n], ref) < tol, (n, ctx)
        r += n


def _edge_case(dtype, D, Dv, i, key, n_rows):
    """A sequence of i + 1 rows in which the query at place i matches the key at place ``key`` by far the best, whose value stands
    out; the last n_rows are the step's rows.  Returns (queries, keys, values)."""
    g = torch.Generator().manual_seed(i * 31 + key)
    k, v = 0.1 * torch.randn(i + 1, 1, D, generator=g), torch.randn(i + 1, 1, Dv, generator=g)
    q = 0.1 * torch.randn(i + 1, 1, D, generator=g)
    star = torch.sign(torch.randn(D, generator=g))
    q[i, 0], k[key, 0] = star, star
    v[key] += 20.0
    return (t.to(dtype) for t in (q[i + 1 - n_rows:], k, v))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,Dv", [(64, 64), (128, 128), (24, 20)])
@pytest.mark.parametrize("size,i", [(40, 159), (40, 120), (40, 121), (64, 127), (64, 128), (64, 191), (100, 250), (100, 200), (37, 36), (37, 37), (1, 5), (500, 499), (500, 505)])
@pytest.mark.parametrize("n_rows", [1, 2, 50])
def test_keys_just_inside_and_just_outside_a_chunk_or_a_window(dtype, D, Dv, size, i, n_rows):
    """A key that would win the softmax stands on the first place the query sees, on the place before it, and on the first
    place of the sequence: it shows in the first case and not in the others (unless that place is seen)."""
    from vllm_hymeta import hip_ops
    n_rows = min(n_rows, i + 1)
    for mode, first in (("chunk", in_chunk(size)(i)), ("window", in_window(size)(i))):
        for key in {first, first - 1, 0, i}:
            if key < 0:
                continue
            q, k, v = _edge_case(dtype, D, Dv, i, key, n_rows)
            page = 64 if D != 24 else 16
            tables = scattered(1, i // page + 1)
            lay = layout_of([n_rows], [i + 1 - n_rows], tables, page)
            out = hip_ops.sink_attention(q.to(DEV), _paged([torch.cat([k, v], -1)], tables, page), lay.block_tables, lay.query_start_loc, lay.seq_lens, 1, D, Dv, 1.0,
                                         lay.max_query_len, lay.max_seq_len, sink=False, **({"chunk": size} if mode == "chunk" else {"window_left": size - 1}))
            full = torch.cat([torch.zeros(i + 1 - n_rows, 1, D, dtype=torch.float64), q.double()])
            ref = attend_ref(full, k.double(), v.double(), 1.0, (in_chunk if mode == "chunk" else in_window)(size))
            assert rel_err(out[-1], ref[i]) < (1e-5 if dtype == torch.float32 else 6e-3), (mode, key)
            assert (float(out[-1].float().mean()) > 10) == (key >= first), (mode, key)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,C,R", [(6, 36, 12), (4, 64, 32), (16, 128, 64), (28, 128, 32), (3, 256, 64), (40, 64, 64), (2, 384, 64), (1, 20, 0)])
@pytest.mark.parametrize("window", [1, 13, 64, 65, 200])
def test_latent_rows_in_a_window_with_a_sink(dtype, H, C, R, window):
    """Values inside the keys; one head's sink outweighs everything, another's nothing; a far row would win where it is seen."""
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(window + C)
    page = 64 if window % 2 == 0 else 16
    portions, contexts = [90, 1, 2, 1], [0, 127, 200, 64]
    totals = [n + c for n, c in zip(portions, contexts)]
    tables = scattered(len(portions), (max(totals) + page - 1) // page, window)
    q = [torch.randn(n, H, C + R, generator=g).to(dtype) for n in portions]
    rows = [torch.randn(n, 1, C + R, generator=g).to(dtype) for n in totals]
    for s, (n, c) in enumerate(zip(portions, contexts)):      # just inside the last row's window, and just outside
        for back, gain in ((window - 1, 0.5), (window, 2.0)):
            if n + c - 1 - back >= 0:
                rows[s][n + c - 1 - back, 0] = gain * q[s][-1, 0]
    sink = torch.randn(H, generator=g)
    sink[0] = 6.0
    sink[-1] = -30.0
    lay = layout_of(portions, contexts, tables, page)
    scale = (C + R) ** -0.5
    out = hip_ops.sink_attention(torch.cat(q).to(DEV), _paged(rows, tables, page), lay.block_tables, lay.query_start_loc, lay.seq_lens, 1, C + R, C, scale,
                                 lay.max_query_len, lay.max_seq_len, sink=True, sink_logits=sink.to(DEV), value_in_key=True, window_left=window - 1)
    r = 0
    for n, ctx, qs, rw in zip(portions, contexts, q, rows):
        full = torch.cat([torch.zeros(ctx, H, C + R, dtype=torch.float64), qs.double()])
        ref = attend_ref(full, rw.double(), rw[:, :, :C].double(), scale, in_window(window), sink.double())[ctx:]
        assert rel_err(out[r:r + n], ref) < (2e-5 if dtype == torch.float32 else 6e-3), (n, ctx)
        r += n


def test_a_chunk_and_a_window_together_are_refused():
    from vllm_hymeta import hip_ops
    from vllm_hymeta.models.rotary_window_attention import PagedWindowAttention
    q, kv = torch.zeros(1, 1, 8, device=DEV), torch.zeros(1, 16, 1, 16, device=DEV)
    with pytest.raises(Exception):
        hip_ops.sink_attention(q, kv, i32([[0]]), i32([0, 1]), i32([1]), 1, 8, 8, 1.0, 1, 1, sink=False, chunk=4, window_left=3)
    with pytest.raises(Exception):
        hip_ops.sink_attention(q, kv, i32([[0]]), i32([0, 1]), i32([1]), 1, 8, 8, 1.0, 1, 1, sink=False, chunk=-1)
    with pytest.raises(ValueError):
        PagedWindowAttention(1, 1, 8, 8, 1.0, "banitar.refused", sliding_window=3, chunk=4)


# --------------------------------------------------------------------------- whole models under the engine
def build_engine(cfg, weights, dtype, max_tokens=512, block_size=16, max_num_seqs=4, max_num_batched_tokens=1 << 30):
    from vllm_hymeta.engine import LLMEngine
    from vllm_hymeta.models.configuration_banitar import BanitarConfig
    from vllm_hymeta.models.modeling_banitar import BanitarForCausalLM
    model = BanitarForCausalLM(BanitarConfig(cfg), max_num_seqs=max_num_seqs, dtype=dtype, device=DEV)
    model.load_weights(weights.items())
    return LLMEngine(model, num_blocks=max_tokens // block_size, block_size=block_size, max_num_seqs=max_num_seqs,
                     max_num_batched_tokens=max_num_batched_tokens, device=DEV)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunked,latent", [(chunked_config(), latent_config()), (chunked_config(heads=4, kv_heads=4, dim=64, vdim=64, chunk=70, rot_dims=32), latent_config(heads=4, dim=32, rot_dim=32, vdim=48, kv_rank=64, window=65)),
                                            (chunked_config(heads=1, kv_heads=1, dim=8, vdim=8, chunk=1, rot_dims=8), latent_config(heads=1, dim=4, rot_dim=2, vdim=3, kv_rank=5, window=1)),
                                            (chunked_config(heads=8, kv_heads=1, dim=128, vdim=64, chunk=64, rot_dims=128, scaling={"factor": 2.0, "original": 32, "fast": 2.0, "slow": 0.1}),
                                             latent_config(heads=20, dim=64, rot_dim=64, vdim=64, kv_rank=128, window=33))])
def test_sublayers_alone_against_the_oracle(dtype, chunked, latent):
    eps, W, T = 1e-5, 64, 140
    cfg = banitar_config(vocab=40, width=W, eps=eps, layers=[("attention", chunked, 48), ("latent_attention", latent, None)], loop=None)
    w = banitar_random_weights(cfg, seed=5)
    eng = build_engine(cfg, w, dtype, max_tokens=192, block_size=16)
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(1)).to(dtype)
    model = eng.model.model
    table = [[7, 3, 0, 11, 5, 2, 9, 1, 10, 4, 8, 6]]
    tol = 2e-5 if dtype == torch.float32 else 2.5e-2
    sub = lambda p: {k[len(p):]: v.double() for k, v in w.items() if k.startswith(p)}      # noqa: E731
    for layer, ref in ((0, chunked_attention_ref(h.double(), sub("l0.mix."), chunked, eps)), (1, latent_attention_ref(h.double(), sub("l1.mix."), latent, eps))):
        attn, at, got = model.attn_layers[f"{layer}_0"], 0, []
        for n in (70, 2, 1, 1, 66):                            # portions, the pages filled as they come
            got.append(model.layers[layer].mixer(h[at:at + n].to(DEV), layout_of([n], [at], table, 16), attn))
            at += n
        assert rel_err(torch.cat(got), ref) < tol, layer
    assert rel_err(model.layers[0].mlp(h.to(DEV)), silu_glu_ref(h.double(), sub("l0.mlp."))) < tol


MODELS = {
    "default": dict(),
    "ones_and_equals": dict(width=40, embed_scale=1.0, loop=(0, 3, 1), layers=[       # one head, a chunk and a window of one token, one pass over everything
        ("attention", chunked_config(heads=1, kv_heads=1, dim=8, vdim=8, chunk=1, rot_dims=2, scaling=None), None),
        ("latent_attention", latent_config(heads=1, dim=8, rot_dim=8, vdim=8, kv_rank=8, window=1), 40),
        ("attention", chunked_config(heads=2, kv_heads=2, dim=40, vdim=40, chunk=9, rot_dims=40, scale=0.1), 16)]),
    "matrix_core_sizes": dict(width=256, vocab=192, loop=(1, 4, 2), layers=[
        ("attention", chunked_config(heads=8, kv_heads=2, dim=64, vdim=64, chunk=70, rot_dims=64), 256),
        ("latent_attention", latent_config(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=64, window=65), 320),
        ("attention", chunked_config(heads=2, kv_heads=1, dim=128, vdim=64, chunk=64, rot_dims=96), None),
        ("latent_attention", latent_config(heads=18, dim=32, rot_dim=64, vdim=32, kv_rank=128, window=33), 256)]),
    "no_loop": dict(width=72, loop=None, layers=[("latent_attention", latent_config(heads=3, window=40), 56),
                                                 ("attention", chunked_config(heads=2, kv_heads=1, chunk=50), 33)]),
    "loop_first_then_a_tail": dict(width=48, loop=(0, 1, 4), layers=[("latent_attention", latent_config(heads=2, dim=10, rot_dim=6, vdim=14, kv_rank=18, window=30), 64),
                                                                     ("attention", chunked_config(heads=4, kv_heads=2, chunk=32), 64)]),
}


def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


TOL = {torch.float32: 5e-5, torch.bfloat16: 0.05}


@pytest.mark.parametrize("name", sorted(MODELS))
def test_model_whole_prompt_against_the_oracle_fp32(name):
    """One step for the whole prompt, every position's logits and the stream after every layer run."""
    cfg = banitar_config(**MODELS[name])
    weights = banitar_random_weights(cfg, seed=len(name))
    toks = _tokens(150, cfg["vocab"], 7)
    stream_ref = []
    ref = banitar_ref(cfg, weights, toks, residual_out=stream_ref)
    eng = build_engine(cfg, weights, torch.float32, max_tokens=256, block_size=16)
    stream = []
    inner = eng.model.model
    plain = inner.forward
    inner.forward = lambda *a, **k: plain(*a, residual_out=stream, **k)
    got = eng.run_batch([("a", toks, list(range(len(toks))))])
    assert len(stream) == len(stream_ref) == len(inner.runs)
    for n, (s, r) in enumerate(zip(stream, stream_ref)):
        assert rel_err(s, r) < 2e-5, (n, inner.runs[n])
    assert rel_err(got, ref) < TOL[torch.float32]


def _replay(eng, seqs, plan):
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    for step in plan:
        out = eng.run_batch([(f"r{k}", seqs[k][at[k]:at[k] + n], list(range(n))) for k, n in step])
        row = 0
        for k, n in step:
            got[k].append(out[row:row + n])
            row += n
            at[k] += n
            if at[k] == len(seqs[k]):
                eng.finish_request(f"r{k}")
    return {k: torch.cat(v) for k, v in got.items() if v}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_model_schedules_agree_with_the_whole_prompt(name, dtype):
    cfg = banitar_config(**MODELS[name])
    weights = banitar_random_weights(cfg, seed=len(name))
    seqs = {k: _tokens(n, cfg["vocab"], 10 + k) for k, n in enumerate([150, 33, 1, 70, 19, 64])}
    refs = {k: banitar_ref(cfg, weights, t) for k, t in seqs.items()}
    tol = TOL[dtype]
    page = 64 if name == "matrix_core_sizes" else 16
    pages = 320 // page
    eng = build_engine(cfg, weights, dtype, max_tokens=pages * page, block_size=page, max_num_seqs=4)
    whole = {}
    for k, t in seqs.items():
        whole[k] = eng.run_batch([(f"w{k}", t, list(range(len(t))))])
        eng.finish_request(f"w{k}")
        assert rel_err(whole[k], refs[k]) < tol, k
    assert eng.pool.num_free == pages
    # token by token after a prompt that ends inside a page
    got = _replay(eng, seqs, [[(0, 85)]] + [[(0, 1)]] * 65)
    assert rel_err(got[0], whole[0]) < tol and rel_err(got[0], refs[0]) < tol
    # token by token from the very first token
    got = _replay(eng, seqs, [[(1, 1)]] * 33)
    assert rel_err(got[1], whole[1]) < tol
    # portions: 2, 1, 3, ... across page borders and the edges of chunks and windows
    got = _replay(eng, seqs, [[(0, n)] for n in (2, 1, 3, 10, 2, 45, 2, 64, 2, 19)])
    assert rel_err(got[0], whole[0]) < tol
    # mixed: up to four live requests, portions beside single tokens, a request that pauses, requests that end and free
    # pages for new ones
    plan = [[(0, 70), (1, 2)], [(0, 1), (1, 31), (2, 1)], [(0, 1), (3, 16), (4, 2)], [(0, 78), (3, 1), (4, 17)], [(3, 53), (5, 3)], [(5, 2)], [(5, 59)]]
    got = _replay(eng, seqs, plan)
    for k in seqs:
        assert rel_err(got[k], whole[k]) < tol and rel_err(got[k], refs[k]) < tol, k
    assert eng.pool.num_free == pages and not eng.requests


def test_every_pass_has_a_cache_of_its_own():
    """Garbage in one pass's pages changes the output; the passes' pages differ."""
    cfg = banitar_config()
    eng = build_engine(cfg, banitar_random_weights(cfg, seed=2), torch.float32, max_tokens=64)
    names = list(eng.kv_caches)
    assert len(names) == len(set(names)) == 2 + 2 * 3 and sum("pass2" in n for n in names) == 2
    toks = _tokens(21, cfg["vocab"], 1)
    eng.run_batch([("a", toks[:20], [])])
    out = eng.run_batch([("a", toks[20:], [0])])
    eng.finish_request("a")
    for n in names:
        for m in names:
            if n < m:
                assert eng.kv_caches[n].shape != eng.kv_caches[m].shape or not torch.equal(eng.kv_caches[n], eng.kv_caches[m])
    for n in names:
        eng.run_batch([("b", toks[:20], [])])
        eng.kv_caches[n].normal_()
        moved = rel_err(eng.run_batch([("b", toks[20:], [0])]), out)
        eng.finish_request("b")
        assert moved > 1e-3, n


@pytest.mark.parametrize("dtype", DTYPES)
def test_positions_may_be_left_out(dtype):
    """A caller that gives no positions: the rows' places in their sequences."""
    cfg = banitar_config()
    eng = build_engine(cfg, banitar_random_weights(cfg, seed=1), dtype, max_tokens=256)
    toks = _tokens(40, cfg["vocab"], 2)
    a = eng.run_batch([("a", toks, list(range(40)))])
    inner = eng.model.model
    plain = inner.forward
    inner.forward = lambda ids, pos=None, **k: plain(ids, None, **k)
    eng.run_batch([("b", toks[:17], [])])
    b = eng.run_batch([("c", toks, list(range(40))), ("b", toks[17:], list(range(23)))])
    assert rel_err(b[:40], a) < TOL[dtype] and rel_err(b[40:], a[17:]) < TOL[dtype]


def test_greedy_generation_through_the_scheduler_matches_the_oracle():
    """engine.generate: six prompts, two places, a token budget that cuts prompts into portions -- the scheduler batches
    portions beside decoded tokens and reuses pages; every generated token is the oracle's argmax."""
    from vllm_hymeta.engine import SamplingParams
    cfg = banitar_config()
    weights = banitar_random_weights(cfg, seed=4)
    prompts = [_tokens(n, cfg["vocab"], 40 + n) for n in (23, 5, 1, 37, 12, 18)]
    new = 5
    eng = build_engine(cfg, weights, torch.float32, max_tokens=128, block_size=16, max_num_seqs=2, max_num_batched_tokens=16)
    outs = eng.generate(prompts, SamplingParams(max_tokens=new))
    assert eng.pool.num_free == 8 and not eng.requests
    for p, o in zip(prompts, outs):
        assert len(o) == new
        logits = banitar_ref(cfg, weights, list(p) + o)
        for j, t in enumerate(o):
            row = logits[len(p) - 1 + j]
            top2 = row.topk(2).values
            if float(top2[0] - top2[1]) > 1e-3:        # a clear winner: the engine must have picked it
                assert t == int(row.argmax())


@pytest.mark.parametrize("dtype,name", [(torch.float32, "default"), (torch.bfloat16, "matrix_core_sizes")])
def test_long_decode_passes_every_window_and_every_chunk(dtype, name):
    """400 tokens decoded one by one after a two-token prompt: every window passes over decoded tokens and every chunk ends
    many times."""
    cfg = banitar_config(**MODELS[name])
    weights = banitar_random_weights(cfg, seed=8)
    toks = _tokens(402, cfg["vocab"], 3)
    page = 64 if dtype == torch.bfloat16 else 32
    eng = build_engine(cfg, weights, dtype, max_tokens=448, block_size=page, max_num_seqs=1)
    places = [17, 69, 70, 139, 140, 200, 333, 401]
    whole = eng.run_batch([("w", toks, places)])
    eng.finish_request("w")
    eng.run_batch([("d", toks[:2], [])])
    for i in range(2, 402):
        out = eng.run_batch([("d", toks[i:i + 1], [0] if i in places else [])])
        if i in places:
            assert rel_err(out, whole[places.index(i):places.index(i) + 1]) < 2 * TOL[dtype], i
    eng.finish_request("d")
    if dtype == torch.float32:
        assert rel_err(eng.run_batch([("x", toks[:201], [200])]), banitar_ref(cfg, weights, toks[:201])[-1:]) < TOL[dtype]


@pytest.mark.parametrize("name", ["default", "matrix_core_sizes"])
def test_a_decode_step_replayed_from_a_graph(name):
    """Three sequences of different lengths decode eight tokens: the step captured once and replayed, with eager work and
    synchronisations between the replays, against the engine's eager steps."""
    from vllm_hymeta.attention.meta_attention import MetaAttentionMetadata
    from vllm_hymeta.models.attention import bind_kv_cache
    cfg = banitar_config(**MODELS[name])
    weights = banitar_random_weights(cfg, seed=3)
    prompts, new, page, blocks = [_tokens(n, cfg["vocab"], n) for n in (90, 5, 64)], 8, 64, 2
    fed = torch.tensor([_tokens(new, cfg["vocab"], 70 + s) for s in range(3)])
    eng = build_engine(cfg, weights, torch.bfloat16, max_tokens=6 * page, block_size=page, max_num_seqs=3)
    for s, p in enumerate(prompts):
        eng.run_batch([(f"s{s}", p, [])])
    model = eng.model
    tables = torch.zeros(3, blocks, dtype=torch.int32)
    for s in range(3):
        r = eng.requests[f"s{s}"]
        eng.pool.grow(r.blocks, len(prompts[s]) + new)
        tables[s, :len(r.blocks)] = torch.tensor(r.blocks, dtype=torch.int32)
    cache_before = {n: t.clone() for n, t in eng.kv_caches.items()}
    want = [eng.run_batch([(f"s{s}", [int(fed[s, t])], [0]) for s in range(3)]) for t in range(new)]

    def rewind():
        for n, t in eng.kv_caches.items():
            t.copy_(cache_before[n])
            bind_kv_cache(eng.attn_layers[n], t)

    lens = torch.tensor([len(p) for p in prompts])
    ids, pos = torch.zeros(3, dtype=torch.int64, device=DEV), torch.zeros(3, dtype=torch.int64, device=DEV)
    seq, ctx, sm = i32([0, 0, 0]), i32([0, 0, 0]), torch.zeros(3, dtype=torch.int64, device=DEV)
    md = MetaAttentionMetadata(
        num_prefills=0, num_prefill_tokens=0, num_decode_tokens=3, slot_mapping=sm, multi_modal_placeholder_index_maps=None,
        enable_kv_scales_calculation=False, seq_lens=None, seq_lens_tensor=seq, max_prefill_seq_len=0, max_decode_seq_len=2 * page,
        context_lens_tensor=ctx, block_tables=tables.to(DEV), use_cuda_graph=True, max_query_len=1, max_decode_query_len=1,
        query_start_loc=i32([0, 1, 2, 3]), seq_start_loc=None)

    def inputs(t):
        p = lens + t
        ids.copy_(fed[:, t]), pos.copy_(p), seq.copy_(p + 1), ctx.copy_(p)
        sm.copy_(torch.tensor([int(tables[s, int(p[s]) // page]) * page + int(p[s]) % page for s in range(3)]))

    with torch.inference_mode():
        step = lambda: model.compute_logits(model(ids, pos, attn_metadata=md))      # noqa: E731
        inputs(0)
        side, graph = torch.cuda.Stream(), torch.cuda.CUDAGraph()
        with torch.cuda.stream(side):
            step()
            with torch.cuda.graph(graph, stream=side):
                logits = step()
        torch.cuda.synchronize()
        rewind()
        for t in range(new):
            inputs(t)
            graph.replay()
            torch.cuda.synchronize()
            assert rel_err(logits, want[t]) < 1e-3, t
            torch.ones(1000, device=DEV).sum().item()


def test_trace_runner_and_generate_command_lines(tmp_path):
    """A checkpoint folder (config.json + model.safetensors) served by the two programs under bin/: the trace replayer
    runs portions, single tokens and two requests side by side, gives pages back at a request's end and writes the logits
    asked for (fp32 against the oracle); the generator's greedy tokens are the oracle's argmax."""
    import json
    import os
    import subprocess
    import sys
    import numpy as np
    from safetensors.torch import save_file
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = banitar_config()
    weights = banitar_random_weights(cfg, seed=12)
    model_dir = tmp_path / "model"
    model_dir.mkdir()
    (model_dir / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, str(model_dir / "model.safetensors"))
    a, b = _tokens(90, cfg["vocab"], 5), _tokens(40, cfg["vocab"], 6)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:50], "want": [0, 49]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[50:52], "want": []}, {"id": "b", "tokens": b[:39], "want": [38]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[39:], "want": [0]}, {"id": "a", "tokens": a[52:53], "want": [0]}], "end": ["b"]},
        {"step": 3, "entries": [{"id": "a", "tokens": a[53:], "want": [36]}, {"id": "c", "tokens": b[:7], "want": [6]}], "end": ["a", "c"]},
    ]
    out_dir = tmp_path / "out"
    run = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(model_dir), "--dtype", "float32", "--out", str(out_dir),
                          "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {k}" for k in range(4)]
    ra, rb = banitar_ref(cfg, weights, a), banitar_ref(cfg, weights, b)
    want = {0: torch.stack([ra[0], ra[49]]), 1: rb[38:39], 2: torch.stack([rb[39], ra[52]]), 3: torch.stack([ra[89], rb[6]])}
    for k, ref in want.items():
        got = torch.from_numpy(np.fromfile(str(out_dir / f"{k}.f32"), dtype="<f4").reshape(ref.shape[0], -1))
        assert rel_err(got, ref) < TOL[torch.float32], k
    gen = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), "--model", str(model_dir), "--dtype", "float32", "--prompt-ids",
                          ",".join(map(str, a[:20])), "--max-new-tokens", "3", "--max-tokens", "128"], capture_output=True, text=True, timeout=100)
    assert gen.returncode == 0, gen.stderr[-2000:]
    line = json.loads([l for l in gen.stdout.splitlines() if l.startswith("{")][-1])
    assert len(line["output"]) == 3
    logits = banitar_ref(cfg, weights, a[:20] + line["output"])
    for j, t in enumerate(line["output"]):
        top2 = logits[19 + j].topk(2).values
        if float(top2[0] - top2[1]) > 1e-3:
            assert t == int(logits[19 + j].argmax())


def _random_model(seed):
    """Sizes drawn at random: layer order and loop, head counts, group sizes, key, value and latent sizes (also such that a layer
    takes the matrix-core kernels), chunks and windows around a page and a tile, rotations."""
    import random
    r = random.Random(seed)
    layers = []
    sizes = [1, 2, 7, 15, 16, 17, 63, 64, 65, 100, 128, 1000]
    for _ in range(r.randint(1, 4)):
        if r.random() < 0.5:
            G = r.choice([1, 2, 3])
            D, Dv = (r.choice([64, 128]), r.choice([64, 128])) if r.random() < 0.5 else (r.randint(3, 50), r.randint(3, 50))
            scaling = r.choice([None, "yarn", {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}, {"factor": 1.0, "original": 16, "fast": 1.0, "slow": 1.0}])
            mixer = ("attention", chunked_config(heads=G * r.choice([1, 2, 3, 5]), kv_heads=G, dim=D, vdim=Dv, chunk=r.choice(sizes), rot_dims=2 * r.randint(1, D // 2),
                                                 base=r.choice([100.0, 1e4, 1e6]), scaling=scaling, scale=r.choice([D ** -0.5, 0.3, 0.05])))
        else:
            C, R = (r.choice([64, 128, 256]), 64) if r.random() < 0.5 else (r.randint(4, 60), 2 * r.randint(1, 12))
            mixer = ("latent_attention", latent_config(heads=r.choice([1, 2, 3, 5, 20]), dim=r.randint(3, 40), rot_dim=R, vdim=r.randint(3, 40), kv_rank=C, window=r.choice(sizes),
                                                       base=r.choice([100.0, 1e4, 1e6])))
        layers.append(mixer + (r.choice([None, 16, 72, 128]),))
    start = r.randint(0, len(layers) - 1)
    loop = None if r.random() < 0.2 else (start, r.randint(start + 1, len(layers)), r.randint(1, 3))
    return banitar_config(vocab=r.choice([50, 130]), width=r.choice([24, 40, 64, 96, 128, 200]), layers=layers, loop=loop, eps=r.choice([1e-5, 1e-6, 1e-3]), embed_scale=r.choice([1.0, 2.5, 12.0]))


@pytest.mark.parametrize("seed", range(12))
def test_models_of_random_sizes_under_the_engine(seed):
    """A prompt of 190 tokens in one step, then in portions and single tokens beside a second request, against the oracle."""
    cfg = _random_model(seed)
    weights = banitar_random_weights(cfg, seed=seed)
    seqs = {0: _tokens(190, cfg["vocab"], 100 + seed), 1: _tokens(75, cfg["vocab"], 200 + seed)}
    refs = {k: banitar_ref(cfg, weights, t) for k, t in seqs.items()}
    page = 64 if seed % 2 else 16
    plan = [[(0, 3)], [(0, 64), (1, 2)], [(0, 1), (1, 1)], [(0, 62), (1, 70)], [(0, 1), (1, 1)], [(0, 2), (1, 1)], [(0, 57)]]
    for dtype in DTYPES:
        eng = build_engine(cfg, weights, dtype, max_tokens=448, block_size=page, max_num_seqs=2)
        whole = eng.run_batch([("w", seqs[0], list(range(190)))])
        eng.finish_request("w")
        got = _replay(eng, seqs, plan)
        assert not eng.requests
        assert rel_err(whole, refs[0]) < TOL[dtype] and all(rel_err(got[k], refs[k]) < TOL[dtype] for k in seqs), dtype
