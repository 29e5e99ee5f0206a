"""The Nilevik building blocks and the model under the engine, against the plain CPU statement in ``oracle/nilevik.py``.

Mechanisms alone first (embedding rows with the position's sinusoid, the normed sum with the stream's copy, the gelu-gated
units, the queries' norm and temperature with the scaled-key cache, the attention over it, the gated delta rule as a step,
in chunks and token by token), then whole models of several shapes: a prompt in one step against the oracle, and the same
tokens cut into steps in every way the engine allows (token by token, portions down to two tokens, unequal requests in one
batch, pages and state slots used again) against the one-step result.
"""
import math

import pytest
import torch
import torch.nn.functional as F

pytestmark = pytest.mark.gpu

from oracle.nilevik import (attention_config, attention_mixer_ref, delta_config, delta_mixer_ref, delta_rule_ref, gelu_tanh_ref,  # noqa: E402
                            nilevik_config, nilevik_random_weights, nilevik_ref, penalised_sink_attention_ref, query_temperature_ref, rms_ref,
                            sinusoid_ref, slope_ref, token_side_ref, unit_ref)

DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


def rel_err(got: torch.Tensor, ref: torch.Tensor) -> float:
    got, ref = got.double().cpu(), ref.double().cpu()
    assert torch.isfinite(got).all()
    return float((got - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


def rows_close(got: torch.Tensor, ref: torch.Tensor, tol: float, exact: bool) -> bool:
    """fp32 (``exact``): the whole tensor within ``tol``.  bf16: the typical row within ``0.6 tol`` and at most one row in ten
    (or one) beyond ``tol``: the norm of what a sublayer adds makes much of a rounding where a head's small output nearly
    cancels (relative noise of 2^-9 on the weights moves the same rows of the oracle as far)."""
    if exact:
        return rel_err(got, ref) < tol
    got, ref = got.double().cpu(), ref.double().cpu()
    err = (got - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt().clamp_min(1e-30)
    return float(err.median()) < 0.6 * tol and int((err > tol).sum()) <= max(1, err.numel() // 10)


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def layout_of(portions, contexts, slots, block_tables=None, block_size=16):
    """A step's layout from (rows, tokens before them, state slot) per sequence."""
    from itertools import accumulate
    from vllm_hymeta.models.stream_block import StepLayout
    qsl = list(accumulate(portions, initial=0))
    slot_mapping = bt = None
    if block_tables is not None:
        width = max(len(t) for t in block_tables)
        bt = torch.zeros(len(block_tables), width, dtype=torch.int32)
        sm = []
        for s, (n, ctx) in enumerate(zip(portions, contexts)):
            bt[s, :len(block_tables[s])] = torch.tensor(block_tables[s], dtype=torch.int32)
            sm += [block_tables[s][p // block_size] * block_size + p % block_size for p in range(ctx, ctx + n)]
        bt, slot_mapping = bt.to(DEV), torch.tensor(sm, dtype=torch.int64, device=DEV)
    positions = torch.tensor(sum((list(range(c, c + n)) for n, c in zip(portions, contexts)), []), dtype=torch.int64, device=DEV)
    return StepLayout(query_start_loc=i32(qsl), context_lens=i32(contexts), seq_lens=i32([c + n for c, n in zip(contexts, portions)]),
                      slot_idx=i32(slots), block_tables=bt, slot_mapping=slot_mapping, max_query_len=max(portions),
                      max_seq_len=max(c + n for c, n in zip(contexts, portions)), positions=positions)


def in_steps(seqs, plan, run):
    """Cut the sequences' rows into the plan's steps (lists of (sequence, rows)), call ``run([(sequence, context, rows)])`` per
    step, and return every sequence's outputs joined."""
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    for step in plan:
        out = run([(k, at[k], n) for k, n in step])
        r = 0
        for k, n in step:
            got[k].append(out[r:r + n])
            r += n
            at[k] += n
    return {k: torch.cat(v) for k, v in got.items() if v}


# --------------------------------------------------------------------------- embedding rows, the normed sum, gelu units
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [56, 33, 1024])
def test_embedding_rows_with_the_positions_sinusoid(dtype, width):
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(width)
    V = 50
    table = torch.randn(V, width, generator=g).to(dtype)
    ids = torch.randint(0, V, (9,), generator=g)
    pos = torch.tensor([0, 1, 2, 63, 64, 1000, 4095, 99999, 5])
    freqs = torch.tensor([10000.0 ** (-2.0 * i / width) for i in range((width + 1) // 2)], dtype=torch.float64, device=DEV)
    wave = sinusoid_ref(100000, width)[pos] if width < 100 else torch.cat([sinusoid_ref(int(p) + 1, width)[-1:] for p in pos[:6]])
    n = wave.shape[0]
    x, h = hip_ops.embed_rows(ids[:n].to(DEV), table.to(DEV), positions=pos[:n].to(DEV), pos_freqs=freqs, copy=True)
    ref = table[ids[:n]].double() + wave
    assert x.dtype == torch.float32 and h.dtype == dtype and float((x.double().cpu() - ref).abs().max()) < 2e-6
    assert torch.equal(h, x.to(dtype))
    assert torch.equal(hip_ops.embed_rows(ids.to(DEV), table.to(DEV)).cpu(), table[ids].float())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,pad", [(56, 0), (33, 0), (64, 3), (1024, 8), (4096, 0), (5000, 0)])
def test_normed_sum_with_the_streams_copy(dtype, width, pad):
    from vllm_hymeta.models.added_norm_block import AddNormed
    g = torch.Generator().manual_seed(width)
    T, eps = 7, 1e-4
    x0, y0 = torch.randn(T, width, generator=g), (torch.randn(T, width + pad, generator=g) * 0.01).to(dtype)[:, :width]
    w = 1 + 0.3 * torch.randn(width, generator=g)
    ref = x0.double() + rms_ref(y0.double(), eps) * w.double()
    x = x0.clone().to(DEV)
    y = torch.zeros(T, width + pad, dtype=dtype)
    y[:, :width] = y0
    h = AddNormed(w.to(DEV), eps)(x, y.to(DEV)[:, :width])
    assert rel_err(x, ref) < 1e-6 and torch.equal(h, x.to(dtype)) and (h is x) == (dtype == torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,pad", [(24, 0), (7, 0), (512, 8), (1500, 1)])
def test_gelu_gated_units_and_rows_of_a_table(dtype, n, pad):
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(n)
    T, V, tol = 13, 29, 2e-6 if dtype == torch.float32 else 4e-3
    x = (torch.randn(T, 2 * n, generator=g) * 3).to(dtype)
    x[0, :4] = torch.tensor([-40.0, 40.0, 0.0, -5.0]).to(dtype)
    out = hip_ops.gelu_mul(x.to(DEV))
    assert rel_err(out, gelu_tanh_ref(x[:, :n].double()) * x[:, n:].double()) < tol
    table = torch.randn(V, 3 * n + pad, generator=g).to(dtype)
    ids = torch.randint(0, V, (T,), generator=g)
    got = hip_ops.gelu_mul_rows(x[:, :n].contiguous().to(DEV), table.to(DEV)[:, n:2 * n], ids.to(DEV))
    assert rel_err(got, gelu_tanh_ref(x[:, :n].double()) * table[ids, n:2 * n].double()) < tol


@pytest.mark.parametrize("dtype", DTYPES)
def test_token_input_picks_the_layers_columns(dtype):
    from vllm_hymeta.linear import HymetaLinear
    from vllm_hymeta.models.added_norm_block import AddNormed, TokenInput
    g = torch.Generator().manual_seed(3)
    W, d, V, L, T, eps = 72, 20, 31, 3, 40, 1e-5
    w = {"gate": torch.randn(d, W, generator=g) * W ** -0.5, "proj": torch.randn(W, d, generator=g) * d ** -0.5, "norm": 1 + 0.2 * torch.randn(W, generator=g)}
    w = {k: v.to(torch.bfloat16).float() for k, v in w.items()}
    table = torch.randn(V, L * d, generator=g).to(torch.bfloat16)
    x0, ids = torch.randn(T, W, generator=g), torch.randint(0, V, (T,), generator=g)
    for i in range(L):
        x = x0.clone().to(DEV)
        side = TokenInput(HymetaLinear.from_weight(w["gate"].to(dtype).to(DEV)), HymetaLinear.from_weight(w["proj"].to(dtype).to(DEV)),
                          table.to(dtype).to(DEV)[:, i * d:(i + 1) * d])
        AddNormed(w["norm"].to(DEV), eps)(x, side(x.to(dtype), ids.to(DEV)))
        ref = token_side_ref(x0.double(), table[ids][:, i * d:(i + 1) * d].double(), {k: v.double() for k, v in w.items()}, eps)
        assert rel_err(x.cpu() - x0, ref) < (5e-6 if dtype == torch.float32 else 1.5e-2), i


# --------------------------------------------------------------------------- queries, temperature, the scaled-key cache
def _unpack(row: torch.Tensor, G: int, D: int):
    """(keys [G, D], factors [G]) of one cache row (CPU)."""
    raw = row.contiguous().view(torch.uint8)
    at = (G * D * row.element_size() + 3) // 4 * 4
    return row[:G * D].view(G, D), raw[at:at + 4 * G].clone().view(torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,extra", [(6, 2, 24, 5), (4, 4, 128, 8), (3, 1, 33, 0), (1, 1, 4, 0), (2, 1, 300, 4), (40, 8, 64, 0), (3, 3, 5, 1)])
def test_query_norm_temperature_and_the_scaled_key_cache(dtype, H, G, D, extra):
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(H * D)
    eps, coef, every, page = 1e-3, 0.7, 8, 16
    portions, contexts, tables = [20, 1, 3], [0, 95, 6], [[3, 1], [9, 2, 8, 4, 0, 7], [5]]
    T = sum(portions)
    qk = (torch.randn(T, (H + G) * D + extra, generator=g) * 0.2).to(dtype)
    qw, kw = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.3 * torch.randn(D, generator=g)
    lay = layout_of(portions, contexts, [0, 1, 2], tables, page)
    row = hip_ops.scaled_key_row(G, D, dtype)
    assert row * dtype.itemsize % 16 == 0
    stale = torch.full((10, page, 1, row), 9.0, dtype=dtype)
    temps = query_temperature_ref(200, coef, every)
    assert float(temps[6]) == 1.0 and float(temps[7]) > 1.4            # the eighth token is the first with another temperature
    for with_temp in (True, False):
        buf, cache = qk.clone().to(DEV), stale.clone().to(DEV)
        hip_ops.scaled_key_cache_(buf, H, G, D, qw.to(DEV), kw.to(DEV), eps, cache, lay.slot_mapping, coef if with_temp else 0.0, every, lay.positions)
        q_ref = rms_ref(qk[:, :H * D].double().view(T, H, D), eps) * qw.double() * kw.double()
        if with_temp:
            q_ref = q_ref * temps[lay.positions.cpu()][:, None, None]
        assert rel_err(buf[:, :H * D].view(T, H, D), q_ref) < (2e-6 if dtype == torch.float32 else 4e-3)
        assert torch.equal(buf[:, H * D:].cpu(), qk[:, H * D:])
        raw = qk[:, H * D:(H + G) * D].view(T, G, D)
        inv = 1 / torch.sqrt(raw.double().pow(2).mean(-1) + eps)
        written = cache.view(-1, row).cpu()
        for t, slot in enumerate(lay.slot_mapping.tolist()):
            keys, factors = _unpack(written[slot], G, D)
            assert torch.equal(keys, raw[t]) and rel_err(factors, inv[t]) < 1e-6
        untouched = torch.ones(written.shape[0], dtype=torch.bool)
        untouched[lay.slot_mapping.cpu()] = False
        assert torch.equal(written[untouched], stale.view(-1, row)[untouched])


def _caches(ks, tables, page, blocks, dtype, eps, g):
    """A paged scaled-key cache (stale rows everywhere else) that holds ``ks [n, G, D]`` per sequence."""
    from vllm_hymeta import hip_ops
    G, D = ks[0].shape[1:]
    cache = torch.randn(blocks, page, 1, hip_ops.scaled_key_row(G, D, dtype), generator=g).to(dtype).to(DEV)
    ones = torch.ones(D, device=DEV)
    for k, tab in zip(ks, tables):
        n = k.shape[0]
        qk = torch.cat([torch.ones(n, D), k.reshape(n, G * D).float()], 1).to(dtype).to(DEV)
        sm = torch.tensor([tab[p // page] * page + p % page for p in range(n)], dtype=torch.int64, device=DEV)
        hip_ops.scaled_key_cache_(qk, 1, G, D, ones, ones, eps, cache, sm)
    return cache


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,window,gated,sink,page", [
    (6, 2, 24, 13, True, True, 16), (8, 4, 64, 70, True, True, 64), (4, 1, 128, 64, True, True, 64), (2, 2, 96, 200, False, True, 16), (8, 8, 32, 17, True, False, 32),
    (3, 1, 20, 1, False, True, 16), (5, 5, 8, None, True, True, 16), (40, 1, 64, 65, True, True, 16), (7, 1, 128, None, True, True, 16), (20, 1, 32, 130, True, True, 64),
    (8, 2, 64, 1, True, True, 16)])
def test_attention_whose_values_are_its_keys(dtype, H, G, D, window, gated, sink, page):
    """Prompts, portions and single rows of three sequences in one launch against the plain attention of each."""
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(H * 100 + D)
    lens, scale, eps, blocks = [330, 70, 33], 1.7 * D ** -0.5, 1e-5, 60
    perm = torch.randperm(blocks, generator=g).tolist()
    tables, used = [], 0
    for n in lens:
        nb = (n + page - 1) // page
        tables.append(perm[used:used + nb])
        used += nb
    qs = [torch.randn(n, H, D, generator=g).to(dtype) for n in lens]
    ks = [(torch.randn(n, G, D, generator=g) * (0.2 + 2 * torch.rand(n, G, 1, generator=g))).to(dtype) for n in lens]      # keys of many lengths
    gates = [torch.randn(n, H * D + 8, generator=g).to(dtype) for n in lens]
    sinks = torch.randn(H, generator=g) + 1
    slopes = torch.tensor([slope_ref(h, H) for h in range(H)])
    cache = _caches(ks, tables, page, blocks, dtype, eps, g)
    refs = []
    for s, n in enumerate(lens):
        o = penalised_sink_attention_ref(qs[s].double(), rms_ref(ks[s].double(), eps), ks[s].double(), scale, window, slopes.tolist(),
                                         sinks.double() if sink else None)
        refs.append(o.reshape(n, H * D) * (torch.sigmoid(gates[s][:, 8:].double()) if gated else 1.0))
    tol = 3e-6 if dtype == torch.float32 else 8e-3
    for plan in ([(330, 0), (70, 0), (33, 0)], [(37, 293), (1, 69), (20, 0)], [(1, 329), (1, 42), (1, 0)], [(2, 200), (64, 6), (1, 32)]):
        q = torch.cat([qs[s][c:c + n] for s, (n, c) in enumerate(plan)]).to(DEV)
        gate = torch.cat([gates[s][c:c + n] for s, (n, c) in enumerate(plan)]).to(DEV)[:, 8:] if gated else None
        lay = layout_of([n for n, _ in plan], [c for _, c in plan], [0, 1, 2], tables, page)
        out = hip_ops.sink_attention(q, cache, lay.block_tables, lay.query_start_loc, lay.seq_lens, G, D, D, scale, lay.max_query_len, lay.max_seq_len,
                                     sink=sink, sink_logits=sinks.to(DEV) if sink else None, window_left=-1 if window is None else window - 1,
                                     scaled_key=True, slopes=slopes.to(DEV), elem_gate=gate)
        assert rel_err(out.view(-1, H * D), torch.cat([refs[s][c:c + n] for s, (n, c) in enumerate(plan)])) < tol, plan


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [48, 64, 128])
@pytest.mark.parametrize("page", [16, 64])
def test_one_key_decides_at_the_edges_of_the_window(dtype, D, page):
    """Among hundreds of keys ONE points along the query and is long: at the window's first position it makes the output,
    one further back it must not be seen; the window's edge falls on, before and behind pages' and tiles' borders.  In
    prompts, in portions of two and decoded."""
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(D + page)
    n, window, H, G, eps = 300, 70, 2, 1, 1e-6
    along = F.normalize(torch.randn(D, generator=g), dim=0)
    slopes = torch.tensor([2.0 ** -6, 2.0 ** -8], device=DEV)
    tables = [list(range(3, 3 + (n + page - 1) // page))]
    for query_pos in (299, 197, 133, 70, 69):
        for back, seen in ((window - 1, True), (window, False), (0, True), (64, True)):
            key_pos = query_pos - back
            if key_pos < 0:
                continue
            k = torch.randn(n, G, D, generator=g) * 0.1
            k -= (k @ along)[:, :, None] * along
            k[key_pos, 0] = along * 5.0
            cache = _caches([k.to(dtype)], tables, page, 30, dtype, eps, g)
            for rows, ctx in ((1, query_pos), (query_pos + 1, 0), (2, query_pos - 1)):
                if ctx < 0:
                    continue
                q = torch.randn(rows, H, D, generator=g)
                q[-1] = along * D ** 0.5
                lay = layout_of([rows], [ctx], [0], tables, page)
                out = hip_ops.sink_attention(q.to(dtype).to(DEV), cache, lay.block_tables, lay.query_start_loc, lay.seq_lens, G, D, D, 20.0 / D,
                                             lay.max_query_len, lay.max_seq_len, sink=True, sink_logits=torch.zeros(H, device=DEV), window_left=window - 1,
                                             scaled_key=True, slopes=slopes)
                got = (out[-1].float().cpu() @ along).tolist()
                assert all((v > 4.5) == seen and (seen or abs(v) < 0.2) for v in got), (query_pos, back, rows, got)


@pytest.mark.parametrize("dtype,D", [(torch.float32, 40), (torch.bfloat16, 64), (torch.bfloat16, 128), (torch.bfloat16, 40)])
def test_sink_penalty_and_gate_each_show(dtype, D):
    """Equal scores everywhere, so that the output is the number of visible keys over that number plus the sink: a sink
    that is left out, scaled, penalised or counted per slice of the keys changes it; a steep slope leaves the nearest keys."""
    from vllm_hymeta import hip_ops
    n, H, page = 260, 2, 64
    g = torch.Generator().manual_seed(0)
    k = torch.ones(n, 1, D)
    tables = [list(range((n + page - 1) // page))]
    cache = _caches([k.to(dtype)], tables, page, 8, dtype, 1e-6, g)
    sinks = torch.tensor([5.0, -2.0])
    gate = torch.full((n, H * D), 1.25).to(dtype)
    q = torch.zeros(n, H, D, dtype=dtype)
    for slopes in ([0.0, 0.0], [1.0, 0.5]):
        for rows, ctx in ((n, 0), (1, n - 1), (3, 100)):
            lay = layout_of([rows], [ctx], [0], tables, page)
            out = hip_ops.sink_attention(q[:rows].to(DEV), cache, lay.block_tables, lay.query_start_loc, lay.seq_lens, 1, D, D, 100.0, lay.max_query_len,
                                         lay.max_seq_len, sink=True, sink_logits=sinks.to(DEV), scaled_key=True, slopes=torch.tensor(slopes, device=DEV),
                                         elem_gate=gate[:rows].to(DEV))
            for h in range(H):
                for r in (0, rows - 1):
                    mass = sum(math.exp(-slopes[h] * d) for d in range(ctx + r + 1))
                    want = mass / (mass + math.exp(sinks[h])) / (1 + math.exp(-1.25))
                    assert float((out[r, h].float() - want).abs().max()) < (1e-5 if dtype == torch.float32 else 6e-3), (slopes, rows, h, r)


# --------------------------------------------------------------------------- the gated delta rule
UNIT_EPS = 1e-6


def _delta_ref(q, k, v, beta_logit, log2_decay, state=None):
    """``q, k [T, G, D]``, ``v [T, H, Dv]``, all double, through the oracle's rule."""
    H, G, D = v.shape[1], q.shape[1], q.shape[2]
    pick = [h // (H // G) for h in range(H)]
    o = delta_rule_ref((unit_ref(q) * D ** -0.5)[:, pick], unit_ref(k)[:, pick], v, torch.sigmoid(beta_logit), 2.0 ** log2_decay, state)
    return o.reshape(v.shape[0], -1)


DELTA_SHAPES = [(2, 1, 16, 24), (3, 3, 32, 32), (4, 2, 64, 64), (2, 2, 128, 128), (4, 1, 96, 32), (2, 1, 32, 96), (1, 1, 20, 7), (2, 2, 160, 64), (1, 1, 128, 256),
                (2, 1, 64, 40)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,Dv", DELTA_SHAPES)
def test_delta_rule_in_portions_and_single_rows(dtype, H, G, D, Dv):
    """Whole sequences, portions of every size, single rows, a state slot used again, the state that is left; the outputs and
    states of a decode step with the norm and gate in the same launch."""
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(H * D + Dv)
    lens = {0: 200, 1: 1, 2: 90, 3: 64}
    # keys that share a direction (neighbours overlap strongly), of many lengths
    common = torch.randn(D, generator=g)
    qs = {s: torch.randn(n, G, D, generator=g).to(dtype) for s, n in lens.items()}
    ks = {s: ((torch.randn(n, G, D, generator=g) + common) * (0.1 + 3 * torch.rand(n, G, 1, generator=g))).to(dtype) for s, n in lens.items()}
    vs = {s: torch.randn(n, H, Dv, generator=g).to(dtype) for s, n in lens.items()}
    bs = {s: (torch.randn(n, H, generator=g) * 2).to(dtype) for s, n in lens.items()}
    lds = {s: -torch.rand(n, H, generator=g) * 0.3 for s, n in lens.items()}
    for s in lens:
        lds[s][::23] = -40.0                      # now and then everything is forgotten
        lds[s][5::37] = 0.0                       # ... or nothing
        lds[s][11::41] = -3.0e4                   # a decay that is zero in any type
    ends = {s: torch.zeros(H, D, Dv, dtype=torch.float64) for s in lens}
    refs = {s: _delta_ref(qs[s].double(), ks[s].double(), vs[s].double(), bs[s].double(), lds[s].double(), ends[s]) for s in lens}
    state = torch.full((5, H, D, Dv), 3.0, dtype=torch.float32, device=DEV)          # stale values: a new sequence must not read them
    slots = {0: 1, 1: 3, 2: 0, 3: 4}

    def run(step, **kw):
        cat = lambda d: torch.cat([d[s][at:at + n] for s, at, n in step]).to(DEV)      # noqa: E731
        lay = layout_of([n for _, _, n in step], [at for _, at, _ in step], [slots[s] for s, _, _ in step])
        return hip_ops.delta_rule(cat(qs), cat(ks), cat(vs), cat(bs), cat(lds), state, lay.query_start_loc, lay.context_lens, lay.slot_idx, lay.max_query_len,
                                  D ** -0.5, UNIT_EPS, **kw)

    tol = 5e-6 if dtype == torch.float32 else 1e-4               # (the inputs are what they are in either type: only the products' parts round)
    whole = in_steps(lens, [[(0, 200), (1, 1), (2, 90), (3, 64)]], run)
    for s in lens:
        assert rel_err(whole[s], refs[s]) < tol and rel_err(state[slots[s]], ends[s]) < tol, s
    assert float((state[2] - 3.0).abs().max()) == 0.0             # nobody's slot
    state.fill_(-2.0)
    plan = [[(0, 2)], [(0, 1), (2, 7)], [(0, 61), (2, 1), (3, 8)], [(0, 64), (1, 1), (2, 2), (3, 1)], [(0, 8), (2, 70), (3, 55)], [(0, 63), (2, 9)], [(0, 1), (2, 1)]]
    cut = in_steps(lens, plan, run)
    for s in lens:
        assert cut[s].shape[0] == lens[s] and rel_err(cut[s], refs[s]) < tol and rel_err(state[slots[s]], ends[s]) < tol, s
    # single rows, the norm and the gate in the same launch, slots used again
    if hip_ops.delta_rule_step_supported(D, Dv):
        w = 1 + 0.2 * torch.randn(Dv, generator=g)
        gates = {s: torch.randn(n, H * Dv, generator=g).to(dtype) for s, n in lens.items()}
        before = state[slots[3]].clone()
        slots.update({0: 3, 2: 1})
        got = {0: [], 2: []}
        for t in range(12):
            step = [(0, t, 1), (2, t, 1)]
            out = run(step, norm_weight=w.to(DEV), gate=torch.cat([gates[s][t:t + 1] for s in (0, 2)]).to(DEV), norm_eps=1e-4)
            assert out.dtype == dtype
            got[0].append(out[:1]), got[2].append(out[1:])
        for s in (0, 2):
            o = refs[s][:12].view(12, H, Dv)
            ref = (rms_ref(o, 1e-4) * w.double()).reshape(12, H * Dv) * F.silu(gates[s][:12].double())
            assert rel_err(torch.cat(got[s]), ref) < (1e-5 if dtype == torch.float32 else 4e-3), s
        assert torch.equal(state[slots[3]], before)                 # a sequence that was left out keeps its state
    # no slot: the outputs are those of a fresh sequence, nothing is stored
    keep = state.clone()
    slots[3] = -1
    assert rel_err(in_steps({3: 64}, [[(3, 64)]], run)[3], refs[3]) < tol and torch.equal(state, keep)


@pytest.mark.parametrize("D,Dv", [(32, 32), (128, 128)])
def test_delta_rule_overwrites_what_a_key_held(D, Dv):
    """The same key again and again with full write strength: the state must hold the LAST value under it, not a sum, at
    every place of a chunk and across chunks (the chunk's triangular system is as full as it gets)."""
    from vllm_hymeta import hip_ops
    g = torch.Generator().manual_seed(D)
    T, H = 150, 2
    key = torch.randn(1, 1, D, generator=g).expand(T, 1, D)
    v = torch.randn(T, H, Dv, generator=g).to(torch.bfloat16)
    k = key.to(torch.bfloat16).contiguous()
    state = torch.zeros(1, H, D, Dv, device=DEV)
    beta, ld = torch.full((T, H), 20.0, dtype=torch.bfloat16, device=DEV), torch.zeros(T, H, device=DEV)
    out = hip_ops.delta_rule(k.to(DEV), k.to(DEV), v.to(DEV), beta, ld, state, i32([0, T]), i32([0]), i32([0]), T, 1.0, UNIT_EPS)
    assert float((out.view(T, H, Dv).cpu() - v.float()).abs().max()) < 2e-3
    ref = torch.zeros(H, D, Dv, dtype=torch.float64)
    _delta_ref(k.double(), k.double(), v.double(), beta.double().cpu(), ld.double().cpu(), ref)
    assert rel_err(state[0], ref) < 1e-4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cfg", [delta_config(), delta_config(heads=4, kv_heads=1, dim=32, vdim=64, conv=2), delta_config(heads=1, kv_heads=1, dim=8, vdim=8, conv=1),
                                 delta_config(heads=2, kv_heads=2, dim=64, vdim=32, conv=3)])
def test_mixers_alone_against_the_oracle(dtype, cfg):
    """The delta mixer (projections, convolution, rule, norm, gate) as a sublayer of a one-layer model, and the attention mixer
    beside it."""
    eps, W, T = 1e-5, 64, 140
    c = nilevik_config(vocab=40, width=W, eps=eps, side=8, layers=[("delta", cfg, None), ("attention", attention_config(heads=4, kv_heads=2, dim=32, window=20), None)])
    w = nilevik_random_weights(c, seed=5)
    eng = build_engine(c, w, dtype, max_tokens=192, block_size=16)
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(1)).to(dtype)
    model = eng.model.model
    (recurrent, conv), _ = model.state_cache.current_run_tensors(request_ids_to_seq_ids={"x": [0]}, finished_requests_ids=[])
    lay = layout_of([T], [0], [0], [list(range(12))], 16)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    sub = lambda p: {k[len(p):]: v.double() for k, v in w.items() if k.startswith(p)}      # noqa: E731
    got = model.layers[0].mixer(h.to(DEV), lay, (recurrent[0][0], conv[0][0]))
    assert rel_err(got, delta_mixer_ref(h.double(), sub("l0.mix."), cfg, eps)) < tol
    got = model.layers[1].mixer(h.to(DEV), lay, model.attn_layers["1"])
    assert rel_err(got, attention_mixer_ref(h.double(), sub("l1.mix."), c["layers"][1]["mixer"], eps)) < tol


# --------------------------------------------------------------------------- whole models under the engine
def build_engine(cfg, weights, dtype, max_tokens=512, block_size=16, max_num_seqs=4, max_num_batched_tokens=1 << 30):
    from vllm_hymeta.engine import LLMEngine
    from vllm_hymeta.models.configuration_nilevik import NilevikConfig
    from vllm_hymeta.models.modeling_nilevik import NilevikForCausalLM
    model = NilevikForCausalLM(NilevikConfig(cfg), max_num_seqs=max_num_seqs, dtype=dtype, device=DEV)
    model.load_weights(weights.items())
    return LLMEngine(model, num_blocks=max_tokens // block_size, block_size=block_size, max_num_seqs=max_num_seqs,
                     max_num_batched_tokens=max_num_batched_tokens, device=DEV)


MODELS = {
    "default": dict(),
    "ones_and_equals": dict(width=40, side=1, layers=[                # one head, a window of one token, one tap, one side column, temperature from the first token on
        ("attention", attention_config(heads=1, kv_heads=1, dim=8, window=1, coef=0.5, every=1), None),
        ("delta", delta_config(heads=1, kv_heads=1, dim=24, vdim=24, conv=1), 40),
        ("attention", attention_config(heads=2, kv_heads=2, dim=40, window=9, coef=0.5, every=3, scale=0.1), 16)]),
    "matrix_core_sizes": dict(width=128, vocab=200, side=32, layers=[
        ("attention", attention_config(heads=8, kv_heads=2, dim=64, window=70, coef=0.4, every=32), 192),
        ("delta", delta_config(heads=4, kv_heads=2, dim=64, vdim=64, conv=4), 160),
        ("attention", attention_config(heads=4, kv_heads=4, dim=128, window=65, coef=0.2, every=50), None),
        ("delta", delta_config(heads=2, kv_heads=1, dim=128, vdim=128, conv=3), None),
        ("attention", attention_config(heads=6, kv_heads=1, dim=32, window=64), 64)]),
    "delta_only": dict(width=72, side=20, layers=[("delta", delta_config(heads=6, kv_heads=3, dim=20, vdim=12, conv=2), 56),
                                                  ("delta", delta_config(heads=2, kv_heads=2, dim=32, vdim=32, conv=5), None)]),
    "attention_only": dict(width=48, side=16, layers=[("attention", attention_config(heads=4, kv_heads=4, dim=20, window=33, every=100), 64),
                                                      ("attention", attention_config(heads=8, kv_heads=1, dim=32, window=2, coef=2.0, every=16), 64)]),
}


def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


TOL = {torch.float32: 5e-5, torch.bfloat16: 0.06}


@pytest.mark.parametrize("name", sorted(MODELS))
def test_model_whole_prompt_against_the_oracle_fp32(name):
    """One step for the whole prompt, every position's logits and the stream after every layer."""
    cfg = nilevik_config(**MODELS[name])
    weights = nilevik_random_weights(cfg, seed=len(name))
    toks = _tokens(150, cfg["vocab"], 7)
    stream_ref = []
    ref = nilevik_ref(cfg, weights, toks, residual_out=stream_ref)
    eng = build_engine(cfg, weights, torch.float32, max_tokens=256, block_size=16)
    stream = []
    inner = eng.model.model
    plain = inner.forward
    inner.forward = lambda *a, **k: plain(*a, residual_out=stream, **k)
    got = eng.run_batch([("a", toks, list(range(len(toks))))])
    assert len(stream) == len(cfg["layers"])
    for i, (s, r) in enumerate(zip(stream, stream_ref)):
        assert rel_err(s, r) < 2e-5, (i, cfg["layers"][i]["type"])
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
    sizes = dict(MODELS[name])
    if dtype == torch.bfloat16 and sizes.get("side") == 1:
        sizes["side"] = 6             # the norm of one column's product is its sign: a rounding around zero flips the whole row
    cfg = nilevik_config(**sizes)
    weights = nilevik_random_weights(cfg, seed=len(name))
    seqs = {k: _tokens(n, cfg["vocab"], 10 + k) for k, n in enumerate([150, 33, 1, 70, 19, 64])}
    refs = {k: nilevik_ref(cfg, weights, t) for k, t in seqs.items()}
    exact, tol = dtype == torch.float32, TOL[dtype]
    page = 64 if name == "matrix_core_sizes" else 16
    pages = 320 // page
    eng = build_engine(cfg, weights, dtype, max_tokens=pages * page, block_size=page, max_num_seqs=4)
    whole = {}
    for k, t in seqs.items():
        whole[k] = eng.run_batch([(f"w{k}", t, list(range(len(t))))])
        eng.finish_request(f"w{k}")
        assert rows_close(whole[k], refs[k], tol, exact), k
    assert eng.pool.num_free == pages
    # token by token after a prompt that ends inside a page
    got = _replay(eng, seqs, [[(0, 85)]] + [[(0, 1)]] * 65)
    assert rows_close(got[0], whole[0], tol, exact) and rows_close(got[0], refs[0], tol, exact)
    # token by token from the very first token
    got = _replay(eng, seqs, [[(1, 1)]] * 33)
    assert rows_close(got[1], whole[1], tol, exact)
    # portions: 2, 1, 3, ... across page borders and multiples of 64 rows
    got = _replay(eng, seqs, [[(0, n)] for n in (2, 1, 3, 10, 2, 45, 2, 64, 2, 19)])
    assert rows_close(got[0], whole[0], tol, exact)
    # mixed: up to four live requests, portions beside single tokens, a request that pauses, requests that end and free
    # pages and slots for new ones
    plan = [[(0, 70), (1, 2)], [(0, 1), (1, 31), (2, 1)], [(0, 1), (3, 16), (4, 2)], [(0, 78), (3, 1), (4, 17)], [(3, 53), (5, 3)], [(5, 2)], [(5, 59)]]
    got = _replay(eng, seqs, plan)
    for k in seqs:
        assert rows_close(got[k], whole[k], tol, exact) and rows_close(got[k], refs[k], tol, exact), k
    assert eng.pool.num_free == pages and not eng.requests


@pytest.mark.parametrize("dtype", DTYPES)
def test_positions_may_be_left_out(dtype):
    """A caller that gives no positions: the rows' places in their sequences."""
    cfg = nilevik_config()
    eng = build_engine(cfg, nilevik_random_weights(cfg, seed=1), dtype, max_tokens=256)
    toks = _tokens(40, cfg["vocab"], 2)
    a = eng.run_batch([("a", toks, list(range(40)))])
    inner = eng.model.model
    plain = inner.forward
    inner.forward = lambda ids, pos=None, **k: plain(ids, None, **k)
    eng.run_batch([("b", toks[:17], [])])
    b = eng.run_batch([("c", toks, list(range(40))), ("b", toks[17:], list(range(23)))])
    assert torch.equal(a, b[:40]) and rows_close(b[40:], a[17:], TOL[dtype], dtype == torch.float32)


@pytest.mark.parametrize("n,stride", [(101, 101), (8, 8), (40001, 40001), (40000, 40003), (3, 7)])
def test_greedy_choice_over_a_vocabulary_of_any_size(n, stride):
    from vllm_hymeta import hip_ops
    x = torch.randn(5, stride, generator=torch.Generator().manual_seed(n))
    x[2, n - 1] = 50.0
    x[:, n:] = 99.0                       # behind a row's columns
    assert hip_ops.argmax_rows(x.to(DEV)[:, :n]).tolist() == x[:, :n].argmax(-1).tolist() and int(x[2, :n].argmax()) == n - 1


def test_greedy_generation_through_the_scheduler_matches_the_oracle():
    """engine.generate: six prompts, two state slots, a token budget that cuts prompts into portions -- the scheduler
    batches portions beside decoded tokens and reuses slots and pages; every generated token is the oracle's argmax."""
    from vllm_hymeta.engine import SamplingParams
    cfg = nilevik_config()
    weights = nilevik_random_weights(cfg, seed=4)
    prompts = [_tokens(n, cfg["vocab"], 40 + n) for n in (23, 5, 1, 37, 12, 18)]
    new = 5
    eng = build_engine(cfg, weights, torch.float32, max_tokens=128, block_size=16, max_num_seqs=2, max_num_batched_tokens=16)
    outs = eng.generate(prompts, SamplingParams(max_tokens=new))
    assert eng.pool.num_free == 8 and not eng.requests
    for p, o in zip(prompts, outs):
        assert len(o) == new
        logits = nilevik_ref(cfg, weights, list(p) + o)
        for j, t in enumerate(o):
            row = logits[len(p) - 1 + j]
            top2 = row.topk(2).values
            if float(top2[0] - top2[1]) > 1e-3:        # a clear winner: the engine must have picked it
                assert t == int(row.argmax())


@pytest.mark.parametrize("dtype,name", [(torch.float32, "default"), (torch.bfloat16, "matrix_core_sizes")])
def test_long_decode_passes_every_window_and_keeps_its_states(dtype, name):
    """400 tokens decoded one by one after a two-token prompt: every window passes over decoded tokens many times, the
    recurrent and convolution states are carried 400 times, the temperature changes many times."""
    cfg = nilevik_config(**MODELS[name])
    weights = nilevik_random_weights(cfg, seed=8)
    toks = _tokens(402, cfg["vocab"], 3)
    page = 64 if dtype == torch.bfloat16 else 32
    eng = build_engine(cfg, weights, dtype, max_tokens=448, block_size=page, max_num_seqs=1)
    places = [17, 200, 333, 401]
    whole = eng.run_batch([("w", toks, places)])
    eng.finish_request("w")
    eng.run_batch([("d", toks[:2], [])])
    for i in range(2, 402):
        out = eng.run_batch([("d", toks[i:i + 1], [0] if i in places else [])])
        if i in places:
            assert rel_err(out, whole[places.index(i):places.index(i) + 1]) < 2 * TOL[dtype], i
    eng.finish_request("d")
    if dtype == torch.float32:
        assert rel_err(eng.run_batch([("x", toks[:201], [200])]), nilevik_ref(cfg, weights, toks[:201])[-1:]) < TOL[dtype]


@pytest.mark.parametrize("name", ["default", "matrix_core_sizes"])
def test_a_decode_step_replayed_from_a_graph(name):
    """Three sequences of different lengths decode eight tokens: the step captured once and replayed, with eager work and
    synchronisations between the replays, against the engine's eager steps."""
    from vllm_hymeta.attention.meta_attention import MetaAttentionMetadata
    from vllm_hymeta.models.attention import bind_kv_cache
    cfg = nilevik_config(**MODELS[name])
    weights = nilevik_random_weights(cfg, seed=3)
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
    states = model.model.state_cache._slot_tensors()
    states_before = [t.clone() for t in states]
    slots = [model.model.state_cache.slots.slot_of(eng.requests[f"s{s}"].state_key, 0) for s in range(3)]
    want = [eng.run_batch([(f"s{s}", [int(fed[s, t])], [0]) for s in range(3)]) for t in range(new)]

    def rewind():
        for n, t in eng.kv_caches.items():
            t.copy_(cache_before[n])
            bind_kv_cache(eng.attn_layers[n], t)
        for t, b in zip(states, states_before):
            t.copy_(b)

    lens = torch.tensor([len(p) for p in prompts])
    ids, pos = torch.zeros(3, dtype=torch.int64, device=DEV), torch.zeros(3, dtype=torch.int64, device=DEV)
    seq, ctx, sm = i32([0, 0, 0]), i32([0, 0, 0]), torch.zeros(3, dtype=torch.int64, device=DEV)
    md = MetaAttentionMetadata(
        num_prefills=0, num_prefill_tokens=0, num_decode_tokens=3, slot_mapping=sm, multi_modal_placeholder_index_maps=None,
        enable_kv_scales_calculation=False, seq_lens=None, seq_lens_tensor=seq, max_prefill_seq_len=0, max_decode_seq_len=2 * page,
        context_lens_tensor=ctx, block_tables=tables.to(DEV), use_cuda_graph=True, max_query_len=1, max_decode_query_len=1,
        query_start_loc=i32([0, 1, 2, 3]), seq_start_loc=None)
    cache, idx = model.get_seqlen_agnostic_capture_inputs(3)
    idx.copy_(i32(slots))

    def inputs(t):
        p = lens + t
        ids.copy_(fed[:, t]), pos.copy_(p), seq.copy_(p + 1), ctx.copy_(p)
        sm.copy_(torch.tensor([int(tables[s, int(p[s]) // page]) * page + int(p[s]) % page for s in range(3)]))

    with torch.inference_mode():
        step = lambda: model.compute_logits(model(ids, pos, attn_metadata=md, seqlen_agnostic_capture_inputs=(cache, idx)))      # noqa: E731
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
    cfg = nilevik_config()
    weights = nilevik_random_weights(cfg, seed=12)
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
    ra, rb = nilevik_ref(cfg, weights, a), nilevik_ref(cfg, weights, b)
    want = {0: torch.stack([ra[0], ra[49]]), 1: rb[38:39], 2: torch.stack([rb[39], ra[52]]), 3: torch.stack([ra[89], rb[6]])}
    for k, ref in want.items():
        got = torch.from_numpy(np.fromfile(str(out_dir / f"{k}.f32"), dtype="<f4").reshape(ref.shape[0], -1))
        assert rel_err(got, ref) < TOL[torch.float32], k
    gen = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), "--model", str(model_dir), "--dtype", "float32", "--prompt-ids",
                          ",".join(map(str, a[:20])), "--max-new-tokens", "3", "--max-tokens", "128"], capture_output=True, text=True, timeout=100)
    assert gen.returncode == 0, gen.stderr[-2000:]
    line = json.loads([l for l in gen.stdout.splitlines() if l.startswith("{")][-1])
    assert len(line["output"]) == 3
    logits = nilevik_ref(cfg, weights, a[:20] + line["output"])
    for j, t in enumerate(line["output"]):
        top2 = logits[19 + j].topk(2).values
        if float(top2[0] - top2[1]) > 1e-3:
            assert t == int(logits[19 + j].argmax())


def _random_model(seed):
    """Sizes drawn at random: layer order, head counts, group sizes, key, value and state sizes (also such that a layer
    takes the matrix-core kernels), windows around a page and a tile, taps, temperatures."""
    import random
    r = random.Random(seed)
    layers = []
    for _ in range(r.randint(1, 4)):
        G = r.choice([1, 2, 3])
        H = G * r.choice([1, 2, 3, 5])
        if r.random() < 0.5:
            D = r.choice([32, 64, 96, 128]) if r.random() < 0.5 else r.randint(3, 50)
            mixer = ("attention", attention_config(heads=H, kv_heads=G, dim=D, window=r.choice([1, 2, 7, 15, 16, 17, 63, 64, 65, 100, 128, 1000]),
                                                   coef=r.choice([0.1, 0.5, 2.0]), every=r.choice([1, 5, 16, 64, 100, 4096]), scale=r.choice([D ** -0.5, 0.3, 0.05])))
        else:
            D, Dv = (r.choice([32, 64, 128]), r.choice([32, 64, 96])) if r.random() < 0.5 else (r.randint(4, 40), r.randint(3, 40))
            mixer = ("delta", delta_config(heads=H, kv_heads=G, dim=D, vdim=Dv, conv=r.choice([1, 2, 3, 4, 6])))
        layers.append(mixer + (r.choice([None, 16, 72, 128]),))
    return nilevik_config(vocab=r.choice([50, 130]), width=r.choice([24, 40, 64, 96, 128, 200]), layers=layers, eps=r.choice([1e-5, 1e-6, 1e-3]), side=r.choice([3, 8, 24, 64]))


@pytest.mark.parametrize("seed", range(12))
def test_models_of_random_sizes_under_the_engine(seed):
    """A prompt of 190 tokens in one step, then in portions and single tokens beside a second request, against the oracle."""
    cfg = _random_model(seed)
    weights = nilevik_random_weights(cfg, seed=seed)
    seqs = {0: _tokens(190, cfg["vocab"], 100 + seed), 1: _tokens(75, cfg["vocab"], 200 + seed)}
    refs = {k: nilevik_ref(cfg, weights, t) for k, t in seqs.items()}
    page = 64 if seed % 2 else 16
    plan = [[(0, 3)], [(0, 64), (1, 2)], [(0, 1), (1, 1)], [(0, 62), (1, 70)], [(0, 1), (1, 1)], [(0, 2), (1, 1)], [(0, 57)]]
    for dtype in DTYPES:
        eng = build_engine(cfg, weights, dtype, max_tokens=448, block_size=page, max_num_seqs=2)
        exact, tol = dtype == torch.float32, TOL[dtype]
        whole = eng.run_batch([("w", seqs[0], list(range(190)))])
        eng.finish_request("w")
        got = _replay(eng, seqs, plan)
        assert not eng.requests
        assert rows_close(whole, refs[0], tol, exact) and all(rows_close(got[k], refs[k], tol, exact) for k in seqs), dtype
