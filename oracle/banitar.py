"""Plain, slow CPU statement of the Banitar decoder, one function per mechanism, in whatever float type the inputs have
(the tests use float64).  TEST INFRASTRUCTURE ONLY: written from the model's equations, shares no code with the product
path, and also makes the random checkpoints the tests load into the product.

Every function sees ONE whole sequence from its first token: no cache, no pages, no batching.

The design: scaled token embedding; layers with a squashing norm on both sides of every sublayer (``x += norm(mixer(norm
x)); x += norm(ff(norm x))`` with ``norm(x) = tanh(alpha x) w + b``); a run of layers repeated with the same weights, each
pass entered through a linear map of the stream beside the embedding output plus a vector of the pass; two mixers, a
windowed latent attention with a sink and a chunked attention with biased projections, interleaved rotation, unit-rms
queries and keys and a gate per head; a silu-gated feed-forward or none; an output projection of its own.
"""
from __future__ import annotations

import math
from typing import Callable, Dict, List, Optional, Tuple

import torch


# ------------------------------------------------------------------------------------------------ small pieces
def tanh_norm_ref(x: torch.Tensor, alpha: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    return torch.tanh(alpha * x) * w + b


def rms_ref(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu_glu_ref(h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    z = h @ w["gate"].T
    return (z * torch.sigmoid(z) * (h @ w["up"].T)) @ w["down"].T


# ------------------------------------------------------------------------------------------------ rotation
def rotation_frequencies_ref(dims: int, base: float, scaling: Optional[dict] = None) -> Tuple[List[float], float]:
    """``(frequency of every pair, factor on cos and sin)``."""
    out, mag = [], 1.0
    for i in range(dims // 2):
        f = base ** (-2 * i / dims)
        if scaling is not None:
            def turn_dim(turns):
                return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
            lo, hi = max(math.floor(turn_dim(scaling["fast"])), 0), min(math.ceil(turn_dim(scaling["slow"])), dims - 1)
            ramp = (i - lo) / max(hi - lo, 0.001)
            ramp = 0.0 if ramp < 0 else 1.0 if ramp > 1 else ramp
            f = f / scaling["factor"] * ramp + f * (1 - ramp)
            mag = 0.1 * math.log(scaling["factor"]) + 1
        out.append(f)
    return out, mag


def rotate_ref(x: torch.Tensor, dims: int, freqs: List[float], mag: float, half_split: bool) -> torch.Tensor:
    """``x [T, heads, D]``, row t at position t: the first ``dims`` dimensions turn in pairs, ``(i, i + dims / 2)`` with
    ``half_split``, else ``(2 i, 2 i + 1)``."""
    out = x.clone()
    t = torch.arange(x.shape[0], dtype=torch.float64)
    for i in range(dims // 2):
        p, r = (i, i + dims // 2) if half_split else (2 * i, 2 * i + 1)
        c, s = ((f(t * freqs[i]) * mag).to(x.dtype)[:, None] for f in (torch.cos, torch.sin))
        u, v = x[:, :, p], x[:, :, r]
        out[:, :, p], out[:, :, r] = u * c - v * s, v * c + u * s
    return out


# ------------------------------------------------------------------------------------------------ attention
def in_window(size: int) -> Callable[[int], int]:
    """First visible key of a query at position i: the last ``size`` tokens, itself included."""
    return lambda i: max(0, i - size + 1)


def in_chunk(size: int) -> Callable[[int], int]:
    """First visible key of a query at position i: the start of its chunk of ``size`` tokens, counted from 0."""
    return lambda i: (i // size) * size


def attend_ref(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, first: Callable[[int], int],
               sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, Dv]`` -> ``[T, H, Dv]``; query i sees keys ``first(i) .. i``."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            lo = first(i)
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            if sink is not None:
                s = torch.cat([s, sink[h].reshape(1)])
            p = torch.softmax(s, 0)[:i + 1 - lo]
            out[i, h] = p @ v[lo:i + 1, g]
    return out


def latent_attention_ref(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """Keys and values written out per head (the product absorbs their up projections)."""
    T, H, D, R, Dv, C = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    freqs, mag = rotation_frequencies_ref(m["rot"]["dims"], m["rot"]["base"])
    q = (h @ w["q"].T).view(T, H, D + R)
    both = h @ w["dkv"].T
    c = rms_ref(both[:, :C], eps) * w["dkv.norm"]
    kr = rotate_ref(both[:, None, C:], m["rot"]["dims"], freqs, mag, True)
    q = torch.cat([q[..., :D], rotate_ref(q[..., D:], m["rot"]["dims"], freqs, mag, True)], -1)
    k = torch.cat([(c @ w["uk"].T).view(T, H, D), kr.expand(T, H, R)], -1)
    v = (c @ w["uv"].T).view(T, H, Dv)
    o = attend_ref(q, k, v, m["scale"], in_window(m["mask"]["size"]), w["sink"])
    return o.reshape(T, H * Dv) @ w["o"].T


def chunked_attention_ref(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    freqs, mag = rotation_frequencies_ref(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    q = (h @ w["q"].T + w["q.b"]).view(T, H, D)
    k = (h @ w["k"].T + w["k.b"]).view(T, G, D)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, Dv)
    q = rms_ref(rotate_ref(q, m["rot"]["dims"], freqs, mag, False), eps)
    k = rms_ref(rotate_ref(k, m["rot"]["dims"], freqs, mag, False), eps)
    o = attend_ref(q, k, v, m["scale"], in_chunk(m["mask"]["size"]))
    o = o * torch.sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, H * Dv) @ w["o"].T


# ------------------------------------------------------------------------------------------------ the model
def _sub(weights: Dict[str, torch.Tensor], prefix: str, dtype) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v.to(dtype) for k, v in weights.items() if k.startswith(prefix)}


def layer_runs_ref(cfg: dict) -> List[Tuple[int, int, bool]]:
    """``(layer, pass, whether the pass starts with it)`` in the order of execution."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, 0, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, 0, False) for i in range(a)] + [(i, t, i == a) for t in range(loop["times"]) for i in range(a, b)]
            + [(i, 0, False) for i in range(b, n)])


def banitar_ref(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
                residual_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence."""
    eps = cfg["norm"]["eps"]

    def norm(x, name):
        return tanh_norm_ref(x, *(weights[name + s].to(dtype) for s in (".alpha", "", ".b")))

    x = x0 = weights["embed"].to(dtype)[torch.tensor(tokens)] * cfg["embedding"]["scale"]
    for i, t, enters in layer_runs_ref(cfg):
        if enters:
            x = torch.cat([x, x0], -1) @ weights["loop.in"].to(dtype).T + weights["loop.step"].to(dtype)[t]
        p, entry = f"l{i}.", cfg["layers"][i]
        mix = latent_attention_ref if entry["type"] == "latent_attention" else chunked_attention_ref
        x = x + norm(mix(norm(x, p + "norm1"), _sub(weights, p + "mix.", dtype), entry["mixer"], eps), p + "norm1b")
        if entry.get("mlp") is not None:
            x = x + norm(silu_glu_ref(norm(x, p + "norm2"), _sub(weights, p + "mlp.", dtype)), p + "norm2b")
        if residual_out is not None:
            residual_out.append(x.clone())
    return norm(x, "final.norm") @ weights["head"].to(dtype).T


# ------------------------------------------------------------------------------------------------ test checkpoints
def latent_config(heads=6, dim=24, rot_dim=12, vdim=20, kv_rank=36, window=13, base=500.0, scale=None) -> dict:
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
            "rot": {"base": base, "dims": rot_dim}, "scale": float(scale if scale is not None else (dim + rot_dim) ** -0.5)}


def chunked_config(heads=6, kv_heads=2, dim=24, vdim=16, chunk=29, rot_dims=16, base=900.0, scaling="yarn", scale=None) -> dict:
    rot = {"base": base, "dims": rot_dims}
    if scaling == "yarn":
        scaling = {"factor": 5.0, "original": 64, "fast": 4.0, "slow": 1.0}
    if scaling is not None:
        rot["scaling"] = dict(scaling)
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "rot": rot,
            "scale": float(scale if scale is not None else dim ** -0.5)}


def banitar_config(vocab=101, width=56, layers=None, loop=(1, 3, 3), eps=1e-5, embed_scale=3.0) -> dict:
    """``layers``: a list of ``(type, mixer config, feed-forward width or None)``; ``loop``: (start, stop, times) or None."""
    if layers is None:
        layers = [("attention", chunked_config(), 72), ("latent_attention", latent_config(), 88),
                  ("attention", chunked_config(heads=3, kv_heads=3, dim=16, vdim=24, chunk=17, rot_dims=16, scaling=None), None),
                  ("latent_attention", latent_config(heads=2, dim=16, rot_dim=8, vdim=32, kv_rank=20, window=5), 40)]
    cfg = {"architecture": "Banitar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
           "layers": [{"type": t, "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}} for t, m, ff in layers]}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def banitar_random_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """bf16-representable random tensors under the checkpoint's names (fp32 tensors whose values survive a bf16 round trip)."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, s=1.0):
        return (torch.randn(shape, generator=g) * s).to(torch.bfloat16).float()

    def lin(o, i, s=1.0):
        return rnd(o, i, s=s * i ** -0.5)

    def near(v, *shape, s=0.2):
        return (v + rnd(*shape, s=s)).to(torch.bfloat16).float()

    w = {"embed": rnd(V, W), "head": lin(V, W)}

    def norm(name, alpha):
        w[name], w[name + ".b"], w[name + ".alpha"] = near(1.0, W), rnd(W, s=0.1), near(alpha, s=0.05)

    norm("final.norm", 0.5)
    if cfg.get("loop"):
        w["loop.in"], w["loop.step"] = lin(W, 2 * W), rnd(cfg["loop"]["times"], W, s=0.5)
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        norm(p + "norm1", 0.4), norm(p + "norm1b", 0.9)
        H = m["heads"]
        if entry["type"] == "latent_attention":
            D, R, Dv, C = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            w[p + "mix.q"], w[p + "mix.dkv"], w[p + "mix.dkv.norm"] = lin(H * (D + R), W, 1.5), lin(C + R, W, 1.5), near(1.0, C)
            w[p + "mix.uk"], w[p + "mix.uv"], w[p + "mix.o"], w[p + "mix.sink"] = lin(H * D, C), lin(H * Dv, C), lin(W, H * Dv, 1.5), rnd(H)
        else:
            G, D, Dv = m["kv_heads"], m["dim"], m["vdim"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                w[p + f"mix.{n}"], w[p + f"mix.{n}.b"] = lin(rows, W), rnd(rows, s=0.5)
            w[p + "mix.g"], w[p + "mix.o"] = lin(H, W), lin(W, H * Dv, 1.5)
        if entry["mlp"] is not None:
            ff = entry["mlp"]["ff"]
            norm(p + "norm2", 0.4), norm(p + "norm2b", 0.9)
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(ff, W, 1.5), lin(ff, W), lin(W, ff, 1.5)
    return w
