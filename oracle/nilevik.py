"""Plain, slow CPU statement of the Nilevik decoder, one function per mechanism, in whatever float type the inputs have
(the tests use float64).  TEST INFRASTRUCTURE ONLY: written from the model's equations, shares no code with the product
path, and also makes the random checkpoints the tests load into the product.

Every function sees ONE whole sequence from its first token: no cache, no state, no batching.

The design: token embedding plus a sinusoidal vector of the position; layers that read the stream itself and norm what
they add (``x += norm(mixer(x)); x += norm(ff(x)); x += norm(proj(gelu(gate x) * table[token]))``); two mixers, a windowed
softmax attention without rotation (normed queries and keys, a temperature on the queries that grows with the position,
a linear distance penalty per head, a sink logit, the unnormed keys as values, an elementwise output gate) and a gated
delta rule; a tanh-gelu gated feed-forward or none; the embedding table is the output projection.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch
import torch.nn.functional as F


# ------------------------------------------------------------------------------------------------ small pieces
def rms_ref(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh_ref(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def sinusoid_ref(T: int, width: int, dtype=torch.float64) -> torch.Tensor:
    """``[T, width]``: sine in the even entries, cosine in the odd ones, of ``t * 10000^(-2 i / width)`` for pair i."""
    out = torch.zeros(T, width, dtype=torch.float64)
    t = torch.arange(T, dtype=torch.float64)
    for d in range(width):
        ang = t * 10000.0 ** (-2.0 * (d // 2) / width)
        out[:, d] = torch.sin(ang) if d % 2 == 0 else torch.cos(ang)
    return out.to(dtype)


# ------------------------------------------------------------------------------------------------ attention
def query_temperature_ref(T: int, coef: float, every: float) -> torch.Tensor:
    return torch.tensor([1.0 + coef * math.log(math.floor((t + 1) / every) + 1) for t in range(T)], dtype=torch.float64)


def slope_ref(h: int, heads: int) -> float:
    return 2.0 ** (-8.0 * (h + 1) / heads)


def penalised_sink_attention_ref(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: Optional[int],
                                 slopes: List[float], sink: Optional[torch.Tensor]) -> torch.Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, Dv]`` -> ``[T, H, Dv]``: scores ``scale q.k - slope_h (i - j)`` over
    ``0 <= i - j < window``; the softmax's denominator has ``exp(sink_h)`` besides."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            lo = 0 if window is None else max(0, i - window + 1)
            s = (k[lo:i + 1, g] @ q[i, h]) * scale - slopes[h] * torch.arange(i - lo, -1, -1, dtype=q.dtype)
            if sink is None:
                p = torch.softmax(s, 0)
            else:
                m = torch.maximum(s.max(), sink[h])
                e = torch.exp(s - m)
                p = e / (e.sum() + torch.exp(sink[h] - m))
            out[i, h] = p @ v[lo:i + 1, g]
    return out


def attention_mixer_ref(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    raw = (h @ w["k"].T).view(T, G, D)
    q = rms_ref((h @ w["q"].T).view(T, H, D), eps) * w["q.norm"]
    k = rms_ref(raw, eps) * w["k.norm"]
    qt = m.get("q_temp")
    if qt:
        q = q * query_temperature_ref(T, qt["coef"], qt["every"]).to(h.dtype)[:, None, None]
    o = penalised_sink_attention_ref(q, k, raw, m["scale"], (m.get("mask") or {}).get("size"), [slope_ref(j, H) for j in range(H)],
                                     w["sink"])
    return (o.reshape(T, H * D) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ------------------------------------------------------------------------------------------------ gated delta rule
def short_conv_ref(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """``x [T, C]``, ``w [C, taps]`` (the last column weighs the current token), zeros before the start; then silu."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            if t - (taps - 1) + j >= 0:
                out[t] = out[t] + w[:, j] * x[t - (taps - 1) + j]
    return F.silu(out)


def unit_ref(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule_ref(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, beta: torch.Tensor, decay: torch.Tensor,
                   state: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``q, k [T, H, D]``, ``v [T, H, Dv]``, ``beta, decay [T, H]`` -> ``[T, H, Dv]``: ``S <- decay S``, ``u = beta (v - S^T k)``,
    ``S <- S + k u^T``, ``o = S^T q``.  ``state [H, D, Dv]``: where to leave the final state."""
    T, H, Dv = v.shape
    out = torch.zeros(T, H, Dv, dtype=v.dtype)
    for h in range(H):
        S = torch.zeros(q.shape[2], Dv, dtype=v.dtype)
        for t in range(T):
            S = decay[t, h] * S
            u = beta[t, h] * (v[t, h] - S.T @ k[t, h])
            S = S + torch.outer(k[t, h], u)
            out[t, h] = S.T @ q[t, h]
        if state is not None:
            state[h] = S
    return out


def delta_mixer_ref(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_ref(short_conv_ref(h @ w["q"].T, w["q.conv"]).view(T, G, D)) * D ** -0.5
    k = unit_ref(short_conv_ref(h @ w["k"].T, w["k.conv"]).view(T, G, D))
    v = short_conv_ref(h @ w["v"].T, w["v.conv"]).view(T, H, Dv)
    beta = torch.sigmoid(h @ w["b"].T)
    decay = torch.exp(-torch.exp(w["A_log"]) * F.softplus(h @ w["a"].T + w["dt_bias"]))
    pick = [j // (H // G) for j in range(H)]
    o = delta_rule_ref(q[:, pick], k[:, pick], v, beta, decay)
    o = rms_ref(o, eps) * w["norm"] * F.silu(h @ w["g"].T).view(T, H, Dv)
    return o.reshape(T, H * Dv) @ w["o"].T


# ------------------------------------------------------------------------------------------------ feed-forward, token input
def geglu_ref(h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    return (gelu_tanh_ref(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def token_side_ref(x: torch.Tensor, e: torch.Tensor, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    """What the per-layer token input adds: ``e [T, d]`` is the layer's part of the tokens' rows of the table."""
    y = (gelu_tanh_ref(x @ w["gate"].T) * e) @ w["proj"].T
    return rms_ref(y, eps) * w["norm"]


# ------------------------------------------------------------------------------------------------ the model
def _sub(weights: Dict[str, torch.Tensor], prefix: str, dtype) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v.to(dtype) for k, v in weights.items() if k.startswith(prefix)}


def nilevik_ref(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
                residual_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence."""
    eps = cfg["norm"]["eps"]
    idx = torch.tensor(tokens)
    x = weights["embed"].to(dtype)[idx] + sinusoid_ref(len(tokens), cfg["width"], dtype)
    side = (cfg.get("token_side") or {}).get("dim", 0)
    for i, entry in enumerate(cfg["layers"]):
        p = f"l{i}."
        mix = attention_mixer_ref if entry["type"] == "attention" else delta_mixer_ref
        x = x + rms_ref(mix(x, _sub(weights, p + "mix.", dtype), entry["mixer"], eps), eps) * weights[p + "norm1"].to(dtype)
        if entry.get("mlp") is not None:
            x = x + rms_ref(geglu_ref(x, _sub(weights, p + "mlp.", dtype)), eps) * weights[p + "norm2"].to(dtype)
        if side:
            e = weights["side.embed"].to(dtype)[idx][:, i * side:(i + 1) * side]
            x = x + token_side_ref(x, e, _sub(weights, p + "side.", dtype), eps)
        if residual_out is not None:
            residual_out.append(x.clone())
    return (rms_ref(x, eps) * weights["final.norm"].to(dtype)) @ weights["embed"].to(dtype).T


# ------------------------------------------------------------------------------------------------ test checkpoints
def attention_config(heads=6, kv_heads=2, dim=24, window=13, coef=0.3, every=7, scale=None) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": float(scale if scale is not None else dim ** -0.5)}
    if window is not None:
        m["mask"] = {"size": window}
    if coef is not None:
        m["q_temp"] = {"coef": coef, "every": every}
    return m


def delta_config(heads=4, kv_heads=2, dim=16, vdim=24, conv=4) -> dict:
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def nilevik_config(vocab=101, width=56, layers=None, eps=1e-5, side=12) -> dict:
    """``layers``: a list of ``(type, mixer config, feed-forward width or None)``."""
    if layers is None:
        layers = [("delta", delta_config(), 72), ("attention", attention_config(), 88), ("attention", attention_config(heads=3, kv_heads=3, dim=16, window=5), None),
                  ("delta", delta_config(heads=3, kv_heads=3, dim=24, vdim=16, conv=2), None)]
    return {"architecture": "Nilevik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "token_side": {"dim": side},
            "layers": [{"type": t, "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}} for t, m, ff in layers]}


def nilevik_random_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """bf16-representable random tensors under the checkpoint's names (fp32 tensors whose values survive a bf16 round trip)."""
    g = torch.Generator().manual_seed(seed)
    W, side = cfg["width"], cfg["token_side"]["dim"]

    def rnd(*shape, s=1.0):
        return (torch.randn(shape, generator=g) * s).to(torch.bfloat16).float()

    def lin(o, i):
        return rnd(o, i, s=i ** -0.5)

    def ones(n):
        return (1 + rnd(n, s=0.2)).to(torch.bfloat16).float()

    w = {"embed": rnd(cfg["vocab"], W), "side.embed": rnd(cfg["vocab"], len(cfg["layers"]) * side), "final.norm": ones(W)}
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        w[p + "norm1"] = ones(W)
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        if entry["type"] == "attention":
            w[p + "mix.q"], w[p + "mix.k"], w[p + "mix.g"], w[p + "mix.o"] = lin(H * D, W), lin(G * D, W), lin(H * D, W), lin(W, H * D)
            w[p + "mix.q.norm"], w[p + "mix.k.norm"], w[p + "mix.sink"] = ones(D), ones(D), rnd(H)
        else:
            Dv, taps = m["vdim"], m["conv"]
            for n, c in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                w[p + f"mix.{n}"], w[p + f"mix.{n}.conv"] = lin(c, W), rnd(c, taps, s=taps ** -0.5)
            w[p + "mix.b"], w[p + "mix.a"], w[p + "mix.g"], w[p + "mix.o"] = lin(H, W), lin(H, W), lin(H * Dv, W), lin(W, H * Dv)
            w[p + "mix.A_log"], w[p + "mix.dt_bias"], w[p + "mix.norm"] = rnd(H, s=0.5) - 1.5, rnd(H, s=0.5), ones(Dv)
            w[p + "mix.A_log"] = w[p + "mix.A_log"].to(torch.bfloat16).float()
        if entry["mlp"] is not None:
            ff = entry["mlp"]["ff"]
            w[p + "norm2"] = ones(W)
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(ff, W), lin(ff, W), lin(W, ff)
        if side:
            w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"] = lin(side, W), lin(W, side), ones(W)
    return w
