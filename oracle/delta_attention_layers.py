"""Plain restatement of the layer mechanisms of the Sugizen decoder (float64, one function per mechanism, token-by-token loops and
explicit sums), which the tests compare ``msa_amd`` with: channel-wise delta rule, rotary chunk attention, clamped gated feed-forward and
output-normed residuals.  It shares no code with the product path and reads a model as ``(config dict, {tensor name: tensor})``."""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

from .recurrent_layers import F64, causal_conv, rms, sigmoid, silu, softplus


def unit(x):
    """Vectors of length one over the last axis (1e-6 under the root)."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, log_decay, beta, S=None):
    """``q / k [T, H, D]`` (unit vectors, q scaled), ``v [T, H, E]``, ``log_decay [T, H, D]``, ``beta [T, H]``: read-outs
    ``[T, H, E]`` and the state ``[H, D, E]``.  Per token and head: decay the rows, replace what the key recalls, read."""
    T, H, D = k.shape
    S = torch.zeros(H, D, v.shape[2], dtype=v.dtype) if S is None else S
    out = torch.zeros_like(v)
    for t in range(T):
        S = torch.exp(log_decay[t])[:, :, None] * S
        recalled = (S * k[t][:, :, None]).sum(1)
        u = beta[t][:, None] * (v[t] - recalled)
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def gated_head_norm(o, w, gate, eps):
    """``o [T, H, E]`` over its root mean square per head, times ``w [E]``, times ``sigmoid(gate)``."""
    return rms(o, eps) * w * sigmoid(gate)


def rotary_frequencies(base: float, dims: int, scaling: Optional[dict] = None) -> List[float]:
    """Radians per position of each rotated pair; ``scaling`` stretches long wavelengths by ``factor``, keeps short ones, and
    blends in between."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling is not None:
            length = 2.0 * math.pi / f
            if length > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            elif length >= scaling["original"] / scaling["high"]:
                s = (scaling["original"] / length - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate(x, positions, freqs):
    """``x [T, heads, D]``: dimension i turned against dimension i + dims/2, ``dims = 2 len(freqs)``; the rest unchanged."""
    n = len(freqs)
    a = torch.as_tensor(positions, dtype=F64)[:, None, None] * torch.tensor(freqs, dtype=F64)
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., 2 * n:]], dim=-1)


def chunk_attention(q, k, v, scale: float, size: Optional[int]):
    """Softmax attention of ``q [T, H, D]`` (the last T of the L tokens) over ``k [L, G, D]``, ``v [L, G, E]``: a position sees
    the positions up to itself in its own stretch of ``size`` (all of them with None)."""
    T, H, _ = q.shape
    L, G, _ = k.shape
    kv = torch.arange(H) // (H // G)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        i = L - T + t
        lo = 0 if size is None else i // size * size
        s = (q[t][None] * k[lo:i + 1, kv]).sum(-1) * scale
        p = torch.exp(s - s.max(dim=0).values)
        out[t] = (p[:, :, None] * v[lo:i + 1, kv]).sum(0) / p.sum(0)[:, None]
    return out


def clamped_glu(gate, up, limit: float):
    g, u = torch.clamp(gate, max=limit), torch.clamp(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


# ------------------------------------------------------------------------------------------------ the mixers
def channel_delta_mixer(w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, h, shared):
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def stream(n):
        x = h @ w[p + n].T
        return silu(causal_conv(x, w[p + n + ".conv"], torch.zeros(x.shape[1], dtype=x.dtype)))
    of = torch.arange(H) // (H // G)
    q = unit(stream("q").view(T, G, D))[:, of] * D ** -0.5
    k = unit(stream("k").view(T, G, D))[:, of]
    v = stream("v").view(T, H, E)
    beta = sigmoid(h @ w[p + "b"].T)
    step = softplus((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]).view(T, H, D)
    o, _ = delta_rule(q, k, v, -torch.exp(w[p + "A_log"])[None, :, None] * step, beta)
    gate = ((h @ w[p + "g1"].T) @ w[p + "g2"].T).view(T, H, E)
    return gated_head_norm(o, w[p + "norm"], gate, eps).reshape(T, H * E) @ w[p + "o"].T


def attention_mixer(w, p, m, eps, h, shared):
    """``shared`` maps a layer to its rotated keys and its values; layers with keys of their own enter theirs."""
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot = m["rot"]
    freqs = rotary_frequencies(rot["base"], rot["dims"], rot.get("scaling"))
    turned = lambda n, heads: rotate(rms((h @ w[p + n].T).view(T, heads, D), eps) * w[p + n + ".norm"], range(T), freqs)
    q = turned("q", H)
    if m.get("kv_from") is None:
        k, v = turned("k", G), (h @ w[p + "v"].T).view(T, G, E)
        shared[p] = (k, v)
    else:
        k, v = shared[f"l{m['kv_from']}.mix."]
    o = chunk_attention(q, k, v, m["scale"], (m.get("mask") or {}).get("size"))
    return (o * sigmoid(h @ w[p + "g"].T)[:, :, None]).reshape(T, H * E) @ w[p + "o"].T


MIXERS = {"channel_delta": channel_delta_mixer, "attention": attention_mixer}


# ------------------------------------------------------------------------------------------------ the decoder
def forward(config: dict, weights: Dict[str, torch.Tensor], tokens, trace: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one whole sequence; ``trace`` collects the residual stream after every layer."""
    w = {n: t.to(F64) for n, t in weights.items() if t.is_floating_point()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    shared: dict = {}
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        x = x + rms(MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], eps, x, shared), eps) * w[p + "norm1"]
        if layer["mlp"] is not None:
            act = clamped_glu(x @ w[p + "mlp.gate"].T, x @ w[p + "mlp.up"].T, layer["mlp"]["limit"])
            x = x + rms(act @ w[p + "mlp.down"].T, eps) * w[p + "norm2"]
        if trace is not None:
            trace.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
