"""Plain restatement of the layer mechanisms of the Gevonex decoder (float64, one function per mechanism, written as
token-by-token loops and explicit sums): the checker of ``msa_amd``'s recurrent and latent-attention layers.  It shares
no code with the product path and reads a model as ``(config dict, {tensor name: tensor})``."""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Root-mean-square normalisation over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def dyn_tanh(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def token_shift(h, mix, before=None):
    """``h [T, W]`` mixed towards the token before it; ``before [W]`` is the last token of the portion before."""
    prev = torch.zeros_like(h)
    prev[1:] = h[:-1]
    if before is not None:
        prev[0] = before
    return h + (prev - h) * mix


def causal_conv(x, taps, bias):
    """Per-channel causal convolution of ``x [T, C]`` with ``taps [C, K]`` (last column: the current token)."""
    T, K = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        acc = bias.clone()
        for j in range(K):
            s = t - (K - 1) + j
            if s >= 0:
                acc = acc + taps[:, j] * x[s]
        out[t] = acc
    return out


def ssd_scan(x, Bm, Cm, dt, A_log, D, S=None):
    """``x [T, H, P]``, ``Bm / Cm [T, G, N]``, ``dt [T, H]`` (after softplus): returns ``y [T, H, P]`` and the state
    ``[H, N, P]``."""
    T, H, P = x.shape
    G, N = Bm.shape[1:]
    S = torch.zeros(H, N, P, dtype=x.dtype) if S is None else S
    grp = torch.arange(H) // (H // G)
    y = torch.zeros_like(x)
    for t in range(T):
        decay = torch.exp(-torch.exp(A_log) * dt[t])
        S = decay[:, None, None] * S + dt[t][:, None, None] * Bm[t][grp][:, :, None] * x[t][:, None, :]
        y[t] = (S * Cm[t][grp][:, :, None]).sum(1) + D[:, None] * x[t]
    return y, S


def gated_group_norm(y, z, w, parts, eps):
    """RMS norm in ``parts`` equal parts of ``y * silu(z)``, times ``w``."""
    v = y * silu(z)
    T, n = v.shape
    return rms(v.view(T, parts, n // parts), eps).reshape(T, n) * w


def min_gru(z, u, S=None):
    """``z`` (gate, after sigmoid) and ``u`` (pre-activation candidate), both ``[T, n]``: the states ``[T, n]``."""
    cand = torch.where(u >= 0, u + 0.5, sigmoid(u))
    S = torch.zeros_like(u[0]) if S is None else S
    out = []
    for t in range(u.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * cand[t]
        out.append(S)
    return torch.stack(out)


def sink_attention(q, k, v, sink, scale):
    """Causal attention of ``q [T, H, D]`` (the last T of the L tokens) over ``k [L, H, D]``, ``v [L, H, E]`` with a
    learned number per head in the denominator."""
    T, H, _ = q.shape
    L = k.shape[0]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        n = L - T + t + 1
        s = (q[t][None] * k[:n]).sum(-1) * scale                     # [n, H]
        m = torch.maximum(s.max(dim=0).values, sink)
        e = torch.exp(s - m)
        out[t] = (e[:, :, None] * v[:n]).sum(0) / (e.sum(0) + torch.exp(sink - m))[:, None]
    return out


# ------------------------------------------------------------------------------------------------ the mixers
def mamba2_mixer(w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, h):
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, T = H * P, h.shape[0]
    z, xbc, dt = torch.split(h @ w[p + "in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, Bm, Cm = torch.split(xbc, [inner, G * N, G * N], dim=-1)
    y, _ = ssd_scan(x.reshape(T, H, P), Bm.reshape(T, G, N), Cm.reshape(T, G, N), softplus(dt + w[p + "dt_bias"]),
                    w[p + "A_log"], w[p + "D"])
    return gated_group_norm(y.reshape(T, inner), z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


def mingru_mixer(w, p, m, eps, h):
    z = sigmoid(h @ w[p + "z"].T + w[p + "z.b"])
    u = h @ w[p + "x"].T + w[p + "x.b"]
    return (min_gru(z, u) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def latent_attention_mixer(w, p, m, eps, h):
    T, H = h.shape[0], m["heads"]
    q = (h @ w[p + "q"].T).view(T, H, m["dim"])
    c = rms(h @ w[p + "dkv"].T, eps) * w[p + "dkv.norm"]
    k = (c @ w[p + "uk"].T).view(T, H, m["dim"])
    v = (c @ w[p + "uv"].T).view(T, H, m["vdim"])
    return sink_attention(q, k, v, w[p + "sink"], m["scale"]).reshape(T, H * m["vdim"]) @ w[p + "o"].T


MIXERS = {"mamba2": mamba2_mixer, "mingru": mingru_mixer, "latent_attention": latent_attention_mixer}


# ------------------------------------------------------------------------------------------------ the decoder
def decoder_layer(w, i: int, layer: dict, eps: float, x):
    p = f"l{i}."
    norm = lambda n: dyn_tanh(x, w[p + n + ".alpha"], w[p + n], w[p + n + ".b"])
    gate = lambda n, h: sigmoid(h @ w[p + n].T + w[p + n + ".b"])
    h = norm("norm1")
    x = x + gate("rg1", h) * MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], eps, token_shift(h, w[p + "shift"]))
    if layer["mlp"] is not None:
        h = norm("norm2")
        x = x + gate("rg2", h) * (gelu_tanh(h @ w[p + "mlp.up"].T) @ w[p + "mlp.down"].T)
    return x


def layer_runs(config: dict) -> List[tuple]:
    """``(layer, pass)`` in the order they run; the pass is None outside the loop."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    return ([(i, None) for i in range(loop["start"])]
            + [(i, t) for t in range(loop["times"]) for i in range(loop["start"], loop["stop"])]
            + [(i, None) for i in range(loop["stop"], n)])


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens, trace: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one whole sequence; ``trace`` collects the residual stream after every layer run."""
    w = {k: v.to(F64) for k, v in weights.items() if v.is_floating_point()}
    eps = config["norm"]["eps"]
    x0 = x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, t in layer_runs(config):
        if t is not None and i == config["loop"]["start"]:
            x = torch.cat([x, x0], dim=-1) @ w["loop.in"].T + w["loop.step"][t]
        x = decoder_layer(w, i, config["layers"][i], eps, x)
        if trace is not None:
            trace.append(x)
    h = dyn_tanh(x, w["final.norm.alpha"], w["final.norm"], w["final.norm.b"])
    logits = h @ w["head"].T
    cap = config.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
