"""Layers of the decoders of mixed layers: token mixers (state space, minimal gated recurrence, latent attention, channel-wise
delta rule, rotary chunk attention), dense feed-forwards, and the two kinds of layer around them (gated residuals behind
dynamic-tanh norms and token shift; residuals with a norm on the sublayer's output).

A mixer projects its input with one matrix (``w_in``, rows padded so that a second matrix can follow in one launch), keeps
its own per-sequence state (``state_specs``) and has two forms of the work between its projections: ``mix`` for any rows of a
step, and ``decode`` for up to 16 sequences' single rows with the projection folded in.  The gated residuals' gates read the norm
output before the token shift, so such a layer's first matrix is ``[w_in ; gate]`` over two operands (``decode`` returns the gate's
columns beside the mixed rows); other layers pass ``w_in`` alone.
"""
from __future__ import annotations

from typing import Callable, Dict, Tuple

import torch
import torch.nn.functional as F

from . import seq_ops
from .cache import StateSpec
from .config import (AttentionConfig, ChannelDeltaConfig, HybridLayerConfig, LatentAttentionConfig, Mamba2Config,
                     MinGRUConfig)

Get = Callable[[str], torch.Tensor]
F32 = torch.float32
ROW_PAD = 32                  # rows of a matrix that another one follows are padded to this


def _pad_rows(w: torch.Tensor, multiple: int = ROW_PAD) -> torch.Tensor:
    pad = -w.shape[0] % multiple
    return torch.cat([w, w.new_zeros(pad, w.shape[1])]) if pad else w


def head_linear(x: torch.Tensor, w: torch.Tensor, heads: int) -> torch.Tensor:
    """Per-head products: ``x [T, heads K]``, ``w [heads N, K]`` -> ``[T, heads N]``."""
    T, K = x.shape[0], w.shape[1]
    if x.dtype == torch.bfloat16 and K % 8 == 0 and x.stride(0) % 8 == 0:
        if T <= seq_ops.MAX_ROWS:
            return seq_ops.rows_linear(x, w, groups=heads)
        return torch.cat([seq_ops.rows_linear(x[i:i + seq_ops.MAX_ROWS], w, groups=heads) for i in range(0, T, seq_ops.MAX_ROWS)])
    y = torch.bmm(x.reshape(T, heads, K).transpose(0, 1).contiguous(), w.view(heads, -1, K).transpose(1, 2).contiguous())
    return y.transpose(0, 1).reshape(T, -1)


class Mamba2Mixer:
    """State-space layer: ``[z | x | B | C | dt]`` from one projection, causal convolution + silu of x, B, C, scalar-decay
    recurrence per head, output gate, grouped RMS norm."""

    def __init__(self, c: Mamba2Config, width: int, eps: float):
        self.c, self.eps = c, eps

    def shapes(self, width: int) -> Dict[str, Tuple[int, ...]]:
        c = self.c
        ch = c.conv_channels
        return {"in": (c.inner + ch + c.heads, width), "conv": (ch, c.conv), "conv.b": (ch,), "dt_bias": (c.heads,),
                "A_log": (c.heads,), "D": (c.heads,), "norm": (c.inner,), "o": (width, c.inner)}

    def load(self, get: Get) -> None:
        self.w_in, self.w_o = _pad_rows(get("in")), get("o")
        self.taps, self.conv_b, self.dt_bias, self.A_log, self.D, self.norm = (
            get(n).to(F32).contiguous() for n in ("conv", "conv.b", "dt_bias", "A_log", "D", "norm"))

    def state_specs(self, dtype) -> Dict[str, StateSpec]:
        c = self.c
        return {"conv": StateSpec((c.conv - 1, c.conv_channels), F32), "ssm": StateSpec((c.heads, c.state, c.vdim), F32)}

    def decode_ok(self) -> bool:
        return self.c.inner % 8 == 0

    def _columns(self, proj):
        c = self.c
        a, b = c.inner, c.inner + c.conv_channels
        return proj[:, :a], proj[:, a:b], proj[:, b:b + c.heads]

    def _scan(self, xbc, z, dt, state, batch):
        c = self.c
        chunked = (xbc.dtype == torch.bfloat16 and batch.max_rows >= seq_ops.SSD_CHUNKED_ROWS and c.state % 8 == 0
                   and c.state <= 256 and c.vdim % 8 == 0)
        v = seq_ops.ssd(xbc, z, dt, self.dt_bias, self.A_log, self.D, c.heads, c.vdim, c.state, c.groups, state["ssm"], batch,
                        chunked=chunked)
        return seq_ops.group_rmsnorm(v, self.norm, c.norm_groups, self.eps)

    def mix(self, proj, state, batch):
        z, xbc, dt = self._columns(proj)
        return self._scan(seq_ops.conv_silu(xbc, self.taps, self.conv_b, state["conv"], batch), z, dt, state, batch)

    def decode(self, w, hs, h, state, batch):
        n_b = self.w_in.shape[0]
        out = seq_ops.rows_conv(hs, w, h, n_b, self.c.inner, self.taps, self.conv_b, state["conv"], batch.slot)
        z, xbc, dt = self._columns(out)
        return self._scan(xbc, z, dt, state, batch), out[:, n_b:]


class MinGRUMixer:
    """Gated recurrence whose gates read only the current token; z, candidate and output gate come from one projection with
    their rows interleaved (16 channels at a time)."""

    def __init__(self, c: MinGRUConfig, width: int, eps: float):
        self.c = c

    def shapes(self, width: int):
        n = self.c.width
        return {"z": (n, width), "z.b": (n,), "x": (n, width), "x.b": (n,), "g": (n, width), "o": (width, n)}

    def load(self, get: Get) -> None:
        self.w_in, self.w_o = seq_ops.interleave_gru(get("z"), get("x"), get("g")), get("o")
        self.z_b, self.u_b = get("z.b").to(F32).contiguous(), get("x.b").to(F32).contiguous()

    def state_specs(self, dtype):
        return {"gru": StateSpec((self.c.width,), F32)}

    def decode_ok(self) -> bool:
        return self.c.width % 8 == 0

    def mix(self, proj, state, batch):
        return seq_ops.min_gru(proj, self.z_b, self.u_b, self.c.width, state["gru"], batch)

    def decode(self, w, hs, h, state, batch):
        act, out = seq_ops.rows_gru(hs, w, h, self.c.width, self.z_b, self.u_b, state["gru"], batch.slot)
        return act, out[:, self.w_in.shape[0]:]


class LatentAttention:
    """Attention without positions over a shared low-rank latent per token (the only thing cached), with a learned sink per
    head.  Long portions expand the latents to keys and values; short ones multiply the queries by the key matrices and
    attend to the latents themselves."""

    ABSORB_ROWS = seq_ops.MAX_ROWS        # portions up to this many tokens

    def __init__(self, c: LatentAttentionConfig, width: int, eps: float):
        self.c, self.eps = c, eps

    def shapes(self, width: int):
        c = self.c
        return {"q": (c.heads * c.dim, width), "dkv": (c.kv_rank, width), "dkv.norm": (c.kv_rank,),
                "uk": (c.heads * c.dim, c.kv_rank), "uv": (c.heads * c.vdim, c.kv_rank), "sink": (c.heads,),
                "o": (width, c.heads * c.vdim)}

    def load(self, get: Get) -> None:
        c = self.c
        q, dkv = get("q"), get("dkv")
        if q.shape[0] % 8:                 # keep the latent columns 16-byte aligned
            q = _pad_rows(q, 8)
        self.c_at = q.shape[0]
        self.w_in, self.w_o = _pad_rows(torch.cat([q, dkv])), get("o")
        self.uk, self.uv = get("uk").contiguous(), get("uv").contiguous()
        self.uk_t = self.uk.view(c.heads, c.dim, c.kv_rank).transpose(1, 2).reshape(c.heads * c.kv_rank, c.dim).contiguous()
        self.c_norm, self.sink = get("dkv.norm").to(F32).contiguous(), get("sink").to(F32).contiguous()

    def state_specs(self, dtype):
        return {"latent": StateSpec((self.c.kv_rank,), dtype, per_token=True)}

    def decode_ok(self) -> bool:
        c = self.c
        return c.dim % 8 == 0 and c.kv_rank % 8 == 0 and (c.heads * c.vdim) % 8 == 0

    def _absorbed(self, q, cache, batch):
        c = self.c
        qa = head_linear(q, self.uk_t, c.heads)
        ctx = seq_ops.latent_attn(qa.view(batch.rows, c.heads, c.kv_rank), cache, self.sink, c.scale, batch, batch.max_keys)
        return head_linear(ctx.view(batch.rows, -1), self.uv, c.heads)

    def mix(self, proj, state, batch):
        c, cache = self.c, state["latent"]
        q = proj[:, :c.heads * c.dim]
        seq_ops.latent_append(proj[:, self.c_at:self.c_at + c.kv_rank], self.c_norm, self.eps, cache, batch)
        if batch.max_rows <= self.ABSORB_ROWS or not seq_ops.flash_ok(q.dtype, c.dim, c.vdim, c.scale) or proj.stride(0) % 8:
            return self._absorbed(q, cache, batch)
        ends = [p + n for p, n in zip(batch.positions, batch.counts)]
        if batch.n_seq == 1:
            lat, off = cache[batch.slots[0], :ends[0]], [0]
        else:
            lat = torch.cat([cache[s, :e] for s, e in zip(batch.slots, ends)])
            off = [sum(ends[:i]) for i in range(batch.n_seq)]
        return seq_ops.flash(q, F.linear(lat, self.uk), F.linear(lat, self.uv),
                             torch.tensor(off, dtype=torch.int64).to(q.device), self.sink, c.scale, c.heads, batch)

    def decode(self, w, hs, h, state, batch):
        c, n_b = self.c, self.w_in.shape[0]
        out = seq_ops.rows_linear(hs, w, x_b=h, n_b=n_b)
        seq_ops.latent_append(out[:, self.c_at:self.c_at + c.kv_rank], self.c_norm, self.eps, state["latent"], batch)
        return self._absorbed(out[:, :c.heads * c.dim], state["latent"], batch), out[:, n_b:]


def _pad_cols(w: torch.Tensor, n: int) -> torch.Tensor:
    return F.pad(w, (0, n - w.shape[1])) if n > w.shape[1] else w


class ChannelDeltaMixer:
    """Delta rule with a decay per key channel: ``[q | k | v | a1 | g1 | b]`` from one projection, causal convolution + silu of q, k
    and v, the decays and the output gate through a low rank, the recurrence, norm and gate per head."""

    def __init__(self, c: ChannelDeltaConfig, width: int, eps: float):
        self.c, self.eps = c, eps

    def shapes(self, width: int):
        c = self.c
        qk, v, a = c.kv_heads * c.dim, c.heads * c.vdim, c.heads * c.dim
        return {"q": (qk, width), "q.conv": (qk, c.conv), "k": (qk, width), "k.conv": (qk, c.conv), "v": (v, width), "v.conv": (v, c.conv),
                "b": (c.heads, width), "A_log": (c.heads,), "norm": (c.vdim,), "a1": ("a_rank", width), "a2": (a, "a_rank"),
                "dt_bias": (a,), "g1": ("g_rank", width), "g2": (v, "g_rank"), "o": (width, v)}

    def default_dims(self) -> Dict[str, int]:
        """Sizes that only the weights tell."""
        return {"a_rank": self.c.vdim, "g_rank": self.c.vdim}

    def load(self, get: Get) -> None:
        a1, a2, g1, g2 = (get(n) for n in ("a1", "a2", "g1", "g2"))
        R = -(-max(a1.shape[0], g1.shape[0]) // 8) * 8          # both ranks padded alike: their second products share a launch
        rank_rows = lambda w: F.pad(w, (0, 0, 0, R - w.shape[0]))
        qkv = _pad_rows(torch.cat([get("q"), get("k"), get("v")]), 8)
        self.a_at, self.g_at, self.b_at = qkv.shape[0], qkv.shape[0] + R, qkv.shape[0] + 2 * R
        self.w_in, self.w_o = _pad_rows(torch.cat([qkv, rank_rows(a1), rank_rows(g1), get("b")])).contiguous(), get("o").contiguous()
        a2 = _pad_rows(_pad_cols(a2, R))
        self.n_a = a2.shape[0]
        self.w_low = torch.cat([a2, _pad_cols(g2, R)]).contiguous()
        self.taps = torch.cat([get(n + ".conv") for n in "qkv"]).to(F32).contiguous()
        self.A_log, self.dt_bias, self.norm = (get(n).to(F32).contiguous() for n in ("A_log", "dt_bias", "norm"))

    def state_specs(self, dtype) -> Dict[str, StateSpec]:
        c = self.c
        return {"conv": StateSpec((c.conv - 1, c.conv_channels), F32), "delta": StateSpec((c.heads, c.dim, c.vdim), F32)}

    def decode_ok(self) -> bool:
        return (self.c.heads * self.c.vdim) % 8 == 0

    def _low(self, proj):
        """The low-rank operands of the decays and the gate."""
        return proj[:, self.a_at:self.g_at], proj[:, self.g_at:self.b_at]

    def _rule(self, qkv, a, gate, proj, state, batch):
        c = self.c
        chunked = batch.max_rows >= seq_ops.DELTA_CHUNKED_ROWS and seq_ops.delta_chunked_ok(qkv.dtype, c.dim, c.vdim)
        return seq_ops.delta(qkv, a[:, :c.heads * c.dim], proj[:, self.b_at:self.b_at + c.heads], gate, self.A_log, self.dt_bias, self.norm,
                             self.eps, c.heads, c.kv_heads, c.dim, c.vdim, state["delta"], batch, chunked)

    def mix(self, proj, state, batch):
        qkv = seq_ops.conv_silu(proj[:, :self.c.conv_channels], self.taps, None, state["conv"], batch)
        a_low, g_low = self._low(proj)
        return self._rule(qkv, F.linear(a_low, self.w_low[:self.n_a]), F.linear(g_low, self.w_low[self.n_a:]), proj, state, batch)

    def decode(self, w, hs, h, state, batch):
        n_b = self.w_in.shape[0]
        out = seq_ops.rows_conv(hs, w, h, n_b, 0, self.taps, None, state["conv"], batch.slot)
        a_low, g_low = self._low(out)
        low = seq_ops.rows_linear(a_low, self.w_low, x_b=g_low, n_b=self.n_a)
        return self._rule(out[:, :self.c.conv_channels], low[:, :self.n_a], low[:, self.n_a:], out, state, batch), out[:, n_b:]


class RotaryAttention:
    """Grouped-query attention with query / key norms, rotary positions, a chunk mask and a gate per head.  The cache holds keys
    (normed and rotated) and values per key head; a layer with ``kv_from`` has none and reads an earlier layer's."""

    SPLIT_ROWS = seq_ops.MAX_ROWS         # portions up to this many tokens take the split-keys form

    def __init__(self, c: AttentionConfig, width: int, eps: float):
        self.c, self.eps, self.kv_from = c, eps, c.kv_from

    def shapes(self, width: int):
        c = self.c
        out = {"q": (c.heads * c.dim, width), "q.norm": (c.dim,), "g": (c.heads, width), "o": (width, c.heads * c.vdim)}
        if self.kv_from is None:
            out.update({"k": (c.kv_heads * c.dim, width), "v": (c.kv_heads * c.vdim, width), "k.norm": (c.dim,)})
        return out

    def load(self, get: Get) -> None:
        parts = [_pad_rows(get(n), 8) for n in (("q", "k", "v", "g") if self.kv_from is None else ("q", "g"))]
        self.at = [sum(p.shape[0] for p in parts[:i]) for i in range(len(parts))]
        self.w_in, self.w_o = _pad_rows(torch.cat(parts)).contiguous(), get("o").contiguous()
        self.q_norm = get("q.norm").to(F32).contiguous()
        self.k_norm = get("k.norm").to(F32).contiguous() if self.kv_from is None else None
        freqs = self.c.rot.frequencies() if self.c.rot is not None else []
        self.freqs = torch.tensor(freqs, dtype=torch.float64, device=self.w_in.device)

    def state_specs(self, dtype):
        c = self.c
        if self.kv_from is not None:
            return {}
        return {"k": StateSpec((c.kv_heads, c.dim), dtype, per_token=True), "v": StateSpec((c.kv_heads, c.vdim), dtype, per_token=True)}

    def decode_ok(self) -> bool:
        return (self.c.heads * self.c.vdim) % 8 == 0

    def mix(self, proj, state, batch):
        c, kc, vc = self.c, state["k"], state["v"]
        cols = lambda i, n: proj[:, self.at[i]:self.at[i] + n]
        own = {} if self.kv_from is not None else {"k": cols(1, c.kv_heads * c.dim), "v": cols(2, c.kv_heads * c.vdim), "k_norm": self.k_norm}
        q = seq_ops.qk_rope_append(cols(0, c.heads * c.dim), self.q_norm, self.freqs, self.eps, kc, vc, batch, **own)
        gate, chunk = cols(len(self.at) - 1, c.heads), c.mask.size if c.mask is not None else 0
        if batch.max_rows > self.SPLIT_ROWS and seq_ops.flash_ok(q.dtype, c.dim, c.vdim, c.scale):
            rows = kc.shape[0] * kc.shape[1]
            return seq_ops.flash(q.view(batch.rows, -1), kc.view(rows, -1), vc.view(rows, -1), batch.cache_rows(kc.shape[1]), None, c.scale,
                                 c.heads, batch, c.kv_heads, chunk, gate)
        return seq_ops.kv_attn(q, kc, vc, c.scale, batch, chunk, gate)

    def decode(self, w, hs, h, state, batch):
        n_b = self.w_in.shape[0]
        out = seq_ops.rows_linear(hs, w, x_b=h, n_b=n_b)
        return self.mix(out, state, batch), out[:, n_b:]


MIXERS = {"mamba2": Mamba2Mixer, "mingru": MinGRUMixer, "latent_attention": LatentAttention, "channel_delta": ChannelDeltaMixer,
          "attention": RotaryAttention}


def norm_shapes(name: str, width: int):
    return {name: (width,), name + ".alpha": (), name + ".b": (width,)}


def load_norm(get: Get, name: str) -> seq_ops.DynTanhNorm:
    return seq_ops.DynTanhNorm(get(name).to(F32).contiguous(), get(name + ".b").to(F32).contiguous(), float(get(name + ".alpha")))


class HybridLayer:
    """Token shift and gated residuals around a mixer and an optional dense feed-forward."""

    def __init__(self, c: HybridLayerConfig, width: int, eps: float):
        self.width, self.mlp = width, c.mlp
        self.mixer = MIXERS[c.type](c.mixer, width, eps)

    def shapes(self) -> Dict[str, Tuple[int, ...]]:
        W = self.width
        out = {**norm_shapes("norm1", W), "shift": (W,), "rg1": (W, W), "rg1.b": (W,)}
        out.update({"mix." + n: s for n, s in self.mixer.shapes(W).items()})
        if self.mlp is not None:
            out.update({**norm_shapes("norm2", W), "rg2": (W, W), "rg2.b": (W,), "mlp.up": (self.mlp.ff, W), "mlp.down": (W, self.mlp.ff)})
        return out

    def load(self, get: Get) -> None:
        self.norm1, self.shift = load_norm(get, "norm1"), get("shift").to(F32).contiguous()
        self.mixer.load(lambda n: get("mix." + n))
        # the mixer's matrix and the gate's lie behind one another: one launch when decoding
        self.w_in = torch.cat([self.mixer.w_in, get("rg1")]).contiguous()
        self.n_mix = self.mixer.w_in.shape[0]
        self.mixer.w_in = self.w_in[:self.n_mix]
        self.w_gate, self.gate_b, self.w_o = self.w_in[self.n_mix:], get("rg1.b").to(F32).contiguous(), self.mixer.w_o.contiguous()
        if self.mlp is not None:
            self.norm2 = load_norm(get, "norm2")
            up = _pad_rows(get("mlp.up"))
            self.n_up = up.shape[0]
            self.w_up, self.w_down = torch.cat([up, get("rg2")]).contiguous(), get("mlp.down").contiguous()
            self.gate2_b = get("rg2.b").to(F32).contiguous()

    def state_specs(self, dtype) -> Dict[str, StateSpec]:
        return {"shift": StateSpec((self.width,), F32), **self.mixer.state_specs(dtype)}

    def decode_ok(self) -> bool:
        return self.width % 8 == 0 and (self.mlp is None or self.mlp.ff % 8 == 0) and self.mixer.decode_ok()


class PostNormLayer:
    """A mixer and an optional clamped gated feed-forward, each with a norm on its output before it joins the stream."""

    def __init__(self, c: HybridLayerConfig, width: int, eps: float):
        self.width, self.mlp = width, c.mlp
        self.mixer = MIXERS[c.type](c.mixer, width, eps)

    def shapes(self):
        W = self.width
        out = {"norm1": (W,), **{"mix." + n: s for n, s in self.mixer.shapes(W).items()}}
        if self.mlp is not None:
            out.update({"norm2": (W,), "mlp.gate": (self.mlp.ff, W), "mlp.up": (self.mlp.ff, W), "mlp.down": (W, self.mlp.ff)})
        return out

    def load(self, get: Get) -> None:
        self.mixer.load(lambda n: get("mix." + n))
        self.norm1, self.w_o = get("norm1").to(F32).contiguous(), self.mixer.w_o
        if self.mlp is not None:
            self.norm2, self.w_down = get("norm2").to(F32).contiguous(), get("mlp.down").contiguous()
            self.w_gate_up = seq_ops.interleave_pairs(get("mlp.gate"), get("mlp.up"))

    def state_specs(self, dtype) -> Dict[str, StateSpec]:
        return self.mixer.state_specs(dtype)

    def decode_ok(self) -> bool:
        return self.width % 8 == 0 and (self.mlp is None or self.mlp.ff % 8 == 0) and self.mixer.decode_ok()
