"""Decoder of mixed layers (state space, minimal gated recurrence, latent attention, ...) with dynamic-tanh norms, token shift,
gated residuals and an optional looped range of layers: the Gevonex architecture.

The residual stream is fp32.  Between two matrices stands one fused step: gated residual, norm and token shift of the next
consumer (``seq_ops.residual_norm``).  Up to 16 sequences that bring one token each (bf16) take the decode form, in which
that step, and everything else that is element-wise, is the epilogue of a weight-streaming product: four launches a layer
besides the state-space / attention step.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from . import seq_ops
from .cache import SequenceStateCache
from .config import HybridConfig
from .hybrid_layers import HybridLayer, load_norm, norm_shapes
from .step_decoder import StepDecoder


class HybridForCausalLM(StepDecoder):
    def __init__(self, config: HybridConfig):
        super().__init__(config, HybridLayer)

    def _outer_shapes(self):
        c = self.config
        out = {"embed": (c.vocab, c.width), "head": (c.vocab, c.width), **norm_shapes("final.norm", c.width)}
        if c.loop is not None:
            out.update({"loop.in": (c.width, 2 * c.width), "loop.step": (c.loop.times, c.width)})
        return out

    def _load_outer(self, get):
        c = self.config
        self.final_norm = load_norm(get, "final.norm")
        if c.loop is not None:
            w = get("loop.in")
            x_part, x0_part = w[:, :c.width], w[:, c.width:]
            # bf16 products take the fp32 stream as high and low part (seq_ops.join)
            self.loop_in = torch.cat([x_part, x_part, x0_part] if self.dtype == torch.bfloat16 else [x_part, x0_part], dim=1).contiguous()
            self.loop_step = get("loop.step").to(torch.float32).contiguous()

    # ---------------------------------------------------------------------------------------- steps
    def _starts_pass(self, r: int) -> bool:
        return r < len(self.runs) and self.runs[r][1] is not None and self.runs[r][0] == self.config.loop.start

    def _consumer(self, r: int, cache: SequenceStateCache) -> dict:
        """What reads the stream in front of run ``r``: norm, token shift and its state, or nothing when a pass starts there
        (the stream is projected first), or the final norm."""
        if r == len(self.runs):
            return {"norm": self.final_norm}
        layer = self.layers[self.runs[r][0]]
        return {"norm": layer.norm1, "shift": layer.shift, "prev": cache.tensors[r]["shift"]}

    def _block_rows(self, tokens, batch, cache, trace=None):
        """Any rows: every element-wise step a kernel of its own between the products."""
        dt = self.dtype
        x0 = x = self._embed(tokens)
        h = hs = None
        for r, (i, t) in enumerate(self.runs):
            layer, state = self.layers[i], self.run_state(cache, r)
            if self._starts_pass(r):
                x = self._product_f32(seq_ops.join(x, x0, dt), self.loop_in).add_(self.loop_step[t])
            if h is None:
                x, h, hs = seq_ops.residual_norm(x, batch, dt, **self._consumer(r, cache))
            after = {} if self._starts_pass(r + 1) else self._consumer(r + 1, cache)
            y = F.linear(layer.mixer.mix(F.linear(hs, layer.mixer.w_in), state, batch), layer.w_o)
            nxt = {"norm": layer.norm2} if layer.mlp is not None else after
            x, h, hs = seq_ops.residual_norm(x, batch, dt, y, F.linear(h, layer.w_gate), layer.gate_b, **nxt)
            if layer.mlp is not None:
                up = F.linear(h, layer.w_up)
                act = seq_ops.gelu_(up[:, :layer.mlp.ff])
                x, h, hs = seq_ops.residual_norm(x, batch, dt, F.linear(act, layer.w_down), up[:, layer.n_up:], layer.gate2_b, **after)
            if trace is not None:
                trace.append(x.clone())
        return h

    def _decode_rows(self, tokens, batch, cache, trace=None):
        """One token for each of up to 16 sequences (bf16)."""
        loop = self.config.loop
        x0 = self._embed(tokens)
        x = x0.clone() if loop is not None and loop.start > 0 else x0
        h = hs = None
        for r, (i, t) in enumerate(self.runs):
            layer, state = self.layers[i], self.run_state(cache, r)
            if self._starts_pass(r):
                x = seq_ops.rows_linear_f32(seq_ops.join(x, x0, self.dtype), self.loop_in, add=self.loop_step[t])
            if h is None:
                _, h, hs = seq_ops.residual_norm(x, batch, self.dtype, **self._consumer(r, cache))
            after = {} if self._starts_pass(r + 1) else self._consumer(r + 1, cache)
            mixed, gate = layer.mixer.decode(layer.w_in, hs, h, state, batch)
            nxt = {"norm": layer.norm2} if layer.mlp is not None else after
            h, hs = seq_ops.rows_residual(mixed, layer.w_o, x, gate, layer.gate_b, batch.slot, **nxt)
            if layer.mlp is not None:
                up = seq_ops.rows_linear(h, layer.w_up, gelu_n=layer.n_up)
                h, hs = seq_ops.rows_residual(up[:, :layer.mlp.ff], layer.w_down, x, up[:, layer.n_up:], layer.gate2_b, batch.slot, **after)
            if trace is not None:
                trace.append(x.clone())
        return h
