"""Decoder of mixed layers (channel-wise delta rule, rotary chunk attention, ...) with RMS norms on the sublayers' outputs only and
clamped gated feed-forwards: the Sugizen architecture.

The residual stream is fp32 and is itself (in the activations' type) what every sublayer reads.  Behind an output projection
stands one fused step, residual + norm + the next operand (``seq_ops.rms_residual``); it needs a row's statistics, so that also
when decoding it is a launch of its own.  The decode form folds the convolution into the mixer's input projection and the gated
unit into the feed-forward's.
"""
from __future__ import annotations

import torch.nn.functional as F

from . import seq_ops
from .config import PostNormConfig
from .hybrid_layers import F32, PostNormLayer
from .step_decoder import StepDecoder


class PostNormForCausalLM(StepDecoder):
    def __init__(self, config: PostNormConfig):
        super().__init__(config, PostNormLayer)

    def _outer_shapes(self):
        c = self.config
        return {"embed": (c.vocab, c.width), "head": (c.vocab, c.width), "final.norm": (c.width,)}

    def _load_outer(self, get):
        self.final_norm = get("final.norm").to(F32).contiguous()

    def _residual(self, x, y, w, last: bool):
        """The stream (in place) and the next operand; behind the last sublayer that is the final norm's output."""
        return seq_ops.rms_residual(x, self.dtype, y, w, self.config.norm_eps, self.final_norm if last else None, out=x)

    def _start(self, tokens):
        x = self._embed(tokens)
        _, h = seq_ops.rms_residual(x, self.dtype, eps=self.config.norm_eps, next_w=None if self.layers else self.final_norm)
        return x, h

    def _layers(self, tokens, trace, mix, product, feed_forward):
        x, h = self._start(tokens)
        for r, layer in enumerate(self.layers):
            last = r + 1 == len(self.layers)
            x, h = self._residual(x, product(mix(r, layer, h), layer.w_o), layer.norm1, last and layer.mlp is None)
            if layer.mlp is not None:
                x, h = self._residual(x, product(feed_forward(layer, h), layer.w_down), layer.norm2, last)
            if trace is not None:
                trace.append(x.clone())
        return h

    def _block_rows(self, tokens, batch, cache, trace=None):
        """Any rows: every element-wise step a kernel of its own between the products."""
        return self._layers(tokens, trace,
                            lambda r, l, h: l.mixer.mix(F.linear(h, l.mixer.w_in), self.run_state(cache, r), batch), F.linear,
                            lambda l, h: seq_ops.clamped_glu(F.linear(h, l.w_gate_up), l.mlp.limit))

    def _decode_rows(self, tokens, batch, cache, trace=None):
        """One token for each of up to 16 sequences (bf16)."""
        return self._layers(tokens, trace,
                            lambda r, l, h: l.mixer.decode(l.mixer.w_in, h, None, self.run_state(cache, r), batch)[0], seq_ops.rows_linear,
                            lambda l, h: seq_ops.rows_glu(h, l.w_gate_up, l.mlp.limit))
