"""Decoder of mixed layers (state space, minimal gated recurrence, latent attention) with dynamic-tanh norms, token shift,
gated residuals and an optional looped range of layers: the Gevonex architecture.

The model works in steps: a step brings the next tokens of any number of sequences, and everything earlier tokens left is in
a :class:`~msa_amd.cache.SequenceStateCache`.  Generation, and anything else that feeds tokens, goes through :meth:`step`.

The residual stream is fp32.  Between two matrices stands one fused step: gated residual, norm and token shift of the next
consumer (``seq_ops.residual_norm``).  Up to 16 sequences that bring one token each (bf16) take the decode form, in which
that step, and everything else that is element-wise, is the epilogue of a weight-streaming product: four launches a layer
besides the state-space / attention step.
"""
from __future__ import annotations

from typing import Dict, Hashable, List, Optional, Sequence, Tuple

import torch
import torch.nn.functional as F

from . import _lib, seq_ops
from .cache import SequenceStateCache
from .config import HybridConfig
from .generation import greedy_decode
from .hybrid_layers import HybridLayer, load_norm, norm_shapes

Entry = Tuple[Hashable, Sequence[int], Sequence[int]]        # (sequence, its next tokens, places whose logits are wanted)


class HybridForCausalLM:
    def __init__(self, config: HybridConfig):
        self.config = config
        self.layers = [HybridLayer(c, config.width, config.norm_eps) for c in config.layers]
        self.runs = config.runs

    # ---------------------------------------------------------------------------------------- weights
    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        """Names and shapes of every tensor the configuration asks for."""
        c = self.config
        out = {"embed": (c.vocab, c.width), "head": (c.vocab, c.width), **norm_shapes("final.norm", c.width)}
        if c.loop is not None:
            out.update({"loop.in": (c.width, 2 * c.width), "loop.step": (c.loop.times, c.width)})
        for i, layer in enumerate(self.layers):
            out.update({f"l{i}.{n}": s for n, s in layer.shapes().items()})
        return out

    @classmethod
    def from_tensors(cls, config: HybridConfig, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cuda:0"):
        """Packs ``tensors`` (names and shapes of :meth:`tensor_shapes`) for the device; matrices in ``dtype``, small vectors
        in fp32."""
        if dtype not in (torch.bfloat16, torch.float32):
            raise TypeError(f"unsupported dtype {dtype}: bfloat16 or float32")
        self = cls(config)
        for name, shape in self.tensor_shapes().items():
            if name not in tensors:
                raise KeyError(f"missing tensor {name!r}")
            if tuple(tensors[name].shape) != tuple(shape):
                raise ValueError(f"tensor {name!r} is {tuple(tensors[name].shape)}, the configuration asks for {tuple(shape)}")
        self.dtype, self.device = dtype, torch.device(device)
        get = lambda n: tensors[n].to(self.device, dtype if tensors[n].dim() > 1 else torch.float32)
        self.embed, self.head = get("embed"), get("head").contiguous()
        self.final_norm = load_norm(get, "final.norm")
        if config.loop is not None:
            w = get("loop.in")
            x_part, x0_part = w[:, :config.width], w[:, config.width:]
            # bf16 products take the fp32 stream as high and low part (seq_ops.join)
            self.loop_in = torch.cat([x_part, x_part, x0_part] if dtype == torch.bfloat16 else [x_part, x0_part], dim=1).contiguous()
            self.loop_step = get("loop.step").to(torch.float32).contiguous()
        for i, layer in enumerate(self.layers):
            layer.load(lambda n, i=i: get(f"l{i}.{n}"))
        self.fused_decode = dtype == torch.bfloat16 and config.width % 8 == 0 and all(l.decode_ok() for l in self.layers)
        return self

    @classmethod
    def random(cls, config: HybridConfig, seed: int = 0, dtype=torch.bfloat16, device="cuda:0"):
        """Random weights on the device (benchmarks): matrices scaled to keep activations of order one."""
        dev = torch.device(device)
        g = torch.Generator(device=dev).manual_seed(seed)
        tensors = {}
        for name, shape in cls(config).tensor_shapes().items():
            t = torch.randn(shape, generator=g, device=dev)
            if len(shape) > 1 and not name.endswith((".conv", "loop.step", "embed")):
                t *= shape[-1] ** -0.5
            elif name.endswith(("norm", "norm1", "norm2", ".alpha")):
                t = torch.ones(shape, device=dev)
            elif name.endswith("A_log"):
                t = torch.rand(shape, generator=g, device=dev)
            elif name.endswith("dt_bias"):
                t = t - 4.0
            elif name.endswith("shift"):
                t = torch.rand(shape, generator=g, device=dev)
            elif name.endswith((".b", "conv", "loop.step")):
                t *= 0.3
            tensors[name] = t.to(torch.bfloat16)
        return cls.from_tensors(config, tensors, dtype, device)

    # ---------------------------------------------------------------------------------------- state
    def create_cache(self, slots: int = 1, capacity: int = 256) -> SequenceStateCache:
        """One set of states per layer run: a looped layer keeps its passes apart."""
        return SequenceStateCache([self.layers[i].state_specs(self.dtype) for i, _ in self.runs], self.device, slots, capacity)

    # ---------------------------------------------------------------------------------------- steps
    @torch.no_grad()
    def step(self, cache: SequenceStateCache, entries: Sequence[Entry]) -> Optional[torch.Tensor]:
        """Feeds every entry's tokens behind what its sequence has been fed before (a key not seen before starts a
        sequence).  Returns fp32 logits ``[wanted, vocab]`` in the order of the entries and their wanted places, or None."""
        entries = [(k, torch.as_tensor(t, dtype=torch.int64).cpu(), w) for k, t, w in entries]
        for key, tokens, want in entries:
            if not len(tokens) or any(not 0 <= w < len(tokens) for w in want):
                raise ValueError(f"sequence {key!r}: no tokens, or a wanted place outside them")
            if not 0 <= int(tokens.min()) <= int(tokens.max()) < self.config.vocab:
                raise ValueError(f"sequence {key!r}: token outside the vocabulary")
        cache.reserve(max(cache.length.get(k, 0) + len(t) for k, t, _ in entries))
        for key, _, _ in entries:
            if key not in cache.slot_of:
                cache.open(key)
        counts = [len(t) for _, t, _ in entries]
        batch = seq_ops.StepBatch(counts, [cache.slot_of[k] for k, _, _ in entries], [cache.length[k] for k, _, _ in entries],
                                  self.device)
        tokens = torch.cat([t for _, t, _ in entries]).to(self.device)
        rows, at = [], 0
        for (_, ts, want) in entries:
            rows += [at + w for w in want]
            at += len(ts)
        logits = self.forward_rows(tokens, batch, cache, rows)
        for key, ts, _ in entries:
            cache.advance(key, len(ts))
        return logits

    def forward_rows(self, tokens: torch.Tensor, batch: seq_ops.StepBatch, cache: SequenceStateCache, rows: List[int],
                     trace: Optional[list] = None) -> Optional[torch.Tensor]:
        """Logits of ``rows`` of a step whose states are reserved.  ``trace`` (a list) receives a copy of the residual stream
        after every layer run."""
        if self.fused_decode and batch.max_rows == 1 and batch.rows <= seq_ops.MAX_ROWS:
            h = self._decode_rows(tokens, batch, cache, trace)
        else:
            h = self._block_rows(tokens, batch, cache, trace)
        if not rows:
            return None
        if rows != list(range(batch.rows)):
            h = h[rows[0]:rows[0] + 1] if len(rows) == 1 else h[torch.tensor(rows, device=h.device)]
        cap = self.config.logit_softcap or 0.0
        if self.fused_decode and len(rows) <= seq_ops.MAX_ROWS:
            return seq_ops.rows_linear_f32(h, self.head, cap)
        return seq_ops.softcap(self._product_f32(h, self.head), cap)

    def _product_f32(self, x, w):
        """Vendor product with fp32 output."""
        return torch.mm(x, w.t(), out_dtype=torch.float32) if x.dtype == torch.bfloat16 else F.linear(x, w)

    def _starts_pass(self, r: int) -> bool:
        return r < len(self.runs) and self.runs[r][1] is not None and self.runs[r][0] == self.config.loop.start

    def _consumer(self, r: int, cache: SequenceStateCache) -> dict:
        """What reads the stream in front of run ``r``: norm, token shift and its state, or nothing when a pass starts there
        (the stream is projected first), or the final norm."""
        if r == len(self.runs):
            return {"norm": self.final_norm}
        layer = self.layers[self.runs[r][0]]
        return {"norm": layer.norm1, "shift": layer.shift, "prev": cache.tensors[r]["shift"]}

    def _embed(self, tokens):
        return self.embed[tokens].to(torch.float32)

    def _block_rows(self, tokens, batch, cache, trace=None):
        """Any rows: every element-wise step a kernel of its own between the products."""
        dt = self.dtype
        x0 = x = self._embed(tokens)
        h = hs = None
        for r, (i, t) in enumerate(self.runs):
            layer, state = self.layers[i], cache.tensors[r]
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
            layer, state = self.layers[i], cache.tensors[r]
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

    # ---------------------------------------------------------------------------------------- generation
    @torch.no_grad()
    def generate_greedy(self, input_ids, attention_mask, max_new_tokens: int, cache: Optional[SequenceStateCache] = None,
                        timings: Optional[dict] = None, use_graph: bool = False):
        """Feeds the prompts ``input_ids [B, S]`` (``attention_mask`` 0 on padding, on either side) and decodes
        ``max_new_tokens`` greedily.  Returns ``(tokens [B, max_new_tokens], cache)``; the sequences ``0 .. B - 1`` stay open
        in the cache, with every token but the last fed."""
        import time
        prompts = [ids[mask != 0] for ids, mask in zip(input_ids.cpu(), attention_mask.cpu())]
        B = len(prompts)
        cache = cache if cache is not None else self.create_cache(B)
        longest = max(len(p) for p in prompts)
        cache.reserve(longest + max_new_tokens)
        if timings is not None:
            torch.cuda.synchronize()
            t0 = time.perf_counter()
        logits = self.step(cache, [(b, p, [len(p) - 1]) for b, p in enumerate(prompts)])
        lib = _lib.load_seq()
        tok = seq_ops.greedy_tokens(logits)
        if timings is not None:
            torch.cuda.synchronize()
            timings["prefill_s"] = time.perf_counter() - t0
            t0 = time.perf_counter()
        batch = seq_ops.StepBatch([1] * B, [cache.slot_of[b] for b in range(B)], [cache.length[b] for b in range(B)], self.device)
        batch.max_keys = max(cache.length.values()) + max_new_tokens        # of the last step: the loop runs on fixed buffers
        rows = list(range(B))
        out = greedy_decode(lambda: self.forward_rows(tok, batch, cache, rows), tok, batch.pos, max_new_tokens, use_graph, lib)
        for b in range(B):
            cache.advance(b, max_new_tokens - 1)
        if timings is not None:
            torch.cuda.synchronize()
            timings["decode_s"] = time.perf_counter() - t0
            timings["decode_steps"] = max_new_tokens - 1
        return out, cache
