"""What the decoders of mixed layers share: weights by name, per-sequence states, steps over any number of sequences, greedy
generation.

A model works in steps: a step brings the next tokens of any number of sequences, and everything earlier tokens left is in a
:class:`~msa_amd.cache.SequenceStateCache`.  Generation, and anything else that feeds tokens, goes through :meth:`StepDecoder.step`.
A model class adds how its layers follow one another: ``_block_rows`` for any rows of a step and ``_decode_rows`` for up to 16
sequences that bring one token each (bf16), where what stands between two products is folded into them as far as it can be.
"""
from __future__ import annotations

from typing import Dict, Hashable, List, Optional, Sequence, Tuple, Union

import torch
import torch.nn.functional as F

from . import _lib, seq_ops
from .cache import SequenceStateCache
from .generation import greedy_decode

Entry = Tuple[Hashable, Sequence[int], Sequence[int]]        # (sequence, its next tokens, places whose logits are wanted)
Shape = Tuple[Union[int, str], ...]                          # a named dimension is whatever the weight file has


class StepDecoder:
    """``layer_type(config, width, eps)`` builds a layer: ``shapes``, ``load``, ``state_specs``, ``decode_ok``, ``mixer``."""

    def __init__(self, config, layer_type):
        self.config = config
        self.layers = [layer_type(c, config.width, config.norm_eps) for c in config.layers]
        self.runs = config.runs
        # layers that read the cache of an earlier one: the run whose states they see
        self._source: Dict[int, int] = {}
        for r, (i, _) in enumerate(self.runs):
            j = getattr(self.layers[i].mixer, "kv_from", None)
            if j is not None:
                self._source[r] = max(q for q in range(r) if self.runs[q][0] == j)

    # ---------------------------------------------------------------------------------------- weights
    def _outer_shapes(self) -> Dict[str, Shape]:
        """Tensors outside the layers."""
        raise NotImplementedError

    def _load_outer(self, get) -> None:
        raise NotImplementedError

    def tensor_shapes(self) -> Dict[str, Shape]:
        """Names and shapes of every tensor the configuration asks for."""
        out = self._outer_shapes()
        for i, layer in enumerate(self.layers):
            out.update({f"l{i}.{n}": s for n, s in layer.shapes().items()})
        return out

    def _check_tensors(self, tensors: Dict[str, torch.Tensor]) -> None:
        named: Dict[Tuple[str, str], int] = {}
        for name, shape in self.tensor_shapes().items():
            if name not in tensors:
                raise KeyError(f"missing tensor {name!r}")
            got, layer = tuple(tensors[name].shape), name.split(".", 1)[0]
            want = tuple(named.setdefault((layer, d), got[i]) if isinstance(d, str) and i < len(got) else d for i, d in enumerate(shape))
            if got != want:
                raise ValueError(f"tensor {name!r} is {got}, the configuration asks for {want}")

    @classmethod
    def from_tensors(cls, config, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cuda:0"):
        """Packs ``tensors`` (names and shapes of :meth:`tensor_shapes`) for the device; matrices in ``dtype``, small vectors
        in fp32."""
        if dtype not in (torch.bfloat16, torch.float32):
            raise TypeError(f"unsupported dtype {dtype}: bfloat16 or float32")
        self = cls(config)
        self._check_tensors(tensors)
        self.dtype, self.device = dtype, torch.device(device)
        get = lambda n: tensors[n].to(self.device, dtype if tensors[n].dim() > 1 else torch.float32)
        self.embed, self.head = get("embed"), get("head").contiguous()
        self._load_outer(get)
        for i, layer in enumerate(self.layers):
            layer.load(lambda n, i=i: get(f"l{i}.{n}"))
        self.fused_decode = dtype == torch.bfloat16 and config.width % 8 == 0 and all(l.decode_ok() for l in self.layers)
        return self

    @classmethod
    def random(cls, config, seed: int = 0, dtype=torch.bfloat16, device="cuda:0"):
        """Random weights on the device (benchmarks): matrices scaled to keep activations of order one."""
        dev = torch.device(device)
        g = torch.Generator(device=dev).manual_seed(seed)
        tensors = {}
        self = cls(config)
        for name, shape in self.tensor_shapes().items():
            if any(isinstance(d, str) for d in shape):
                dims = self.layers[int(name[1:].split(".", 1)[0])].mixer.default_dims()
                shape = tuple(dims[d] if isinstance(d, str) else d for d in shape)
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

    def run_state(self, cache: SequenceStateCache, r: int) -> Dict[str, torch.Tensor]:
        """The states run ``r`` works on: its own, and those it reads from an earlier run."""
        return {**cache.tensors[self._source[r]], **cache.tensors[r]} if r in self._source else cache.tensors[r]

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
        cap = getattr(self.config, "logit_softcap", None) or 0.0
        if self.fused_decode and len(rows) <= seq_ops.MAX_ROWS:
            return seq_ops.rows_linear_f32(h, self.head, cap)
        logits = self._product_f32(h, self.head)
        return seq_ops.softcap(logits, cap) if cap else logits

    def _product_f32(self, x, w):
        """Vendor product with fp32 output."""
        return torch.mm(x, w.t(), out_dtype=torch.float32) if x.dtype == torch.bfloat16 else F.linear(x, w)

    def _embed(self, tokens):
        return self.embed[tokens].to(torch.float32)

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
