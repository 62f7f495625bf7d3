"""The greedy decode loop the models share: argmax + token bookkeeping on the device, one step captured as a HIP graph."""
from __future__ import annotations

from typing import Callable, Optional

import torch

from . import ops


def greedy_decode(step_logits: Callable[[], torch.Tensor], tok: torch.Tensor, pos: torch.Tensor, max_new_tokens: int,
                  use_graph: bool = False, lib=None) -> torch.Tensor:
    """``tok`` (the first new token of each of B sequences) and ``pos`` are fixed int64 device buffers of B elements that
    ``step_logits()`` reads; it enqueues one decode step on fixed buffers and returns logits with ``B`` rows.  After each
    step the argmax goes to ``tok`` and into the returned ``[B, max_new_tokens]``, and ``pos`` advances by one.  With
    ``use_graph`` one step is captured as a HIP graph after two eager ones and replayed for the rest."""
    B, dev = tok.numel(), tok.device
    out = torch.zeros((B, max_new_tokens), dtype=torch.int64, device=dev)
    out[:, :1] = tok.view(B, 1)
    col = torch.ones((B, 1), dtype=torch.int64, device=dev)
    n_steps = max_new_tokens - 1
    native = dev.type == "cuda" and tok.is_contiguous() and pos.is_contiguous() and pos.dtype == torch.int64 and pos.numel() == B
    scratch = torch.empty(B * 32, dtype=torch.int64, device=dev) if native else None

    def step():
        # everything is in-place on fixed buffers so the same launches can be replayed as a graph
        logits = step_logits().view(B, -1)
        if native:                             # argmax + token bookkeeping in two small launches
            ops.greedy_sample(logits, tok, pos, out, col, scratch, lib=lib)
            return
        new_tok = logits.argmax(-1, keepdim=True)
        tok.copy_(new_tok.view_as(tok))
        pos.add_(1)
        out.scatter_(1, col, new_tok)
        col.add_(1)

    done = 0
    if use_graph and n_steps > 3:
        for _ in range(2):                     # warm-up: workspaces and library handles exist before capture
            step()
            done += 1
        torch.cuda.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):          # records the launches without running them
            step()
        while done < n_steps:
            graph.replay()
            done += 1
    else:
        while done < n_steps:
            step()
            done += 1
    return out
