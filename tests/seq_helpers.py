"""Shared by the GPU tests of the sequence-layer kernels: random operands with their exact float64 copies, comparison, batches."""
import torch

from msa_amd import seq_ops

F64, F32, BF16 = torch.float64, torch.float32, torch.bfloat16


class Rand:
    def __init__(self, seed=0):
        self.g = torch.Generator().manual_seed(seed)

    def __call__(self, *shape, dtype=F32, scale=1.0, add=0.0):
        """Device values and their exact float64 copy."""
        t = (torch.randn(shape, generator=self.g) * scale + add).to(dtype)
        return t.cuda(), t.to(F64)


def close(got, want, dtype, tol=None):
    want = want.cpu().to(F64)
    err = (got.cpu().to(F64) - want).abs().max().item()
    lim = (2e-5 if dtype == F32 else 1.2e-2) if tol is None else tol
    size = max(want.abs().max().item(), 1e-3)
    assert err <= lim * size, f"error {err:.3e} at size {size:.3e}"


def portions(n, sizes):
    out, i = [], 0
    while n:
        k = min(n, sizes[i % len(sizes)])
        out.append(k)
        n, i = n - k, i + 1
    return out


def batch(counts, slots=None, pos=None):
    return seq_ops.StepBatch(counts, list(range(len(counts))) if slots is None else slots, [0] * len(counts) if pos is None else pos, "cuda")
