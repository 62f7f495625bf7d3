"""Torch-tensor front end of ``include/msa_seq.h`` (the layers of the decoders of mixed layers).  As in :mod:`msa_amd.ops`
PyTorch owns memory and names streams only; every function enqueues on the current stream and raises on any failure."""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass
from typing import Optional, Sequence

import torch

from . import _lib
from ._lib import dtype_code, ptr

MAX_ROWS = 16           # rows of a step that the weight-streaming kernels take
SSD_CHUNKED_ROWS = 64   # portions from this many tokens on are cut into chunks


def _check(code: int, where: str) -> None:
    _lib.check(code, where, _lib.load_seq())


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _cuda(*ts):
    for t in ts:
        if t is not None and not t.is_cuda:
            raise ValueError("expected a device tensor (the HIP path has no CPU fallback)")


def _dense(*ts):
    _cuda(*ts)
    for t in ts:
        if t is not None and not t.is_contiguous():
            raise ValueError("expected a contiguous tensor")


def _rows(t: torch.Tensor) -> int:
    """Row stride of a 2-D tensor (possibly a column range of a wider one)."""
    _cuda(t)
    if t.dim() != 2 or (t.shape[1] > 1 and t.stride(1) != 1):
        raise ValueError("expected rows with unit column stride")
    return t.stride(0) if t.shape[0] > 1 else max(t.stride(0), t.shape[1])


def _f32(n: int, *ts):
    for t in ts:
        if t is not None and (t.dtype != torch.float32 or t.numel() != n or not t.is_contiguous() or not t.is_cuda):
            raise ValueError(f"expected {n} contiguous fp32 values on the device, got {t.dtype} {tuple(t.shape)}")


class StepBatch:
    """Device-side description of a step's rows (``msa_seq_batch``): ``counts[s]`` new tokens of the sequence in
    ``slots[s]`` that has already been fed ``positions[s]`` tokens."""

    def __init__(self, counts: Sequence[int], slots: Sequence[int], positions: Sequence[int], device):
        n = len(counts)
        if not n or min(counts) < 1 or len(set(slots)) != n:
            raise ValueError("a step needs at least one token per sequence and one slot each")
        self.counts, self.slots, self.positions = list(counts), list(slots), list(positions)
        self.rows, self.max_rows, self.n_seq = sum(counts), max(counts), n
        host = [0]
        for c in counts:
            host.append(host[-1] + c)
        cu = list(host)
        ints = torch.tensor(cu + list(slots), dtype=torch.int32).to(device)
        self.cu, self.slot = ints[:n + 1], ints[n + 1:]
        self.pos = torch.tensor(list(positions), dtype=torch.int64).to(device)
        self.row_seq = (torch.zeros(self.rows, dtype=torch.int32, device=device) if n == 1 else
                        torch.repeat_interleave(torch.arange(n, dtype=torch.int32), torch.tensor(self.counts)).to(device))
        self.c = _lib.SeqBatch(ptr(self.cu), ptr(self.row_seq), ptr(self.slot), ptr(self.pos), n, self.rows, self.max_rows, 0)
        self.ref = C.byref(self.c)
        self.max_keys = max(p + c for p, c in zip(positions, counts))     # longest sequence at the end of the step
        self._row_at = {}

    def cache_rows(self, capacity: int) -> torch.Tensor:
        """First row of every sequence in a cache of ``capacity`` rows a slot (int64, on the device)."""
        if capacity not in self._row_at:
            self._row_at[capacity] = self.slot.to(torch.int64) * capacity
        return self._row_at[capacity]


@dataclass
class DynTanhNorm:
    """``tanh(alpha x) w + b``."""
    w: torch.Tensor
    b: torch.Tensor
    alpha: float

    def __post_init__(self):
        self.c = _lib.DynTanh(ptr(self.w), ptr(self.b), self.alpha, 0)


_NO_NORM = _lib.DynTanh(None, None, 0.0, 0)
_scratch = {}


def _workspace(device, need: int) -> torch.Tensor:
    ws = _scratch.get(device)
    if ws is None or ws.numel() < need:
        ws = _scratch[device] = torch.empty(max(need, 1), dtype=torch.uint8, device=device)
    return ws


def residual_norm(x: torch.Tensor, batch: StepBatch, dtype: torch.dtype, y=None, gate=None, gate_bias=None,
                  norm: Optional[DynTanhNorm] = None, shift=None, prev=None, want_h: bool = True):
    """``(x', h, h_shift)``: ``x' = x + sigmoid(gate + gate_bias) * y`` (``x`` itself without ``y``), ``h = norm(x')``
    and the token-shifted ``h`` (``prev [slots, W]`` holds every sequence's last ``h`` and is updated)."""
    _dense(x, prev)
    T, W = x.shape
    if x.dtype != torch.float32 or T != batch.rows:
        raise ValueError("the residual stream is fp32 [rows, W]")
    if norm is not None:
        _f32(W, norm.w, norm.b)
    if y is not None:
        _f32(W, gate_bias)
        if y.shape != x.shape or gate.shape != x.shape or y.dtype != dtype or gate.dtype != dtype:
            raise ValueError("sublayer output and gate must be [rows, W] of the activations' type")
    if shift is not None:
        _f32(W, shift)
        if prev.dtype != torch.float32 or prev.shape[1] != W or prev.shape[0] <= max(batch.slots):
            raise ValueError("prev must be fp32 [slots, W]")
    x_out = torch.empty_like(x) if y is not None else None
    h = torch.empty((T, W), dtype=dtype, device=x.device) if norm is not None and want_h else None
    hs = torch.empty((T, W), dtype=dtype, device=x.device) if shift is not None else None
    _check(_lib.load_seq().msa_seq_residual_norm(
        ptr(x), ptr(y), _rows(y) if y is not None else 0, ptr(gate), _rows(gate) if gate is not None else 0, ptr(gate_bias),
        ptr(x_out), dtype_code(dtype), W, C.byref(norm.c if norm is not None else _NO_NORM), ptr(h), ptr(shift), ptr(prev),
        ptr(hs), batch.ref, _stream()), "msa_seq_residual_norm")
    return (x if y is None else x_out), h, hs


def rms_residual(x: torch.Tensor, dtype: torch.dtype, y=None, w=None, eps: float = 0.0, next_w=None, out=None, want_h: bool = True):
    """``(x', h)``: ``x' = x + rms_norm(y) * w`` (``x`` itself without ``y``; into ``out``, which may be ``x``), and ``h = x'``, or
    ``rms_norm(x') * next_w``, in ``dtype``."""
    _dense(x, out)
    T, W = x.shape
    if x.dtype != torch.float32 or (out is not None and (out.shape != x.shape or out.dtype != torch.float32)):
        raise ValueError("the residual stream is fp32 [rows, W]")
    if y is not None:
        _f32(W, w)
        if y.shape != x.shape or y.dtype != dtype:
            raise ValueError("sublayer output must be [rows, W] of the activations' type")
        out = torch.empty_like(x) if out is None else out
    _f32(W, next_w)
    h = torch.empty((T, W), dtype=dtype, device=x.device) if want_h or next_w is not None else None
    _check(_lib.load_seq().msa_seq_rms_residual(ptr(x), ptr(y), _rows(y) if y is not None else 0, ptr(w), eps, ptr(out), ptr(next_w), ptr(h),
                                                dtype_code(dtype), T, W, _stream()), "msa_seq_rms_residual")
    return (x if y is None else out), h


GLU_ALPHA, GLU_SHIFT = 1.702, 1.0


def interleave_pairs(gate_w: torch.Tensor, up_w: torch.Tensor) -> torch.Tensor:
    """Weight rows in (gate, up) pairs."""
    return torch.stack([gate_w, up_w], dim=1).reshape(2 * gate_w.shape[0], gate_w.shape[1]).contiguous()


def clamped_glu(gu: torch.Tensor, limit: float, alpha: float = GLU_ALPHA, shift: float = GLU_SHIFT) -> torch.Tensor:
    """``g sigmoid(alpha g) (u + shift)`` of rows of (gate, up) pairs, the gate capped at ``limit``, up clamped to ``+-limit``."""
    T, n = gu.shape[0], gu.shape[1] // 2
    out = torch.empty((T, n), dtype=gu.dtype, device=gu.device)
    _check(_lib.load_seq().msa_seq_clamped_glu(ptr(gu), _rows(gu), dtype_code(gu.dtype), T, n, limit, alpha, shift, ptr(out), _stream()),
           "msa_seq_clamped_glu")
    return out


def gelu_(y: torch.Tensor) -> torch.Tensor:
    """tanh-form gelu in place on a ``[rows, n]`` column range."""
    _check(_lib.load_seq().msa_seq_gelu(ptr(y), _rows(y), dtype_code(y.dtype), y.shape[0], y.shape[1], _stream()), "msa_seq_gelu")
    return y


def softcap(x: torch.Tensor, cap: float) -> torch.Tensor:
    """fp32 ``cap * tanh(x / cap)`` (a plain copy for ``cap`` 0)."""
    _dense(x)
    out = torch.empty(x.shape, dtype=torch.float32, device=x.device)
    _check(_lib.load_seq().msa_seq_softcap(ptr(x), dtype_code(x.dtype), x.numel(), float(cap), ptr(out), _stream()), "msa_seq_softcap")
    return out


def join(x: torch.Tensor, x0: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """Operand of a projection of ``[x ; x0]`` (fp32 streams): ``[hi(x) | lo(x) | x0]`` in bf16, ``[x | x0]`` in fp32."""
    _dense(x, x0)
    T, W = x.shape
    if x.shape != x0.shape or x.dtype != torch.float32 or x0.dtype != torch.float32:
        raise ValueError("x and x0 must be fp32 and of one shape")
    out = torch.empty((T, W * (3 if dtype == torch.bfloat16 else 2)), dtype=dtype, device=x.device)
    _check(_lib.load_seq().msa_seq_join(ptr(x), ptr(x0), dtype_code(dtype), T, W, ptr(out), _stream()), "msa_seq_join")
    return out


def conv_silu(x: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor], state: torch.Tensor, batch: StepBatch) -> torch.Tensor:
    """Causal per-channel convolution + silu of ``x [rows, C]``; ``state [slots, K - 1, C]`` is updated."""
    T, Cn = x.shape
    K = taps.shape[1]
    _f32(Cn * K, taps)
    _f32(Cn, bias)
    _dense(state)
    if state.dtype != torch.float32 or tuple(state.shape[1:]) != (K - 1, Cn) or state.shape[0] <= max(batch.slots):
        raise ValueError("state must be fp32 [slots, K - 1, C]")
    out = torch.empty((T, Cn), dtype=x.dtype, device=x.device)
    _check(_lib.load_seq().msa_seq_conv_silu(ptr(x), _rows(x), ptr(taps), ptr(bias), dtype_code(x.dtype), Cn, K, ptr(state), ptr(out),
                                             Cn, batch.ref, _stream()), "msa_seq_conv_silu")
    return out


def ssd(xbc, z, dt_raw, dt_bias, A_log, D, H: int, P: int, N: int, G: int, state, batch: StepBatch, chunked: bool = False):
    """Gated output ``[rows, H P]`` of the state-space recurrence; ``state [slots, H, N, P]`` fp32 is updated.  ``chunked``
    takes the matrix-core form (bf16)."""
    _f32(H, dt_bias, A_log, D)
    _dense(state)
    T = batch.rows
    if state.dtype != torch.float32 or tuple(state.shape[1:]) != (H, N, P) or state.shape[0] <= max(batch.slots):
        raise ValueError("state must be fp32 [slots, H, N, P]")
    if xbc.shape != (T, H * P + 2 * G * N) or z.shape != (T, H * P) or dt_raw.shape != (T, H) or not (xbc.dtype == z.dtype == dt_raw.dtype):
        raise ValueError("xbc [rows, H P + 2 G N], z [rows, H P] and dt [rows, H] of one type")
    v = torch.empty((T, H * P), dtype=xbc.dtype, device=xbc.device)
    lib = _lib.load_seq()
    args = [ptr(xbc), _rows(xbc), ptr(z), _rows(z), ptr(dt_raw), _rows(dt_raw), ptr(dt_bias), ptr(A_log), ptr(D),
            dtype_code(xbc.dtype), H, P, N, G, ptr(state), ptr(v), batch.ref]
    if chunked:
        ws = _workspace(xbc.device, lib.msa_seq_ssd_chunked_workspace_bytes(batch.max_rows, batch.n_seq, H, P, N))
        _check(lib.msa_seq_ssd_chunked(*args, ptr(ws), ws.numel(), _stream()), "msa_seq_ssd_chunked")
    else:
        _check(lib.msa_seq_ssd_scan(*args, _stream()), "msa_seq_ssd_scan")
    return v


def group_rmsnorm(v: torch.Tensor, w: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    """RMS norm of ``v [rows, n]`` in ``parts`` equal parts, times ``w``."""
    _dense(v)
    T, n = v.shape
    _f32(n, w)
    out = torch.empty_like(v)
    _check(_lib.load_seq().msa_seq_group_rmsnorm(ptr(v), dtype_code(v.dtype), T, n, parts, ptr(w), eps, ptr(out), _stream()),
           "msa_seq_group_rmsnorm")
    return out


DELTA_CHUNKED_ROWS = 64    # portions from this many tokens on are cut into chunks


def delta_chunked_ok(dtype, D: int, E: int) -> bool:
    return dtype == torch.bfloat16 and D % 8 == 0 and E % 8 == 0 and D <= 128


def delta(qkv, a, b, gate, A_log, dt_bias, norm, eps: float, H: int, G: int, D: int, E: int, state, batch: StepBatch,
          chunked: bool = False) -> torch.Tensor:
    """Normed and gated read-outs ``[rows, H E]`` of the delta rule with a decay per key channel; ``qkv [rows, 2 G D + H E]``,
    ``a [rows, H D]``, ``b [rows, H]``, ``gate [rows, H E]``; ``state [slots, H, D, E]`` fp32 is updated.  ``chunked`` takes the
    matrix-core form (bf16)."""
    T = batch.rows
    _f32(H, A_log)
    _f32(H * D, dt_bias)
    _f32(E, norm)
    _dense(state)
    if state.dtype != torch.float32 or tuple(state.shape[1:]) != (H, D, E) or state.shape[0] <= max(batch.slots):
        raise ValueError("state must be fp32 [slots, H, D, E]")
    if qkv.shape != (T, 2 * G * D + H * E) or a.shape != (T, H * D) or b.shape != (T, H) or gate.shape != (T, H * E) or \
            not (qkv.dtype == a.dtype == b.dtype == gate.dtype):
        raise ValueError("qkv [rows, 2 G D + H E], a [rows, H D], b [rows, H] and gate [rows, H E] of one type")
    out = torch.empty((T, H * E), dtype=qkv.dtype, device=qkv.device)
    c = _lib.DeltaArgs(ptr(qkv), ptr(a), ptr(b), ptr(gate), _rows(qkv), _rows(a), _rows(b), _rows(gate), ptr(A_log), ptr(dt_bias), ptr(norm),
                       ptr(state), ptr(out), H, G, D, E, eps, 0)
    lib = _lib.load_seq()
    if chunked:
        ws = _workspace(qkv.device, lib.msa_seq_delta_chunked_workspace_bytes(C.byref(c), batch.max_rows, batch.n_seq))
        _check(lib.msa_seq_delta_chunked(C.byref(c), batch.ref, ptr(ws), ws.numel(), _stream()), "msa_seq_delta_chunked")
    else:
        _check(lib.msa_seq_delta_scan(C.byref(c), dtype_code(qkv.dtype), batch.ref, _stream()), "msa_seq_delta_scan")
    return out


GRU_GROUP = 16


def interleave_gru(z_w: torch.Tensor, u_w: torch.Tensor, g_w: torch.Tensor) -> torch.Tensor:
    """Weight rows in groups of 48 ``[16 z | 16 u | 16 g]`` of the same 16 channels, zero rows behind the last channel."""
    n, K = z_w.shape
    pad = -n % GRU_GROUP
    parts = [torch.cat([w, w.new_zeros(pad, K)]).view(-1, GRU_GROUP, K) for w in (z_w, u_w, g_w)]
    return torch.stack(parts, dim=1).reshape(3 * (n + pad), K).contiguous()


def min_gru(zug: torch.Tensor, z_bias, u_bias, n: int, state, batch: StepBatch) -> torch.Tensor:
    """``S * silu(g)`` of the minimal gated recurrence; ``zug`` rows in the layout of :func:`interleave_gru`,
    ``state [slots, n]`` fp32 is updated."""
    _f32(n, z_bias, u_bias)
    _dense(state)
    if state.dtype != torch.float32 or state.dim() != 2 or state.shape[1] != n or state.shape[0] <= max(batch.slots):
        raise ValueError("state must be fp32 [slots, n]")
    if zug.shape != (batch.rows, (n + GRU_GROUP - 1) // GRU_GROUP * 3 * GRU_GROUP):
        raise ValueError("zug must hold 48 columns per 16 channels")
    out = torch.empty((batch.rows, n), dtype=zug.dtype, device=zug.device)
    lib = _lib.load_seq()
    need = lib.msa_seq_min_gru_workspace_bytes(batch.rows, batch.n_seq, batch.max_rows, n)
    ws = _workspace(zug.device, need) if need else None
    _check(lib.msa_seq_min_gru(ptr(zug), _rows(zug), ptr(z_bias), ptr(u_bias), dtype_code(zug.dtype), n, ptr(state), ptr(out),
                               batch.ref, ptr(ws), ws.numel() if ws is not None else 0, _stream()), "msa_seq_min_gru")
    return out


def _latent_cache(cache: torch.Tensor, rank: int, dtype, batch: StepBatch) -> int:
    _dense(cache)
    if cache.dim() != 3 or cache.shape[2] != rank or cache.dtype != dtype or cache.shape[0] <= max(batch.slots):
        raise ValueError("the latent cache must be [slots, capacity, rank] of the activations' type")
    return cache.shape[1]


def latent_append(x: torch.Tensor, w: torch.Tensor, eps: float, cache: torch.Tensor, batch: StepBatch) -> None:
    """RMS-normed rows of ``x [rows, rank]`` go to the latent cache at their positions."""
    rank = x.shape[1]
    _f32(rank, w)
    Lcap = _latent_cache(cache, rank, x.dtype, batch)
    if batch.max_keys > Lcap:
        raise ValueError(f"latent cache of {Lcap} rows cannot take {batch.max_keys} tokens")
    _check(_lib.load_seq().msa_seq_latent_append(ptr(x), _rows(x), ptr(w), eps, dtype_code(x.dtype), rank, ptr(cache), Lcap, batch.ref,
                                                 _stream()), "msa_seq_latent_append")


def latent_attn(q: torch.Tensor, cache: torch.Tensor, sink: torch.Tensor, scale: float, batch: StepBatch,
                max_keys: Optional[int] = None) -> torch.Tensor:
    """Causal attention of ``q [rows, H, rank]`` over the cached latents, with the sinks in the denominators.  bf16 rows of
    at most 512 (a multiple of 8) dimensions take the split matrix-core kernel; ``max_keys`` bounds the keys of any row."""
    _dense(q)
    T, H, rank = q.shape
    _f32(H, sink)
    Lcap = _latent_cache(cache, rank, q.dtype, batch)
    if T != batch.rows:
        raise ValueError("one query row per row of the step")
    ctx = torch.empty_like(q)
    lib = _lib.load_seq()
    if q.dtype == torch.bfloat16 and rank % 8 == 0 and rank <= 512 and T <= 65535:
        keys = batch.max_keys if max_keys is None else max_keys
        ws = _workspace(q.device, lib.msa_seq_latent_decode_workspace_bytes(T, H, rank, keys))
        _check(lib.msa_seq_latent_decode(ptr(q), ptr(cache), Lcap, ptr(sink), scale, dtype_code(q.dtype), H, rank, keys, ptr(ctx),
                                         batch.ref, ptr(ws), ws.numel(), _stream()), "msa_seq_latent_decode")
    else:
        _check(lib.msa_seq_latent_attn(ptr(q), ptr(cache), Lcap, ptr(sink), scale, dtype_code(q.dtype), H, rank, ptr(ctx), batch.ref,
                                       _stream()), "msa_seq_latent_attn")
    return ctx


def flash_ok(dtype, D: int, E: int, scale: float) -> bool:
    return dtype == torch.bfloat16 and D % 8 == 0 and E % 8 == 0 and max(D, E) <= 256 and scale > 0


def flash(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, kv_off: torch.Tensor, sink: Optional[torch.Tensor], scale: float, H: int,
          batch: StepBatch, kv_heads: Optional[int] = None, chunk: int = 0, gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Causal attention of ``q [rows, H D]`` over ``k [keys, G D]``, ``v [keys, G E]`` (``G = kv_heads``, H without); sequence ``s``
    owns the rows from ``kv_off[s]`` on.  ``chunk``: a position sees its own stretch of that many positions only; ``gate [rows, H]``:
    head outputs times its sigmoid."""
    G = H if kv_heads is None else kv_heads
    _f32(H, sink)
    D, E = q.shape[1] // H, v.shape[1] // G
    if k.shape[1] != G * D or k.shape[0] != v.shape[0] or k.shape[0] < sum(p + c for p, c in zip(batch.positions, batch.counts)):
        raise ValueError("k and v must hold every sequence's keys")
    if kv_off.dtype != torch.int64 or kv_off.numel() != batch.n_seq:
        raise ValueError("kv_off must be int64, one entry per sequence")
    if gate is not None and (gate.shape != (batch.rows, H) or gate.dtype != q.dtype):
        raise ValueError("gate must be [rows, H] of the activations' type")
    out = torch.empty((batch.rows, H * E), dtype=q.dtype, device=q.device)
    _check(_lib.load_seq().msa_seq_flash(ptr(q), _rows(q), ptr(k), _rows(k), ptr(v), _rows(v), ptr(kv_off), ptr(sink), scale,
                                         dtype_code(q.dtype), H, G, D, E, chunk, ptr(gate), _rows(gate) if gate is not None else 0, ptr(out),
                                         batch.ref, _stream()), "msa_seq_flash")
    return out


def _kv_caches(k_cache, v_cache, dtype, batch: StepBatch):
    """``(capacity, G, D, E)`` of ``k_cache [slots, capacity, G, D]`` and ``v_cache [slots, capacity, G, E]``."""
    _dense(k_cache, v_cache)
    if k_cache.dim() != 4 or v_cache.dim() != 4 or k_cache.shape[:3] != v_cache.shape[:3] or not (k_cache.dtype == v_cache.dtype == dtype) \
            or k_cache.shape[0] <= max(batch.slots):
        raise ValueError("the caches must be [slots, capacity, G, D] and [slots, capacity, G, E] of the activations' type")
    if batch.max_keys > k_cache.shape[1]:
        raise ValueError(f"a cache of {k_cache.shape[1]} rows does not hold {batch.max_keys} tokens")
    return k_cache.shape[1], k_cache.shape[2], k_cache.shape[3], v_cache.shape[3]


def qk_rope_append(q, q_norm, freqs, eps: float, k_cache, v_cache, batch: StepBatch, k=None, v=None, k_norm=None) -> torch.Tensor:
    """Normed and rotated queries ``[rows, H, D]`` of ``q [rows, H D]``; with ``k [rows, G D]`` and ``v [rows, G E]`` the normed and
    rotated keys and the values go to the caches at their positions.  ``freqs`` (fp64): radians per position of each pair."""
    Lcap, G, D, E = _kv_caches(k_cache, v_cache, q.dtype, batch)
    H = q.shape[1] // D
    _f32(D, q_norm)
    if q.shape != (batch.rows, H * D) or freqs.dtype != torch.float64 or not freqs.is_cuda or 2 * freqs.numel() > D:
        raise ValueError("q must be [rows, H D], freqs fp64 on the device")
    if k is not None:
        _f32(D, k_norm)
        if k.shape != (batch.rows, G * D) or v.shape != (batch.rows, G * E) or not (k.dtype == v.dtype == q.dtype):
            raise ValueError("k must be [rows, G D] and v [rows, G E] of the queries' type")
    out = torch.empty((batch.rows, H, D), dtype=q.dtype, device=q.device)
    c = _lib.QKRopeArgs(ptr(q), ptr(k), ptr(v), _rows(q), _rows(k) if k is not None else 0, _rows(v) if k is not None else 0, ptr(q_norm),
                        ptr(k_norm), ptr(freqs), ptr(out), ptr(k_cache), ptr(v_cache), Lcap, H, G, D, E, freqs.numel(), eps)
    _check(_lib.load_seq().msa_seq_qk_rope_append(C.byref(c), dtype_code(q.dtype), batch.ref, _stream()), "msa_seq_qk_rope_append")
    return out


def kv_attn(q: torch.Tensor, k_cache, v_cache, scale: float, batch: StepBatch, chunk: int = 0, gate: Optional[torch.Tensor] = None,
            split: Optional[bool] = None) -> torch.Tensor:
    """Causal attention ``[rows, H E]`` of prepared queries ``q [rows, H, D]`` over the caches, a few rows a sequence, with the chunk
    mask and the gate of :func:`flash`.  bf16 of aligned sizes takes the split matrix-core kernel (``split`` chooses by hand)."""
    _dense(q)
    Lcap, G, D, E = _kv_caches(k_cache, v_cache, q.dtype, batch)
    T, H = q.shape[:2]
    if T != batch.rows or q.shape[2] != D or H % G:
        raise ValueError("one query row [H, D] per row of the step")
    if gate is not None and (gate.shape != (T, H) or gate.dtype != q.dtype):
        raise ValueError("gate must be [rows, H] of the activations' type")
    out = torch.empty((T, H * E), dtype=q.dtype, device=q.device)
    c = _lib.KVAttnArgs(ptr(q), ptr(k_cache), ptr(v_cache), ptr(gate), ptr(out), Lcap, _rows(gate) if gate is not None else 0, batch.max_keys,
                        H, G, D, E, chunk, scale)
    lib = _lib.load_seq()
    if split is None:
        split = flash_ok(q.dtype, D, E, scale) and T <= 65535
    if split:
        need = lib.msa_seq_kv_decode_workspace_bytes(C.byref(c), T)
        ws = _workspace(q.device, need) if need else None
        _check(lib.msa_seq_kv_decode(C.byref(c), batch.ref, ptr(ws), ws.numel() if need else 0, _stream()), "msa_seq_kv_decode")
    else:
        _check(lib.msa_seq_kv_attn(C.byref(c), dtype_code(q.dtype), batch.ref, _stream()), "msa_seq_kv_attn")
    return out


def _rows_args(x, w, groups: int = 1, x_b=None, n_b: Optional[int] = None) -> _lib.RowsArgs:
    M = x.shape[0]
    K = w.shape[1]
    N = w.shape[0] // groups
    _dense(w)
    if w.dtype != torch.bfloat16 or x.dtype != torch.bfloat16 or x.shape[1] != K * groups or N * groups != w.shape[0]:
        raise ValueError("rows_linear: bf16 x [M, groups K] and w [groups N, K]")
    if x_b is not None and (x_b.shape != (M, K) or x_b.dtype != torch.bfloat16):
        raise ValueError("rows_linear: the second operand must be bf16 [M, K]")
    a = _lib.RowsArgs()
    a.x, a.w, a.x_stride, a.M, a.N, a.K, a.groups = ptr(x), ptr(w), _rows(x), M, N, K, groups
    a.n_b = N if n_b is None else n_b
    if x_b is not None:
        a.x_b, a.x_b_stride = ptr(x_b), _rows(x_b)
    return a


def _run_rows(a: _lib.RowsArgs, epilogue: int) -> None:
    _check(_lib.load_seq().msa_rows_linear(C.byref(a), epilogue, _stream()), "msa_rows_linear")


def rows_linear(x, w, groups: int = 1, x_b=None, n_b: Optional[int] = None, gelu_n: int = 0) -> torch.Tensor:
    """bf16 ``[M, groups N]`` products of up to 16 rows; weight rows from ``n_b`` on multiply ``x_b``; the first ``gelu_n``
    columns leave through gelu."""
    a = _rows_args(x, w, groups, x_b, n_b)
    out = torch.empty((x.shape[0], w.shape[0]), dtype=torch.bfloat16, device=x.device)
    a.out, a.out_stride, a.gelu_n = ptr(out), out.shape[1], gelu_n
    _run_rows(a, _lib.ROWS_PLAIN)
    return out


def rows_linear_f32(x, w, cap: float = 0.0, add: Optional[torch.Tensor] = None) -> torch.Tensor:
    """fp32 products of up to 16 rows, softcapped, plus ``add [N]``."""
    a = _rows_args(x, w)
    out = torch.empty((x.shape[0], w.shape[0]), dtype=torch.float32, device=x.device)
    if add is not None:
        _f32(w.shape[0], add)
    a.out, a.out_stride, a.cap, a.add = ptr(out), out.shape[1], cap, ptr(add)
    _run_rows(a, _lib.ROWS_F32)
    return out


def rows_glu(x, w, limit: float, alpha: float = GLU_ALPHA, shift: float = GLU_SHIFT) -> torch.Tensor:
    """:func:`clamped_glu` of up to 16 rows' products with weights in the layout of :func:`interleave_pairs`."""
    a = _rows_args(x, w)
    out = torch.empty((x.shape[0], w.shape[0] // 2), dtype=torch.bfloat16, device=x.device)
    a.out, a.out_stride, a.glu_limit, a.glu_alpha, a.glu_shift = ptr(out), out.shape[1], limit, alpha, shift
    _run_rows(a, _lib.ROWS_GLU)
    return out


def rows_residual(x, w, stream: torch.Tensor, gate, gate_bias, slot, norm: Optional[DynTanhNorm] = None, shift=None, prev=None,
                  want_h: bool = True):
    """The output projection of a sublayer for up to 16 sequences' single rows, with :func:`residual_norm` behind it: the fp32
    stream is updated in place, ``(h, h_shift)`` returned."""
    a = _rows_args(x, w)
    M, N = x.shape[0], w.shape[0]
    _dense(stream, prev)
    _f32(N, gate_bias, shift)
    if stream.dtype != torch.float32 or stream.shape != (M, N) or gate.shape != (M, N) or gate.dtype != torch.bfloat16:
        raise ValueError("rows_residual: fp32 stream [M, N], bf16 gate [M, N]")
    if slot.dtype != torch.int32 or slot.numel() != M:
        raise ValueError("rows_residual: one int32 slot per row")
    a.x_in = a.x_out = ptr(stream)
    a.gate, a.gate_stride, a.gate_bias, a.slot = ptr(gate), _rows(gate), ptr(gate_bias), ptr(slot)
    h = hs = None
    if norm is not None:
        _f32(N, norm.w, norm.b)
        a.norm = norm.c
        if want_h:
            h = torch.empty((M, N), dtype=torch.bfloat16, device=x.device)
    if shift is not None:
        if prev.dtype != torch.float32 or prev.shape[1] != N:
            raise ValueError("prev must be fp32 [slots, N]")
        hs = torch.empty((M, N), dtype=torch.bfloat16, device=x.device)
    a.h, a.shift, a.prev, a.h_shift = ptr(h), ptr(shift), ptr(prev), ptr(hs)
    _run_rows(a, _lib.ROWS_RESIDUAL)
    return h, hs


def rows_conv(x, w, x_b, n_b: Optional[int], conv_lo: int, taps, bias, state, slot) -> torch.Tensor:
    """Input projection of a layer with a convolution for up to 16 sequences' single rows: columns ``conv_lo ..`` leave through the
    causal convolution + silu, whose ``state [slots, K - 1, C]`` is updated."""
    a = _rows_args(x, w, 1, x_b, n_b)
    Cn, K = taps.shape
    _f32(Cn * K, taps)
    _f32(Cn, bias)
    _dense(state)
    if state.dtype != torch.float32 or tuple(state.shape[1:]) != (K - 1, Cn) or slot.dtype != torch.int32 or slot.numel() != x.shape[0]:
        raise ValueError("state must be fp32 [slots, K - 1, C] and slot int32, one per row")
    out = torch.empty((x.shape[0], w.shape[0]), dtype=torch.bfloat16, device=x.device)
    a.out, a.out_stride, a.taps, a.conv_bias, a.conv_state = ptr(out), out.shape[1], ptr(taps), ptr(bias), ptr(state)
    a.conv_lo, a.conv_n, a.conv_k, a.slot = conv_lo, Cn, K, ptr(slot)
    _run_rows(a, _lib.ROWS_MAMBA)
    return out


def rows_gru(x, w, x_b, n: int, z_bias, u_bias, state, slot):
    """Input projection and recurrence of the minimal gated layer for up to 16 sequences' single rows (weights in the layout of
    :func:`interleave_gru`, then the rows that multiply ``x_b``): ``(S * silu(g) [M, n], all columns [M, N])``, of which only the
    ``x_b`` columns are written."""
    n_b = (n + GRU_GROUP - 1) // GRU_GROUP * 3 * GRU_GROUP
    a = _rows_args(x, w, 1, x_b, n_b)
    _f32(n, z_bias, u_bias)
    _dense(state)
    if state.dtype != torch.float32 or state.shape[1] != n or slot.dtype != torch.int32 or slot.numel() != x.shape[0]:
        raise ValueError("state must be fp32 [slots, n] and slot int32, one per row")
    M = x.shape[0]
    out = torch.empty((M, w.shape[0]), dtype=torch.bfloat16, device=x.device)
    act = torch.empty((M, n), dtype=torch.bfloat16, device=x.device)
    a.out, a.out_stride, a.out2, a.gru_n = ptr(out), out.shape[1], ptr(act), n
    a.z_bias, a.u_bias, a.gru_state, a.slot = ptr(z_bias), ptr(u_bias), ptr(state), ptr(slot)
    _run_rows(a, _lib.ROWS_GRU)
    return act, out


def greedy_tokens(logits: torch.Tensor) -> torch.Tensor:
    """int64 ``[B]`` argmax of ``[B, V]`` logits."""
    from . import ops
    return ops.greedy_sample(logits, torch.empty(logits.shape[0], dtype=torch.int64, device=logits.device), lib=_lib.load_seq())
