"""Torch-tensor front end of ``include/msa_seq.h`` (recurrent and latent-attention layers).  As in :mod:`msa_amd.ops`
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


def conv_silu(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor, state: torch.Tensor, batch: StepBatch) -> torch.Tensor:
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


def flash(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, kv_off: torch.Tensor, sink: torch.Tensor, scale: float, H: int,
          batch: StepBatch) -> torch.Tensor:
    """Causal attention of ``q [rows, H D]`` over expanded ``k [keys, H D]``, ``v [keys, H E]``; sequence ``s`` owns the rows
    from ``kv_off[s]`` on."""
    _f32(H, sink)
    D, E = q.shape[1] // H, v.shape[1] // H
    if k.shape[1] != H * D or k.shape[0] != v.shape[0] or k.shape[0] < sum(p + c for p, c in zip(batch.positions, batch.counts)):
        raise ValueError("k and v must hold every sequence's keys")
    if kv_off.dtype != torch.int64 or kv_off.numel() != batch.n_seq:
        raise ValueError("kv_off must be int64, one entry per sequence")
    out = torch.empty((batch.rows, H * E), dtype=q.dtype, device=q.device)
    _check(_lib.load_seq().msa_seq_flash(ptr(q), _rows(q), ptr(k), _rows(k), ptr(v), _rows(v), ptr(kv_off), ptr(sink), scale,
                                         dtype_code(q.dtype), H, D, E, ptr(out), batch.ref, _stream()), "msa_seq_flash")
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


def rows_conv(x, w, x_b, n_b: int, conv_lo: int, taps, bias, state, slot) -> torch.Tensor:
    """Input projection of the state-space layer for up to 16 sequences' single rows: columns ``conv_lo ..`` leave through the
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
