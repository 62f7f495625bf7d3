"""Every kernel of libmsa_seq.so against the plain float64 mechanisms of oracle/recurrent_layers.py: each alone, in whole
sequences, in portions and in ragged batches, in fp32 and bf16."""
import math

import pytest
import torch

pytestmark = pytest.mark.gpu

from msa_amd import _lib, seq_ops
from oracle import recurrent_layers as R
from seq_helpers import Rand, batch, close, portions

F64, F32, BF16 = torch.float64, torch.float32, torch.bfloat16
DTYPES = [pytest.param(F32, id="f32"), pytest.param(BF16, id="bf16")]


@pytest.fixture(scope="module", autouse=True)
def gpu():
    assert torch.cuda.is_available()
    _lib.load_seq()
    torch.cuda.set_device(0)


# ------------------------------------------------------------------------------------------------ element-wise steps
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [136, 51])
def test_residual_norm_shift(dtype, W):
    r = Rand(1)
    counts, slots = [1, 19, 2, 300], [3, 0, 4, 1]
    T = sum(counts)
    (x, x_), (y, y_), (g, g_) = r(T, W), r(T, W, dtype=dtype), r(T, W, dtype=dtype)
    (gb, gb_), (w, w_), (b, b_), (sh, sh_) = r(W), r(W), r(W), r(W)
    prev, prev_ = r(6, W)
    norm = seq_ops.DynTanhNorm(w, b, 0.7)
    xo, h, hs = seq_ops.residual_norm(x, batch(counts, slots), dtype, y, g, gb, norm, sh, prev)
    want_x = x_ + R.sigmoid(g_ + gb_) * y_
    want_h = R.dyn_tanh(want_x, 0.7, w_, b_)
    close(xo, want_x, F32)
    close(h, want_h, dtype)
    at = 0
    keep = prev_.clone()
    for c, s in zip(counts, slots):
        close(hs[at:at + c], R.token_shift(want_h[at:at + c], sh_, prev_[s]), dtype)
        keep[s] = want_h[at + c - 1]
        at += c
    close(prev, keep, F32)
    # no sublayer output: the norm alone, over the same stream, and the norm without a shift
    x2, h2, none = seq_ops.residual_norm(xo, batch(counts, slots), dtype, norm=norm)
    assert x2 is xo and none is None and torch.equal(h2, h)
    x3, h3, _ = seq_ops.residual_norm(x, batch(counts, slots), dtype, y, g, gb)
    assert h3 is None and torch.equal(x3, xo)


def test_token_shift_in_portions_equals_whole():
    r = Rand(2)
    W, T = 72, 41
    (x, _), (w, _), (b, _), (sh, _) = r(T, W), r(W), r(W), r(W)
    norm = seq_ops.DynTanhNorm(w, b, 1.3)
    whole = torch.zeros(2, W, device="cuda")
    _, _, want = seq_ops.residual_norm(x, batch([T], [1]), F32, norm=norm, shift=sh, prev=whole)
    keep, at = torch.zeros(2, W, device="cuda"), 0
    for n in portions(T, [1, 2, 9, 3]):
        _, _, got = seq_ops.residual_norm(x[at:at + n].contiguous(), batch([n], [1]), F32, norm=norm, shift=sh, prev=keep)
        assert torch.equal(got, want[at:at + n])
        at += n
    assert torch.equal(keep, whole)


@pytest.mark.parametrize("dtype", DTYPES)
def test_gelu_softcap_join_group_norm(dtype):
    r = Rand(3)
    big, big_ = r(7, 100, dtype=dtype, scale=3.0)
    for n in (64, 61):
        y = big.clone()
        seq_ops.gelu_(y[:, :n])
        close(y[:, :n], R.gelu_tanh(big_[:, :n]), dtype, 1e-5 if dtype == F32 else 4e-3)
        assert torch.equal(y[:, n:], big[:, n:])
    close(seq_ops.softcap(big, 2.5), 2.5 * torch.tanh(big_ / 2.5), F32)
    assert torch.equal(seq_ops.softcap(big, 0.0), big.float())
    (x, x_), (x0, x0_) = r(5, 48), r(5, 48, dtype=dtype)
    j = seq_ops.join(x, x0.float(), dtype).cpu().to(F64)
    if dtype == BF16:
        assert (j[:, :48] + j[:, 48:96] - x_).abs().max() < 2e-5 * x_.abs().max() and torch.equal(j[:, :48].to(BF16), x.cpu().to(BF16))
    else:
        assert torch.equal(j[:, :48], x_)
    assert torch.equal(j[:, -48:], x0_)
    for parts in (1, 4, 48):
        (v, v_), (w, w_) = r(9, 48, dtype=dtype), r(48)
        close(seq_ops.group_rmsnorm(v, w, parts, 0.01), R.rms(v_.view(9, parts, -1), 0.01).reshape(9, 48) * w_, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("K", [1, 2, 4, 6])
def test_convolution_portions_and_batches(dtype, K):
    r = Rand(4 + K)
    C, lens = 40, [50, 3, 33]
    seqs = [r(n, 64, dtype=dtype) for n in lens]                # wider rows: the input is a column range
    (taps, taps_), (b, b_) = r(C, K), r(C)
    want = [R.silu(R.causal_conv(s[:, 5:5 + C], taps_, b_)) for _, s in seqs]
    state = torch.zeros(4, K - 1, C, device="cuda")
    at = [0] * 3
    for sizes in ([1, 2, 1], [2, 1, 17], [5, 0, 1], [1, 0, 3], [41, 0, 11]):
        live = [i for i in range(3) if sizes[i]]
        rows = torch.cat([seqs[i][0][at[i]:at[i] + sizes[i]] for i in live])
        got = seq_ops.conv_silu(rows[:, 5:5 + C], taps, b, state, batch([sizes[i] for i in live], [3 - i for i in live]))
        o = 0
        for i in live:
            close(got[o:o + sizes[i]], want[i][at[i]:at[i] + sizes[i]], dtype)
            at[i], o = at[i] + sizes[i], o + sizes[i]
    assert at == lens
    for i in range(3):
        if K > 1:
            kept = torch.cat([torch.zeros(K, C, dtype=F64), seqs[i][1][:, 5:5 + C]])[-(K - 1):]
            assert torch.equal(state[3 - i].cpu().to(F64), kept)


# ------------------------------------------------------------------------------------------------ recurrences
def run_ssd(dtype, H, P, N, G, plan, seed=0, chunked=False, dt_add=-1.0):
    """``plan``: per sequence its portion sizes; sequences advance together."""
    r = Rand(seed)
    lens = [sum(p) for p in plan]
    width = H * P + 2 * G * N
    seqs = [(r(n, width, dtype=dtype), r(n, H * P, dtype=dtype), r(n, H + 8, dtype=dtype)) for n in lens]
    (dtb, dtb_), (al, al_), (D, D_) = r(H, add=dt_add), r(H, scale=0.7), r(H)
    state = torch.zeros(len(plan) + 1, H, N, P, device="cuda")
    got = [[] for _ in plan]
    at = [0] * len(plan)
    for k in range(max(len(p) for p in plan)):
        live = [i for i in range(len(plan)) if k < len(plan[i])]
        cut = lambda j, i: seqs[i][j][0][at[i]:at[i] + plan[i][k]]
        rows = [torch.cat([cut(j, i) for i in live]) for j in range(3)]
        b = batch([plan[i][k] for i in live], [len(plan) - i for i in live])
        v = seq_ops.ssd(rows[0], rows[1], rows[2][:, 4:4 + H], dtb, al, D, H, P, N, G, state, b, chunked=chunked)
        o = 0
        for i in live:
            got[i].append(v[o:o + plan[i][k]])
            o += plan[i][k]
            at[i] += plan[i][k]
    for i, ((_, xbc), (_, z), (_, dt)) in enumerate(seqs):
        T = lens[i]
        x, B, C = torch.split(xbc, [H * P, G * N, G * N], dim=1)
        y, S = R.ssd_scan(x.view(T, H, P), B.view(T, G, N), C.view(T, G, N), R.softplus(dt[:, 4:4 + H] + dtb_), al_, D_)
        close(torch.cat(got[i]), y.reshape(T, -1) * R.silu(z), dtype, None if dtype == F32 else 6e-3)
        close(state[len(plan) - i], S, F32, 3e-5 if dtype == F32 or not chunked else 1e-4)
    assert torch.all(state[0] == 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,P,N,G", [(4, 16, 8, 2), (3, 70, 40, 1), (2, 8, 130, 2), (6, 5, 9, 3), (1, 1, 1, 1), (2, 16, 300, 1)])
def test_state_space_scan(dtype, H, P, N, G):
    run_ssd(dtype, H, P, N, G, [[1, 2, 30, 1, 7], [9], [1, 1, 1]], seed=H + N)


@pytest.mark.parametrize("H,P,N,G", [(4, 16, 8, 2), (3, 72, 40, 1), (2, 64, 128, 1), (2, 24, 200, 2), (4, 136, 64, 4)])
@pytest.mark.parametrize("plan", [[[300]], [[64, 65, 127, 128, 129]], [[70, 1, 200], [1, 66, 2], [130]]], ids=["whole", "edges", "ragged"])
def test_state_space_chunked(H, P, N, G, plan):
    run_ssd(BF16, H, P, N, G, plan, seed=H + P, chunked=True)


@pytest.mark.parametrize("dt_add", [-9.0, 6.0])
def test_state_space_chunked_extreme_steps(dt_add):
    """Decays next to one (a state that lives for the whole sequence) and next to zero."""
    run_ssd(BF16, 2, 32, 32, 1, [[520]], seed=5, chunked=True, dt_add=dt_add)
    run_ssd(F32, 2, 32, 32, 1, [[520]], seed=5, dt_add=dt_add)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [32, 21, 300])
def test_min_gru(dtype, n):
    r = Rand(n)
    lens = [200, 64, 66]
    cols = -(-n // 16) * 48
    seqs = [r(m, cols, dtype=dtype, scale=1.5) for m in lens]
    (zb, zb_), (ub, ub_) = r(n), r(n)
    pick = lambda s, k: torch.stack([s[:, c // 16 * 48 + 16 * k + c % 16] for c in range(n)], 1)
    state = torch.zeros(5, n, device="cuda")
    at, got = [0] * 3, [[] for _ in lens]
    for sizes in ([1, 64, 2], [63, 0, 63], [65, 0, 1], [64, 0, 0], [7, 0, 0]):
        live = [i for i in range(3) if sizes[i]]
        rows = torch.cat([seqs[i][0][at[i]:at[i] + sizes[i]] for i in live])
        out = seq_ops.min_gru(rows, zb, ub, n, state, batch([sizes[i] for i in live], [i + 1 for i in live]))
        o = 0
        for i in live:
            got[i].append(out[o:o + sizes[i]])
            at[i], o = at[i] + sizes[i], o + sizes[i]
    for i, (_, s) in enumerate(seqs):
        S = R.min_gru(R.sigmoid(pick(s, 0) + zb_), pick(s, 1) + ub_)
        close(torch.cat(got[i]), S * R.silu(pick(s, 2)), dtype)
        close(state[i + 1], S[-1], F32)
    assert torch.all(state[0] == 0) and torch.all(state[4] == 0)


# ------------------------------------------------------------------------------------------------ attention
def test_latent_append_places_rows_at_their_positions():
    r = Rand(11)
    for dtype in (F32, BF16):
        (x, x_), (w, w_) = r(6, 80, dtype=dtype), r(24)
        cache = torch.zeros(3, 70, 24, dtype=dtype, device="cuda")
        seq_ops.latent_append(x[:, 8:32], w, 0.02, cache, batch([1, 3, 2], [2, 0, 1], [69, 62, 0]))
        want = torch.zeros(3, 70, 24, dtype=F64)
        c = R.rms(x_[:, 8:32], 0.02) * w_
        want[2, 69], want[0, 62:65], want[1, 0:2] = c[0], c[1:4], c[4:6]
        close(cache, want, dtype)
        with pytest.raises(ValueError, match="cannot take"):
            seq_ops.latent_append(x[:, 8:32], w, 0.02, cache, batch([1, 3, 2], [2, 0, 1], [69, 62, 69]))


def latent_case(dtype, H, rank, lens, news, seed=0, scale=0.3, cap=None, sharpen=None):
    """Query rows that are the last ``news`` tokens of sequences of ``lens``; ``sharpen[(seq, row)] = key`` points a row's
    query of head 0 at one key so that its score stands out."""
    r = Rand(seed)
    cap = max(lens) + 3 if cap is None else cap
    cache, cache_ = r(len(lens) + 1, cap, rank, dtype=dtype)
    q, q_ = r(sum(news), H, rank, dtype=dtype)
    slots = [len(lens) - i for i in range(len(lens))]
    at = 0
    for s, n in enumerate(news):
        for (i, row), key in (sharpen or {}).items():
            if i == s:
                c = cache_[slots[s], key]
                q_[at + row, 0] = (c * (30.0 / scale / (c * c).sum())).to(dtype).to(F64)
        at += n
    q = q_.to(dtype).cuda()
    sink, sink_ = r(H, scale=2.0)
    b = batch(news, slots, [l - n for l, n in zip(lens, news)])
    got = seq_ops.latent_attn(q, cache, sink, scale, b)
    want, at = [], 0
    for s, (l, n) in enumerate(zip(lens, news)):
        c = cache_[slots[s], :l]
        k = c[:, None].expand(l, H, rank)
        want.append(R.sink_attention(q_[at:at + n], k, k, sink_, scale))
        at += n
    want = torch.cat(want)
    close(got, want, dtype)
    return got, q, cache, sink, b, want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,rank", [(1, 8), (5, 72), (16, 128), (40, 96), (3, 512), (2, 27), (2, 520)])
def test_latent_attention(dtype, H, rank):
    latent_case(dtype, H, rank, [1, 65, 300, 128], [1, 1, 3, 2], seed=H)


@pytest.mark.parametrize("key", [0, 1, 62, 63, 64, 65, 127, 128, 700, 997, 998, 999])
def test_latent_decode_sees_one_far_key(key):
    """A single key with a score far above the rest: the output is that key's latent, wherever it lies (tile and split edges,
    the first keys, the row's own)."""
    got, *_, want = latent_case(BF16, 4, 64, [1000, 65], [1, 1], seed=key, sharpen={(0, 0): key})
    assert (got[0, 0].cpu().to(F64) - want[0, 0]).abs().max() < 0.05


def test_rows_of_a_portion_do_not_see_later_keys():
    """The keys behind a row's own are set apart by huge values: they must not show in it."""
    for dtype, rank in ((F32, 32), (BF16, 32), (BF16, 30)):
        r = Rand(3)
        cache, _ = r(1, 80, rank, dtype=dtype)
        q, q_ = r(5, 2, rank, dtype=dtype)
        sink = torch.zeros(2, device="cuda")
        b = batch([5], [0], [62])
        base = seq_ops.latent_attn(q, cache, sink, 0.2, b)
        for row in range(4):
            poked = cache.clone()
            poked[:, 62 + row + 1:] = 1e4
            assert torch.equal(seq_ops.latent_attn(q, poked, sink, 0.2, b)[:row + 1], base[:row + 1])


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_takes_its_share(dtype):
    """Scores of zero: every key and the sink weigh exp(0) and exp(sink); an ever larger sink takes everything."""
    cache = torch.ones(1, 64, 16, dtype=dtype, device="cuda")
    q = torch.zeros(1, 3, 16, dtype=dtype, device="cuda")
    sink = torch.tensor([0.0, math.log(5.0), 80.0], device="cuda")
    got = seq_ops.latent_attn(q, cache, sink, 1.0, batch([1], [0], [4])).float().cpu()
    for h, w in enumerate((5 / 6, 0.5, 0.0)):
        assert torch.allclose(got[0, h], torch.full((16,), w), atol=4e-3)


def flash_case(H, D, E, lens, news, seed=0, scale=0.25, sharpen=None):
    r = Rand(seed)
    T = sum(news)
    q, q_ = r(T, H * D + 16, dtype=BF16)
    off = [sum(lens[:i]) for i in range(len(lens))]
    (k, k_), (v, v_), (sink, sink_) = r(sum(lens), H * D, dtype=BF16), r(sum(lens), H * E, dtype=BF16), r(H, scale=2.0)
    for (row, h), key in (sharpen or {}).items():
        c = k_[key, h * D:(h + 1) * D]
        q_[row, 8 + h * D:8 + (h + 1) * D] = (c * (30.0 / scale / (c * c).sum())).to(BF16).to(F64)
    q = q_.to(BF16).cuda()
    b = batch(news, None, [l - n for l, n in zip(lens, news)])
    got = seq_ops.flash(q[:, 8:8 + H * D], k, v, torch.tensor(off, device="cuda"), sink, scale, H, b)
    at = 0
    for i, (l, n) in enumerate(zip(lens, news)):
        want = R.sink_attention(q_[at:at + n, 8:8 + H * D].view(n, H, D), k_[off[i]:off[i] + l].view(l, H, D),
                                v_[off[i]:off[i] + l].view(l, H, E), sink_, scale)
        close(got[at:at + n], want.reshape(n, -1), BF16)
        at += n


@pytest.mark.parametrize("H,D,E", [(2, 40, 24), (3, 64, 64), (1, 128, 128), (2, 72, 48), (2, 168, 104), (1, 256, 200), (1, 8, 8)])
def test_flash_shapes(H, D, E):
    flash_case(H, D, E, [200], [200], seed=D)


@pytest.mark.parametrize("lens,news", [([130, 65, 40], [1, 65, 17]), ([300], [129]), ([64, 128], [64, 128]), ([257], [2])])
def test_flash_portions_and_batches(lens, news):
    flash_case(2, 48, 40, lens, news, seed=lens[0])


def test_flash_far_keys_at_every_edge():
    """Rows pointed at single keys: the first, tile edges, their own, far and near."""
    keys = [0, 1, 31, 32, 63, 64, 127, 128, 191, 192, 255, 299]
    flash_case(2, 64, 64, [300], [300], seed=9, sharpen={(r, r % 2): k for k in keys for r in {k, 299, min(299, k + 64), min(299, k + 1)}})


# ------------------------------------------------------------------------------------------------ decode products
@pytest.mark.parametrize("M,N,K", [(1, 16, 8), (16, 37, 136), (3, 200, 72), (7, 2600, 264), (16, 6200, 128), (5, 48, 1000), (16, 8200, 520), (3, 9001, 1032),
                                   (5, 8192, 2560), (2, 8300, 1800), (9, 20000, 4096), (1, 8192, 3000)])
def test_rows_linear_plain_and_f32(M, N, K):
    r = Rand(M + K)
    (x, x_), (w, w_) = r(M, K, dtype=BF16), r(N, K, dtype=BF16, scale=K ** -0.5)
    want = x_ @ w_.T
    close(seq_ops.rows_linear(x, w), want, BF16, 4e-3)
    gn = N // 2
    close(seq_ops.rows_linear(x, w, gelu_n=gn), torch.cat([R.gelu_tanh(want[:, :gn]), want[:, gn:]], 1), BF16, 4e-3)
    add, add_ = r(N)
    close(seq_ops.rows_linear_f32(x, w, add=add), want + add_, F32)
    close(seq_ops.rows_linear_f32(x, w, cap=0.8), 0.8 * torch.tanh(want / 0.8), F32)


@pytest.mark.parametrize("N_a,N_b,K", [(32, 40, 80), (64, 6200, 80), (3200, 3000, 80), (8192, 200, 648), (32, 9000, 1160), (6400, 6000, 2568)])
def test_rows_linear_two_operands(N_a, N_b, K):
    r = Rand(N_a)
    (x, x_), (y, y_), (w, w_) = r(9, K, dtype=BF16), r(9, K, dtype=BF16), r(N_a + N_b, K, dtype=BF16, scale=K ** -0.5)
    got = seq_ops.rows_linear(x, w, x_b=y, n_b=N_a)
    close(got, torch.cat([x_ @ w_[:N_a].T, y_ @ w_[N_a:].T], 1), BF16, 4e-3)


@pytest.mark.parametrize("groups,N,K", [(5, 72, 40), (3, 16, 8), (36, 200, 24), (4, 512, 136)])
def test_rows_linear_per_head(groups, N, K):
    r = Rand(groups)
    (x, x_), (w, w_) = r(13, groups * K, dtype=BF16), r(groups * N, K, dtype=BF16, scale=K ** -0.5)
    want = torch.bmm(x_.view(13, groups, K).transpose(0, 1), w_.view(groups, N, K).transpose(1, 2)).transpose(0, 1).reshape(13, -1)
    close(seq_ops.rows_linear(x, w, groups=groups), want, BF16, 4e-3)


@pytest.mark.parametrize("M,N,K", [(4, 120, 64), (16, 51, 200), (1, 2600, 136)])
def test_rows_residual(M, N, K):
    r = Rand(N)
    (x, x_), (w, w_), (g, g_) = r(M, K, dtype=BF16), r(N, K, dtype=BF16, scale=K ** -0.5), r(M, N + 16, dtype=BF16)
    (s, s_), (gb, gb_), (nw, nw_), (nb, nb_), (sh, sh_), (prev, prev_) = r(M, N), r(N), r(N), r(N), r(N), r(20, N)
    slot = torch.arange(19, 19 - M, -1, dtype=torch.int32, device="cuda")
    h, hs = seq_ops.rows_residual(x, w, s, g[:, 5:5 + N], gb, slot, seq_ops.DynTanhNorm(nw, nb, 0.9), sh, prev)
    want = s_ + R.sigmoid(g_[:, 5:5 + N] + gb_) * (x_ @ w_.T)
    wh = R.dyn_tanh(want, 0.9, nw_, nb_)
    before = prev_[slot.cpu().long()]
    close(s, want, F32)
    close(h, wh, BF16, 4e-3)
    close(hs, wh + (before - wh) * sh_, BF16, 4e-3)
    prev_[slot.cpu().long()] = wh
    close(prev, prev_, F32)


@pytest.mark.parametrize("W,rows", [(64, 32), (600, 8200)])
@pytest.mark.parametrize("K", [1, 2, 5])
def test_rows_conv_equals_the_block_form(K, W, rows):
    r = Rand(K)
    lo, C = 40, 56
    (w, _), (taps, _), (b, _) = r(128 + rows, W, dtype=BF16, scale=1.6 * W ** -0.5), r(C, K), r(C)
    s1, s2 = torch.zeros(4, K - 1, C, device="cuda"), torch.zeros(4, K - 1, C, device="cuda")
    for step in range(6):
        (x, x_), (y, _) = r(3, W, dtype=BF16), r(3, W, dtype=BF16)
        slot = torch.tensor([2, 0, 3], dtype=torch.int32, device="cuda")
        out = seq_ops.rows_conv(x, w, y, 128, lo, taps, b, s1, slot)
        plain = seq_ops.rows_linear(x, w, x_b=y, n_b=128)
        conv = seq_ops.conv_silu(plain[:, lo:lo + C], taps, b, s2, batch([1, 1, 1], [2, 0, 3]))
        assert torch.equal(out[:, :lo], plain[:, :lo]) and torch.equal(out[:, lo + C:], plain[:, lo + C:])
        close(out[:, lo:lo + C], conv, BF16)
    if K > 1:
        close(s1, s2, BF16, 4e-3)
        assert torch.all(s1[1] == 0)


@pytest.mark.parametrize("n", [24, 16, 72])
def test_rows_gru_equals_the_block_form(n):
    r = Rand(n)
    W = 48
    (wz, _), (wu, _), (wg, _), (wr, _) = (r(m, W, dtype=BF16, scale=0.3) for m in (n, n, n, 40))
    w = torch.cat([seq_ops.interleave_gru(wz, wu, wg), wr]).contiguous()
    n_b = w.shape[0] - 40
    (zb, _), (ub, _) = r(n), r(n)
    s1, s2 = torch.zeros(3, n, device="cuda"), torch.zeros(3, n, device="cuda")
    for step in range(5):
        (x, _), (y, y_) = r(2, W, dtype=BF16), r(2, W, dtype=BF16)
        slot = torch.tensor([2, 0], dtype=torch.int32, device="cuda")
        act, out = seq_ops.rows_gru(x, w, y, n, zb, ub, s1, slot)
        plain = seq_ops.rows_linear(x, w, x_b=y, n_b=n_b)
        want = seq_ops.min_gru(plain[:, :n_b], zb, ub, n, s2, batch([1, 1], [2, 0]))
        close(act, want, BF16, 2e-2)
        assert torch.equal(out[:, n_b:], plain[:, n_b:])
    close(s1, s2, BF16)
    assert torch.all(s1[1] == 0)
