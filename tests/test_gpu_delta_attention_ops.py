"""The kernels of the channel-wise delta rule, rotary chunk attention, clamped gated units and output-normed residuals against the
plain float64 mechanisms of oracle/delta_attention_layers.py: each alone, in portions, in ragged batches, in fp32 and bf16."""
import pytest
import torch

pytestmark = pytest.mark.gpu

from msa_amd import _lib, seq_ops
from msa_amd.config import RotaryConfig
from oracle import delta_attention_layers as O
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
@pytest.mark.parametrize("W", [8, 51, 136, 4500, 4501])
def test_rms_residual(dtype, W):
    r = Rand(W)
    T, eps = 7, 0.02
    (x, x_), (wide, wide_), (w, w_), (n, n_) = r(T, W), r(T, W + 8, dtype=dtype), r(W), r(W)
    y, y_ = wide[:, :W], wide_[:, :W]
    want = x_ + O.rms(y_, eps) * w_
    xo, h = seq_ops.rms_residual(x, dtype, y, w, eps)
    close(xo, want, F32)
    close(h, want, dtype)
    xo2, h2 = seq_ops.rms_residual(x, dtype, y, w, eps, next_w=n)
    assert torch.equal(xo2, xo)
    close(h2, O.rms(want, eps) * n_, dtype)
    same, h3 = seq_ops.rms_residual(x, dtype)
    assert same is x and torch.equal(h3, x.to(dtype))
    _, h4 = seq_ops.rms_residual(x, dtype, eps=eps, next_w=n)
    close(h4, O.rms(x_, eps) * n_, dtype)
    out = x.clone()
    back, none = seq_ops.rms_residual(out, dtype, y, w, eps, out=out, want_h=False)
    assert back is out and none is None and torch.equal(out, xo)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 37, 64])
def test_clamped_glu(dtype, n):
    r = Rand(n)
    (wide, wide_) = r(9, 2 * n + 8, dtype=dtype, scale=3.0)
    for limit in (0.5, 2.0, 50.0):
        got = seq_ops.clamped_glu(wide[:, :2 * n], limit)
        close(got, O.clamped_glu(wide_[:, 0:2 * n:2], wide_[:, 1:2 * n:2], limit), dtype, 1e-5 if dtype == F32 else 6e-3)
    # a constant pair on each side of each clamp
    x = torch.tensor([[3.0, 1.0, -3.0, 1.0, 1.0, 3.0, 1.0, -3.0]], device="cuda").to(dtype)
    want = O.clamped_glu(x.cpu().to(F64)[:, 0::2], x.cpu().to(F64)[:, 1::2], 2.0)
    close(seq_ops.clamped_glu(x, 2.0), want, dtype, 1e-5 if dtype == F32 else 6e-3)
    assert want[0, 3] < 0 and want[0, 1] < 0        # up may fall below -1, and a low gate is not clamped


@pytest.mark.parametrize("M", [1, 5, 16])
@pytest.mark.parametrize("ff,K", [(9, 24), (200, 256), (4200, 64), (4200, 768), (4103, 1032)])
def test_rows_glu(M, ff, K):
    """Both forms of the weight-streaming product (few rows a workgroup; many)."""
    r = Rand(M + ff)
    (x, x_), (g, g_), (u, u_) = r(M, K, dtype=BF16), r(ff, K, dtype=BF16, scale=2 * K ** -0.5), r(ff, K, dtype=BF16, scale=2 * K ** -0.5)
    w = seq_ops.interleave_pairs(g, u)
    assert torch.equal(w[0::2], g) and torch.equal(w[1::2], u)
    close(seq_ops.rows_glu(x, w, 1.5), O.clamped_glu(x_ @ g_.T, x_ @ u_.T, 1.5), BF16)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E", [1, 24, 64, 72, 130, 136, 1040])
def test_head_norm_gate(dtype, E):
    r = Rand(E)
    T, H, eps = 5, 3, 1e-3
    (o, o_), (g, g_), (w, w_) = r(T, H * E, dtype=dtype), r(T, H * E + 8, dtype=dtype), r(E)
    lib = _lib.load_seq()
    rc = lib.msa_seq_head_norm_gate(o.data_ptr(), g.data_ptr(), H * E + 8, w.data_ptr(), eps, _lib.dtype_code(dtype), T, H, E, 0)
    assert rc == 0
    close(o, O.gated_head_norm(o_.view(T, H, E), w_, g_[:, :H * E].view(T, H, E), eps).reshape(T, -1), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_convolution_without_bias(dtype):
    r = Rand(4)
    for C, K in ((40, 4), (37, 3), (16, 1), (24, 7)):
        (x, x_), (taps, taps_) = r(30, C, dtype=dtype), r(C, K)
        want = O.silu(O.causal_conv(x_, taps_, torch.zeros(C, dtype=F64)))
        state, at = torch.zeros(1, K - 1, C, device="cuda"), 0
        for n in portions(30, [2, 1, 20, 3]):
            close(seq_ops.conv_silu(x[at:at + n], taps, None, state, batch([n], [0])), want[at:at + n], dtype)
            at += n


def test_projection_with_convolution_without_bias():
    r = Rand(5)
    M, K, C, taps_n = 3, 64, 40, 4
    (w, w_), (taps, taps_) = r(64, K, dtype=BF16, scale=K ** -0.5), r(C, taps_n)
    xs = [r(M, K, dtype=BF16) for _ in range(6)]
    state = torch.zeros(4, taps_n - 1, C, device="cuda")
    slot = torch.tensor([3, 0, 2], dtype=torch.int32, device="cuda")
    conv = [O.silu(O.causal_conv(torch.stack([x_[m] @ w_[:C].T for _, x_ in xs]), taps_, torch.zeros(C, dtype=F64))) for m in range(M)]
    for t, (x, x_) in enumerate(xs):
        got = seq_ops.rows_conv(x, w, None, 64, 0, taps, None, state, slot)
        close(got[:, C:], x_ @ w_[C:].T, BF16)
        close(got[:, :C], torch.stack([conv[m][t] for m in range(M)]), BF16)


# ------------------------------------------------------------------------------------------------ delta rule
class DeltaCase:
    """Operands of a few sequences and the oracle's outputs and final states."""

    def __init__(self, H, G, D, E, lens, dtype, seed=0, a_scale=1.0, rate=0.0, bias=-2.0):
        r = Rand(seed)
        self.dims, self.lens, self.dtype, self.eps = (H, G, D, E), lens, dtype, 1e-3
        n = sum(lens)
        self.qkv, qkv = r(n, 2 * G * D + H * E, dtype=dtype)
        self.a, a = r(n, H * D, dtype=dtype, scale=a_scale)
        self.b, b = r(n, H, dtype=dtype)
        self.gate, gate = r(n, H * E, dtype=dtype)
        self.A_log, A_log = r(H, scale=0.3, add=rate)
        self.dt_bias, dt_bias = r(H * D, scale=0.7, add=bias)
        self.norm, norm = r(E, scale=0.2, add=1.0)
        of = torch.arange(H) // (H // G)
        self.want, self.states, at = [], [], 0
        for L in lens:
            rows = slice(at, at + L)
            q, k, v = torch.split(qkv[rows], [G * D, G * D, H * E], dim=1)
            step = O.softplus(a[rows] + dt_bias).view(L, H, D)
            o, S = O.delta_rule(O.unit(q.view(L, G, D))[:, of] * D ** -0.5, O.unit(k.view(L, G, D))[:, of], v.reshape(L, H, E),
                                -torch.exp(A_log)[None, :, None] * step, O.sigmoid(b[rows]))
            self.want.append(O.gated_head_norm(o, norm, gate[rows].view(L, H, E), self.eps).reshape(L, H * E))
            self.states.append(S)
            at += L
        self.starts = [sum(lens[:i]) for i in range(len(lens))]
        self.fed = [0] * len(lens)
        self.slots = [len(lens) - i for i in range(len(lens))]
        self.state = torch.zeros(len(lens) + 2, H, D, E, device="cuda")

    def step(self, counts, chunked, tol=None):
        """The next ``counts[i]`` tokens of every sequence (0: none), checked."""
        live = [i for i, n in enumerate(counts) if n]
        rows = torch.cat([torch.arange(self.starts[i] + self.fed[i], self.starts[i] + self.fed[i] + counts[i]) for i in live]).cuda()
        b = batch([counts[i] for i in live], [self.slots[i] for i in live], [self.fed[i] for i in live])
        got = seq_ops.delta(self.qkv[rows], self.a[rows], self.b[rows], self.gate[rows], self.A_log, self.dt_bias, self.norm, self.eps,
                            *self.dims, self.state, b, chunked)
        at = 0
        for i in live:
            close(got[at:at + counts[i]], self.want[i][self.fed[i]:self.fed[i] + counts[i]], self.dtype, tol)
            self.fed[i] += counts[i]
            at += counts[i]

    def finish(self, tol=None):
        assert self.fed == self.lens
        for i, S in enumerate(self.states):
            close(self.state[self.slots[i]], S, F32, tol)
        assert not self.state[0].any() and not self.state[-1].any()          # nobody's slots


SCAN_SIZES = [(4, 2, 24, 40), (3, 1, 7, 5), (2, 2, 128, 128), (6, 3, 64, 72), (2, 1, 136, 130), (1, 1, 1, 1), (2, 1, 260, 70), (2, 2, 500, 9)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", SCAN_SIZES, ids=str)
def test_delta_scan(dtype, sizes):
    c = DeltaCase(*sizes, [37, 1, 12, 20], dtype)
    for counts in ([30, 1, 2, 0], [1, 0, 8, 1], [6, 0, 2, 19]):
        c.step(counts, False)
    c.finish()


CHUNK_SIZES = [(4, 2, 24, 40), (2, 2, 128, 128), (3, 3, 64, 72), (6, 3, 72, 16), (2, 1, 8, 8), (2, 1, 96, 136), (1, 1, 128, 264), (8, 1, 32, 64)]


@pytest.mark.parametrize("sizes", CHUNK_SIZES, ids=str)
def test_delta_chunked(sizes):
    """Ragged portions that end inside chunks and blocks, states carried between forms."""
    c = DeltaCase(*sizes, [200, 1, 83, 64], BF16)
    for counts, chunked in (([130, 1, 17, 0], True), ([1, 0, 1, 0], False), ([69, 0, 64, 64], True), ([0, 0, 1, 0], True)):
        c.step(counts, chunked)
    c.finish(2e-4)


@pytest.mark.parametrize("L", [2, 15, 16, 17, 47, 48, 63, 64, 65, 128, 129])
def test_delta_chunked_lengths(L):
    c = DeltaCase(2, 1, 40, 24, [L], BF16, seed=L)
    c.step([L], True)
    c.finish(2e-4)


@pytest.mark.parametrize("rate,bias,a_scale", [(0.0, -6.0, 1.0), (2.0, 0.0, 2.0), (3.0, 3.0, 3.0), (4.0, -1.0, 8.0), (1.0, 12.0, 1.0), (-9.0, -9.0, 1.0)])
def test_delta_chunked_decays(rate, bias, a_scale):
    """From hardly any decay to states that are gone after a token, and both in neighbouring channels and tokens: blocks that are
    multiplied with their decays factored and blocks that are summed pair by pair."""
    c = DeltaCase(3, 3, 56, 40, [150], BF16, seed=3, rate=rate, bias=bias, a_scale=a_scale)
    c.step([150], True)
    c.finish(3e-4)
    s = DeltaCase(3, 3, 56, 40, [150], BF16, seed=3, rate=rate, bias=bias, a_scale=a_scale)
    s.step([150], False)
    s.finish()


def test_delta_reads_a_far_write():
    """No decay: a value written under a key of its own is read back hundreds of tokens later, across chunks and portions."""
    D, E, L = 64, 32, 400
    qkv = torch.zeros(L, 2 * D + E)
    qkv[:, D + 1] = 1.0                                        # every key the same ...
    qkv[3, D:2 * D] = 0
    qkv[3, D] = 1.0                                            # ... but one,
    qkv[:, 2 * D:] = 0.1 * torch.randn(L, E, generator=torch.Generator().manual_seed(1))
    qkv[3, 2 * D:] = torch.arange(E) / E + 1.0
    qkv[L - 1, 0] = 1.0                                        # which the last query asks for
    qkv = qkv.to(BF16).cuda()
    a, b, gate = torch.full((L, D), -100.0), torch.full((L, 1), 30.0), torch.full((L, E), 30.0)
    a, b, gate = a.to(BF16).cuda(), b.to(BF16).cuda(), gate.to(BF16).cuda()
    zeros = lambda n: torch.zeros(n, device="cuda")
    want = qkv[3, 2 * D:].cpu().to(F64)
    want = want / torch.sqrt((want * want).mean())
    for sizes in ([400], [399, 1], [100, 2, 1], [64], [65, 63]):
        state, at = torch.zeros(1, 1, D, E, device="cuda"), 0
        for n in portions(L, sizes):
            rows = slice(at, at + n)
            out = seq_ops.delta(qkv[rows], a[rows], b[rows], gate[rows], zeros(1), zeros(D), torch.ones(E, device="cuda"), 1e-6, 1, 1, D, E, state,
                                batch([n], [0], [at]), chunked=n >= 2)
            at += n
        close(out[-1], want, BF16)


def test_delta_chunked_in_segments():
    """More chunks than are prepared at a time, in few and in many segments: as the token-by-token form."""
    H, G, D, E, T = 32, 4, 128, 128, 9300
    g = torch.Generator(device="cuda").manual_seed(2)
    bf = lambda *s: torch.randn(s, generator=g, device="cuda").to(BF16)
    qkv, a, b, gate = bf(T, 2 * G * D + H * E), bf(T, H * D), bf(T, H), bf(T, H * E)
    A_log, bias, norm = torch.rand(H, device="cuda"), torch.randn(H * D, device="cuda") - 3, torch.ones(E, device="cuda")
    outs, states = [], []
    for chunked in (False, True):
        state = torch.zeros(1, H, D, E, device="cuda")
        outs.append(seq_ops.delta(qkv, a, b, gate, A_log, bias, norm, 1e-5, H, G, D, E, state, batch([T], [0]), chunked))
        states.append(state)
    close(outs[1], outs[0], BF16)
    close(states[1], states[0], F32, 2e-4)


def test_delta_chunked_segments_of_a_ragged_batch():
    """Sequences that end in different segments."""
    c = DeltaCase(2, 1, 32, 24, [1700, 3, 1408, 1409, 900], BF16, seed=11)
    c.step(c.lens, True)
    c.finish(3e-4)


# ------------------------------------------------------------------------------------------------ rotary attention
def frequencies(pairs, base=1e4):
    return RotaryConfig(base, 2 * pairs).frequencies()


class Cache:
    """Keys and values of a few sequences in scattered slots, and the positions the queries stand at."""

    def __init__(self, G, D, E, pos, counts, dtype, seed=0, spare=3):
        r = Rand(seed)
        self.pos, self.counts = pos, counts
        cap = max(p + n for p, n in zip(pos, counts)) + spare
        self.k, self.k_ = r(len(pos) + 1, cap, G, D, dtype=dtype)
        self.v, self.v_ = r(len(pos) + 1, cap, G, E, dtype=dtype)
        self.slots = [len(pos) - i for i in range(len(pos))]
        self.batch = batch(counts, self.slots, pos)

    def attend(self, q_, scale, chunk):
        out, at = [], 0
        for s, p, n in zip(self.slots, self.pos, self.counts):
            out.append(O.chunk_attention(q_[at:at + n], self.k_[s, :p + n], self.v_[s, :p + n], scale, chunk or None))
            at += n
        return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,E,pairs", [(8, 2, 88, 104, 24), (4, 4, 40, 24, 20), (3, 1, 13, 11, 5), (5, 5, 16, 8, 0), (2, 1, 200, 136, 16), (9, 3, 64, 64, 32),
                                           (2, 2, 512, 16, 256), (1, 1, 1, 1, 0)])
def test_norm_rotation_and_cache_rows(dtype, H, G, D, E, pairs):
    r = Rand(D)
    pos, counts, slots, eps = [0, 3000, 7], [3, 1, 5], [2, 0, 3], 1e-3
    T = sum(counts)
    at8 = lambda n: -(-n // 8) * 8
    (proj, proj_) = r(T, at8(H * D) + at8(G * D) + G * E + 8, dtype=dtype)
    ko, vo = at8(H * D), at8(H * D) + at8(G * D)
    (qn, qn_), (kn, kn_) = r(D), r(D)
    fr = frequencies(pairs)
    freqs = torch.tensor(fr, dtype=F64, device="cuda")
    kc, vc = torch.full((5, 3010, G, D), 7.0, dtype=dtype, device="cuda"), torch.full((5, 3010, G, E), 7.0, dtype=dtype, device="cuda")
    b = batch(counts, slots, pos)
    where = [(s, p + j) for s, p, n in zip(slots, pos, counts) for j in range(n)]
    at = [p for _, p in where]
    turn = lambda x, heads, w: O.rotate(O.rms(x.reshape(T, heads, D), eps) * w, at, fr)
    want_q, want_k = turn(proj_[:, :H * D], H, qn_), turn(proj_[:, ko:ko + G * D], G, kn_)
    got = seq_ops.qk_rope_append(proj[:, :H * D], qn, freqs, eps, kc, vc, b, proj[:, ko:ko + G * D], proj[:, vo:vo + G * E], kn)
    close(got, want_q, dtype)
    close(torch.stack([kc[s, p] for s, p in where]), want_k, dtype)
    assert torch.equal(torch.stack([vc[s, p] for s, p in where]).view(T, -1), proj[:, vo:vo + G * E])
    for s, p in where:                                        # and nothing else is written
        kc[s, p], vc[s, p] = 7.0, 7.0
    assert bool((kc == 7).all()) and bool((vc == 7).all())
    again = seq_ops.qk_rope_append(proj[:, :H * D], qn, freqs, eps, kc, vc, b)
    assert torch.equal(again, got) and bool((kc == 7).all())


def test_rotation_far_out():
    """Angles of a million positions stay exact."""
    r = Rand(1)
    (q, q_), (w, w_) = r(2, 64), r(64)
    fr = frequencies(32)
    kc = torch.zeros(1, 1 << 20, 1, 64, device="cuda")
    vc = torch.zeros(1, 1 << 20, 1, 1, device="cuda")
    pos = (1 << 20) - 2
    got = seq_ops.qk_rope_append(q, w, torch.tensor(fr, dtype=F64, device="cuda"), 1e-5, kc, vc, batch([2], [0], [pos]))
    close(got, O.rotate(O.rms(q_.view(2, 1, 64), 1e-5) * w_, [pos, pos + 1], fr), F32)


ATTN_SIZES = [(8, 2, 88, 104), (4, 4, 40, 24), (20, 1, 64, 128), (2, 1, 200, 136), (1, 1, 8, 8), (34, 2, 128, 128)]


@pytest.mark.parametrize("chunk", [0, 1, 7, 64, 100])
@pytest.mark.parametrize("H,G,D,E", ATTN_SIZES + [(3, 1, 13, 11)], ids=str)
@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_of_a_few_rows(dtype, H, G, D, E, chunk):
    r = Rand(chunk)
    c = Cache(G, D, E, [0, 262, 99, 63, 6], [2, 1, 3, 1, 2], dtype, seed=H)
    T = sum(c.counts)
    (q, q_), (g, g_) = r(T, H, D, dtype=dtype), r(T, H + 3, dtype=dtype)
    want = c.attend(q_, 0.2, chunk)
    close(seq_ops.kv_attn(q, c.k, c.v, 0.2, c.batch, chunk), want.reshape(T, -1), dtype)
    gated = (want * O.sigmoid(g_[:, :H])[:, :, None]).reshape(T, -1)
    close(seq_ops.kv_attn(q, c.k, c.v, 0.2, c.batch, chunk, g[:, :H]), gated, dtype)
    if dtype == BF16 and D % 8 == 0:
        close(seq_ops.kv_attn(q, c.k, c.v, 0.2, c.batch, chunk, g[:, :H], split=False), gated, dtype)


def test_split_attention_long():
    """Thousands of keys over many workgroups, with one key that outweighs the rest at a range's edge."""
    r = Rand(9)
    H, G, D, E = 8, 2, 64, 64
    c = Cache(G, D, E, [4099, 31, 2047], [1, 1, 1], BF16, seed=2)
    q, q_ = r(3, H, D, dtype=BF16)
    for key in (0, 31, 32, 1023, 1024, 2047, 4099):
        k, k_ = c.k.clone(), c.k_.clone()
        for i, s in enumerate(c.slots):
            if key <= c.pos[i]:
                k[s, key] = (4 * q[i].view(G, H // G, D)[:, 0]).to(BF16)
        k_ = k.cpu().to(F64)
        want = torch.cat([O.chunk_attention(q_[i:i + 1], k_[s, :c.pos[i] + 1], c.v_[s, :c.pos[i] + 1], 0.3, None) for i, s in enumerate(c.slots)])
        close(seq_ops.kv_attn(q, k, c.v, 0.3, c.batch), want.reshape(3, -1), BF16)


@pytest.mark.parametrize("chunk", [0, 5, 32, 100, 128, 300])
@pytest.mark.parametrize("H,G,D,E", [(8, 2, 88, 104), (4, 4, 40, 24), (8, 1, 64, 128), (2, 1, 200, 136), (3, 3, 8, 8)], ids=str)
def test_prefill_attention(H, G, D, E, chunk):
    r = Rand(chunk + D)
    c = Cache(G, D, E, [0, 77, 0, 130], [150, 129, 1, 40], BF16, seed=H)
    T = sum(c.counts)
    (q, q_), (g, g_) = r(T, H * D, dtype=BF16), r(T, H, dtype=BF16)
    n = c.k.shape[0] * c.k.shape[1]
    got = seq_ops.flash(q, c.k.view(n, -1), c.v.view(n, -1), c.batch.cache_rows(c.k.shape[1]), None, 0.15, H, c.batch, G, chunk, g)
    want = c.attend(q_.view(T, H, D), 0.15, chunk) * O.sigmoid(g_)[:, :, None]
    close(got, want.reshape(T, -1), BF16)


@pytest.mark.parametrize("size", [3, 16, 63, 64, 65, 130])
def test_chunk_edges(size):
    """One key outweighs all others wherever it is seen: queries on both sides of every border, in prompts, portions and decoding."""
    H, G, D, E, L = 2, 1, 64, 64, 300
    r = Rand(size)
    (k, k_), (v, v_) = r(1, L, G, D, dtype=BF16, scale=0.1), r(1, L, G, E, dtype=BF16)
    q = torch.ones(L, H, D).to(BF16).cuda()
    for key in {0, size - 1, size, 2 * size - 1, 2 * size, 200 // size * size, 200 // size * size + size - 1} & set(range(L)):
        kk = k.clone()
        kk[0, key] = 2.0
        want = O.chunk_attention(q.cpu().to(F64), kk[0].cpu().to(F64), v_[0], 0.25, size)
        seen = [i for i in range(key, L) if i // size == key // size]
        assert (want[seen] - v_[0, key]).abs().max() < 1e-3                  # (the key decides)
        hidden = [i for i in range(L) if i not in seen]
        assert not hidden or (want[hidden] - v_[0, key]).abs().amax(dim=(1, 2)).min() > 0.1
        got = seq_ops.flash(q.view(L, -1), kk.view(L, -1), v.view(L, -1), torch.zeros(1, dtype=torch.int64, device="cuda"), None, 0.25, H,
                            batch([L], [0]), G, size)
        close(got, want.reshape(L, -1), BF16)
        for at, n in ((key, 1), (max(0, key - 1), 3), (min(L - 2, seen[-1]), 2), (seen[-1], 1), (min(L - 1, seen[-1] + 1), 1)):
            n = min(n, L - at)
            got = seq_ops.kv_attn(q[at:at + n].contiguous(), kk, v, 0.25, batch([n], [0], [at]), size)
            close(got, want[at:at + n].reshape(n, -1), BF16)


def test_bad_arguments_raise():
    z = lambda *s, dtype=BF16: torch.zeros(s, dtype=dtype, device="cuda")
    f = lambda n: z(n, dtype=F32)
    b = batch([2], [0])
    with pytest.raises(ValueError):
        seq_ops.rms_residual(z(2, 8, dtype=F32), BF16, z(2, 8), f(7), 1e-5)
    with pytest.raises(ValueError):                            # the cache does not hold the step's tokens
        seq_ops.kv_attn(z(2, 1, 8), z(1, 1, 1, 8), z(1, 1, 1, 8), 1.0, b)
    with pytest.raises(ValueError):
        seq_ops.kv_attn(z(2, 3, 8), z(1, 4, 2, 8), z(1, 4, 2, 8), 1.0, b)
    with pytest.raises(_lib.MsaError):
        seq_ops.kv_attn(z(2, 2, 12), z(1, 4, 2, 12), z(1, 4, 2, 12), 1.0, b, split=True)
    with pytest.raises(ValueError):
        seq_ops.delta(z(2, 24), z(2, 8), z(2, 1), z(2, 8), f(1), f(8), f(8), 1e-5, 1, 1, 8, 8, z(1, 1, 8, 7, dtype=F32), b)
    with pytest.raises(_lib.MsaError):
        seq_ops.delta(z(2, 18), z(2, 6), z(2, 1), z(2, 6), f(1), f(6), f(6), 1e-5, 1, 1, 6, 6, z(1, 1, 6, 6, dtype=F32), b, chunked=True)
    with pytest.raises(ValueError):
        seq_ops.qk_rope_append(z(2, 8), f(8), z(5, dtype=F64), 1e-5, z(1, 4, 1, 8), z(1, 4, 1, 8), b)
