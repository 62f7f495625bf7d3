"""The output-normed decoder on the GPU against oracle/delta_attention_layers.py: whole prompts, token by token, portions, ragged
batches, slots used again, chunk borders, long decoding, greedy generation, and the trace runner."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

from hybrid_models import save_model
from msa_amd import seq_ops
from msa_amd.config import PostNormConfig
from msa_amd.postnorm import PostNormForCausalLM
from oracle import delta_attention_layers as O
from postnorm_models import ATTN, CONFIGS, DELTA, RANKS, config, layer, random_weights, tensor_shapes

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [pytest.param(F32, id="f32"), pytest.param(BF16, id="bf16")]
_made = {}


def build(cfg, w, dtype):
    return PostNormForCausalLM.from_tensors(PostNormConfig.from_dict(cfg), w, dtype, "cuda:0")


def made(name, dtype):
    """(config, weights, model), built once."""
    if (name, "w") not in _made:
        _made[name, "w"] = random_weights(tensor_shapes(CONFIGS[name], RANKS[name]), seed=len(name))
    if (name, dtype) not in _made:
        _made[name, dtype] = build(CONFIGS[name], _made[name, "w"], dtype)
    return CONFIGS[name], _made[name, "w"], _made[name, dtype]


def oracle_logits(name, tokens):
    key = (name, tuple(tokens))
    if key not in _made:
        _made[key] = O.forward(CONFIGS[name], _made[name, "w"], tokens)
    return _made[key]


def tokens_for(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def check(got, want, dtype):
    """Logits with their mean taken off, rms over the vocabulary relative to the logits' own size.  In bf16 a position whose sublayer
    output happens to be small has its rounding blown up by the norm behind it: one in thirty may be three times as far off."""
    d = got.cpu().double() - want
    d = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()
    scale = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    err, lim = d / scale, 4e-5 if dtype == F32 else 0.06
    far = int((err > lim).sum())
    assert err.max() < (lim if dtype == F32 else 3 * lim) and far <= max(1, d.numel() // 30), \
        f"error {err.max():.3e} (worst of {d.numel()} positions: {int(d.argmax())}), {far} over {lim}"


def feed(model, cache, key, tokens, sizes):
    """Portions of ``sizes`` in turn; the logits of every token."""
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(sizes[i % len(sizes)], len(tokens) - at)
        out.append(model.step(cache, [(key, tokens[at:at + n], list(range(n)))]))
        at, i = at + n, i + 1
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_layers(name, dtype):
    cfg, w, m = made(name, dtype)
    toks = tokens_for(cfg, 150)
    want = oracle_logits(name, toks)
    check(feed(m, m.create_cache(), "a", toks, [150]), want, dtype)
    check(feed(m, m.create_cache(), "a", toks[:1], [1]), want[:1], dtype)
    trace_want, trace = [], []
    O.forward(cfg, w, toks[:40], trace_want)
    c = m.create_cache()
    b = seq_ops.StepBatch([40], [c.open("a")], [0], m.device)
    m.forward_rows(torch.tensor(toks[:40]).cuda(), b, c, [], trace)
    assert len(trace) == len(trace_want) == len(m.runs)
    for got, ref in zip(trace, trace_want):
        check(got, ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("sizes", [[1], [2], [64, 1, 17], [3, 65, 1, 2, 16]], ids=str)
def test_portions_equal_the_whole(name, dtype, sizes):
    cfg, w, m = made(name, dtype)
    toks = tokens_for(cfg, 150)
    check(feed(m, m.create_cache(), "a", toks, sizes), oracle_logits(name, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
def test_unequal_batch_equals_each_alone(name, dtype):
    """Prompts of very different lengths in one step, then steps that mix decoding with portions, joiners and leavers."""
    cfg, w, m = made(name, dtype)
    seqs = {k: tokens_for(cfg, n, seed=n) for k, n in (("a", 150), ("b", 5), ("c", 37), ("d", 90), ("e", 2))}
    c = m.create_cache()
    plan = [[("a", 80), ("b", 1), ("c", 30)], [("a", 1), ("b", 1), ("c", 1)], [("d", 65), ("b", 2), ("a", 30)],
            [("b", 1), ("e", 1), ("c", 6), ("d", 1)], [("e", 1), ("d", 24), ("a", 39)]]
    at = dict.fromkeys(seqs, 0)
    for step in plan:
        entries = [(k, seqs[k][at[k]:at[k] + n], [0, n - 1] if n > 1 else [0]) for k, n in step]
        got = m.step(c, entries)
        want = torch.cat([oracle_logits(name, seqs[k])[[at[k] + j for j in e[2]]] for (k, n), e in zip(step, entries)])
        check(got, want, dtype)
        for k, n in step:
            at[k] += n
            if at[k] == len(seqs[k]):
                c.close(k)
    assert at == {k: len(s) for k, s in seqs.items()} and not c.slot_of


@pytest.mark.parametrize("dtype", DTYPES)
def test_twenty_sequences_decode_together(dtype):
    """More rows than the weight-streaming form takes."""
    cfg, w, m = made("mixed", dtype)
    toks = [tokens_for(cfg, 6, seed=100 + i) for i in range(20)]
    c = m.create_cache()
    for t in range(6):
        got = m.step(c, [(i, toks[i][t:t + 1], [0]) for i in range(20)])
        check(got, torch.stack([oracle_logits("mixed", toks[i])[t] for i in range(20)]), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_slots_are_used_again_and_the_cache_grows(dtype):
    cfg, w, m = made("mixed", dtype)
    c = m.create_cache(slots=1, capacity=8)
    first = tokens_for(cfg, 150)
    feed(m, c, "old", first, [100, 1])
    slot = c.slot_of["old"]
    c.close("old")
    toks = tokens_for(cfg, 37, seed=37)
    got = feed(m, c, "new", toks, [2, 1, 20])
    assert c.slot_of["new"] == slot and c.slots == 1 and c.capacity >= 150
    check(got, oracle_logits("mixed", toks), dtype)
    other = feed(m, c, "other", first, [33])               # a second slot appears beside a live sequence
    check(other, oracle_logits("mixed", first), dtype)
    more = tokens_for(cfg, 40, seed=1)
    check(feed(m, c, "new", more, [1]), oracle_logits("mixed", toks + more)[37:], dtype)


@pytest.mark.parametrize("name", ["mixed", "ones"])
def test_long_decoding(name):
    """Hundreds of single tokens from states and caches alone, over many chunk borders."""
    cfg, w, m = made(name, BF16)
    toks = tokens_for(cfg, 420, seed=4)
    want = oracle_logits(name, toks)
    check(feed(m, m.create_cache(), "a", toks, [1]), want, BF16)
    check(feed(m, m.create_cache(), "a", toks, [420]), want, BF16)
    m32 = made(name, F32)[2]
    check(feed(m32, m32.create_cache(), "a", toks, [300, 1]), want, F32)


def spread(rows):
    return (rows - rows.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt().max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shared", [False, True])
def test_a_chunk_border_shows(dtype, shared):
    """Queries and keys of one head all point along the token's first channel, which one token has with the other sign: wherever it is
    seen it decides the logits, and a token behind the border must not see it.  A layer with shared keys has borders of its own."""
    size, D = 40, 16
    att = {"heads": 1, "kv_heads": 1, "dim": D, "vdim": D, "scale": 3.0, "mask": {"size": size}, "rot": {"base": 1e5, "dims": 4}}
    layers = [layer("attention", att, None)] + ([layer("attention", att, None, kv_from=0, mask={"size": 25})] if shared else [])
    cfg = config(layers, width=64, vocab=50)
    w = random_weights(tensor_shapes(cfg), seed=3)
    w["embed"][:, 0] = -1.0
    w["embed"][7, 0] = 1.0
    for i in range(len(layers)):
        for n in ("q", "k"):
            if f"l{i}.mix.{n}" in w:
                w[f"l{i}.mix.{n}"] = torch.zeros_like(w[f"l{i}.mix.{n}"])
                w[f"l{i}.mix.{n}"][D - 1, 0] = 1.0 if n == "k" else 0.0
                w[f"l{i}.mix.{n}.norm"] = torch.ones(D, dtype=BF16)
        w[f"l{i}.mix.q"][D - 1, 0] = -1.0
    m = build(cfg, w, dtype)
    plain = [t for t in tokens_for(cfg, 130, seed=6)]
    plain = [t if t != 7 else 8 for t in plain]
    base = O.forward(cfg, w, plain)
    for at in (0, size - 1, size, 2 * size - 1, 2 * size, 49, 50):
        toks = plain[:at] + [7] + plain[at + 1:]
        want = O.forward(cfg, w, toks)
        changed = [(want[i] - base[i]).abs().max().item() > 1e-9 for i in range(130)]
        last = max(i for i in range(130) if changed[i])
        reach = max((at // n + 1) * n - 1 for n in ((size, 25) if shared else (size,)))
        assert last == reach                                   # the borders, and only they, end the token's reach
        assert spread(want[last] - base[last]) > 0.15 * spread(base[last])
        for sizes in ([130], [1], [at + 1, 1], [max(1, last), 2], [last + 1, 2], [33, 2]):
            check(feed(m, m.create_cache(), "a", toks, sizes), want, dtype)


@pytest.mark.parametrize("name", ["mixed", "wide", "odd"])
def test_greedy_generation(name):
    """Left-padded prompts through generate_greedy: tokens agree with the oracle's argmax wherever that is clear, graph replays
    equal eager decoding, and decoding can go on from the cache."""
    cfg, w, m = made(name, BF16)
    prompts = [tokens_for(cfg, n, seed=n) for n in (9, 40, 2)]
    S, n_new = 40, 24
    ids, mask = torch.zeros(3, S, dtype=torch.long), torch.zeros(3, S, dtype=torch.long)
    for b, p in enumerate(prompts):
        ids[b, S - len(p):] = torch.tensor(p)
        mask[b, S - len(p):] = 1
    eager, cache = m.generate_greedy(ids, mask, n_new)
    graph, _ = m.generate_greedy(ids, mask, n_new, use_graph=True)
    assert torch.equal(eager, graph)
    for b, p in enumerate(prompts):
        toks = p + eager[b].tolist()
        want = O.forward(cfg, w, toks)
        for i in range(n_new):
            row = want[len(p) - 1 + i]
            size = (row - row.mean()).pow(2).mean().sqrt()
            top = row.topk(2).values
            if top[0] - top[1] > 0.3 * size:
                assert int(row.argmax()) == toks[len(p) + i], (b, i)
            else:
                assert row.max() - row[toks[len(p) + i]] < 0.3 * size
        assert cache.length[b] == len(toks) - 1
        check(m.step(cache, [(b, toks[-1:], [0])]), want[-1:], BF16)


def test_step_refuses_bad_entries():
    cfg, w, m = made("ones", F32)
    c = m.create_cache()
    for entry in (("a", [], []), ("a", [1], [1]), ("a", [cfg["vocab"]], [0]), ("a", [-1], [])):
        with pytest.raises(ValueError):
            m.step(c, [entry])
    assert not c.slot_of and m.step(c, [("a", [1, 2], [])]) is None and c.length["a"] == 2


def test_new_mixers_inside_gated_residuals():
    """The mixers belong to the framework, not to one layer kind: a gated-residual decoder runs them too, in all its forms."""
    import hybrid_models as H
    from msa_amd.config import HybridConfig
    from msa_amd.hybrid import HybridForCausalLM
    from oracle import recurrent_layers as R
    cfg = H.config([H.layer("channel_delta", DELTA), H.layer("attention", ATTN), H.layer("mingru", H.GRU)])
    shapes = {n: tuple({"a_rank": 11, "g_rank": 20}.get(d, d) for d in s) for n, s in HybridForCausalLM(HybridConfig.from_dict(cfg)).tensor_shapes().items()}
    w = H.random_weights(shapes, seed=5)
    toks = tokens_for(cfg, 90, seed=2)
    wrap = lambda f: lambda w_, p, m_, eps, h: f(w_, p, m_, eps, h, {})
    R.MIXERS.update({n: wrap(f) for n, f in O.MIXERS.items()})
    try:
        want = R.forward(cfg, w, toks)
    finally:
        for n in O.MIXERS:
            del R.MIXERS[n]
    for dtype in (F32, BF16):
        m = HybridForCausalLM.from_tensors(HybridConfig.from_dict(cfg), w, dtype, "cuda:0")
        for sizes in ([90], [1], [70, 2, 1]):
            check(feed(m, m.create_cache(), "a", toks, sizes), want, dtype)


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(tmp_path, dtype):
    cfg, w, m = made("mixed", BF16)
    save_model(tmp_path / "model", cfg, w)
    a, b = tokens_for(cfg, 77, seed=77), tokens_for(cfg, 5, seed=5)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:70], "want": [0, 69]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": a[70:76], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[76:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "x", "tokens": b, "want": [4, 2]}], "end": ["x"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "77"], input="".join(json.dumps(s) + "\n" for s in steps), text=True, capture_output=True, timeout=200)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (tmp_path / "1.f32").exists()
    A, B = oracle_logits("mixed", a), oracle_logits("mixed", b)
    for i, want in ((0, A[[0, 69]]), (2, A[[76]]), (3, B[[4, 2]])):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", dtype="<f4")).view(-1, cfg["vocab"])
        check(got, want, getattr(torch, dtype))
