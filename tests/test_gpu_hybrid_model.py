"""The hybrid decoder on the GPU against oracle/recurrent_layers.py: whole prompts, token by token, portions, ragged batches,
slots used again, long decoding, greedy generation, and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

from hybrid_models import CONFIGS, config, layer, random_weights, save_model, tensor_shapes
from msa_amd.config import HybridConfig
from msa_amd.hybrid import HybridForCausalLM
from oracle import recurrent_layers as R

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [pytest.param(F32, id="f32"), pytest.param(BF16, id="bf16")]
_made = {}


def made(name, dtype):
    """(config, weights, model), built once."""
    if (name, "w") not in _made:
        _made[name, "w"] = random_weights(tensor_shapes(CONFIGS[name]), seed=len(name))
    cfg, w = CONFIGS[name], _made[name, "w"]
    if (name, dtype) not in _made:
        _made[name, dtype] = HybridForCausalLM.from_tensors(HybridConfig.from_dict(cfg), w, dtype, "cuda:0")
    return cfg, w, _made[name, dtype]


def oracle_logits(name, tokens):
    key = (name, tuple(tokens))
    if key not in _made:
        _made[key] = R.forward(CONFIGS[name], _made[name, "w"], tokens)
    return _made[key]


def tokens_for(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def check(got, want, dtype):
    """Logits with their mean taken off, rms over the vocabulary relative to the logits' own size."""
    d = got.cpu().double() - want
    d = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()
    scale = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    err = (d / scale).max().item()
    assert err < (2e-5 if dtype == F32 else 0.04), f"error {err:.3e} (worst of {d.numel()} positions: {int(d.argmax())})"


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
    R.forward(cfg, w, toks[:40], trace_want)
    from msa_amd import seq_ops
    c = m.create_cache()
    b = seq_ops.StepBatch([40], [c.open("a")], [0], m.device)
    m.forward_rows(torch.tensor(toks[:40]).cuda(), b, c, [], trace)
    assert len(trace) == len(trace_want) == len(m.runs)
    for got, ref in zip(trace, trace_want):
        assert (got.cpu().double() - ref).abs().max() < (2e-5 if dtype == F32 else 0.05) * ref.abs().max()


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
    whole = toks + more
    check(feed(m, c, "new", more, [1]), oracle_logits("mixed", whole)[37:], dtype)


@pytest.mark.parametrize("name", ["mixed", "ones"])
def test_long_decoding(name):
    """Hundreds of single tokens from the states alone."""
    cfg, w, m = made(name, BF16)
    toks = tokens_for(cfg, 420, seed=4)
    want = oracle_logits(name, toks)
    check(feed(m, m.create_cache(), "a", toks, [1]), want, BF16)
    check(feed(m, m.create_cache(), "a", toks, [420]), want, BF16)
    m32 = made(name, F32)[2]
    check(feed(m32, m32.create_cache(), "a", toks, [300, 1]), want, F32)


def test_a_far_token_shows():
    """The last token's query is pointed at the keys of two tokens: whichever of them starts the sequence decides the last
    logits, hundreds of tokens later.  A cache that lost or shifted its first row would not follow."""
    lat = {"heads": 2, "dim": 16, "vdim": 16, "kv_rank": 24, "scale": 0.25}
    cfg = config([layer("latent_attention", lat, None)], width=64, vocab=90)
    w = random_weights(tensor_shapes(cfg), seed=8)
    toks = [0] + [5, 9] * 129 + [11]
    f = {n: t.double() for n, t in w.items()}

    def mixer_input(seq):
        h = R.dyn_tanh(f["embed"][torch.tensor(seq)], f["l0.norm1.alpha"], f["l0.norm1"], f["l0.norm1.b"])
        return R.token_shift(h, f["l0.shift"])
    keys, aim = [], []
    for first in (3, 77):
        c = R.rms(mixer_input([first] + toks[1:]) @ f["l0.mix.dkv"].T, cfg["norm"]["eps"]) * f["l0.mix.dkv.norm"]
        keys.append((c @ f["l0.mix.uk"].T)[:, :16])
        aim.append(torch.tensor([1.0] + [0.0] * (len(toks) - 1)))
    point = torch.linalg.pinv(torch.cat(keys), rtol=1e-6) @ torch.cat(aim).double()    # one on the first keys, zero on the rest
    h = mixer_input(toks)[-1]
    w["l0.mix.q"][:16] += (16.0 / lat["scale"] * torch.outer(point, h / (h * h).sum())).to(BF16)
    for dtype in (F32, BF16):
        m = HybridForCausalLM.from_tensors(HybridConfig.from_dict(cfg), w, dtype, "cuda:0")
        last = []
        for first in (3, 77):
            seq = [first] + toks[1:]
            want = R.forward(cfg, w, seq)
            for sizes in ([260], [200, 1], [64, 2]):
                check(feed(m, m.create_cache(), "a", seq, sizes), want, dtype)
            last.append(want[-1])
        spread = (last[0] - last[0].mean()).pow(2).mean().sqrt()
        assert (last[0] - last[1]).abs().max() > 0.3 * spread          # the two must be told apart for the test to mean anything


@pytest.mark.parametrize("name", ["mixed", "wide", "odd"])
def test_greedy_generation(name):
    """Left-padded prompts through generate_greedy: tokens agree with the oracle's argmax wherever that is clear, graph replays
    equal eager decoding, and decoding can go on from the cache."""
    cfg, w, m = made(name, BF16)
    prompts = [tokens_for(cfg, n, seed=n) for n in (9, 30, 2)]
    S, n_new = 30, 14
    ids, mask = torch.zeros(3, S, dtype=torch.long), torch.zeros(3, S, dtype=torch.long)
    for b, p in enumerate(prompts):
        ids[b, S - len(p):] = torch.tensor(p)
        mask[b, S - len(p):] = 1
    eager, cache = m.generate_greedy(ids, mask, n_new)
    graph, _ = m.generate_greedy(ids, mask, n_new, use_graph=True)
    assert torch.equal(eager, graph)
    for b, p in enumerate(prompts):
        toks = p + eager[b].tolist()
        want = R.forward(cfg, w, toks)
        for i in range(n_new):
            row = want[len(p) - 1 + i]
            top = row.topk(2).values
            if top[0] - top[1] > 0.25 * (row - row.mean()).pow(2).mean().sqrt():
                assert int(row.argmax()) == toks[len(p) + i], (b, i)
            else:
                assert row.max() - row[toks[len(p) + i]] < 0.25 * (row - row.mean()).pow(2).mean().sqrt()
        assert cache.length[b] == len(toks) - 1
        check(m.step(cache, [(b, toks[-1:], [0])]), want[-1:], BF16)


def test_step_refuses_bad_entries():
    cfg, w, m = made("ones", F32)
    c = m.create_cache()
    for entry in (("a", [], []), ("a", [1], [1]), ("a", [cfg["vocab"]], [0]), ("a", [-1], [])):
        with pytest.raises(ValueError):
            m.step(c, [entry])
    assert not c.slot_of and m.step(c, [("a", [1, 2], [])]) is None and c.length["a"] == 2


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(tmp_path, dtype):
    cfg, w, m = made("mixed", BF16)
    save_model(tmp_path / "model", cfg, w)
    a, b = tokens_for(cfg, 37, seed=37), tokens_for(cfg, 5, seed=5)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": a[20:36], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[36:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "x", "tokens": b, "want": [4, 2]}], "end": ["x"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "37"], input="".join(json.dumps(s) + "\n" for s in steps), text=True, capture_output=True, timeout=200)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (tmp_path / "1.f32").exists()
    A, B = oracle_logits("mixed", a), oracle_logits("mixed", b)
    for i, want in ((0, A[[0, 19]]), (2, A[[36]]), (3, B[[4, 2]])):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", dtype="<f4")).view(-1, cfg["vocab"])
        check(got, want, getattr(torch, dtype))
