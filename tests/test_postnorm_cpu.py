"""CPU tests of the output-normed decoder's host side (configuration, weights, registry, shared caches) and pins of its plain
mechanisms against independent formulations."""
import json
import math

import pytest
import torch

from hybrid_models import save_model
from msa_amd import registry, seq_ops
from msa_amd.config import ClampedGLUConfig, PostNormConfig, RotaryConfig
from msa_amd.postnorm import PostNormForCausalLM
from oracle import delta_attention_layers as O
from postnorm_models import ATTN, CONFIGS, DELTA, RANKS, config, layer, random_weights, tensor_shapes


def rnd(*shape, seed=0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_config_reads_every_key_and_refuses_others():
    c = PostNormConfig.from_dict(CONFIGS["mixed"])
    assert c.layers[0].mixer.rot.scaling.original == 300 and c.layers[2].mixer.kv_from == 0 and c.layers[2].mixer.mask.size == 31
    assert c.layers[1].mixer.conv_channels == 2 * 3 * 40 + 6 * 24 and c.layers[3].mlp is None and c.layers[4].mlp == ClampedGLUConfig(104, limit=0.7)
    assert c.runs == [(i, None) for i in range(5)]
    for change, match in (({"sink": True}, "unknown keys .*sink"), ({"rot": {"base": 1.0, "dims": 3}}, "rotated"),
                          ({"rot": {"base": 1.0, "dims": 48}}, "rotated"), ({"mask": {"size": 0}}, "chunks of 0"),
                          ({"mask": {"window": 4}}, "unknown keys"), ({"heads": 5}, "heads over")):
        with pytest.raises(ValueError, match=match):
            PostNormConfig.from_dict(config([layer("attention", {**ATTN, **change})]))
    with pytest.raises(ValueError, match="missing keys .*scale"):
        PostNormConfig.from_dict(config([layer("attention", {k: v for k, v in ATTN.items() if k != "scale"})]))
    with pytest.raises(ValueError, match="missing keys .*limit"):
        PostNormConfig.from_dict(config([{**layer("channel_delta", DELTA), "mlp": {"kind": "dense", "ff": 8}}]))
    with pytest.raises(NotImplementedError, match="feed-forward"):
        PostNormConfig.from_dict(config([{**layer("channel_delta", DELTA), "mlp": {"kind": "experts", "ff": 8, "limit": 1.0}}]))
    for j, what in ((1, "no keys"), (2, "no keys"), (-1, "no keys"), (5, "no keys")):          # itself, another kind, a sharer, nowhere
        with pytest.raises(ValueError, match=what):
            PostNormConfig.from_dict(config([layer("attention", ATTN), layer("channel_delta", DELTA), layer("attention", ATTN, kv_from=0),
                                             layer("attention", ATTN, kv_from=j)]))
    with pytest.raises(ValueError, match="heads differ"):
        PostNormConfig.from_dict(config([layer("attention", ATTN), layer("attention", ATTN, kv_from=0, kv_heads=3)]))


def test_frequencies():
    assert RotaryConfig(1e4, 8).frequencies() == pytest.approx([1.0, 0.1, 0.01, 0.001])
    s = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}
    got = RotaryConfig(5e5, 128, s).frequencies()
    assert got == pytest.approx(O.rotary_frequencies(5e5, 128, s), rel=1e-14)
    plain = RotaryConfig(5e5, 128).frequencies()
    turns = [8192 * f / (2 * math.pi) for f in plain]
    for f, p, t in zip(got, plain, turns):
        assert f == pytest.approx(p) if t > 4 else f == pytest.approx(p / 8) if t < 1 else p / 8 <= f <= p
    assert any(1 < t < 4 for t in turns) and any(t < 1 for t in turns) and any(t > 4 for t in turns)
    assert RotaryConfig(1e4, 0).frequencies() == []


@pytest.mark.parametrize("name", list(CONFIGS))
def test_registry_loads_the_weights(tmp_path, name):
    cfg = CONFIGS[name]
    w = random_weights(tensor_shapes(cfg, RANKS[name]))
    save_model(tmp_path / name, cfg, w)
    m = registry.load_model(str(tmp_path / name), torch.float32, "cpu")
    assert isinstance(m, PostNormForCausalLM) and len(m.layers) == len(cfg["layers"])
    for i, l in enumerate(m.layers):
        if cfg["layers"][i]["mlp"] is not None:
            assert torch.equal(l.w_gate_up[0::2], w[f"l{i}.mlp.gate"].float()) and torch.equal(l.w_gate_up[1::2], w[f"l{i}.mlp.up"].float())
        if cfg["layers"][i]["type"] == "channel_delta":
            x = l.mixer
            assert torch.equal(x.w_in[x.b_at:x.b_at + x.c.heads], w[f"l{i}.mix.b"].float()) and x.a_at % 8 == x.g_at % 8 == x.b_at % 8 == x.n_a % 32 == 0
            h = rnd(3, cfg["width"]).float()
            low = h @ x.w_in[x.a_at:x.g_at].T @ x.w_low[:x.n_a].T
            assert torch.allclose(low[:, :x.c.heads * x.c.dim], h @ w[f"l{i}.mix.a1"].float().T @ w[f"l{i}.mix.a2"].float().T, atol=1e-5)
            gate = h @ x.w_in[x.g_at:x.b_at].T @ x.w_low[x.n_a:].T
            assert torch.allclose(gate, h @ w[f"l{i}.mix.g1"].float().T @ w[f"l{i}.mix.g2"].float().T, atol=1e-5)
    bad = dict(w)
    del bad["l0.norm1"]
    save_model(tmp_path / "short", cfg, bad)
    with pytest.raises(KeyError, match="l0.norm1"):
        registry.load_model(str(tmp_path / "short"), torch.float32, "cpu")


def test_ranks_come_from_the_weights_and_have_to_agree(tmp_path):
    cfg = config([layer("channel_delta", DELTA)])
    w = random_weights(tensor_shapes(cfg, (9, 33)))
    w["l0.mix.a2"] = w["l0.mix.a2"][:, :8]
    save_model(tmp_path / "m", cfg, w)
    with pytest.raises(ValueError, match="l0.mix.a2"):
        registry.load_model(str(tmp_path / "m"), torch.float32, "cpu")


def test_shared_layers_read_their_sources_cache():
    cfg = CONFIGS["mixed"]
    m = PostNormForCausalLM.from_tensors(PostNormConfig.from_dict(cfg), random_weights(tensor_shapes(cfg, RANKS["mixed"])), torch.float32, "cpu")
    cache = m.create_cache(slots=2, capacity=9)
    assert cache.tensors[2] == {} and set(cache.tensors[0]) == {"k", "v"} and cache.tensors[0]["k"].shape == (2, 9, 2, 40)
    assert cache.tensors[1]["delta"].shape == (2, 6, 40, 24) and cache.tensors[1]["conv"].shape == (2, 2, 384)
    for r in (2, 4):
        assert m.run_state(cache, r)["k"] is cache.tensors[0]["k"]
    assert m.run_state(cache, 1) is cache.tensors[1]
    cache.reserve(20)                                          # growing replaces the tensors: sharers follow
    assert m.run_state(cache, 4)["v"] is cache.tensors[0]["v"] and cache.tensors[0]["v"].shape[1] == 20


def test_interleaved_pairs():
    g, u = rnd(5, 3), rnd(5, 3, seed=1)
    w = seq_ops.interleave_pairs(g, u)
    assert w.shape == (10, 3) and torch.equal(w[0::2], g) and torch.equal(w[1::2], u)


# ------------------------------------------------------------------------------------------------ pins of the plain mechanisms
def test_delta_rule_is_a_regression_step_and_carries_its_state():
    T, H, D, E = 9, 2, 5, 4
    q, k, v, la, b = O.unit(rnd(T, H, D)), O.unit(rnd(T, H, D, seed=1)), rnd(T, H, E, seed=2), -rnd(T, H, D, seed=3).abs(), torch.sigmoid(rnd(T, H, seed=4))
    o, S = O.delta_rule(q, k, v, la, b)
    o1, S1 = O.delta_rule(q[:4], k[:4], v[:4], la[:4], b[:4])
    o2, S2 = O.delta_rule(q[4:], k[4:], v[4:], la[4:], b[4:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    # as products of transition matrices: S_t = (1 - b k k^T) diag(g) S + b k v^T
    for h in range(H):
        M = torch.zeros(D, E, dtype=torch.float64)
        for t in range(T):
            kk = k[t, h][:, None]
            M = (torch.eye(D, dtype=torch.float64) - b[t, h] * kk @ kk.T) @ torch.diag(torch.exp(la[t, h])) @ M + b[t, h] * kk @ v[t, h][None]
            assert torch.allclose(M.T @ q[t, h], o[t, h])
    # full step, no decay: the state answers the last key with the last value, whatever was there
    o, S = O.delta_rule(k, k, v, torch.zeros_like(la), torch.ones_like(b))
    assert torch.allclose(o[-1], v[-1], atol=1e-5)


def test_chunk_attention_is_softmax_over_the_chunk():
    L, T, H, G, D, E = 11, 4, 6, 2, 3, 5
    q, k, v = rnd(T, H, D), rnd(L, G, D, seed=1), rnd(L, G, E, seed=2)
    for size in (None, 1, 4, 20):
        out = O.chunk_attention(q, k, v, 0.7, size)
        for t in range(T):
            i = L - T + t
            seen = [j for j in range(i + 1) if size is None or j // size == i // size]
            for h in range(H):
                p = torch.softmax(k[seen, h // 3] @ q[t, h] * 0.7, 0)
                assert torch.allclose(out[t, h], p @ v[seen, h // 3])


def test_rotation_depends_on_distance():
    fr = O.rotary_frequencies(100.0, 6)
    q, k = rnd(1, 1, 8), rnd(1, 1, 8, seed=1)
    dot = lambda a, b: (O.rotate(q, [a], fr) * O.rotate(k, [b], fr)).sum()
    assert torch.allclose(dot(5, 2), dot(105, 102)) and not torch.allclose(dot(5, 2), dot(5, 3))
    assert torch.equal(O.rotate(q, [7], fr)[..., 6:], q[..., 6:]) and torch.allclose(O.rotate(q, [0], fr), q)
    x = O.rotate(torch.tensor([[[1.0, 0, 0, 0]]], dtype=torch.float64), [2], [0.5, 0.1])
    assert torch.allclose(x[0, 0], torch.tensor([math.cos(1.0), 0, math.sin(1.0), 0], dtype=torch.float64))


def test_clamped_unit_and_head_norm():
    g, u = rnd(50) * 3, rnd(50, seed=1) * 3
    want = []
    for x, y in zip(g.tolist(), u.tolist()):
        x, y = min(x, 1.5), max(-1.5, min(1.5, y))
        want.append(x / (1 + math.exp(-1.702 * x)) * (y + 1))
    assert torch.allclose(O.clamped_glu(g, u, 1.5), torch.tensor(want, dtype=torch.float64))
    o = rnd(3, 2, 8)
    y = O.gated_head_norm(o, torch.ones(8, dtype=torch.float64), torch.full((3, 2, 8), 50.0, dtype=torch.float64), 0.0)
    assert torch.allclose((y * y).mean(-1), torch.ones(3, 2, dtype=torch.float64))


def test_plain_forward_is_causal():
    cfg = CONFIGS["mixed"]
    w = random_weights(tensor_shapes(cfg, RANKS["mixed"]))
    toks = torch.randint(0, cfg["vocab"], (60,), generator=torch.Generator().manual_seed(1)).tolist()
    whole = O.forward(cfg, w, toks)
    assert torch.allclose(O.forward(cfg, w, toks[:23]), whole[:23])
    trace = []
    O.forward(cfg, w, toks[:5], trace)
    assert len(trace) == 5 and json.dumps(cfg)
