"""CPU tests of the hybrid decoder's host side (configuration, weight files, registry, state cache, weight packing) and pins of
its oracle's mechanisms against independent formulations."""
import json

import pytest
import torch

from hybrid_models import CONFIGS, GRU, config, layer, random_weights, save_model, tensor_shapes
from msa_amd import registry, seq_ops
from msa_amd.cache import SequenceStateCache, StateSpec
from msa_amd.config import HybridConfig
from msa_amd.weights import SafetensorsFile, load_tensors
from oracle import recurrent_layers as R


def test_config_runs_and_errors():
    c = HybridConfig.from_dict(CONFIGS["mixed"])
    assert c.runs == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (1, 2), (2, 2), (3, None)] == R.layer_runs(CONFIGS["mixed"])
    assert HybridConfig.from_dict(CONFIGS["ones"]).runs == [(0, None), (1, None), (2, None)]
    bad = json.loads(json.dumps(CONFIGS["mixed"]))
    bad["layers"][0]["mixer"]["window"] = 4
    with pytest.raises(ValueError, match=r"layers\[0\].mixer.*window"):
        HybridConfig.from_dict(bad)
    with pytest.raises(NotImplementedError, match="mixer 'conv'"):
        HybridConfig.from_dict(config([layer("conv", GRU)]))
    with pytest.raises(NotImplementedError, match="feed-forward"):
        HybridConfig.from_dict(config([{**layer("mingru", GRU), "mlp": {"kind": "moe", "ff": 8}}]))
    with pytest.raises(ValueError, match="loop"):
        HybridConfig.from_dict(config([layer("mingru", GRU)], loop={"start": 0, "stop": 2, "times": 1}))
    with pytest.raises(ValueError, match="missing|required"):
        HybridConfig.from_dict(config([layer("mingru", {})]))


def test_safetensors_reader(tmp_path):
    w = {"a": torch.randn(3, 5).to(torch.bfloat16), "b": torch.arange(6, dtype=torch.int32).view(2, 3), "c": torch.tensor(1.5),
         "d": torch.zeros(0, 4)}
    save_model(tmp_path, {}, w)
    got = load_tensors(str(tmp_path))
    assert set(got) == set(w)
    for n, t in w.items():
        assert got[n].dtype == t.dtype and got[n].shape == t.shape and torch.equal(got[n], t)
    f = SafetensorsFile(str(tmp_path / "model.safetensors"))
    assert "a" in f and "x" not in f
    with pytest.raises(KeyError):
        f["x"]
    from safetensors.torch import load_file, save_file           # the format as others write it
    save_file({"q": w["a"]}, str(tmp_path / "model.safetensors"))
    assert torch.equal(load_tensors(str(tmp_path))["q"], w["a"])
    (tmp_path / "model.safetensors").write_bytes(b"\xff" * 32)
    with pytest.raises(ValueError, match="not a safetensors"):
        load_tensors(str(tmp_path))


def test_registry_picks_the_model(tmp_path):
    assert registry.architecture(CONFIGS["mixed"]) == "Gevonex"
    assert registry.architecture({"architectures": ["MSAForCausalLM"]}) == "MSAForCausalLM"
    with pytest.raises(NotImplementedError, match="unknown architecture"):
        registry.architecture({"architecture": "Other"})
    from msa_amd.config import MSAConfig
    from msa_amd.model import MSAForCausalLM
    small = dict(hidden_size=64, num_hidden_layers=1, num_attention_heads=1, num_key_value_heads=1, head_dim=128, intermediate_size=64,
                 vocab_size=50, msa_config={"router_layer_idx": "0", "decouple_router": True, "top_k_docs": 2, "pooling_kernel_size": 8})
    want = MSAForCausalLM(MSAConfig(**small)).init_random(seed=3).to(torch.bfloat16)
    save_model(tmp_path / "m", {"architectures": ["MSAForCausalLM"], **small}, dict(want.state_dict()))
    got = registry.load_model(str(tmp_path / "m"), torch.bfloat16, "cpu")
    assert isinstance(got, MSAForCausalLM)
    for (n, a), (_, b) in zip(want.state_dict().items(), got.state_dict().items()):
        assert torch.equal(a, b), n


@pytest.mark.parametrize("name", list(CONFIGS))
def test_registry_loads_hybrid_weights(tmp_path, name):
    cfg = CONFIGS[name]
    w = random_weights(tensor_shapes(cfg))
    save_model(tmp_path / name, cfg, w)
    m = registry.load_model(str(tmp_path / name), torch.float32, "cpu")
    assert m.config.width == cfg["width"] and len(m.layers) == len(cfg["layers"])
    assert torch.equal(m.layers[0].w_gate, w["l0.rg1"].float())
    del w["l0.rg1.b"]
    save_model(tmp_path / "short", cfg, w)
    with pytest.raises(KeyError, match="l0.rg1.b"):
        registry.load_model(str(tmp_path / "short"), torch.float32, "cpu")
    w["l0.rg1.b"] = torch.zeros(3)
    save_model(tmp_path / "bent", cfg, w)
    with pytest.raises(ValueError, match="l0.rg1.b"):
        registry.load_model(str(tmp_path / "bent"), torch.float32, "cpu")


def test_state_cache_slots_growth_and_reuse():
    specs = [{"s": StateSpec((3,), torch.float32), "rows": StateSpec((2,), torch.float32, per_token=True)}] * 2
    c = SequenceStateCache(specs, "cpu", slots=2, capacity=4)
    a, b = c.open("a"), c.open("b")
    assert {a, b} == {0, 1}
    with pytest.raises(KeyError):
        c.open("a")
    c.tensors[1]["s"][a] = 7.0
    c.tensors[0]["rows"][b, 3] = 5.0
    d = c.open("d")                                    # no slot left: doubled, contents kept
    assert d == 2 and c.slots == 4 and c.tensors[1]["s"].shape == (4, 3)
    assert torch.all(c.tensors[1]["s"][a] == 7) and torch.all(c.tensors[0]["rows"][b, 3] == 5)
    c.advance("b", 4)
    c.reserve(9)
    assert c.capacity == 9 and c.tensors[0]["rows"].shape == (4, 9, 2) and torch.all(c.tensors[0]["rows"][b, 3] == 5)
    c.reserve(10)
    assert c.capacity == 13                            # grows by half at least
    c.close("a")
    assert "a" not in c.length
    got = [c.open(i) for i in range(2)]
    assert a in got and torch.all(c.tensors[1]["s"][a] == 0)      # the slot comes back cleared


def test_step_batch_describes_rows():
    b = seq_ops.StepBatch([3, 1, 2], [4, 0, 2], [10, 0, 5], "cpu")
    assert b.cu.tolist() == [0, 3, 4, 6] and b.row_seq.tolist() == [0, 0, 0, 1, 2, 2] and b.slot.tolist() == [4, 0, 2]
    assert b.pos.tolist() == [10, 0, 5] and (b.rows, b.max_rows, b.max_keys) == (6, 3, 13)
    for counts, slots in (([], []), ([0], [0]), ([1, 1], [2, 2])):
        with pytest.raises(ValueError):
            seq_ops.StepBatch(counts, slots, [0] * len(counts), "cpu")


def test_interleaved_gru_rows():
    n, K = 21, 4
    z, u, g = (torch.full((n, K), float(i)) + torch.arange(n).view(n, 1) / 100 for i in (1, 2, 3))
    w = seq_ops.interleave_gru(z, u, g)
    assert w.shape == (2 * 48, K)
    for c in range(n):
        at = c // 16 * 48 + c % 16
        assert torch.equal(w[at], z[c]) and torch.equal(w[at + 16], u[c]) and torch.equal(w[at + 32], g[c])
    assert torch.all(w[48 + 5:48 + 16] == 0)


# ------------------------------------------------------------------------------------------------ oracle pins
def rnd(*shape, seed=0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_oracle_norms_and_activations():
    x = rnd(5, 12)
    assert torch.allclose(R.rms(x, 1e-5), torch.nn.functional.rms_norm(x, (12,), eps=1e-5))
    assert torch.allclose(R.gelu_tanh(x), torch.nn.functional.gelu(x, approximate="tanh"))
    assert torch.allclose(R.softplus(x * 40), torch.nn.functional.softplus(x * 40), atol=1e-12)
    y = R.gated_group_norm(x, rnd(5, 12, seed=1), torch.ones(12, dtype=torch.float64), 3, 0.0)
    assert torch.allclose((y.view(5, 3, 4) ** 2).mean(-1), torch.ones(5, 3, dtype=torch.float64))


def test_oracle_convolution_and_shift():
    x, taps, b = rnd(9, 4), rnd(4, 3, seed=1), rnd(4, seed=2)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (2, 0)), taps[:, None], b, groups=4)[0].T
    assert torch.allclose(R.causal_conv(x, taps, b), want)
    mix = torch.tensor([0.0, 1.0, 0.5, 0.25], dtype=torch.float64)
    y = R.token_shift(x, mix)
    assert torch.equal(y[:, 0], x[:, 0]) and torch.allclose(y[1:, 1], x[:-1, 1]) and y[0, 1] == 0
    assert torch.allclose(y[0], x[0] * (1 - mix))
    assert torch.allclose(torch.cat([R.token_shift(x[:4], mix), R.token_shift(x[4:], mix, x[3])]), y)


def test_oracle_recurrences_have_their_closed_forms():
    T, H, P, N, G = 7, 4, 3, 5, 2
    x, B, C, dt = rnd(T, H, P), rnd(T, G, N, seed=1), rnd(T, G, N, seed=2), rnd(T, H, seed=3).abs()
    A_log, D = rnd(H, seed=4), rnd(H, seed=5)
    y, S = R.ssd_scan(x, B, C, dt, A_log, D)
    for h in range(H):
        la = torch.cumsum(-torch.exp(A_log[h]) * dt[:, h], 0)
        M = torch.tril(torch.exp(la[:, None] - la[None, :])) * (C[:, h // 2] @ B[:, h // 2].T) * dt[:, h]
        assert torch.allclose(y[:, h], M @ x[:, h] + D[h] * x[:, h])
    y2, S2 = R.ssd_scan(x[3:], B[3:], C[3:], dt[3:], A_log, D, R.ssd_scan(x[:3], B[:3], C[:3], dt[:3], A_log, D)[1])
    assert torch.allclose(y2, y[3:]) and torch.allclose(S2, S)
    z, u = torch.sigmoid(rnd(T, 6)), rnd(T, 6, seed=1)
    S = R.min_gru(z, u)
    keep = torch.cumprod(1 - z, 0)
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    assert torch.allclose(S[-1], sum(keep[-1] / keep[t] * z[t] * cand[t] for t in range(T)))


def test_oracle_sink_is_a_key_without_a_value():
    T, L, H, D, E = 4, 9, 3, 5, 6
    q, k, v, sink = rnd(T, H, D), rnd(L, H, D, seed=1), rnd(L, H, E, seed=2), rnd(H, seed=3) * 3
    out = R.sink_attention(q, k, v, sink, 0.7)
    for t in range(T):
        n = L - T + t + 1
        s = torch.einsum("hd,jhd->hj", q[t], k[:n]) * 0.7
        p = torch.softmax(torch.cat([s, sink[:, None]], 1), 1)[:, :n]
        assert torch.allclose(out[t], torch.einsum("hj,jhe->he", p, v[:n]))
    far = R.sink_attention(q, k, v, torch.full((H,), 60.0, dtype=torch.float64), 0.7)
    assert far.abs().max() < 1e-12
