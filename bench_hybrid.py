"""Throughput of the hybrid decoder (state-space, minimal gated and latent-attention layers) at sizes of real models, random
weights, beside the attention model of this framework at equal width, feed-forward, vocabulary and number of layers; and every
kernel of a layer alone, as a fraction of its roofline, beside the attention model's like kernels.

    python bench.py --hybrid            # or: python bench_hybrid.py [--size 4b|1b] [--kernels-only|--models-only]

Prints one JSON line.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

HBM_GBS, MFMA_TFLOPS = 8000.0, 2500.0
SIZES = {
    "4b": {"width": 2560, "ff": 9728, "vocab": 151936, "heads": 32, "kv_heads": 8, "kv_rank": 512, "ssm_heads": 80, "state": 128, "gru": 2560},
    "1b": {"width": 1024, "ff": 3072, "vocab": 151936, "heads": 16, "kv_heads": 4, "kv_rank": 256, "ssm_heads": 32, "state": 128, "gru": 1024},
}
LAYERS, PREFILL, CONTEXT, STEPS = 8, 8192, 4096, 64


def hybrid_config(z: dict):
    from msa_amd.config import HybridConfig
    mlp = {"kind": "dense", "ff": z["ff"]}
    ssm = {"type": "mamba2", "mlp": mlp, "mixer": {"heads": z["ssm_heads"], "vdim": 64, "state": z["state"], "groups": 8, "conv": 4,
                                                   "norm_groups": 8}}
    gru = {"type": "mingru", "mlp": mlp, "mixer": {"width": z["gru"]}}
    att = {"type": "latent_attention", "mlp": mlp, "mixer": {"heads": z["heads"], "dim": 128, "vdim": 128, "kv_rank": z["kv_rank"],
                                                             "scale": 128 ** -0.5}}
    return HybridConfig.from_dict({"vocab": z["vocab"], "width": z["width"], "layers": [ssm, gru, ssm, att] * (LAYERS // 4), "loop": None,
                                   "norm": {"eps": 1e-5}, "logit_softcap": 30.0})


def time_us(fn, reps=20, warm=3):
    """GPU time of a call, measured over a HIP graph of `reps` of them (no launch cost of the host in between)."""
    for _ in range(warm):
        fn()
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        for _ in range(reps):
            fn()
    graph.replay()
    best = 1e30
    for _ in range(3):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        graph.replay()
        b.record()
        torch.cuda.synchronize()
        best = min(best, a.elapsed_time(b))
    return best * 1e3 / reps


def row(us: float, bytes_: float = 0.0, flops: float = 0.0) -> dict:
    """A kernel's line: time and the fraction of whichever roofline binds it."""
    hbm, mfma = bytes_ / (HBM_GBS * 1e3), flops / (MFMA_TFLOPS * 1e6)
    bound, floor = ("hbm", hbm) if hbm >= mfma else ("mfma", mfma)
    return {"us": round(us, 2), "bound": bound, "roofline_us": round(floor, 2), "frac": round(floor / us, 3)}


class Ring:
    """Successive operand sets, so that a set has left the caches when its turn comes again."""

    def __init__(self, make, nbytes):
        self.sets = [make() for _ in range(max(1, min(24, int(600e6 / max(nbytes, 1)))))]
        self.i = 0

    def __call__(self):
        self.i = (self.i + 1) % len(self.sets)
        return self.sets[self.i]


def kernels(size: str, dev) -> dict:
    """Every kernel of the three layer kinds at prefill (one sequence of PREFILL tokens) and decode (16 sequences at CONTEXT
    tokens), and the attention model's like kernels at the same shapes.  Operands rotate through copies larger than the last-level
    cache where a launch is short."""
    from msa_amd import ops, seq_ops
    z = SIZES[size]
    W, ff, H, rank, SH, N, P, G, n = z["width"], z["ff"], z["heads"], z["kv_rank"], z["ssm_heads"], z["state"], 64, 8, z["gru"]
    g = torch.Generator(device=dev).manual_seed(5)
    bf = lambda *s, scale=1.0: (torch.randn(s, generator=g, device=dev) * scale).to(torch.bfloat16)
    f32 = lambda *s: torch.randn(s, generator=g, device=dev)
    T, B, L = PREFILL, 16, CONTEXT
    inner, C = SH * P, SH * P + 2 * G * N
    out = {"prefill": {}, "decode": {}, "prefill_like": {}, "decode_like": {}}

    # ---------------------------------------------------------------- prefill
    pb = seq_ops.StepBatch([T], [0], [0], dev)
    norm = seq_ops.DynTanhNorm(f32(W), f32(W), 0.8)
    gb, sh, prev = f32(W), f32(W), torch.zeros(1, W, device=dev)
    x, y, gate = f32(T, W), bf(T, W), bf(T, W)
    p = out["prefill"]
    p["residual + norm + shift"] = row(time_us(lambda: seq_ops.residual_norm(x, pb, torch.bfloat16, y, gate, gb, norm, sh, prev)),
                                       T * W * (4 + 2 + 2 + 4 + 2 + 2))
    up = bf(T, ff + W)
    p["gelu"] = row(time_us(lambda: seq_ops.gelu_(up[:, :ff])), T * ff * 4)
    xbc_in, taps, cb, cs = bf(T, C), f32(C, 4), f32(C), torch.zeros(1, 3, C, device=dev)
    p["convolution + silu"] = row(time_us(lambda: seq_ops.conv_silu(xbc_in, taps, cb, cs, pb)), T * C * 4)
    zz, dtr = bf(T, inner), bf(T, SH)
    dtb, al, D = f32(SH) - 4.0, torch.rand(SH, device=dev), f32(SH)
    st = torch.zeros(1, SH, N, P, device=dev)
    Q = 128 if N <= 128 else 64
    ssd_fl = SH * T * (2.0 * Q / 2 * (N + 2 * P) + 2.0 * N * P * 4)      # (two products per decay- or state-carrying operand)
    p["state-space scan (4 launches)"] = row(time_us(lambda: seq_ops.ssd(xbc_in, zz, dtr, dtb, al, D, SH, P, N, G, st, pb, chunked=True)),
                                             T * (C + 2 * inner + SH) * 2, ssd_fl)
    v, nw = bf(T, inner), f32(inner)
    p["grouped rms norm"] = row(time_us(lambda: seq_ops.group_rmsnorm(v, nw, 8, 1e-5)), T * inner * 4)
    cols = -(-n // 16) * 48
    zug, zb, ub, gs = bf(T, cols), f32(n), f32(n), torch.zeros(1, n, device=dev)
    p["minimal gated recurrence (3 launches)"] = row(time_us(lambda: seq_ops.min_gru(zug, zb, ub, n, gs, pb)), T * n * 2 * 4)
    dkv, lw, cache = bf(T, rank), f32(rank), torch.zeros(1, T, rank, dtype=torch.bfloat16, device=dev)
    p["latent norm + append"] = row(time_us(lambda: seq_ops.latent_append(dkv, lw, 1e-5, cache, pb)), T * rank * 4)
    q, k, vv, sink = bf(T, H * 128), bf(T, H * 128), bf(T, H * 128), f32(H)
    off = torch.zeros(1, dtype=torch.int64, device=dev)
    pairs = T * (T + 1) / 2
    p["attention (expanded keys)"] = row(time_us(lambda: seq_ops.flash(q, k, vv, off, sink, 128 ** -0.5, H, pb), reps=5),
                                         T * H * 128 * 2 * 4, 4 * pairs * H * 128)
    for name, (N_, K_) in {"vendor product [up | gate]": (ff + W, W), "vendor product down": (W, ff)}.items():
        a_, w_ = bf(T, K_), bf(N_, K_, scale=K_ ** -0.5)
        p[name] = row(time_us(lambda: torch.nn.functional.linear(a_, w_), reps=5), 0, 2.0 * T * N_ * K_)

    l = out["prefill_like"]
    xb, rb, wn = bf(T, W), bf(T, W), torch.ones(W, dtype=torch.bfloat16, device=dev)
    l["rms norm + residual"] = row(time_us(lambda: ops.rmsnorm(xb, wn, 1e-6, residual=rb)), T * W * 8)
    gu = bf(T, 2 * ff)
    l["silu * up"] = row(time_us(lambda: ops.silu_mul(gu)), T * ff * 6)
    kv_off, kv_len = torch.zeros(1, dtype=torch.int64, device=dev), torch.full((1,), T, dtype=torch.int32, device=dev)
    cu = torch.tensor([0, T], dtype=torch.int32, device=dev)
    q3, kc, vc = bf(T, H, 128), bf(T, z["kv_heads"], 128), bf(T, z["kv_heads"], 128)
    l["flash attention (GQA)"] = row(time_us(lambda: ops.sparse_attn(q3, kc, vc, kv_off, kv_len, T, cu_q=cu, max_sq=T), reps=5),
                                     T * H * 128 * 4, 4 * pairs * H * 128)

    # ---------------------------------------------------------------- decode
    db = seq_ops.StepBatch([1] * B, list(range(B)), [L - 1] * B, dev)
    d = out["decode"]
    stream, prevs = f32(B, W), torch.zeros(B, W, device=dev)
    gates = bf(B, W)

    def rows_case(name, N_, K_, call, extra=0.0):
        ring = Ring(lambda: bf(N_, K_, scale=K_ ** -0.5), N_ * K_ * 2)
        d[name] = row(time_us(lambda: call(ring()), reps=24), N_ * K_ * 2 + extra)

    pad = lambda v_: -(-v_ // 32) * 32
    hB = bf(B, W)
    ssm_rows = pad(inner + C + SH)
    cst = torch.zeros(B, 3, C, device=dev)
    rows_case("in projection + convolution (state space)", ssm_rows + W, W,
              lambda w_: seq_ops.rows_conv(hB, w_, hB, ssm_rows, inner, taps, cb, cst, db.slot), B * C * 24)
    gst = torch.zeros(B, n, device=dev)
    rows_case("in projection + recurrence (minimal gated)", cols + W, W, lambda w_: seq_ops.rows_gru(hB, w_, hB, n, zb, ub, gst, db.slot))
    att_rows = pad(H * 128 + rank)
    rows_case("in projection (attention)", att_rows + W, W, lambda w_: seq_ops.rows_linear(hB, w_, x_b=hB, n_b=att_rows))
    rows_case("[up | gate] + gelu", ff + W, W, lambda w_: seq_ops.rows_linear(hB, w_, gelu_n=ff))
    actB = bf(B, ff)
    rows_case("down + residual + norm + shift", W, ff, lambda w_: seq_ops.rows_residual(actB, w_, stream, gates, gb, db.slot, norm, sh, prevs))
    oB = bf(B, H * 128)
    rows_case("attention output + residual + norm", W, H * 128, lambda w_: seq_ops.rows_residual(oB, w_, stream, gates, gb, db.slot, norm))
    iB = bf(B, inner)
    rows_case("state-space output + residual + norm", W, inner, lambda w_: seq_ops.rows_residual(iB, w_, stream, gates, gb, db.slot, norm))
    rows_case("head + softcap", z["vocab"], W, lambda w_: seq_ops.rows_linear_f32(hB, w_, 30.0))
    qB = bf(B, H * 128)
    rows_case("queries to latent space", H * rank, 128, lambda w_: seq_ops.rows_linear(qB, w_, groups=H), B * H * rank * 2)
    ctxB = bf(B, H * rank)
    rows_case("latent to values", H * 128, rank, lambda w_: seq_ops.rows_linear(ctxB, w_, groups=H), B * H * rank * 2)
    xbcB, zB, dtB = bf(B, C), bf(B, inner), bf(B, SH)
    ring = Ring(lambda: torch.zeros(B, SH, N, P, device=dev), B * SH * N * P * 4)
    d["state-space update"] = row(time_us(lambda: seq_ops.ssd(xbcB, zB, dtB, dtb, al, D, SH, P, N, G, ring(), db), reps=24),
                                  2.0 * B * SH * N * P * 4)
    qa = bf(B, H, rank)
    ring = Ring(lambda: bf(B, L, rank), B * L * rank * 2)
    d["latent attention + combine"] = row(time_us(lambda: seq_ops.latent_attn(qa, ring(), sink, 0.1, db, L), reps=24), B * L * rank * 2)
    long = seq_ops.StepBatch([1] * B, list(range(B)), [4 * L - 1] * B, dev)
    far = Ring(lambda: bf(B, 4 * L, rank), B * 4 * L * rank * 2)
    d[f"latent attention + combine at {4 * L} tokens"] = row(time_us(lambda: seq_ops.latent_attn(qa, far(), sink, 0.1, long, 4 * L), reps=12),
                                                             B * 4 * L * rank * 2)
    vB = bf(B, inner)
    d["grouped rms norm"] = row(time_us(lambda: seq_ops.group_rmsnorm(vB, nw, 8, 1e-5)), B * inner * 4)
    d["latent norm + append"] = row(time_us(lambda: seq_ops.latent_append(dkv[:B], lw, 1e-5, ring(), db)), B * rank * 4)

    l = out["decode_like"]
    rb16 = bf(B, W)

    def like_case(name, N_, K_, call):
        ring = Ring(lambda: bf(N_, K_, scale=K_ ** -0.5), N_ * K_ * 2)
        l[name] = row(time_us(lambda: call(ring()), reps=24), N_ * K_ * 2)
    like_case("qkv (norm folded)", (H + 2 * z["kv_heads"]) * 128, W, lambda w_: ops.skinny_linear(hB, w_, norm_weight=wn, eps=1e-6))
    like_case("gate/up + silu-mul (norm folded)", 2 * ff, W, lambda w_: ops.skinny_linear(hB, w_, silu_mul=True, norm_weight=wn, eps=1e-6))
    like_case("down + residual", W, ff, lambda w_: ops.skinny_linear(actB, w_, residual=rb16))
    like_case("attention output + residual", W, H * 128, lambda w_: ops.skinny_linear(oB, w_, residual=rb16))
    like_case("head (norm folded)", z["vocab"], W, lambda w_: ops.skinny_linear(hB, w_, norm_weight=wn, eps=1e-6))
    for nm, (N_, K_) in {"plain, rows and columns of the state-space in projection": (ssm_rows + W, W),
                         "plain, of the minimal gated in projection": (cols + W, W), "plain, of [up | gate]": (ff + W, W)}.items():
        like_case(nm, N_, K_, lambda w_: ops.skinny_linear(hB, w_))
    kv = z["kv_heads"]
    ring = Ring(lambda: (bf(B, L + 64, kv, 128), bf(B, L + 64, kv, 128)), B * L * kv * 128 * 4)
    qkv = bf(B, (H + 2 * kv) * 128)
    pos, hw = torch.full((B,), L, dtype=torch.int64, device=dev), torch.ones(128, dtype=torch.bfloat16, device=dev)
    rope = ops.rope_tables(L + 128, 128, 1e6, device=dev)
    klen = torch.full((B,), L, dtype=torch.int32, device=dev)

    def attn():
        kc_, vc_ = ring()
        klen.fill_(L)
        ops.decode_attn_fused(qkv, H, kv, 128, pos, hw, hw, 1e-6, rope, kc_, vc_, klen)
    l["decode attention (norm, rotary, append folded in; with one fill launch)"] = row(time_us(attn, reps=24), B * L * kv * 128 * 4)
    w_in = torch.ones(inner, dtype=torch.bfloat16, device=dev)
    l["rms norm"] = row(time_us(lambda: ops.rmsnorm(iB, w_in, 1e-6)), B * inner * 4)
    return out


def model_throughput(size: str, dev, others=None) -> dict:
    """Prefill of one prompt of PREFILL tokens and greedy decoding (HIP graph) of 1 and 16 sequences behind CONTEXT tokens, both
    models (and ``others``: name -> function of batch, prompt length, new tokens and generator that returns the timings) at equal
    width, feed-forward, vocabulary and number of layers; timed in turn."""
    from msa_amd.cache import create_cache
    from msa_amd.config import MSAConfig
    from msa_amd.hybrid import HybridForCausalLM
    from msa_amd.model import MSAForCausalLM
    z = SIZES[size]
    hybrid = HybridForCausalLM.random(hybrid_config(z), 1, torch.bfloat16, dev)
    mc = MSAConfig(hidden_size=z["width"], num_hidden_layers=LAYERS, num_attention_heads=z["heads"], num_key_value_heads=z["kv_heads"],
                   intermediate_size=z["ff"], vocab_size=z["vocab"])
    mc.msa_config.router_layer_idx = "-1"                       # no memory: every layer plain attention
    with torch.device(dev):
        msa = MSAForCausalLM(mc).to(torch.bfloat16)
    msa.init_random_(0.02, seed=1).eval()
    for layer in msa.model.layers:
        layer.self_attn.decode_reserve = STEPS + 8
    g = torch.Generator(device=dev).manual_seed(2)

    def run_hybrid(B, S, new, g):
        ids = torch.randint(0, z["vocab"], (B, S), generator=g, device=dev)
        t = {}
        hybrid.generate_greedy(ids, torch.ones_like(ids), new, timings=t, use_graph=True)
        return t

    def run_msa(B, S, new, g):
        ids = torch.randint(0, z["vocab"], (B, S), generator=g, device=dev)
        cache = create_cache()
        empty = torch.zeros((1, z["kv_heads"], 1, 128), dtype=torch.bfloat16, device=dev)
        for i in range(LAYERS):
            cache.record_kwargs(i, {"template_prefix_kcache": empty, "template_prefix_vcache": empty})
        t = {}
        msa.generate_greedy(ids, torch.ones_like(ids), torch.zeros_like(ids), new, past_key_values=cache, timings=t, use_graph=True)
        return t
    res = {}
    for name, B, S, new in (("prefill", 1, PREFILL, 2), ("decode_1", 1, CONTEXT, STEPS), ("decode_16", 16, CONTEXT, STEPS)):
        best = {}
        for _ in range(3):
            for who, fn in {"hybrid": run_hybrid, "attention_model": run_msa, **(others or {})}.items():
                t = fn(B, S, new, g)
                v = B * S / t["prefill_s"] if name == "prefill" else B * t["decode_steps"] / t["decode_s"]
                best[who] = max(best.get(who, 0.0), v)
        res[name + "_tokens_per_s"] = {k: round(v, 1) for k, v in best.items()}
    return res


def main(argv=None) -> dict:
    ap = argparse.ArgumentParser()
    ap.add_argument("--size", choices=list(SIZES), action="append")
    ap.add_argument("--kernels-only", action="store_true")
    ap.add_argument("--models-only", action="store_true")
    args = ap.parse_args(argv)
    if not torch.cuda.is_available():
        sys.exit("bench_hybrid: no GPU visible; the HIP path has no CPU fallback")
    dev = torch.device("cuda:0")
    out = {"metric": "hybrid decoder prefill / decode throughput", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic",
           "config": {"layers": LAYERS, "prefill_tokens": PREFILL, "decode_context": CONTEXT, "pattern": "ssm, gru, ssm, attention",
                      "sizes": {s: SIZES[s] for s in args.size or SIZES}}, "models": {}, "kernels": {}}
    t0 = time.time()
    for size in args.size or SIZES:
        if not args.kernels_only:
            out["models"][size] = model_throughput(size, dev)
            print(f"[bench_hybrid] models {size} {time.time() - t0:.0f} s", file=sys.stderr, flush=True)
        if not args.models_only:
            out["kernels"][size] = kernels(size, dev)
            print(f"[bench_hybrid] kernels {size} {time.time() - t0:.0f} s", file=sys.stderr, flush=True)
        torch.cuda.empty_cache()
    print(json.dumps(out), flush=True)
    return out


if __name__ == "__main__":
    main()
