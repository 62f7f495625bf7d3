"""Throughput of the output-normed decoder (channel-wise delta rule, rotary chunk attention, clamped gated feed-forward) at sizes of
real models, random weights, beside this framework's closest models at equal width, feed-forward, vocabulary and number of
layers: the hybrid recurrent decoder and the attention model.  And every kernel of a layer alone, as a fraction of its roofline,
beside the like kernels of those models.

    python bench.py --postnorm          # or: python bench_postnorm.py [--size 4b|1b] [--kernels-only|--models-only]

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

import bench_hybrid
from bench_hybrid import CONTEXT, LAYERS, PREFILL, STEPS, Ring, row, time_us

# the delta layers' heads; everything else is bench_hybrid.SIZES
SIZES = {"4b": {"delta_heads": 32, "delta_kv_heads": 16, "delta_dim": 128, "delta_vdim": 128, "rank": 128},
         "1b": {"delta_heads": 16, "delta_kv_heads": 16, "delta_dim": 64, "delta_vdim": 128, "rank": 64}}
CHUNK, LIMIT = 8192, 7.0


def sizes(name: str) -> dict:
    return {**bench_hybrid.SIZES[name], **SIZES[name]}


def postnorm_config(z: dict):
    from msa_amd.config import PostNormConfig
    mlp = {"kind": "dense", "ff": z["ff"], "limit": LIMIT}
    delta = {"type": "channel_delta", "mlp": mlp, "mixer": {"heads": z["delta_heads"], "kv_heads": z["delta_kv_heads"], "dim": z["delta_dim"],
                                                           "vdim": z["delta_vdim"], "conv": 4}}
    mixer = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": CHUNK},
             "rot": {"base": 1e6, "dims": 128, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    layers = []
    for i in range(LAYERS // 4):                               # every second attention layer reads the keys of the one before
        share = {"kv_from": 4 * i - 1} if i % 2 else {}
        layers += [delta, delta, delta, {"type": "attention", "mlp": mlp, "mixer": {**mixer, **share}}]
    return PostNormConfig.from_dict({"vocab": z["vocab"], "width": z["width"], "layers": layers, "norm": {"eps": 1e-5}})


def kernels(name: str, dev) -> dict:
    """Every kernel of the two layer kinds at prefill (one sequence of PREFILL tokens) and decode (16 sequences at CONTEXT tokens)."""
    from msa_amd import seq_ops
    from msa_amd.config import RotaryConfig
    z = sizes(name)
    W, ff, H, G = z["width"], z["ff"], z["heads"], z["kv_heads"]
    DH, DG, D, E, R = z["delta_heads"], z["delta_kv_heads"], z["delta_dim"], z["delta_vdim"], z["rank"]
    g = torch.Generator(device=dev).manual_seed(5)
    bf = lambda *s, scale=1.0: (torch.randn(s, generator=g, device=dev) * scale).to(torch.bfloat16)
    f32 = lambda *s: torch.randn(s, generator=g, device=dev)
    T, B, L = PREFILL, 16, CONTEXT
    C = 2 * DG * D + DH * E
    BF = torch.bfloat16

    # ---------------------------------------------------------------- prefill
    p = {}
    pb = seq_ops.StepBatch([T], [0], [0], dev)
    x, y, nw = f32(T, W), bf(T, W), f32(W)
    p["residual + norm"] = row(time_us(lambda: seq_ops.rms_residual(x, BF, y, nw, 1e-5, out=x)), T * W * (4 + 2 + 4 + 2))
    gu = bf(T, 2 * ff)
    p["clamped gated unit"] = row(time_us(lambda: seq_ops.clamped_glu(gu, LIMIT)), T * ff * 6)
    conv_in, taps, cs = bf(T, C), f32(C, 4), torch.zeros(1, 3, C, device=dev)
    p["convolution + silu"] = row(time_us(lambda: seq_ops.conv_silu(conv_in, taps, None, cs, pb)), T * C * 4)
    a, b, gate = bf(T, DH * D), bf(T, DH), bf(T, DH * E)
    A_log, bias, hn = torch.rand(DH, device=dev), f32(DH * D) - 4.0, torch.ones(E, device=dev)
    st = torch.zeros(1, DH, D, E, device=dev)
    Q = 64                                                     # per token and head: scores, T on [values | keys], state, read-out
    flops = DH * T * (2.0 * Q / 2 * 2 * D + 2.0 * Q / 2 * (D + E) + 2.0 * D * E * 3 + 2.0 * Q / 2 * E)
    p["delta rule, chunked, norm, gate"] = row(
        time_us(lambda: seq_ops.delta(conv_in, a, b, gate, A_log, bias, hn, 1e-5, DH, DG, D, E, st, pb, True), reps=10),
        T * (C + DH * D + DH + 2 * DH * E) * 2, flops)
    o = bf(T, DH * E)

    def head_norm():
        seq_ops._check(seq_ops._lib.load_seq().msa_seq_head_norm_gate(o.data_ptr(), gate.data_ptr(), DH * E, hn.data_ptr(), 1e-5, 0, T, DH, E,
                                                                     seq_ops._stream()), "msa_seq_head_norm_gate")
    p["of it: head norm + gate"] = row(time_us(head_norm), T * DH * E * 6)
    qkv = bf(T, (H + 2 * G) * 128)
    kc, vc = torch.zeros(1, T, G, 128, dtype=BF, device=dev), torch.zeros(1, T, G, 128, dtype=BF, device=dev)
    hw = torch.ones(128, device=dev)
    freqs = torch.tensor(RotaryConfig(1e6, 128).frequencies(), dtype=torch.float64, device=dev)
    cols = lambda t, i, n: t[:, i * 128:(i + n) * 128]
    prepare = lambda t, k_, v_, bt: seq_ops.qk_rope_append(cols(t, 0, H), hw, freqs, 1e-5, k_, v_, bt, cols(t, H, G), cols(t, H + G, G), hw)
    p["head norms + rotation + append"] = row(time_us(lambda: prepare(qkv, kc, vc, pb)), T * (H + 2 * G) * 128 * 4)
    q = prepare(qkv, kc, vc, pb).view(T, -1)
    hg = bf(T, H)
    pairs = T * (T + 1) / 2
    flash = lambda chunk: seq_ops.flash(q, kc.view(T, -1), vc.view(T, -1), pb.cache_rows(T), None, 128 ** -0.5, H, pb, G, chunk, hg)
    p["attention"] = row(time_us(lambda: flash(CHUNK), reps=5), T * H * 128 * 4, 4 * pairs * H * 128)
    n = T // 2048
    p["attention, chunks of 2048"] = row(time_us(lambda: flash(2048), reps=5), T * H * 128 * 4, 4 * n * 2048 * 2049 / 2 * H * 128)
    a_low, w_low = bf(T, R), bf(DH * D, R, scale=R ** -0.5)
    p["vendor product, low rank to decays"] = row(time_us(lambda: torch.nn.functional.linear(a_low, w_low)), T * (R + DH * D) * 2, 2.0 * T * R * DH * D)

    # ---------------------------------------------------------------- decode
    d = {}
    db = seq_ops.StepBatch([1] * B, list(range(B)), [L - 1] * B, dev)
    hB = bf(B, W)

    def rows_case(label, N_, K_, call, extra=0.0):
        ring = Ring(lambda: bf(N_, K_, scale=K_ ** -0.5), N_ * K_ * 2)
        d[label] = row(time_us(lambda: call(ring()), reps=24), N_ * K_ * 2 + extra)
    pad = lambda v_: -(-v_ // 32) * 32
    cst = torch.zeros(B, 3, C, device=dev)
    in_rows = pad(C + 2 * R + DH)
    rows_case("in projection + convolution (delta)", in_rows, W, lambda w_: seq_ops.rows_conv(hB, w_, None, in_rows, 0, taps, None, cst, db.slot), B * C * 24)
    lowB = bf(B, R)
    rows_case("low rank to decays and gates", DH * D + DH * E, R, lambda w_: seq_ops.rows_linear(lowB, w_, x_b=lowB, n_b=DH * D))
    qB, aB, bB, gB = bf(B, C), bf(B, DH * D), bf(B, DH), bf(B, DH * E)
    ring = Ring(lambda: torch.zeros(B, DH, D, E, device=dev), B * DH * D * E * 4)
    d["delta update, norm, gate"] = row(
        time_us(lambda: seq_ops.delta(qB, aB, bB, gB, A_log, bias, hn, 1e-5, DH, DG, D, E, ring(), db), reps=24), 2.0 * B * DH * D * E * 4)
    one = seq_ops.StepBatch([1], [0], [L - 1], dev)
    d["delta update, norm, gate, 1 sequence"] = row(
        time_us(lambda: seq_ops.delta(qB[:1], aB[:1], bB[:1], gB[:1], A_log, bias, hn, 1e-5, DH, DG, D, E, ring(), one), reps=24), 2.0 * DH * D * E * 4)
    oB, iB, actB = bf(B, DH * E), bf(B, H * 128), bf(B, ff)
    rows_case("delta output", W, DH * E, lambda w_: seq_ops.rows_linear(oB, w_))
    xB, yB = f32(B, W), bf(B, W)
    d["residual + norm"] = row(time_us(lambda: seq_ops.rms_residual(xB, BF, yB, nw, 1e-5, out=xB)), B * W * 12)
    rows_case("[gate, up] + clamped unit", 2 * ff, W, lambda w_: seq_ops.rows_glu(hB, w_, LIMIT))
    rows_case("down", W, ff, lambda w_: seq_ops.rows_linear(actB, w_))
    att_rows = pad((H + 2 * G) * 128 + H)
    rows_case("in projection (attention)", att_rows, W, lambda w_: seq_ops.rows_linear(hB, w_))
    rows_case("attention output", W, H * 128, lambda w_: seq_ops.rows_linear(iB, w_))
    rows_case("head", z["vocab"], W, lambda w_: seq_ops.rows_linear_f32(hB, w_))
    ring = Ring(lambda: (bf(B, L, G, 128), bf(B, L, G, 128)), B * L * G * 128 * 4)
    qkvB, hgB = bf(B, (H + 2 * G) * 128), bf(B, H)
    d["head norms + rotation + append"] = row(time_us(lambda: prepare(qkvB, *ring(), db), reps=24), B * (H + 2 * G) * 128 * 4)
    q3 = bf(B, H, 128)
    d["attention + combine"] = row(time_us(lambda: seq_ops.kv_attn(q3, *ring(), 128 ** -0.5, db, CHUNK, hgB), reps=24), B * L * G * 128 * 4)
    d["attention + combine, 1 sequence"] = row(time_us(lambda: seq_ops.kv_attn(q3[:1], *ring(), 128 ** -0.5, one, CHUNK, hgB[:1]), reps=24), L * G * 128 * 4)
    return {"prefill": p, "decode": d}


def single_rows(name: str, dev) -> dict:
    """The hybrid decoder's state update and attention for one sequence."""
    from msa_amd import seq_ops
    z = sizes(name)
    SH, N, P, G, H, rank, L = z["ssm_heads"], z["state"], 64, 8, z["heads"], z["kv_rank"], CONTEXT
    g = torch.Generator(device=dev).manual_seed(6)
    bf = lambda *s: torch.randn(s, generator=g, device=dev).to(torch.bfloat16)
    f32 = lambda *s: torch.randn(s, generator=g, device=dev)
    one = seq_ops.StepBatch([1], [0], [L - 1], dev)
    xbc, zz, dt = bf(1, SH * P + 2 * G * N), bf(1, SH * P), bf(1, SH)
    bias, al, D, sink, qa = f32(SH) - 4.0, torch.rand(SH, device=dev), f32(SH), f32(H), bf(1, H, rank)
    st = Ring(lambda: torch.zeros(1, SH, N, P, device=dev), 16 * SH * N * P * 4)
    cache = Ring(lambda: bf(1, L, rank), 16 * L * rank * 2)
    return {"state-space update, 1 sequence": row(time_us(lambda: seq_ops.ssd(xbc, zz, dt, bias, al, D, SH, P, N, G, st(), one), reps=24),
                                                  2.0 * SH * N * P * 4),
            "latent attention + combine, 1 sequence": row(time_us(lambda: seq_ops.latent_attn(qa, cache(), sink, 0.1, one, L), reps=24),
                                                          L * rank * 2)}


def model_throughput(name: str, dev) -> dict:
    """Prefill of one prompt of PREFILL tokens and greedy decoding (HIP graph) of 1 and 16 sequences behind CONTEXT tokens, the three
    models timed in turn."""
    from msa_amd.postnorm import PostNormForCausalLM
    z = sizes(name)
    model = PostNormForCausalLM.random(postnorm_config(z), 1, torch.bfloat16, dev)

    def run(B, S, new, g):
        ids = torch.randint(0, z["vocab"], (B, S), generator=g, device=dev)
        t = {}
        model.generate_greedy(ids, torch.ones_like(ids), new, timings=t, use_graph=True)
        return t
    return bench_hybrid.model_throughput(name, dev, {"postnorm": run})


def main(argv=None) -> dict:
    ap = argparse.ArgumentParser()
    ap.add_argument("--size", choices=list(SIZES), action="append")
    ap.add_argument("--kernels-only", action="store_true")
    ap.add_argument("--models-only", action="store_true")
    ap.add_argument("--no-like", action="store_true", help="leave the other models' kernels out")
    args = ap.parse_args(argv)
    if not torch.cuda.is_available():
        sys.exit("bench_postnorm: no GPU visible; the HIP path has no CPU fallback")
    dev = torch.device("cuda:0")
    names = args.size or list(SIZES)
    out = {"metric": "output-normed decoder prefill / decode throughput", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic",
           "config": {"layers": LAYERS, "prefill_tokens": PREFILL, "decode_context": CONTEXT, "pattern": "delta, delta, delta, attention",
                      "sizes": {s: sizes(s) for s in names}}, "models": {}, "kernels": {}}
    t0 = time.time()
    for name in names:
        if not args.kernels_only:
            out["models"][name] = model_throughput(name, dev)
            print(f"[bench_postnorm] models {name} {time.time() - t0:.0f} s", file=sys.stderr, flush=True)
        if not args.models_only:
            out["kernels"][name] = kernels(name, dev)
            print(f"[bench_postnorm] kernels {name} {time.time() - t0:.0f} s", file=sys.stderr, flush=True)
            if not args.no_like:
                like = bench_hybrid.kernels(name, dev)
                like["decode"].update(single_rows(name, dev))
                out["kernels"][name]["like"] = {"hybrid": {k: like[k] for k in ("prefill", "decode")},
                                                "attention_model": {"prefill": like["prefill_like"], "decode": like["decode_like"]}}
                print(f"[bench_postnorm] like kernels {name} {time.time() - t0:.0f} s", file=sys.stderr, flush=True)
        torch.cuda.empty_cache()
    print(json.dumps(out), flush=True)
    return out


if __name__ == "__main__":
    main()
