"""Small configurations and random weights of the hybrid decoder for the tests."""
import json

import torch

MAMBA = {"heads": 6, "vdim": 24, "state": 40, "groups": 3, "conv": 3, "norm_groups": 2}
GRU = {"width": 104}
LATENT = {"heads": 5, "dim": 40, "vdim": 24, "kv_rank": 72, "scale": 0.21}


def layer(kind, mixer, ff=152):
    return {"type": kind, "mixer": dict(mixer), "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, width=120, vocab=203, loop=None, cap=11.0, eps=1e-5):
    return {"architecture": "Gevonex", "layers": layers, "loop": loop, "norm": {"eps": eps}, "logit_softcap": cap, "vocab": vocab,
            "width": width}


CONFIGS = {
    # every mixer, a loop in the middle, a layer without feed-forward
    "mixed": config([layer("mingru", GRU), layer("latent_attention", LATENT), layer("mamba2", MAMBA, None), layer("mamba2", MAMBA)],
                    loop={"start": 1, "stop": 3, "times": 3}),
    # sizes that are one, no loop, no softcap
    "ones": config([layer("mamba2", {"heads": 3, "vdim": 8, "state": 8, "groups": 1, "conv": 1, "norm_groups": 3}, 8),
                    layer("latent_attention", {"heads": 1, "dim": 8, "vdim": 16, "kv_rank": 8, "scale": 1.0}),
                    layer("mingru", {"width": 8}, 24)], width=48, cap=None),
    # nothing a multiple of eight: every kernel's unaligned form
    "odd": config([layer("latent_attention", {"heads": 3, "dim": 13, "vdim": 11, "kv_rank": 27, "scale": 0.4}, 45),
                   layer("mamba2", {"heads": 6, "vdim": 7, "state": 9, "groups": 2, "conv": 5, "norm_groups": 3}, 33),
                   layer("mingru", {"width": 35}, None)], width=51, vocab=77, loop={"start": 0, "stop": 3, "times": 1}, cap=5.0),
    # wide heads and ranks: two column blocks of state, more heads than a matrix tile, loop over everything
    "wide": config([layer("mamba2", {"heads": 4, "vdim": 72, "state": 136, "groups": 2, "conv": 4, "norm_groups": 4}, 264),
                    layer("latent_attention", {"heads": 36, "dim": 16, "vdim": 24, "kv_rank": 200, "scale": 0.3}),
                    layer("mingru", {"width": 328})], width=136, loop={"start": 0, "stop": 2, "times": 2}),
}


def random_weights(shapes, seed=0):
    """bf16 weights that keep activations of order one; biases, gates and shifts all different."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes.items():
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last == "alpha":
            t = 0.5 + torch.rand(shape, generator=g)
        elif last in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.3 * t
        elif last == "shift":
            t = torch.rand(shape, generator=g)
        elif last == "A_log":
            t = torch.log(0.3 + torch.rand(shape, generator=g) * 4)
        elif last == "dt_bias":
            t = t - 2.0
        elif last == "sink":
            t = 2.0 * t
        elif last == "head":
            t = t * 2.0 * shape[-1] ** -0.5
        elif len(shape) > 1 and last not in ("embed", "conv"):
            t = t * shape[-1] ** -0.5
        elif last not in ("embed", "D"):
            t = 0.5 * t
        out[name] = t.to(torch.bfloat16)
    return out


def tensor_shapes(cfg):
    from msa_amd.config import HybridConfig
    from msa_amd.hybrid import HybridForCausalLM
    return HybridForCausalLM(HybridConfig.from_dict(cfg)).tensor_shapes()


def save_model(path, cfg, weights):
    """config.json + model.safetensors, written by hand."""
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    header, blobs, at = {}, [], 0
    kinds = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}
    for name, t in weights.items():
        raw = t.contiguous().view(-1).view(torch.uint8).numpy().tobytes()
        header[name] = {"dtype": kinds[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    (path / "model.safetensors").write_bytes(len(head).to_bytes(8, "little") + head + b"".join(blobs))
