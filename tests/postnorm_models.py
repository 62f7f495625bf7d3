"""Small configurations and random weights of the output-normed decoder for the tests."""
import torch

DELTA = {"heads": 6, "kv_heads": 3, "dim": 40, "vdim": 24, "conv": 3}
ATTN = {"heads": 6, "kv_heads": 2, "dim": 40, "vdim": 24, "scale": 0.31, "mask": {"size": 50},
        "rot": {"base": 5000.0, "dims": 32, "scaling": {"factor": 3.0, "low": 1.0, "high": 5.0, "original": 300}}}


def layer(kind, mixer, ff=104, limit=1.5, **more):
    return {"type": kind, "mixer": {**mixer, **more}, "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def config(layers, width=120, vocab=203, eps=1e-5):
    return {"architecture": "Sugizen", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


CONFIGS = {
    # both mixers, shared keys under another mask, layers without feed-forward, shared q / k heads of the delta rule
    "mixed": config([layer("attention", ATTN), layer("channel_delta", DELTA), layer("attention", ATTN, None, kv_from=0, mask={"size": 31}),
                     layer("channel_delta", DELTA, None), layer("attention", ATTN, kv_from=0, heads=4, limit=0.7)]),
    # sizes that are one; one rotated pair; no scaling; chunks of one token
    "ones": config([layer("channel_delta", {"heads": 1, "kv_heads": 1, "dim": 8, "vdim": 16, "conv": 1}, 8),
                    layer("attention", {"heads": 1, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 1.0, "mask": {"size": 1}, "rot": {"base": 10.0, "dims": 2}}, 16),
                    layer("attention", {"heads": 8, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 0.5, "mask": {"size": 500}, "rot": {"base": 100.0, "dims": 8}})],
                   width=48),
    # nothing a multiple of eight: every kernel's unaligned form
    "odd": config([layer("channel_delta", {"heads": 3, "kv_heads": 1, "dim": 13, "vdim": 11, "conv": 5}, 45),
                   layer("attention", {"heads": 3, "kv_heads": 3, "dim": 13, "vdim": 7, "scale": 0.3, "mask": {"size": 33},
                                       "rot": {"base": 1000.0, "dims": 10, "scaling": {"factor": 2.0, "low": 1.0, "high": 2.0, "original": 100}}}, 33),
                   layer("channel_delta", {"heads": 2, "kv_heads": 2, "dim": 5, "vdim": 70, "conv": 2}, None)], width=51, vocab=77),
    # wide heads, many heads a key, value sizes over several column blocks
    "wide": config([layer("channel_delta", {"heads": 4, "kv_heads": 4, "dim": 128, "vdim": 136, "conv": 4}, 264),
                    layer("attention", {"heads": 36, "kv_heads": 2, "dim": 64, "vdim": 128, "scale": 0.125, "mask": {"size": 128},
                                        "rot": {"base": 1e6, "dims": 64}}),
                    layer("attention", {"heads": 18, "kv_heads": 2, "dim": 64, "vdim": 128, "scale": 0.125, "mask": {"size": 70},
                                        "rot": {"base": 1e6, "dims": 64}, "kv_from": 1}, 328)], width=136),
}
RANKS = {"mixed": (11, 20), "ones": (1, 3), "odd": (7, 5), "wide": (64, 24)}        # of the decays and of the gates


def tensor_shapes(cfg, ranks=(11, 20)):
    from msa_amd.config import PostNormConfig
    from msa_amd.postnorm import PostNormForCausalLM
    named = {"a_rank": ranks[0], "g_rank": ranks[1]}
    shapes = PostNormForCausalLM(PostNormConfig.from_dict(cfg)).tensor_shapes()
    return {n: tuple(named.get(d, d) for d in s) for n, s in shapes.items()}


def random_weights(shapes, seed=0):
    """bf16 weights that keep activations of order one; norms, decays and step sizes all different, some decays hardly noticeable."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes.items():
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.3 * t
        elif last == "A_log":
            t = t - 1.0
        elif last == "dt_bias":
            t = t - 2.5
        elif last == "head":
            t = t * 2.0 * shape[-1] ** -0.5
        elif len(shape) > 1 and last not in ("embed", "conv"):
            t = t * shape[-1] ** -0.5
        elif last == "conv":
            t = 0.6 * t
        out[name] = t.to(torch.bfloat16)
    return out
