"""Configuration dataclasses, named and shaped like the reference's (src/config/memory_config.py:6-55
and the msa_config block of the checkpoint's config.json, src/utils/resave_model.py:33-50)."""
from __future__ import annotations

import math
from dataclasses import MISSING, dataclass, field
from typing import Dict, List, Optional, Union

QWEN3_TEMPLATE = {"prompt": "<|im_start|>user\n{prompt}<|im_end|>\n",
                  "response": "<|im_start|>assistant\n<think>\n{think_content}\n</think>\n\n{output}<|im_end|>"}
QWEN3_INSTRUCT_TEMPLATE = {"prompt": "<|im_start|>user\n{prompt}<|im_end|>\n",
                           "response": "<|im_start|>assistant\n{output}<|im_end|>"}
_TEMPLATES = {"QWEN3_TEMPLATE": QWEN3_TEMPLATE, "QWEN3_INSTRUCT_TEMPLATE": QWEN3_INSTRUCT_TEMPLATE}


@dataclass
class GenerateConfig:
    devices: List[int] = None
    template: Union[str, Dict] = None
    max_generate_tokens: int = 256
    max_seq_len: int = 0
    max_query_seq_len: int = 0
    max_batch_size: int = 0
    top_p: float = 0.9
    temperature: float = 0.0
    qa_mode: bool = False

    def __post_init__(self):
        if isinstance(self.template, str):
            if self.template not in _TEMPLATES:
                raise ValueError(f"unknown template {self.template!r}")
            self.template = _TEMPLATES[self.template]
        if self.template is not None and not isinstance(self.template, dict):
            raise TypeError("template must be a dict or a known template name")

    @property
    def world(self) -> int:
        return len(self.devices) if self.devices else 0


@dataclass
class ModelConfig:
    model_path: str = "EverMind-AI/MSA-4B"
    doc_top_k: int = 16
    pooling_kernel_size: int = 64
    router_layer_idx: str = "all"
    template_token_id: int = -2
    template_id_num: int = 3


@dataclass
class MemoryConfig:
    block_size: int = 16000
    slice_chunk_size: int = 16 * 1024
    pooling_kernel_size: int = 64
    memory_file_path: str = ""
    socket_ip: str = ""
    socket_port: int = 0


class DotDict(dict):
    """dict with attribute access (src/msa/configuration_msa.py:6-16)."""
    __setattr__ = dict.__setitem__
    __delattr__ = dict.__delitem__

    def __getattr__(self, name):
        if name.startswith("__"):             # keep copy / pickle protocol lookups honest
            raise AttributeError(name)
        return self.get(name)


def default_msa_config() -> DotDict:
    """The shipped hyper-parameters (scripts/resave_model.sh:2-33)."""
    return DotDict(pooling_kernel_size=64, top_k_docs=16, router_layer_idx=",".join(str(i) for i in range(18, 36)),
                   head_reduce_method="mean", query_reduce_method="max", chunk_reduce_method="max",
                   decouple_pooling_mode="mean", aux_loss_method="INFONCE", decouple_router=True)


@dataclass
class MSAConfig:
    """The Qwen3 fields the layer reads plus ``msa_config`` (src/msa/configuration_msa.py:19-53).
    Defaults are Qwen3-4B's."""
    hidden_size: int = 2560
    num_hidden_layers: int = 36
    num_attention_heads: int = 32
    num_key_value_heads: int = 8
    head_dim: int = 128
    intermediate_size: int = 9728
    vocab_size: int = 151936
    rms_norm_eps: float = 1e-6
    rope_theta: float = 1_000_000.0
    max_position_embeddings: int = 40960
    attention_bias: bool = False
    attention_dropout: float = 0.0
    msa_config: DotDict = field(default_factory=default_msa_config)

    def __post_init__(self):
        if isinstance(self.msa_config, dict) and not isinstance(self.msa_config, DotDict):
            self.msa_config = DotDict(self.msa_config)


# ------------------------------------------------------------------------------ recurrent / latent-attention decoders
def _fields(cls, d: dict, where: str):
    """Builds dataclass ``cls`` from ``d``; unknown or missing keys are an error that names the place."""
    fields = cls.__dataclass_fields__
    unknown = sorted(set(d) - set(fields))
    if unknown:
        raise ValueError(f"{where}: unknown keys {unknown}")
    missing = [n for n, f in fields.items() if n not in d and f.default is MISSING and f.default_factory is MISSING]
    if missing:
        raise ValueError(f"{where}: missing keys {missing}")
    try:
        return cls(**d)
    except ValueError as e:
        raise ValueError(f"{where}: {e}") from None


@dataclass
class Mamba2Config:
    """State-space mixer: ``heads`` of ``vdim`` value and ``state`` state dimensions, ``groups`` of heads sharing B / C,
    ``conv`` taps, output norm in ``norm_groups`` parts."""
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    def __post_init__(self):
        if self.heads % self.groups or self.inner % self.norm_groups:
            raise ValueError(f"mamba2: {self.heads} heads in {self.groups} groups, {self.inner} columns in {self.norm_groups} parts")

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def conv_channels(self) -> int:
        return self.inner + 2 * self.groups * self.state


@dataclass
class MinGRUConfig:
    width: int


@dataclass
class LatentAttentionConfig:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float


@dataclass
class ChannelDeltaConfig:
    """Delta rule with a decay per key channel: ``heads`` of ``vdim`` value dimensions over ``kv_heads`` queries and keys of
    ``dim``, ``conv`` taps in front."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads over {self.kv_heads} keys")

    @property
    def conv_channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


@dataclass
class RotaryScalingConfig:
    """Wavelengths above ``original / low`` are stretched by ``factor``, those below ``original / high`` kept, others blended."""
    factor: float
    low: float
    high: float
    original: float


@dataclass
class RotaryConfig:
    """Rotary positions on the first ``dims`` dimensions of a head, dimension i paired with i + dims / 2."""
    base: float
    dims: int
    scaling: Optional[RotaryScalingConfig] = None

    def __post_init__(self):
        if isinstance(self.scaling, dict):
            self.scaling = _fields(RotaryScalingConfig, self.scaling, "scaling")
        if self.dims < 0 or self.dims % 2:
            raise ValueError(f"{self.dims} rotated dimensions")

    def frequencies(self) -> List[float]:
        """Radians per position of every pair."""
        c, out = self.scaling, []
        for i in range(self.dims // 2):
            f = float(self.base) ** (-2 * i / self.dims)
            if c is not None:
                turns = c.original * f / (2 * math.pi)          # full turns over the original context
                if turns < c.low:
                    f /= c.factor
                elif turns <= c.high:
                    s = (turns - c.low) / (c.high - c.low) if c.high > c.low else 1.0
                    f = (1 - s) * f / c.factor + s * f
            out.append(f)
        return out


@dataclass
class ChunkMaskConfig:
    """A position sees the positions up to itself in its own stretch of ``size``, counted from the sequence's start."""
    size: int

    def __post_init__(self):
        if self.size < 1:
            raise ValueError(f"chunks of {self.size}")


@dataclass
class AttentionConfig:
    """Grouped-query attention with query / key norms, rotary positions, a chunk mask (none: causal) and a sigmoid gate per
    head; with ``kv_from`` the keys and values are those of an earlier layer."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[RotaryConfig] = None
    mask: Optional[ChunkMaskConfig] = None
    kv_from: Optional[int] = None

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads over {self.kv_heads} keys")
        if isinstance(self.rot, dict):
            self.rot = _fields(RotaryConfig, self.rot, "rot")
        if isinstance(self.mask, dict):
            self.mask = _fields(ChunkMaskConfig, self.mask, "mask")
        if self.rot is not None and self.rot.dims > self.dim:
            raise ValueError(f"{self.rot.dims} rotated of {self.dim} dimensions")


@dataclass
class DenseMLPConfig:
    ff: int
    kind: str = "dense"

    def __post_init__(self):
        if self.kind != "dense":
            raise NotImplementedError(f"unsupported feed-forward {self.kind!r}")


@dataclass
class ClampedGLUConfig(DenseMLPConfig):
    """``g sigmoid(1.702 g) (u + 1)`` with the gate capped at ``limit`` and the up projection clamped to ``+-limit``."""
    limit: float = field(kw_only=True)


MIXER_CONFIGS = {"mamba2": Mamba2Config, "mingru": MinGRUConfig, "latent_attention": LatentAttentionConfig,
                 "channel_delta": ChannelDeltaConfig, "attention": AttentionConfig}
MixerConfig = Union[Mamba2Config, MinGRUConfig, LatentAttentionConfig, ChannelDeltaConfig, AttentionConfig]


@dataclass
class HybridLayerConfig:
    type: str
    mixer: MixerConfig
    mlp: Union[DenseMLPConfig, None]


def _layers(entries: List[dict], mlp_config=DenseMLPConfig) -> List[HybridLayerConfig]:
    """The layer list of a ``config.json``."""
    layers = []
    for i, e in enumerate(entries):
        where = f"layers[{i}]"
        if e["type"] not in MIXER_CONFIGS:
            raise NotImplementedError(f"{where}: unsupported mixer {e['type']!r}")
        mlp = e.get("mlp")
        layers.append(HybridLayerConfig(e["type"], _fields(MIXER_CONFIGS[e["type"]], e["mixer"], where + ".mixer"),
                                        None if mlp is None else _fields(mlp_config, mlp, where + ".mlp")))
    for i, layer in enumerate(layers):
        m, j = layer.mixer, getattr(layer.mixer, "kv_from", None)
        if j is None:
            continue
        if not 0 <= j < i or layers[j].type != layer.type or layers[j].mixer.kv_from is not None:
            raise ValueError(f"layers[{i}]: no keys of its own in layer {j}")
        if any(getattr(m, n) != getattr(layers[j].mixer, n) for n in ("kv_heads", "dim", "vdim")):
            raise ValueError(f"layers[{i}]: heads differ from those of layer {j}")
    return layers


@dataclass
class LoopConfig:
    """Layers ``start .. stop - 1`` run ``times`` times in a row with the same weights."""
    start: int
    stop: int
    times: int


@dataclass
class HybridConfig:
    """A decoder whose layers each name their mixer and feed-forward, with an optional looped range of layers, dynamic-tanh
    norms, token shift and gated residuals (the Gevonex architecture)."""
    vocab: int
    width: int
    layers: List[HybridLayerConfig]
    norm_eps: float
    loop: Union[LoopConfig, None] = None
    logit_softcap: Union[float, None] = None

    @classmethod
    def from_dict(cls, d: dict) -> "HybridConfig":
        layers = _layers(d["layers"])
        loop = d.get("loop")
        loop = None if loop is None else _fields(LoopConfig, loop, "loop")
        if loop is not None and not (0 <= loop.start < loop.stop <= len(layers) and loop.times >= 1):
            raise ValueError(f"loop: {loop} over {len(layers)} layers")
        return cls(d["vocab"], d["width"], layers, d["norm"]["eps"], loop, d.get("logit_softcap"))

    @property
    def runs(self) -> List[tuple]:
        """``(layer, pass)`` in the order they run; the pass is None outside the loop.  Each run has its own state."""
        n, lp = len(self.layers), self.loop
        if lp is None:
            return [(i, None) for i in range(n)]
        return ([(i, None) for i in range(lp.start)] + [(i, t) for t in range(lp.times) for i in range(lp.start, lp.stop)]
                + [(i, None) for i in range(lp.stop, n)])


@dataclass
class PostNormConfig:
    """A decoder whose layers each name their mixer and feed-forward, with RMS norms on the sublayers' outputs only (the Sugizen
    architecture)."""
    vocab: int
    width: int
    layers: List[HybridLayerConfig]
    norm_eps: float

    @classmethod
    def from_dict(cls, d: dict) -> "PostNormConfig":
        return cls(d["vocab"], d["width"], _layers(d["layers"], ClampedGLUConfig), d["norm"]["eps"])

    @property
    def runs(self) -> List[tuple]:
        return [(i, None) for i in range(len(self.layers))]
