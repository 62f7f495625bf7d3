"""Configuration dataclasses, named and shaped like the reference's (src/config/memory_config.py:6-55
and the msa_config block of the checkpoint's config.json, src/utils/resave_model.py:33-50)."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Union

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
    names = [f for f in cls.__dataclass_fields__]
    unknown = sorted(set(d) - set(names))
    if unknown:
        raise ValueError(f"{where}: unknown keys {unknown}")
    try:
        return cls(**d)
    except TypeError as e:
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
class DenseMLPConfig:
    ff: int
    kind: str = "dense"

    def __post_init__(self):
        if self.kind != "dense":
            raise NotImplementedError(f"unsupported feed-forward {self.kind!r}")


MIXER_CONFIGS = {"mamba2": Mamba2Config, "mingru": MinGRUConfig, "latent_attention": LatentAttentionConfig}


@dataclass
class HybridLayerConfig:
    type: str
    mixer: Union[Mamba2Config, MinGRUConfig, LatentAttentionConfig]
    mlp: Union[DenseMLPConfig, None]


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
        layers = []
        for i, e in enumerate(d["layers"]):
            where = f"layers[{i}]"
            if e["type"] not in MIXER_CONFIGS:
                raise NotImplementedError(f"{where}: unsupported mixer {e['type']!r}")
            mlp = e.get("mlp")
            layers.append(HybridLayerConfig(e["type"], _fields(MIXER_CONFIGS[e["type"]], e["mixer"], where + ".mixer"),
                                            None if mlp is None else _fields(DenseMLPConfig, mlp, where + ".mlp")))
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
