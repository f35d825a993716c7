"""Engine configuration (reference: tinyvllm/config.py:5-26).

The reference needs a local HuggingFace directory and ``transformers.AutoConfig``.  Here
``model`` may also be a plain dict (or a ``ModelConfig``) of architecture numbers, so that
random-init benchmarks and tests need no files; a directory is read through its
``config.json`` only.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field, fields
from typing import Any

import torch


@dataclass
class ModelConfig:
    """The architecture fields the reference reads from ``hf_config`` (models/qwen3.py:139-153)."""
    # what the engine has to know about a design (class attributes, one set per configuration class)
    portioned = False        # prompts may run in portions, in one batch with single decoded tokens
    recurrent = False        # some layers carry a per-sequence state besides the KV cache
    float32 = False          # the design's kernels exist in 32-bit
    position_quirk = True    # the reference's decode position (len instead of len - 1) applies
    long_portion = None      # portions of at least this many tokens run a form of attention of their own
    windows = ()             # the distinct attention windows of that form
    hidden_size: int
    num_hidden_layers: int
    num_attention_heads: int
    num_key_value_heads: int
    intermediate_size: int
    vocab_size: int = 151936
    head_dim: int | None = None
    rms_norm_eps: float = 1e-6
    rope_theta: float = 1e6
    max_position_embeddings: int = 40960
    tie_word_embeddings: bool = False
    hidden_act: str = "silu"
    attention_bias: bool = False
    rope_scaling: Any = None
    torch_dtype: Any = torch.bfloat16

    def __post_init__(self):
        if self.head_dim is None:
            self.head_dim = self.hidden_size // self.num_attention_heads
        if isinstance(self.torch_dtype, str):
            self.torch_dtype = getattr(torch, self.torch_dtype.replace("torch.", ""))

    @classmethod
    def from_any(cls, src) -> "ModelConfig":
        if isinstance(src, cls):
            return src
        if isinstance(src, str):
            with open(os.path.join(src, "config.json")) as f:
                src = json.load(f)
        names = {f.name for f in fields(cls)}
        return cls(**{k: v for k, v in dict(src).items() if k in names})


@dataclass
class LayeredConfig:
    """A design whose ``config.json`` lists its layers one by one, each with its own mixer, sizes and feed-forward."""
    vocab: int
    width: int
    norm: dict
    layers: list
    torch_dtype: Any = torch.bfloat16
    max_position_embeddings: int | None = None    # no limit of its own: the engine's max_model_len

    portioned = True
    recurrent = False
    float32 = True
    position_quirk = False
    tie_word_embeddings = False
    long_portion = None
    windows = ()

    def __post_init__(self):
        if isinstance(self.torch_dtype, str):
            self.torch_dtype = getattr(torch, self.torch_dtype.replace("torch.", ""))
        self.check_layers()

    def check_layers(self):
        raise NotImplementedError

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def layer_runs(self) -> list[int]:
        """Indices of the layers in the order they run."""
        return list(range(len(self.layers)))

    @classmethod
    def from_dict(cls, src: dict, directory: str | None = None):
        import copy
        names = {f.name for f in fields(cls)}
        return cls(**{k: copy.deepcopy(v) for k, v in src.items() if k in names})


@dataclass
class GitopelConfig(LayeredConfig):
    """A Gitopel model: a list of layers, each with its own mixer ('attention' or 'gla') and sizes.

    Keys of ``config.json``: ``vocab``, ``width``, ``norm`` (``groups``, ``eps``) and ``layers``; a layer has ``type``,
    ``mixer`` and ``mlp`` (``kind``, ``ff``, or null).  ``mixer`` of an attention layer: ``heads``, ``kv_heads``, ``dim``,
    ``vdim``, ``scale``, ``rot`` (``dims``, ``base``), ``mask`` (``size``, ``pool``); of a gla layer: ``heads``, ``dim``,
    ``vdim``, ``tau``.  The rank of a gla layer's decay projection is not in the file: it is the row count of its
    first factor (``mixer["rank"]`` once known, 16 if no checkpoint says otherwise)."""
    recurrent = True

    def check_layers(self):
        assert self.width % self.norm["groups"] == 0
        for layer in self.layers:
            m = layer["mixer"]
            if layer["type"] == "attention":
                assert m["heads"] % m["kv_heads"] == 0
                assert m["vdim"] == m["dim"], "the values are the keys: one size"
                assert m["rot"]["dims"] <= m["dim"] and m["mask"]["size"] >= 1 and m["mask"]["pool"] >= 1
            else:
                assert layer["type"] == "gla", f"unknown mixer {layer['type']!r}"
            assert not layer.get("mlp") or layer["mlp"]["kind"] == "dense"

    @classmethod
    def from_dict(cls, src: dict, directory: str | None = None) -> "GitopelConfig":
        cfg = super().from_dict(src)
        if directory is not None:
            shapes = tensor_shapes(directory)
            for i, layer in enumerate(cfg.layers):
                if layer["type"] == "gla":
                    layer["mixer"].setdefault("rank", shapes[f"l{i}.mix.a1"][0])
        return cfg


@dataclass
class GigopelConfig(LayeredConfig):
    """A Gigopel model: parallel layers of windowed latent attention beside a dense or a mixture-of-experts feed-forward.

    Keys of ``config.json``: ``vocab``, ``width``, ``residual_mult``, ``norm`` (``eps``) and ``layers``; a layer has
    ``type`` ('latent_attention'), ``mixer`` (``heads``, ``dim``, ``rot_dim``, ``vdim``, ``kv_rank``, ``scale``, ``rot``:
    ``dims``, ``base``, ``mask``: ``size``) and ``mlp``: null, ``kind`` 'dense' with ``ff``, or ``kind`` 'moe' with
    ``expert`` (``ff``, ``limit``) and ``router`` (``experts``, ``top``)."""
    residual_mult: float = 1.0

    # from about this many tokens on it costs less to expand the keys and values of every head than to attend in the
    # latent space (2 rank + rot_dim instead of dim + rot_dim + vdim products per head, query and key)
    long_portion = 128

    def check_layers(self):
        for layer in self.layers:
            assert layer["type"] == "latent_attention", f"unknown mixer {layer['type']!r}"
            m, mlp = layer["mixer"], layer.get("mlp")
            assert m["rot"]["dims"] == m["rot_dim"] and m["rot_dim"] % 2 == 0 and m["mask"]["size"] >= 1
            assert not mlp or mlp["kind"] in ("dense", "moe")
            if mlp and mlp["kind"] == "moe":
                assert 1 <= mlp["router"]["top"] <= mlp["router"]["experts"]
        self.windows = tuple(sorted({layer["mixer"]["mask"]["size"] for layer in self.layers}))


@dataclass
class ZuzunexConfig(LayeredConfig):
    """A Zuzunex model: grouped-query attention with sinks and output gates, and SwiGLU feed-forwards or mixtures of experts.

    Keys of ``config.json``: ``vocab``, ``width``, ``logit_scale``, ``norm`` (``eps``), ``loop`` (null, or layers ``start`` ..
    ``stop - 1`` run ``times`` times in a row) and ``layers``; a layer has ``type``, ``mixer`` and ``mlp``.  Mixers have ``heads``,
    ``kv_heads``, ``dim``, ``vdim``, ``scale``; 'attention' also ``q_temp`` (``coef``, ``every``) and ``softcap``, 'attention_2'
    ``conv`` (taps) and ``rot`` (``dims``, ``base``, ``scaling``: null or ``factor``, ``original``, ``fast``, ``slow``).  ``mlp``:
    null, ``kind`` 'dense' with ``ff``, or ``kind`` 'moe' with ``expert`` (``ff``), ``router`` (``experts``, ``identity``, ``top``)
    and ``shared`` (``ff``)."""
    logit_scale: float = 1.0
    loop: dict | None = None

    # from this many tokens on a portion's rows share the keys of a tile; shorter portions run row by row
    long_portion = 16

    def check_layers(self):
        for layer in self.layers:
            assert layer["type"] in ("attention", "attention_2"), f"unknown mixer {layer['type']!r}"
            m, mlp = layer["mixer"], layer.get("mlp")
            assert m["heads"] % m["kv_heads"] == 0
            rot = m.get("rot")
            assert not rot or (rot["dims"] % 2 == 0 and rot["dims"] <= m["dim"])
            assert not mlp or mlp["kind"] in ("dense", "moe")
            if mlp and mlp["kind"] == "moe":
                r = mlp["router"]
                assert 1 <= r["top"] <= r["experts"] + (r.get("identity") or 0)
        if self.loop:
            assert 0 <= self.loop["start"] <= self.loop["stop"] <= len(self.layers) and self.loop["times"] >= 1
        # a convolution has a state
        self.recurrent = any(layer["type"] == "attention_2" and layer["mixer"].get("conv") for layer in self.layers)

    def layer_runs(self) -> list[int]:
        if not self.loop:
            return super().layer_runs()
        start, stop = self.loop["start"], self.loop["stop"]
        return [*range(start), *list(range(start, stop)) * self.loop["times"], *range(stop, len(self.layers))]


NO_WINDOW = 1 << 30      # an attention window that every position is inside of


@dataclass
class TibenexConfig(LayeredConfig):
    """A Tibenex model: post-norm layers of latent attention, of attention whose heads mix their weights or of a state-space
    recurrence, each with an optional dense feed-forward, and a token shift in front of every mixer.

    Keys of ``config.json``: ``vocab``, ``width``, ``embedding`` (``scale``), ``postln_alpha``, ``norm`` (``eps``) and ``layers``; a
    layer has ``type``, ``mixer`` and ``mlp`` (null, or ``kind`` 'dense' with ``ff``).  ``mixer`` of 'latent_attention': ``heads``,
    ``dim``, ``rot_dim``, ``vdim``, ``q_rank``, ``kv_rank``, ``scale``, ``rot`` (``dims``, ``base``, ``scaling``: null or ``factor``,
    ``original``, ``fast``, ``slow``); of 'attention': ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``rot``; of 'mamba2':
    ``heads``, ``vdim``, ``state``, ``groups``, ``conv`` (taps), ``norm_groups``."""
    embedding: dict | None = None
    postln_alpha: float = 1.0

    recurrent = True         # every layer keeps the row before

    # portions from about this many tokens on expand the keys and values of latent attention, and share the keys of a tile
    # in the others; shorter ones run row by row
    long_portion = 128

    @property
    def embedding_scale(self) -> float:
        return float((self.embedding or {}).get("scale", 1.0))

    def check_layers(self):
        for layer in self.layers:
            m, kind, mlp = layer["mixer"], layer["type"], layer.get("mlp")
            if kind == "latent_attention":
                assert m["rot"]["dims"] == m["rot_dim"] and m["rot_dim"] % 2 == 0 and m["q_rank"] >= 1
            elif kind == "attention":
                assert m["heads"] % m["kv_heads"] == 0
                assert not m.get("rot") or (m["rot"]["dims"] % 2 == 0 and m["rot"]["dims"] <= m["dim"])
            else:
                assert kind == "mamba2", f"unknown mixer {kind!r}"
                assert m["heads"] % m["groups"] == 0 and m["conv"] >= 1 and m["heads"] * m["vdim"] % m["norm_groups"] == 0
            assert not mlp or mlp["kind"] == "dense"
        if any(layer["type"] == "latent_attention" for layer in self.layers):
            self.windows = (NO_WINDOW,)


def tensor_shapes(directory: str) -> dict:
    """name -> shape of every tensor in ``directory/*.safetensors``, from the files' headers."""
    from glob import glob
    out = {}
    for file in sorted(glob(os.path.join(directory, "*.safetensors"))):
        with open(file, "rb") as f:
            header = json.loads(f.read(int.from_bytes(f.read(8), "little")))
        out.update({k: tuple(v["shape"]) for k, v in header.items() if k != "__metadata__"})
    return out


LAYERED_DESIGNS = {"Gitopel": GitopelConfig, "Gigopel": GigopelConfig, "Zuzunex": ZuzunexConfig, "Tibenex": TibenexConfig}


def architecture_of(src: dict) -> str:
    """The design a ``config.json`` names: ``architecture``, or the first of ``architectures``; Qwen3 when it names none."""
    name = src.get("architecture") or (src.get("architectures") or ["Qwen3ForCausalLM"])[0]
    return name.removesuffix("ForCausalLM")


def model_config(src):
    """Configuration object from a configuration object, a dict of its keys or a checkpoint directory."""
    if isinstance(src, (ModelConfig, LayeredConfig)):
        return src
    directory = None
    if isinstance(src, str):
        directory = src
        with open(os.path.join(src, "config.json")) as f:
            src = json.load(f)
    name = architecture_of(src)
    if name in LAYERED_DESIGNS:
        return LAYERED_DESIGNS[name].from_dict(src, directory)
    if name == "Qwen3":
        return ModelConfig.from_any(src)
    raise ValueError(f"no model of this framework has the architecture {name!r}")


# Architectures named by the benchmark configurations (Qwen3 family shapes).
QWEN3_SHAPES = {
    "qwen3-0.6b": dict(hidden_size=1024, num_hidden_layers=28, num_attention_heads=16, num_key_value_heads=8,
                       head_dim=128, intermediate_size=3072, tie_word_embeddings=True),
    "qwen3-8b": dict(hidden_size=4096, num_hidden_layers=36, num_attention_heads=32, num_key_value_heads=8,
                     head_dim=128, intermediate_size=12288, tie_word_embeddings=False),
    "qwen3-32b": dict(hidden_size=5120, num_hidden_layers=64, num_attention_heads=64, num_key_value_heads=8,
                      head_dim=128, intermediate_size=25600, tie_word_embeddings=False),
}


@dataclass
class Config:
    model: Any                              # directory, dict, ModelConfig or a key of QWEN3_SHAPES
    max_num_batched_tokens: int = 16384
    max_num_seqs: int = 512
    max_model_len: int = 4096
    gpu_memory_utilization: float = 0.9
    tensor_parallel_size: int = 1
    enforce_eager: bool = False
    hf_config: ModelConfig | None = None
    eos: int = -1
    kvcache_block_size: int = 256
    num_kvcache_blocks: int = -1
    # additions of this build (the reference has neither)
    quantization: str | None = None         # None (bf16 linears) or "w8a16"
    kv_cache_dtype: str = "bf16"            # "bf16" or "fp8_e4m3"
    # static scales of an e4m3 cache, c = e4m3(sat(x / scale)): a float, [Hkv] values or [L][Hkv] values.
    # 1/16 represents |x| <= 28 (448 / 16); larger K or V entries saturate.
    kv_k_scale: Any = 1.0 / 16
    kv_v_scale: Any = 1.0 / 16
    dtype: str | None = None                # "bfloat16" or "float32" instead of the model configuration's own
    num_state_slots: int = -1               # recurrent designs: sequences that can be live at once (-1: max_num_seqs)
    seed: int = 0                           # random-init seed when no weights are given
    decode_position_quirk: bool = True      # reference feeds positions = len(seq) in decode (model_runner.py:219)
    # Decode steps of sequences that can only end by length (ignore_eos) are launched before the token ids of
    # the step before them have been read back: the ids stay on the device as the next step's input, the host
    # keeps two steps in flight and patches the values into its sequences as they arrive.  Same tokens, same
    # block ids and step counts as the step-by-step loop; False restores that loop.
    run_ahead: bool = True
    # The decode attention kernel's split of the step's work over the workgroups is made once per step (one small
    # kernel at the head of the step) instead of by every layer's call: same results, a shorter start per layer.
    decode_plan: bool = True

    def __post_init__(self):
        if isinstance(self.model, str) and self.model.lower() in QWEN3_SHAPES:
            self.hf_config = ModelConfig.from_any(QWEN3_SHAPES[self.model.lower()])
        elif isinstance(self.model, str):
            assert os.path.isdir(self.model), f"{self.model} is neither a known shape nor a directory"
            self.hf_config = model_config(self.model)
        else:
            self.hf_config = model_config(self.model)
        hf = self.hf_config
        if self.dtype is not None:
            hf.torch_dtype = getattr(torch, self.dtype)
        if hf.torch_dtype != torch.bfloat16 and not (hf.float32 and hf.torch_dtype == torch.float32):
            raise ValueError(f"no {hf.torch_dtype} kernels for this model")
        assert self.kvcache_block_size % (64 if hf.portioned else 256) == 0
        assert self.tensor_parallel_size == 1, "this build runs one GPU, no tensor parallelism"
        assert self.quantization in (None, "w8a16")
        assert self.kv_cache_dtype in ("bf16", "fp8_e4m3")
        if hf.portioned:
            assert self.kv_cache_dtype == "bf16", "the caches of this design are held in its own dtype"
            assert self.quantization is None or hf.torch_dtype == torch.bfloat16
        if not hf.position_quirk:
            self.decode_position_quirk = False
        if hf.max_position_embeddings is None:
            hf.max_position_embeddings = self.max_model_len
        if self.num_state_slots < 0:
            self.num_state_slots = self.max_num_seqs
        self.max_model_len = min(self.max_model_len, hf.max_position_embeddings)
        # a design that takes its prompts whole must fit the longest one into a step
        assert hf.portioned or self.max_num_batched_tokens >= self.max_model_len
