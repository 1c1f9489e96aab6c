"""Model shape: the reference's RavenConfig (recpre/raven_config_minimal.py:7-99) as a transformers configuration
class, with the same field names, defaults, `attribute_map` and derived values, so a reference `config.json` loads
unchanged and `AutoConfig` resolves the model type `huginn_raven` to it (registration: raven_modeling_minimal.py:2312-2323).
Only the fields that shape inference are declared; the training-only keys of a reference file are kept as plain
attributes and written back on save."""

from __future__ import annotations

from math import sqrt

from transformers import PretrainedConfig

_NOISE_TYPES = ("geom", "sqrt", "line", "chi", "fixed")  # RMM:818-833


class RavenConfig(PretrainedConfig):
    model_type = "huginn_raven"
    keys_to_ignore_at_inference = [""]
    attribute_map = {"num_attention_heads": "n_heads", "hidden_size": "n_embd", "num_hidden_layers": "n_layers"}

    n_embd: int = 5280
    n_heads: int = 55
    n_layers: int = 8  # prelude + recurrent block + coda
    block_size: int = 4096
    vocab_size: int = 65536
    padding_multiple: int = 4096
    tie_embeddings: bool = True
    intermediate_size: int = 17920
    bias: bool = False
    norm_eps: float = 0.000001
    n_layers_in_recurrent_block: int = 4
    mean_recurrence: int = 32
    mean_backprop_depth: int = 8
    n_layers_in_prelude: int = 2
    n_layers_in_coda: int = 2
    qk_bias: bool = True
    rope_base: float = 50_000
    test_time_noise: float = 0
    test_time_noise_type: str = "fixed"

    def __post_init__(self, **kwargs):
        for alias, field in self.attribute_map.items():  # a file may name a field by its transformers-wide alias
            if kwargs.get(alias) is not None:
                setattr(self, field, kwargs[alias])
        if self.test_time_noise_type not in _NOISE_TYPES:
            raise ValueError(f"unknown test_time_noise_type {self.test_time_noise_type!r}")
        if self.test_time_noise < 0:
            raise ValueError("test_time_noise must not be negative")
        if self.bias:
            raise ValueError("bias=True is not supported: the reference model family has no Linear biases")
        if self.n_embd % self.n_heads:
            raise ValueError(f"n_embd {self.n_embd} is not divisible by n_heads {self.n_heads}")
        # derived values (raven_config_minimal.py:78-91); a file that stores them stores the same numbers
        for derived in ("padded_vocab_size", "num_key_value_heads", "num_attention_heads", "head_dim", "effective_expected_depth",
                        "init_values", "hidden_size", "num_hidden_layers"):
            kwargs.pop(derived, None)
        self.padded_vocab_size = self.vocab_size
        self.num_key_value_heads = self.n_heads
        self.head_dim = self.n_embd // self.n_heads
        self.effective_expected_depth = (self.n_layers_in_prelude + self.n_layers_in_coda
                                         + self.n_layers_in_recurrent_block * self.mean_recurrence)
        std = sqrt(2 / (5 * self.n_embd))
        self.init_values = {"std": std, "out_proj": std / sqrt(2 * self.effective_expected_depth), "embedding": std,
                            "embed_scale": sqrt(self.n_embd)}
        kwargs.pop("model_type", None)
        kwargs["tie_word_embeddings"] = self.tie_embeddings  # raven_config_minimal.py:93-99
        if self.dtype is None and kwargs.get("torch_dtype") is None:
            self.dtype = "bfloat16"  # the reference's default `torch_dtype`
        super().__post_init__(**kwargs)

    @classmethod
    def tiny(cls) -> "RavenConfig":
        """The CPU-runnable plumbing shape."""
        return cls(n_embd=256, n_heads=4, n_layers=4, n_layers_in_prelude=1, n_layers_in_recurrent_block=2,
                   n_layers_in_coda=1, intermediate_size=704, vocab_size=1024, mean_recurrence=4)


class GitipelConfig(PretrainedConfig):
    """Shape of a Gitipel decoder, with the field names of its `config.json`: an embedding scale, a list of layers (each a mixer
    with its sizes and a feed-forward or none), an optional stretch of layers that runs several times with a state per
    pass, and the constants of norm, input convolution and output.  Every size comes from here, except the rank of the delta
    rule's decay projection, which the weights give (`mixer["rank"]`)."""

    model_type = "gitipel"
    attribute_map = {"vocab_size": "vocab", "hidden_size": "width", "n_embd": "width"}

    architecture: str = "Gitipel"
    vocab: int = 256
    width: int = 64
    layers: list | None = None
    embedding: dict | None = None
    norm: dict | None = None
    canon: dict | None = None
    loop: dict | None = None
    logit_scale: float = 1.0

    def __post_init__(self, **kwargs):
        for alias, field in self.attribute_map.items():
            if kwargs.get(alias) is not None:
                setattr(self, field, kwargs[alias])
            kwargs.pop(alias, None)
        kwargs.pop("model_type", None)
        kwargs.pop("num_hidden_layers", None)
        self.layers = [dict(x) for x in (self.layers or [])]
        self.embedding = self.embedding or {"scale": 1.0}
        self.norm = self.norm or {"eps": 1e-5}
        if self.architecture != "Gitipel":
            raise ValueError(f"not a Gitipel configuration: architecture {self.architecture!r}")
        for i, layer in enumerate(self.layers):
            m = layer["mixer"]
            if layer["type"] == "attention":
                if m["heads"] % m["kv_heads"]:
                    raise ValueError(f"layer {i}: {m['heads']} query heads over {m['kv_heads']} key heads")
                if m.get("vdim", m["dim"]) != m["dim"]:
                    raise ValueError(f"layer {i}: the keys are the values, so vdim {m['vdim']} must be dim {m['dim']}")
            elif layer["type"] != "general_delta":
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer.get("mlp") is not None and layer["mlp"]["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp']['kind']!r}")
        if self.loop is not None and not 0 <= self.loop["start"] < self.loop["stop"] <= len(self.layers):
            raise ValueError(f"loop {self.loop} over {len(self.layers)} layers")
        self.num_hidden_layers = len(self.layers)
        kwargs["tie_word_embeddings"] = False
        if self.dtype is None and kwargs.get("torch_dtype") is None:
            self.dtype = "bfloat16"
        super().__post_init__(**kwargs)

    def runs(self) -> list:
        """(layer, pass) in the order they run; pass is None outside the loop."""
        n, loop = len(self.layers), self.loop
        if loop is None:
            return [(i, None) for i in range(n)]
        inside = [(i, t) for t in range(loop["times"]) for i in range(loop["start"], loop["stop"])]
        return [(i, None) for i in range(loop["start"])] + inside + [(i, None) for i in range(loop["stop"], n)]


class GupitarConfig(PretrainedConfig):
    """Shape of a Gupitar decoder, with the field names of its `config.json`: a list of layers, each a mixer (latent attention or a real-gated
    linear recurrent unit) with its sizes and a feed-forward (dense, a mixture of experts, or none).  Every size and constant comes
    from here."""

    model_type = "gupitar"
    attribute_map = {"vocab_size": "vocab", "hidden_size": "width", "n_embd": "width"}

    architecture: str = "Gupitar"
    vocab: int = 256
    width: int = 64
    layers: list | None = None
    norm: dict | None = None

    def __post_init__(self, **kwargs):
        for alias, field in self.attribute_map.items():
            if kwargs.get(alias) is not None:
                setattr(self, field, kwargs[alias])
            kwargs.pop(alias, None)
        kwargs.pop("model_type", None)
        kwargs.pop("num_hidden_layers", None)
        self.layers = [dict(x) for x in (self.layers or [])]
        self.norm = self.norm or {"eps": 1e-6}
        if self.architecture != "Gupitar":
            raise ValueError(f"not a Gupitar configuration: architecture {self.architecture!r}")
        for i, layer in enumerate(self.layers):
            self._check_mixer(i, layer["type"], layer["mixer"])
            mlp = layer.get("mlp")
            if mlp is None or mlp["kind"] == "dense":
                continue
            if mlp["kind"] != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            if not 1 <= mlp["router"]["top"] <= mlp["router"]["experts"]:
                raise ValueError(f"layer {i}: top {mlp['router']['top']} of {mlp['router']['experts']} experts")
        self.num_hidden_layers = len(self.layers)
        kwargs["tie_word_embeddings"] = False
        if self.dtype is None and kwargs.get("torch_dtype") is None:
            self.dtype = "bfloat16"
        super().__post_init__(**kwargs)

    def _check_mixer(self, i: int, kind: str, m: dict) -> None:
        if kind == "rglru":
            if m["width"] % m["blocks"]:
                raise ValueError(f"layer {i}: {m['blocks']} blocks over {m['width']} channels")
            return
        if kind != "latent_attention":
            raise ValueError(f"layer {i}: unknown mixer {kind!r}")
        if m["rot_dim"] % 2 or m["rot"]["dims"] != m["rot_dim"]:
            raise ValueError(f"layer {i}: a rotation of {m['rot']['dims']} of {m['rot_dim']} rotated dimensions")
        if m.get("mask") is not None and m["mask"]["size"] < 1:
            raise ValueError(f"layer {i}: a window of {m['mask']['size']}")
        source = m.get("kv_from")
        if source is None:
            return
        if not 0 <= source < i or self.layers[source]["type"] != "latent_attention" or self.layers[source]["mixer"].get("kv_from") is not None:
            raise ValueError(f"layer {i}: reads the latents of layer {source}, which must come earlier and have latents of its own")
        other = self.layers[source]["mixer"]
        if any(other[k] != m[k] for k in ("kv_rank", "rot_dim")) or other["rot"]["base"] != m["rot"]["base"]:
            raise ValueError(f"layer {i}: kv_rank, rot_dim and rotation must equal those of layer {source}")
