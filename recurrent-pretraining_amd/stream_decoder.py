"""Decoders over an fp32 residual stream: a list of pre-norm layers, each a choice of mixer and feed-forward, described to the kernels
by one structure per layer (hip.MixerLayer) and run by one call into libraven_hip.so per layer.

StreamDecoderForCausalLM holds what such models share: weights in the kernels' layout, loading and saving, the pass over token
rows, the cache (cache.MixerStateCache), generation and sampling (generation.MinimalGeneration) and graph replay of decode steps
(generation.GraphedStep).  A model family (gitipel.py, gupitar.py) builds the layers.

Weights are kept as the kernels read them: the projections of a mixer fused into one matrix, every width rounded up to a multiple
of 8 with zeros (so that any size gives 16-byte rows), heads likewise.  `Weights.placements` maps each tensor of a checkpoint to the
strided views of those buffers it fills."""

from __future__ import annotations

from typing import Callable, Dict, List, Optional, Union

import torch
from transformers import GenerationMixin, PretrainedConfig, PreTrainedModel

from . import checkpoint, hip
from .cache import MixerStateCache
from .generation import CausalLMOutputRecurrentLatents, GraphedStep, MinimalGeneration


def pad8(n: int) -> int:
    return (n + 7) // 8 * 8


class Placement:
    """Where a checkpoint tensor goes: `parts`, views that together hold it (each with the part of the tensor, seen in `seen_as` shape,
    that it takes), and `derived`, buffers that hold a function of it."""

    def __init__(self, shape: tuple):
        self.shape = shape
        self.parts: List[tuple] = []    # (view, seen_as, index)
        self.derived: List[tuple] = []  # (view, function of the float tensor)

    def fill(self, tensor: torch.Tensor) -> None:
        for view, seen_as, index in self.parts:
            view.copy_(tensor.reshape(seen_as)[index].reshape(view.shape))
        for view, fn in self.derived:
            view.copy_(fn(tensor.float()).reshape(view.shape))

    def read(self) -> torch.Tensor:
        view, seen_as, index = self.parts[0]
        if len(self.parts) == 1 and view.numel() == torch.Size(self.shape).numel():
            return view.reshape(self.shape)
        out = torch.empty(seen_as, dtype=view.dtype, device=view.device)
        for view, seen_as, index in self.parts:
            part = out.view(seen_as)[index]
            part.copy_(view.reshape(part.shape))
        return out.view(self.shape)


class Weights:
    """Zero-initialised buffers and the checkpoint tensors that fill parts of them."""

    def __init__(self, device, dtype):
        self.device, self.dtype = device, dtype
        self.placements: Dict[str, Placement] = {}

    def matrix(self, *shape) -> torch.Tensor:
        return torch.zeros(*shape, dtype=self.dtype, device=self.device)

    def vector(self, *shape) -> torch.Tensor:
        return torch.zeros(*shape, dtype=torch.float32, device=self.device)

    def place(self, name: str, view: torch.Tensor, *shape, seen_as: Optional[tuple] = None, index=slice(None)) -> None:
        """`view` takes the whole tensor of `shape`, or tensor.view(seen_as)[index]; several calls for one name add up."""
        self.placements.setdefault(name, Placement(tuple(shape))).parts.append((view, tuple(seen_as or shape), index))

    def derive(self, name: str, view: torch.Tensor, fn: Callable) -> None:
        """`view` holds fn(tensor) of a placed tensor."""
        self.placements[name].derived.append((view, fn))

    def fill(self, name: str, tensor: torch.Tensor) -> None:
        p = self.placements[name]
        if tuple(tensor.shape) != p.shape:
            raise ValueError(f"{name}: checkpoint shape {tuple(tensor.shape)} != model shape {p.shape}")
        p.fill(tensor)


class StreamDecoderForCausalLM(MinimalGeneration, PreTrainedModel, GenerationMixin):
    """A family sets config_class and KERNEL_SOURCES and implements build(weights), which creates embed, layers (each with `native`, a
    hip.MixerLayer, and `plan`, what the cache keeps for it), final_norm and head; where layers run several times, layer_runs() and
    enter_run()."""

    base_model_prefix = "model"
    _tied_weights_keys = {}
    KERNEL_SOURCES: tuple = ()        # the csrc files a library for this family alone is built from
    max_positions = None              # no positional table: the cache alone bounds a sequence
    ROWS_PER_CALL = 16384             # token rows of one pass through the layers; longer prompts run in portions
    embed_scale = 1.0
    logit_scale = 1.0
    keeps_embedding = False           # the rounded embedding rows stay available to enter_run()

    def __init__(self, config: PretrainedConfig, device: Union[str, torch.device, None] = None, dtype: Optional[torch.dtype] = None):
        super().__init__(config)
        if device is None:
            device = "cuda" if torch.cuda.is_available() else "cpu"
        dtype = dtype if dtype is not None else (config.dtype if isinstance(config.dtype, torch.dtype) else torch.bfloat16)
        self._device, self._dtype = torch.device(device), dtype
        self.weights = Weights(self._device, dtype)
        self.dims = hip.StreamDims(config.width, pad8(config.width), config.norm["eps"], hip.dtype_code(dtype))
        self.build(self.weights)
        self.runs = self.layer_runs()
        self._scratch_cache: Optional[MixerStateCache] = None
        self.eval()

    # ---- what a family supplies --------------------------------------------------------------------
    def build(self, w: Weights) -> None:
        raise NotImplementedError

    def layer_runs(self) -> list:
        """(layer, pass) in the order they run; pass is None outside a loop."""
        return [(i, None) for i in range(len(self.layers))]

    def enter_run(self, layer: int, turn: Optional[int], buf: dict) -> None:
        """Called before a layer runs in pass `turn`."""

    def initial_mean(self, name: str) -> float:
        """Mean of the synthetic values of a checkpoint tensor (init_weights)."""
        return 0.0

    @classmethod
    def complete_config(cls, raw: dict, path: str) -> dict:
        """Sizes that only the weights give, added to a configuration read from `path`."""
        return raw

    @property
    def dtype(self) -> torch.dtype:
        return self._dtype

    @property
    def device(self) -> torch.device:
        return self._device

    # ---- weights ---------------------------------------------------------------------------------
    def state_dict(self, *args, **kwargs) -> Dict[str, torch.Tensor]:
        """The checkpoint's tensors, read back out of the kernels' buffers (matrices in the model's dtype, vectors float)."""
        return {name: p.read() for name, p in self.weights.placements.items()}

    @torch.no_grad()
    def load_state_dict(self, state, strict: bool = True, assign: bool = False):
        missing = [n for n in self.weights.placements if n not in state]
        unexpected = [n for n in state if n not in self.weights.placements]
        if strict and (missing or unexpected):
            raise KeyError(f"checkpoint does not match the model: missing {missing[:8]}, unexpected {unexpected[:8]}")
        for name, tensor in state.items():
            if name in self.weights.placements:
                self.weights.fill(name, tensor)
        return torch.nn.modules.module._IncompatibleKeys(missing, unexpected)

    @classmethod
    @torch.no_grad()
    def from_pretrained(cls, path: str, *args, device: Union[str, torch.device, None] = None, dtype: Optional[torch.dtype] = None,
                        config: Optional[PretrainedConfig] = None, **kwargs) -> "StreamDecoderForCausalLM":
        """A local directory with config.json and safetensors (checkpoint.py)."""
        dtype = dtype if dtype is not None else kwargs.pop("torch_dtype", None)
        if isinstance(dtype, str):
            dtype = None if dtype == "auto" else getattr(torch, dtype)
        raw = checkpoint.read_config(path) if config is None else config.to_dict()
        model = cls(cls.config_class(**cls.complete_config(raw, path)), device=device if device is not None else kwargs.get("device_map"), dtype=dtype)
        seen = set()
        for name, tensor in checkpoint.tensors(path):
            if name not in model.weights.placements:
                raise KeyError(f"checkpoint does not match the model: unexpected {name}")
            model.weights.fill(name, tensor)
            seen.add(name)
        missing = [n for n in model.weights.placements if n not in seen]
        if missing:
            raise KeyError(f"checkpoint does not match the model: missing {missing[:8]}")
        return model

    def save_pretrained(self, path: str, max_shard_bytes: int = 5 * 2 ** 30, **unused) -> None:
        cfg = self.config.to_dict()
        cfg.update(architectures=[type(self).__name__], torch_dtype=str(self.dtype).replace("torch.", ""))
        cfg["dtype"] = cfg["torch_dtype"]
        checkpoint.write(path, cfg, self.state_dict(), max_shard_bytes)

    @torch.no_grad()
    def init_weights(self, seed: Optional[int] = None, std: float = 0.02) -> None:
        """Synthetic weights drawn on the model's device: every tensor ~ N(initial_mean(name), std)."""
        if seed is None:
            return
        g = torch.Generator(device=self.device).manual_seed(seed)
        for name, p in self.weights.placements.items():
            p.fill(torch.empty(p.shape, dtype=torch.float32, device=self.device).normal_(self.initial_mean(name), std, generator=g))

    # ---- cache -----------------------------------------------------------------------------------
    def new_cache(self, max_length: Optional[int] = None) -> MixerStateCache:
        return MixerStateCache([self.layers[i].plan for i, _ in self.runs], max_length=max_length)

    def _generation_cache(self, model_kwargs: dict, cache_lookup_strategy: str, batch: int, max_length: Optional[int] = None):
        given = model_kwargs.get("past_key_values")
        return given if given is not None else self.new_cache(max_length)

    @classmethod
    def _supports_default_dynamic_cache(cls) -> bool:
        return False

    # ---- the pass over token rows ------------------------------------------------------------------
    def _row_buffers(self, B: int, S: int, pos0: int = 0) -> dict:
        M, Dp = B * S, self.dims.ld
        if self._device.type != "cuda":
            raise hip.RavenHipError("the forward runs on the GPU; there is no CPU path")
        row = lambda dt: torch.empty(M, Dp, dtype=dt, device=self.device)
        n = max((hip.mixer_layer_workspace_bytes(self.dims, layer.native, B, S, pos0) for layer in self.layers), default=0)
        lin = hip.load().raven_linear_workspace_bytes(M, max(Dp, self.config.vocab)) if 1 < M <= 32 else 0
        keep = self.keeps_embedding
        return {"x": row(torch.float32), "x0": row(self.dtype) if keep else None, "xr": row(self.dtype) if keep else None,
                "ws": torch.empty(max(n, lin, 256), dtype=torch.uint8, device=self.device)}

    def _stream(self, ids: torch.Tensor, buf: dict, cache: MixerStateCache, B: int, S: int, pos0: int, pos_dev=None, trail: Optional[list] = None):
        """Embedding and every layer run for rows ids [B*S]; leaves the stream in buf["x"]."""
        x = buf["x"]
        hip.embed_stream(self.embed, ids, self.embed_scale, x, buf["x0"])
        for run, (i, t) in enumerate(self.runs):
            self.enter_run(i, t, buf)
            hip.mixer_layer(self.dims, self.layers[i].native, cache.native(run), x, B, S, pos0, buf["ws"], pos_dev=pos_dev)
            if trail is not None:
                trail.append(x[:, :self.config.width].clone())
        return x

    def _logits(self, x: torch.Tensor, h: torch.Tensor, out: torch.Tensor, ws) -> torch.Tensor:
        cfg = self.config
        if x.shape[0] == 1 and hip.gemv_stream_fits(self.dims.ld, self.dtype):
            return hip.gemv_stream(x, self.final_norm, cfg.width, cfg.norm["eps"], self.head, self.dtype, scale=self.logit_scale, out=out)
        hip.norm_conv(x, self.final_norm, cfg.width, cfg.norm["eps"], x.shape[0], 1, self.dtype, out=h)
        return hip.linear_epilogue(h, self.head, scale=self.logit_scale, out=out, workspace=ws)

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor, past_key_values: Optional[MixerStateCache] = None, use_cache: bool = False,
                logit_positions=None, logits_to_keep: int = 0, labels: Optional[torch.Tensor] = None, output_hidden_states: bool = False,
                output_details: Optional[dict] = None, **unused) -> CausalLMOutputRecurrentLatents:
        """input_ids [B, S]: the next tokens of B sequences of equal length.  logit_positions: the places among the S tokens whose
        logits are wanted (None: all, or the last `logits_to_keep`).  hidden_states: the stream after every layer run.  Positions
        follow from the cache; attention masks, position ids and the recurrent family's keywords have nothing to act on."""
        B, S = input_ids.shape
        cache = past_key_values
        if cache is None:
            cache = self.new_cache() if use_cache else self._private_cache()
        if not isinstance(cache, MixerStateCache):
            raise TypeError("past_key_values must be this package's MixerStateCache")
        if logit_positions is None:
            logit_positions = range(S - logits_to_keep, S) if logits_to_keep else range(S)
        wanted = list(logit_positions)
        V = self.config.vocab
        logits = torch.empty(B, len(wanted), V, dtype=torch.float32, device=self.device)
        trails = []
        cache.ensure(B, cache.get_seq_length() + S, self.dtype, self.device)
        portion = max(1, self.ROWS_PER_CALL // B)
        ids = input_ids.to(self.device, torch.int64)
        for lo in range(0, S, portion):
            n = min(portion, S - lo)
            buf = self._row_buffers(B, n, cache.get_seq_length())
            trail: Optional[list] = [] if output_hidden_states else None
            x = self._stream(ids[:, lo:lo + n].reshape(-1).contiguous(), buf, cache, B, n, cache.get_seq_length(), trail=trail)
            cache.advance(n)
            if trail is not None:
                trails.append(torch.stack(trail).view(len(trail), B, n, -1))
            here = [k for k, p in enumerate(wanted) if lo <= p < lo + n]
            if here:
                rows = x.view(B, n, -1)
                if [wanted[k] for k in here] != list(range(lo, lo + n)):
                    rows = rows[:, torch.tensor([wanted[k] - lo for k in here], device=self.device)]
                rows = rows.reshape(B * len(here), -1).contiguous()
                h = torch.empty(rows.shape, dtype=self.dtype, device=self.device)
                lws = hip.linear_workspace(rows.shape[0], V, self.device) if 1 < rows.shape[0] <= 32 else None
                straight = here == list(range(here[0], here[-1] + 1)) and (B == 1 or len(here) == len(wanted))
                y = (logits[:, here[0]:here[-1] + 1].view(rows.shape[0], V) if straight else
                     torch.empty(rows.shape[0], V, dtype=torch.float32, device=self.device))
                self._logits(rows, h, y, lws)
                if not straight:
                    logits[:, here] = y.view(B, len(here), V)
        loss = torch.as_tensor(0.0)
        if labels is not None:
            loss = torch.nn.functional.cross_entropy(logits.view(-1, V), labels.to(self.device).view(-1), ignore_index=-100)
        return CausalLMOutputRecurrentLatents(loss=loss, log_ppl=loss.clone(), logits=logits,
                                              past_key_values=cache if (use_cache or past_key_values is not None) else None,
                                              hidden_states=torch.cat(trails, 2) if output_hidden_states else None)

    def _private_cache(self) -> MixerStateCache:
        """For a forward without a cache: one that is used again."""
        if self._scratch_cache is None:
            self._scratch_cache = self.new_cache()
        self._scratch_cache.reset()
        return self._scratch_cache

    # ---- generation ------------------------------------------------------------------------------
    def decode_runner(self, cache, batch: int, num_steps=None, greedy: bool = True, use_graph: bool = True) -> "MixerDecodeRunner":
        return MixerDecodeRunner(self, cache, batch, use_graph=use_graph)

    def prepare_inputs_for_generation(self, input_ids, past_key_values=None, **kwargs):
        """What transformers' loop calls before every forward: the tokens the cache has not seen."""
        if past_key_values is not None and not isinstance(past_key_values, MixerStateCache):
            if past_key_values.get_seq_length() != 0:
                raise ValueError("only an empty cache of another class can be replaced by a MixerStateCache")
            past_key_values = None
        if past_key_values is None:
            past_key_values = self.new_cache()
        return {"input_ids": input_ids[:, past_key_values.get_seq_length():].contiguous(), "past_key_values": past_key_values, "use_cache": True}

    @torch.no_grad()
    def generate(self, input_ids: Optional[torch.Tensor] = None, generation_config=None, **kwargs):
        """GenerationSettings or one of the minimal loop's keywords: generate_minimal; every other call: transformers' loop over
        this forward."""
        from .generation import GenerationSettings
        if any(k in kwargs for k in self._MINIMAL_LOOP_KEYS) or isinstance(generation_config, GenerationSettings):
            return self.generate_minimal(input_ids, generation_config, **kwargs)
        if generation_config is not None:
            kwargs["generation_config"] = generation_config
        return super().generate(input_ids, **kwargs)


class MixerDecodeRunner(GraphedStep):
    """One decode step (a token per sequence) with every buffer preallocated, replayed as a HIP graph from the second step on."""

    def __init__(self, model: StreamDecoderForCausalLM, cache: MixerStateCache, batch: int, use_graph: bool = True):
        super().__init__(use_graph, model.device)
        self.model, self.cache, self.B = model, cache, batch
        need = cache.max_length if cache.max_length is not None else cache.get_seq_length() + 1
        cache.ensure(batch, need, model.dtype, model.device)
        dev = model.device
        self.ids = torch.zeros(batch, dtype=torch.int64, device=dev)
        self.buf = model._row_buffers(batch, 1)
        self.h = torch.empty(batch, model.dims.ld, dtype=model.dtype, device=dev)
        self.logits = torch.empty(batch, model.config.vocab, dtype=torch.float32, device=dev)
        self.next_ids = torch.zeros(batch, dtype=torch.int64, device=dev)

    def _enqueue(self, hint: int) -> None:
        m = self.model
        x = m._stream(self.ids, self.buf, self.cache, self.B, 1, hint, pos_dev=self.pos)
        m._logits(x, self.h, self.logits, self.buf["ws"])
        hip.argmax(self.logits, out=self.next_ids)
        hip.advance_pos(self.pos, 1)

    def _position_bound(self, pos0: int) -> int:
        """The by-value position that sizes a step's grids: the next power of two, so that a capture lasts until the sequence has
        doubled and a cache sized for a long generation does not split a short sequence's attention."""
        bound = 1024
        while bound < pos0 + 1:
            bound *= 2
        return min(bound, self.cache.t_max) - 1

    def step(self, ids: torch.Tensor, state=None, init_scale: float = 1.0):
        """Feeds one token per sequence; returns (logits [B, V], next ids [B], None): the runner's own buffers."""
        c, m = self.cache, self.model
        pos0 = c.get_seq_length()
        c.ensure(self.B, pos0 + 1, m.dtype, m.device)
        self.ids.copy_(ids.view(-1))
        hint = self._position_bound(pos0)
        self.launch(pos0, hint, (c.generation, hint))
        c.advance(1)
        return self.logits, self.next_ids, None
