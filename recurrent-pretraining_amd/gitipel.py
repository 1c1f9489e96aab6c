"""The Gitipel decoder: pre-norm layers over an fp32 residual stream, each with an input convolution over time and one of two
mixers -- attention with capped scores, a logarithmic distance bias and keys that serve as values, or a generalised delta
rule -- and an exact-gelu feed-forward; a stretch of layers may run several times with the same weights, each pass with
its own cache and state and re-entered through a product over [stream, embedding].

The arithmetic of a layer is one call into libraven_hip.so (hip.mixer_layer).  What a sequence leaves behind lives in
cache.MixerStateCache; generation, sampling and graph replay are the package's own (generation.MinimalGeneration, GraphedStep).

Weights are kept as the kernels read them: the projections of a mixer fused into one matrix, every width rounded up to a multiple
of 8 with zeros (so that any size gives 16-byte rows), heads likewise.  `placements` maps each tensor of a checkpoint to the
strided view of those buffers it fills."""

from __future__ import annotations

from typing import Dict, Optional, Union

import torch
from transformers import AutoConfig, AutoModelForCausalLM, GenerationMixin, PreTrainedModel

from . import checkpoint, hip
from .cache import MixerStateCache
from .config import GitipelConfig
from .generation import CausalLMOutputRecurrentLatents, GraphedStep, MinimalGeneration


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


class _Weights:
    """Zero-initialised buffers and the checkpoint tensors that fill parts of them."""

    def __init__(self, device, dtype):
        self.device, self.dtype = device, dtype
        self.placements: Dict[str, tuple] = {}  # name -> (view, checkpoint shape)

    def matrix(self, *shape) -> torch.Tensor:
        return torch.zeros(*shape, dtype=self.dtype, device=self.device)

    def vector(self, *shape) -> torch.Tensor:
        return torch.zeros(*shape, dtype=torch.float32, device=self.device)

    def place(self, name: str, view: torch.Tensor, *shape) -> None:
        self.placements[name] = (view, tuple(shape))

    def fill(self, name: str, tensor: torch.Tensor) -> None:
        view, shape = self.placements[name]
        if tuple(tensor.shape) != shape:
            raise ValueError(f"{name}: checkpoint shape {tuple(tensor.shape)} != model shape {shape}")
        view.copy_(tensor.reshape(view.shape))


class MixerLayer:
    """Buffers of one layer, their checkpoint names, and the descriptor the kernels take."""

    def __init__(self, w: _Weights, cfg: GitipelConfig, index: int):
        spec = cfg.layers[index]
        m, p = spec["mixer"], f"l{index}."
        D, Dp = cfg.width, _pad8(cfg.width)
        taps = cfg.canon["taps"] if cfg.canon is not None else 0
        H, d = m["heads"], m["dim"]
        dp = _pad8(d)
        inner = H * dp
        attention = spec["type"] == "attention"
        G = m["kv_heads"] if attention else 0
        self.plan = {"taps": max(taps, 1), "ld": Dp, "heads": H, "head_dim": dp, "kv_heads": G}

        def vec(name, n):
            t = w.vector(_pad8(n))
            w.place(p + name, t[:n], n)
            return t

        def head_vec(name, n_heads=H):
            t = w.vector(n_heads * dp)
            w.place(p + name, t.view(n_heads, dp)[:, :d], n_heads * d)
            return t

        def head_rows(name, buf, first, n_heads):
            """Rows of a fused projection: n_heads heads from row `first` on."""
            w.place(p + name, buf[first:first + n_heads * dp].view(n_heads, dp, buf.shape[1])[:, :d, :D], n_heads * d, D)

        self.norm1 = vec("norm1", D)
        self.conv = w.vector(taps, Dp) if taps else None
        if taps:
            w.place(p + "canon1", self.conv.t()[:D], D, taps)
        self.w_out = w.matrix(Dp, inner)
        w.place(p + "mix.o", self.w_out[:D].view(D, H, dp)[:, :, :d], D, H * d)
        desc = hip.MixerLayer(heads=H, kv_heads=G, dim=d, head_dim=dp, taps=taps)
        if attention:
            self.w_in = w.matrix((H + G) * dp, Dp)
            head_rows("mix.q", self.w_in, 0, H)
            head_rows("mix.k", self.w_in, inner, G)
            self.r1, self.r2 = (w.vector(H) for _ in range(2))
            w.place(p + "mix.r1", self.r1, H)
            w.place(p + "mix.r2", self.r2, H)
            desc.mixer = hip.MIXER_ATTENTION
            desc.score = hip.Score(m["scale"], m.get("softcap") or 0.0, self.r1.data_ptr(), self.r2.data_ptr())
        else:
            rank, rp = m["rank"], _pad8(m["rank"])
            self.w_in = w.matrix(5 * inner + rp, Dp)
            for i, name in enumerate(("r", "k", "v", "g", "a")):
                head_rows("mix." + name, self.w_in, i * inner, H)
            w.place(p + "mix.w1", self.w_in[5 * inner:5 * inner + rank, :D], rank, D)
            self.w_decay = w.matrix(inner, rp)
            w.place(p + "mix.w2", self.w_decay.view(H, dp, rp)[:, :d, :rank], H * d, rank)
            self.decay_bias, self.a_bias, self.out_norm = head_vec("mix.w0"), head_vec("mix.a.b"), head_vec("mix.norm")
            desc.mixer, desc.rank = hip.MIXER_GENERAL_DELTA, rp
            desc.w_decay = self.w_decay.data_ptr()
            desc.decay_bias, desc.a_bias, desc.out_norm = self.decay_bias.data_ptr(), self.a_bias.data_ptr(), self.out_norm.data_ptr()
        if spec.get("mlp") is not None:
            ff, fp = spec["mlp"]["ff"], _pad8(spec["mlp"]["ff"])
            self.norm2 = vec("norm2", D)
            self.up, self.down = w.matrix(fp, Dp), w.matrix(Dp, fp)
            w.place(p + "mlp.up", self.up[:ff, :D], ff, D)
            w.place(p + "mlp.down", self.down[:D, :ff], D, ff)
            desc.norm2, desc.up, desc.down, desc.ff = self.norm2.data_ptr(), self.up.data_ptr(), self.down.data_ptr(), fp
        desc.norm1, desc.w_in, desc.w_out = self.norm1.data_ptr(), self.w_in.data_ptr(), self.w_out.data_ptr()
        desc.conv = self.conv.data_ptr() if taps else None
        self.native = desc


class GitipelForCausalLM(MinimalGeneration, PreTrainedModel, GenerationMixin):
    config_class = GitipelConfig
    base_model_prefix = "model"
    _tied_weights_keys = {}
    KERNEL_SOURCES = ("gemm_skinny.hip", "gemm_splitk.hip", "gemm_tiled.hip", "gemv_decode.hip", "norm_conv.hip", "attention_capped.hip",
                      "delta_rule.hip", "compose_mixer.hip", "misc.hip")
    max_positions = None              # no positional table: the cache alone bounds a sequence
    ROWS_PER_CALL = 16384             # token rows of one pass through the layers; longer prompts run in portions

    def __init__(self, config: GitipelConfig, device: Union[str, torch.device, None] = None, dtype: Optional[torch.dtype] = None):
        super().__init__(config)
        if device is None:
            device = "cuda" if torch.cuda.is_available() else "cpu"
        dtype = dtype if dtype is not None else (config.dtype if isinstance(config.dtype, torch.dtype) else torch.bfloat16)
        self._device, self._dtype = torch.device(device), dtype
        cfg, w = config, _Weights(self._device, dtype)
        V, D, Dp = cfg.vocab, cfg.width, _pad8(cfg.width)
        self.weights = w
        self.embed = w.matrix(V, Dp)
        w.place("embed", self.embed[:, :D], V, D)
        if cfg.loop is not None:
            self.loop_in = w.matrix(Dp, 2 * Dp)
            w.place("loop.in", self.loop_in[:D].view(D, 2, Dp)[:, :, :D], D, 2 * D)
            self.loop_step = w.vector(cfg.loop["times"], Dp)
            w.place("loop.step", self.loop_step[:, :D], cfg.loop["times"], D)
        self.layers = [MixerLayer(w, cfg, i) for i in range(len(cfg.layers))]
        self.final_norm = w.vector(Dp)
        w.place("final.norm", self.final_norm[:D], D)
        self.head = w.matrix(V, Dp)
        w.place("head", self.head[:, :D], V, D)
        self.runs = cfg.runs()
        self.dims = hip.StreamDims(D, Dp, cfg.norm["eps"], hip.dtype_code(dtype))
        self._scratch_cache: Optional[MixerStateCache] = None
        self.eval()

    @property
    def dtype(self) -> torch.dtype:
        return self._dtype

    @property
    def device(self) -> torch.device:
        return self._device

    # ---- weights ---------------------------------------------------------------------------------
    def state_dict(self, *args, **kwargs) -> Dict[str, torch.Tensor]:
        """The checkpoint's tensors, read back out of the kernels' buffers (matrices in the model's dtype, vectors float)."""
        return {name: view.reshape(shape) for name, (view, shape) in self.weights.placements.items()}

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
                        config: Optional[GitipelConfig] = None, **kwargs) -> "GitipelForCausalLM":
        """A local directory with config.json and safetensors (checkpoint.py); the decay rank of a delta-rule layer comes from its
        tensor."""
        dtype = dtype if dtype is not None else kwargs.pop("torch_dtype", None)
        if isinstance(dtype, str):
            dtype = None if dtype == "auto" else getattr(torch, dtype)
        raw = checkpoint.read_config(path) if config is None else config.to_dict()
        shapes = checkpoint.shapes(path)
        for i, layer in enumerate(raw["layers"]):
            name = f"l{i}.mix.w1"
            if name in shapes:
                layer["mixer"]["rank"] = shapes[name][0]
        model = cls(GitipelConfig(**raw), device=device if device is not None else kwargs.get("device_map"), dtype=dtype)
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
        """Synthetic weights drawn on the model's device: matrices and vectors ~ N(0, std), norms ~ N(1, std)."""
        if seed is None:
            return
        g = torch.Generator(device=self.device).manual_seed(seed)
        for name, (view, _) in self.weights.placements.items():
            mean = 1.0 if name.rsplit(".", 1)[-1] in ("norm", "norm1", "norm2", "r1", "r2") else 0.0
            view.copy_(torch.empty(view.shape, dtype=torch.float32, device=self.device).normal_(mean, std, generator=g))

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
    def _row_buffers(self, B: int, S: int) -> dict:
        M, Dp = B * S, self.dims.ld
        if self._device.type != "cuda":
            raise hip.RavenHipError("the forward runs on the GPU; there is no CPU path")
        row = lambda dt: torch.empty(M, Dp, dtype=dt, device=self.device)
        n = max(hip.mixer_layer_workspace_bytes(self.dims, layer.native, B, S) for layer in self.layers) if self.layers else 0
        loop = self.config.loop is not None
        lin = hip.load().raven_linear_workspace_bytes(M, max(Dp, self.config.vocab)) if 1 < M <= 32 else 0
        return {"x": row(torch.float32), "x0": row(self.dtype) if loop else None, "xr": row(self.dtype) if loop else None,
                "ws": torch.empty(max(n, lin, 256), dtype=torch.uint8, device=self.device)}

    def _stream(self, ids: torch.Tensor, buf: dict, cache: MixerStateCache, B: int, S: int, pos0: int, pos_dev=None, trail: Optional[list] = None):
        """Embedding and every layer run for rows ids [B*S]; leaves the stream in buf["x"]."""
        cfg, x, ws = self.config, buf["x"], buf["ws"]
        hip.embed_stream(self.embed, ids, cfg.embedding["scale"], x, buf["x0"])
        for run, (i, t) in enumerate(self.runs):
            if t is not None and i == cfg.loop["start"]:  # a pass begins: x <- W [x; embedding] + the pass's vector
                hip.round_rows(x, buf["xr"])
                hip.linear_epilogue(buf["xr"], self.loop_in, x1=buf["x0"], bias=self.loop_step[t], out=x, workspace=ws)
            hip.mixer_layer(self.dims, self.layers[i].native, cache.native(run), x, B, S, pos0, ws, pos_dev=pos_dev)
            if trail is not None:
                trail.append(x[:, :cfg.width].clone())
        return x

    def _logits(self, x: torch.Tensor, h: torch.Tensor, out: torch.Tensor, ws) -> torch.Tensor:
        cfg = self.config
        if x.shape[0] == 1 and hip.gemv_stream_fits(self.dims.ld, self.dtype):
            return hip.gemv_stream(x, self.final_norm, cfg.width, cfg.norm["eps"], self.head, self.dtype, scale=cfg.logit_scale, out=out)
        hip.norm_conv(x, self.final_norm, cfg.width, cfg.norm["eps"], x.shape[0], 1, self.dtype, out=h)
        return hip.linear_epilogue(h, self.head, scale=cfg.logit_scale, out=out, workspace=ws)

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
            buf = self._row_buffers(B, n)
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

    def __init__(self, model: GitipelForCausalLM, cache: MixerStateCache, batch: int, use_graph: bool = True):
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


AutoConfig.register("gitipel", GitipelConfig, exist_ok=True)
AutoModelForCausalLM.register(GitipelConfig, GitipelForCausalLM, exist_ok=True)
