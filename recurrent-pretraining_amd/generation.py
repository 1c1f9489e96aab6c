"""What the model families share around their forward: the generation settings and outputs, the token pick, the minimal decode
loop (recpre/raven_modeling_minimal.py:1165-1232) and the capture of a decode step as a HIP graph."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Callable, Optional

import torch
from transformers.utils import ModelOutput

from . import hip


@dataclass
class CausalLMOutputRecurrentLatents(ModelOutput):  # RMM:113-123
    loss: Optional[torch.Tensor] = None
    log_ppl: Optional[torch.Tensor] = None
    logits: Optional[torch.Tensor] = None
    past_key_values: Optional[Any] = None
    latent_states: Optional[torch.Tensor] = None
    hidden_states: Optional[torch.Tensor] = None
    attention_maps: Optional[dict] = None
    stats: Optional[dict] = None


@dataclass
class GenerationSettings:
    """The fields of transformers.GenerationConfig that the generate loops read."""
    max_length: int = 4096
    max_new_tokens: Optional[int] = None
    do_sample: bool = False
    temperature: Optional[float] = None
    top_k: Optional[int] = None
    top_p: Optional[float] = None
    min_p: Optional[float] = None
    repetition_penalty: Optional[float] = None
    dry_multiplier: float = 0.0        # > 0 selects the n-gram penalty instead (RMM:2003-2046)
    dry_base: float = 1.75
    dry_allowed_length: int = 2
    eos_token_id: Any = None
    return_dict_in_generate: bool = False


@dataclass
class GenerateOutput:
    sequences: torch.Tensor
    past_key_values: Optional[Any] = None
    scores: Optional[dict] = None


class MinimalGeneration:
    """The token pick and the decode loop of a model.  A model supplies forward(), decode_runner(cache, batch, num_steps, greedy,
    use_graph) -> an object whose step(ids, state, init_scale) returns (logits, next ids, latents or None), _generation_cache(),
    max_positions (None: unbounded) and DEFAULT_STOPS."""

    DEFAULT_STOPS: frozenset = frozenset()
    _MINIMAL_LOOP_KEYS = ("continuous_compute", "input_states_fn", "stop_tokens", "use_graph")

    def _get_stops(self, generation_config, model_kwargs=None) -> set:
        stops = set(self.DEFAULT_STOPS)
        eos = getattr(generation_config, "eos_token_id", None)
        if eos is not None:
            try:
                stops.update(eos)
            except TypeError:
                stops.add(eos)
        return stops

    def _default_max_length(self, gc) -> int:
        """`max_length` of the generation settings; transformers 5 leaves it unset by default, then the model's own bound."""
        for src in (gc, getattr(self, "generation_config", None)):
            if getattr(src, "max_length", None):
                return src.max_length
        return self.max_positions if self.max_positions is not None else GenerationSettings.max_length

    def _apply_repetition_penalty(self, original_logits, input_ids, generation_config, use_candidates: bool = False):
        """RMM:1991-2070; see sampling.apply_repetition_penalty."""
        from .sampling import apply_repetition_penalty
        return apply_repetition_penalty(original_logits, input_ids, generation_config, use_candidates)

    def _sample_next_token(self, next_token_logits: torch.Tensor, input_ids, generation_config) -> torch.Tensor:
        """RMM:1944-1989.  Greedy selection runs in the HIP argmax kernel."""
        gc = generation_config
        if getattr(gc, "repetition_penalty", None) is not None and gc.repetition_penalty != 1.0:
            next_token_logits = self._apply_repetition_penalty(next_token_logits, input_ids, gc)
        if not getattr(gc, "do_sample", False):
            return hip.argmax(next_token_logits.float().contiguous()).unsqueeze(-1)
        logits = next_token_logits.to(torch.float32)
        if gc.temperature:
            logits = logits / gc.temperature
        probs = torch.softmax(logits, dim=-1)
        if gc.top_k:
            kth = torch.topk(probs, gc.top_k, dim=-1).values[:, -1:]
            probs = torch.where(probs < kth, torch.zeros_like(probs), probs)
        if gc.top_p:
            sp, si = torch.sort(probs, descending=True, dim=-1)
            remove = torch.cumsum(sp, dim=-1) > gc.top_p
            remove[:, 0] = False
            mask = torch.zeros_like(probs, dtype=torch.bool).scatter(1, si, remove)
            probs = torch.where(mask, torch.zeros_like(probs), probs)
        if gc.min_p:
            probs = torch.where(probs < gc.min_p * probs.max(dim=-1, keepdim=True).values, torch.zeros_like(probs), probs)
        probs = probs / probs.sum(dim=-1, keepdim=True).clamp(min=1e-10)
        return torch.multinomial(probs, num_samples=1)

    @torch.no_grad()
    def generate_minimal(self, input_ids: torch.Tensor, generation_config=None, tokenizer=None, streamer=None,
                         continuous_compute: bool = False, init_scale: float = 1.0, cache_lookup_strategy: str = "full",
                         input_states_fn: Optional[Callable] = None, stop_tokens: Optional[set] = None,
                         use_graph: bool = True, **model_kwargs):
        """RMM:1165-1232, for any model family of the package (hooks: forward, decode_runner, _generation_cache, max_positions,
        _get_stops).  Prefill through forward(), then one token per step through the decode
        runner (all kernels of a token on one stream, optionally replayed as a HIP graph).

        input_states_fn(call_index, (B, S, h)) -> latent state to inject into that forward (an
        extension for reproducible runs: the reference re-draws the state from the device RNG on
        every call, RMM:738).  stop_tokens overrides the reference's fixed stop set."""
        gc = generation_config if generation_config is not None else self.generation_config
        B, prompt_len = input_ids.shape
        if "max_new_tokens" in model_kwargs and model_kwargs["max_new_tokens"] is not None:
            max_new = model_kwargs["max_new_tokens"]
            if "max_length" in model_kwargs:
                max_new = min(max_new, model_kwargs["max_length"] - prompt_len)
        elif getattr(gc, "max_new_tokens", None):
            max_new = gc.max_new_tokens
        else:
            max_new = model_kwargs.get("max_length", self._default_max_length(gc)) - prompt_len
        num_steps = model_kwargs.get("num_steps", None)
        stops = self._get_stops(gc) if stop_tokens is None else set(stop_tokens)
        input_ids = input_ids.to(self.device)
        if max_new <= 0:
            return input_ids
        total = prompt_len + max_new if self.max_positions is None else min(prompt_len + max_new, self.max_positions)
        cache = self._generation_cache(model_kwargs, cache_lookup_strategy, B, total)

        def state_for(call: int, S: int, embeds_like=None):
            if input_states_fn is not None:
                return input_states_fn(call, (B, S, self.config.n_embd)).to(self.device, self.dtype)
            return None

        # prefill
        seen = cache.get_seq_length()
        pos = torch.arange(seen, prompt_len, device=self.device)
        out = self.forward(input_ids=input_ids[:, seen:], input_states=state_for(0, prompt_len - seen), num_steps=num_steps,
                           past_key_values=cache, use_cache=True, cache_position=pos, init_scale=init_scale)
        next_tok = self._sample_next_token(out.logits[:, -1, :], input_ids, gc)
        carried = out.latent_states[:, -1:, :] if continuous_compute else None
        tokens = [next_tok]
        alive = torch.ones(B, dtype=torch.bool)
        if streamer:
            streamer.put(next_tok.cpu())

        def update_alive(tok) -> bool:
            if stops:
                for b, v in enumerate(tok.view(-1).tolist()):
                    if alive[b] and v in stops:
                        alive[b] = False
            return bool(alive.any())

        runner = None
        call = 1
        # the penalties look at the growing sequence on every step (RMM:1198-1201, 1946-1947); with one configured the
        # pick is made from the penalised logits on the greedy path too
        penalised = getattr(gc, "repetition_penalty", None) is not None and gc.repetition_penalty != 1.0
        pick_on_host = bool(getattr(gc, "do_sample", False)) or penalised
        all_ids = torch.cat([input_ids, next_tok], dim=-1) if pick_on_host else None
        while len(tokens) < max_new and update_alive(tokens[-1]) and cache.get_seq_length() + 1 <= total:
            if runner is None:
                runner = self.decode_runner(cache, B, num_steps, greedy=not getattr(gc, "do_sample", False), use_graph=use_graph)
            state = carried if continuous_compute else state_for(call, 1)
            logits, nxt, latents = runner.step(tokens[-1].view(-1), state, init_scale)
            if pick_on_host:
                nxt = self._sample_next_token(logits, all_ids, gc).view(-1)
                all_ids = torch.cat([all_ids, nxt.view(B, 1)], dim=-1)
            tokens.append(nxt.view(B, 1).clone())
            if continuous_compute:
                carried = latents.view(B, 1, -1).clone()
            if streamer:
                streamer.put(tokens[-1].cpu())
            call += 1
        if streamer:
            streamer.end()
        sequences = torch.cat([input_ids] + tokens, dim=-1)
        if getattr(gc, "return_dict_in_generate", False):
            return GenerateOutput(sequences=sequences, past_key_values=cache, scores={})
        return sequences


class GraphedStep:
    """A decode step whose launches are the same for every token (the position is read from `self.pos` on the device): eager the
    first time, then captured once per `key` and replayed.  Subclasses implement _enqueue(hint)."""

    def __init__(self, use_graph: bool, device):
        self.pos = torch.zeros(1, dtype=torch.int32, device=device)
        self.use_graph = use_graph
        self.graph: Optional[torch.cuda.CUDAGraph] = None
        self._graph_key = None
        self._warm = False

    def _enqueue(self, hint: int) -> None:
        raise NotImplementedError

    def launch(self, pos0: int, hint: int, key) -> None:
        """Runs the step at position pos0.  hint bounds the position (it sizes grids); key is everything a captured launch holds
        by value -- pointers, capacities, the hint: a change makes the capture stale."""
        self.pos.fill_(pos0)
        if not (self.use_graph and self._warm):
            self._enqueue(hint)
            self._warm = True
            return
        if self.graph is None or self._graph_key != key:
            self.graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(self.graph):
                self._enqueue(hint)
            self._graph_key = key
            self.pos.fill_(pos0)  # capture does not execute; make sure the counter is what this step needs
        self.graph.replay()
