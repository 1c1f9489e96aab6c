"""The Gitipel decoder: pre-norm layers over an fp32 residual stream, each with an input convolution over time and one of two
mixers -- attention with capped scores, a logarithmic distance bias and keys that serve as values, or a generalised delta
rule -- and an exact-gelu feed-forward; a stretch of layers may run several times with the same weights, each pass with
its own cache and state and re-entered through a product over [stream, embedding]."""

from __future__ import annotations

from typing import Optional

from transformers import AutoConfig, AutoModelForCausalLM

from . import checkpoint, hip
from .config import GitipelConfig
from .stream_decoder import StreamDecoderForCausalLM, Weights, pad8


class GitipelLayer:
    """Buffers of one layer, their checkpoint names, and the descriptor the kernels take."""

    def __init__(self, w: Weights, cfg: GitipelConfig, index: int):
        spec = cfg.layers[index]
        m, p = spec["mixer"], f"l{index}."
        D, Dp = cfg.width, pad8(cfg.width)
        taps = cfg.canon["taps"] if cfg.canon is not None else 0
        H, d = m["heads"], m["dim"]
        dp = pad8(d)
        inner = H * dp
        attention = spec["type"] == "attention"
        G = m["kv_heads"] if attention else 0
        self.plan = {"taps": max(taps, 1), "ld": Dp, "heads": H, "head_dim": dp, "kv_heads": G}

        def vec(name, n):
            t = w.vector(pad8(n))
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
            rank, rp = m["rank"], pad8(m["rank"])
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
            ff, fp = spec["mlp"]["ff"], pad8(spec["mlp"]["ff"])
            self.norm2 = vec("norm2", D)
            self.up, self.down = w.matrix(fp, Dp), w.matrix(Dp, fp)
            w.place(p + "mlp.up", self.up[:ff, :D], ff, D)
            w.place(p + "mlp.down", self.down[:D, :ff], D, ff)
            desc.norm2, desc.up, desc.down, desc.ff = self.norm2.data_ptr(), self.up.data_ptr(), self.down.data_ptr(), fp
        desc.norm1, desc.w_in, desc.w_out = self.norm1.data_ptr(), self.w_in.data_ptr(), self.w_out.data_ptr()
        desc.conv = self.conv.data_ptr() if taps else None
        self.native = desc


class GitipelForCausalLM(StreamDecoderForCausalLM):
    config_class = GitipelConfig
    KERNEL_SOURCES = ("gemm_skinny.hip", "gemm_splitk.hip", "gemm_tiled.hip", "gemv_decode.hip", "norm_conv.hip", "attention_capped.hip",
                      "delta_rule.hip", "compose_mixer.hip", "misc.hip")

    def build(self, w: Weights) -> None:
        cfg = self.config
        V, D, Dp = cfg.vocab, cfg.width, pad8(cfg.width)
        self.embed_scale, self.logit_scale, self.keeps_embedding = cfg.embedding["scale"], cfg.logit_scale, cfg.loop is not None
        self.embed = w.matrix(V, Dp)
        w.place("embed", self.embed[:, :D], V, D)
        if cfg.loop is not None:
            self.loop_in = w.matrix(Dp, 2 * Dp)
            w.place("loop.in", self.loop_in[:D].view(D, 2, Dp)[:, :, :D], D, 2 * D)
            self.loop_step = w.vector(cfg.loop["times"], Dp)
            w.place("loop.step", self.loop_step[:, :D], cfg.loop["times"], D)
        self.layers = [GitipelLayer(w, cfg, i) for i in range(len(cfg.layers))]
        self.final_norm = w.vector(Dp)
        w.place("final.norm", self.final_norm[:D], D)
        self.head = w.matrix(V, Dp)
        w.place("head", self.head[:, :D], V, D)

    def layer_runs(self) -> list:
        return self.config.runs()

    def enter_run(self, layer: int, turn: Optional[int], buf: dict) -> None:
        if turn is not None and layer == self.config.loop["start"]:  # a pass begins: x <- W [x; embedding] + the pass's vector
            hip.round_rows(buf["x"], buf["xr"])
            hip.linear_epilogue(buf["xr"], self.loop_in, x1=buf["x0"], bias=self.loop_step[turn], out=buf["x"], workspace=buf["ws"])

    def initial_mean(self, name: str) -> float:
        return 1.0 if name.rsplit(".", 1)[-1] in ("norm", "norm1", "norm2", "r1", "r2") else 0.0

    @classmethod
    def complete_config(cls, raw: dict, path: str) -> dict:
        """The rank of a delta-rule layer's decay projection comes from its tensor."""
        shapes = checkpoint.shapes(path)
        for i, layer in enumerate(raw["layers"]):
            name = f"l{i}.mix.w1"
            if name in shapes:
                layer["mixer"]["rank"] = shapes[name][0]
        return raw


AutoConfig.register("gitipel", GitipelConfig, exist_ok=True)
AutoModelForCausalLM.register(GitipelConfig, GitipelForCausalLM, exist_ok=True)
