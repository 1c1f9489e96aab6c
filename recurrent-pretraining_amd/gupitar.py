"""The Gupitar decoder: pre-norm layers over an fp32 residual stream (norm weights as distances from one), each with one of two mixers --
windowed attention over low-rank key latents with a rotated part shared by all heads and an output gate, where a layer may read
another layer's latents, or a real-gated linear recurrent unit behind a short convolution -- and a gated feed-forward: dense, or a mixture
of experts with sigmoid scores on the experts' inputs and an optional gated shared expert."""

from __future__ import annotations

import ctypes

import torch
from transformers import AutoConfig, AutoModelForCausalLM

from . import hip
from .config import GupitarConfig
from .stream_decoder import StreamDecoderForCausalLM, Weights, pad8


def _ptr(t):
    return None if t is None else t.data_ptr()


class GupitarLayer:
    """Buffers of one layer, their checkpoint names, the descriptor the kernels take and what the cache keeps for it."""

    def __init__(self, w: Weights, cfg: GupitarConfig, index: int):
        spec = cfg.layers[index]
        self.w, self.p, self.D, self.Dp = w, f"l{index}.", cfg.width, pad8(cfg.width)
        self.native = hip.MixerLayer()
        self.norm1 = self._centred_norm("norm1")
        self.native.norm1 = self.norm1.data_ptr()
        if spec["type"] == "latent_attention":
            self._latent(spec["mixer"], cfg.norm["eps"])
        else:
            self._rglru(spec["mixer"])
        self.native.w_in, self.native.w_out = self.w_in.data_ptr(), self.w_out.data_ptr()
        mlp = spec.get("mlp")
        if mlp is not None:
            self.norm2 = self._centred_norm("norm2")
            self.native.norm2 = self.norm2.data_ptr()
            if mlp["kind"] == "dense":
                self.native.ff_kind = hip.FF_SWIGLU
                self.up, self.down = self._gated("mlp.", mlp["ff"])
                self.native.up, self.native.down, self.native.ff = self.up.data_ptr(), self.down.data_ptr(), pad8(mlp["ff"])
            else:
                self._mixture(mlp)

    def _centred_norm(self, name: str) -> torch.Tensor:
        stored, weight = self.w.vector(self.Dp), self.w.vector(self.Dp)
        self.w.place(self.p + name, stored[:self.D], self.D)
        self.w.derive(self.p + name, weight[:self.D], lambda t: 1.0 + t)
        return weight

    def _norm(self, name: str, n: int) -> torch.Tensor:
        t = self.w.vector(pad8(n))
        self.w.place(self.p + name, t[:n], n)
        return t

    def _rows(self, name: str, buf: torch.Tensor, first: int, n: int) -> None:
        self.w.place(self.p + name, buf[first:first + n, :self.D], n, self.D)

    def _latent(self, m: dict, eps: float) -> None:
        w, p, D, Dp = self.w, self.p + "mix.", self.D, self.Dp
        H, dim, rot, vdim, qr, kr = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"]
        np_, rp, vp, qp, kp = (pad8(n) for n in (dim, rot, vdim, qr, kr))
        own = m.get("kv_from") is None
        # rows of z: query latent | key latent | rotated key part | gate
        gate = qp + (kp + rp if own else 0)
        self.w_in = w.matrix(gate + H * vp, Dp)
        self._rows("mix.dq", self.w_in, 0, qr)
        w.place(p + "g", self.w_in[gate:].view(H, vp, Dp)[:, :vdim, :D], H * vdim, D)
        self.q_norm = self._norm("mix.dq.norm", qr)
        pairs = lambda rows: rows.unflatten(-2, (rot // 2, 2)).transpose(-3, -2)  # stored pair by pair, seen as two halves
        if own:
            w.place(p + "dkv", self.w_in[qp:qp + kr, :D], kr + rot, D, index=slice(0, kr))
            w.place(p + "dkv", pairs(self.w_in[qp + kp:qp + kp + rot, :D]), kr + rot, D, index=slice(kr, None))
            self.kv_norm = self._norm("mix.dkv.norm", kr)
        self.w_uq = w.matrix(H * (np_ + rp), qp)
        q = self.w_uq.view(H, np_ + rp, qp)[:, :, :qr]
        heads = (H, dim + rot, qr)
        w.place(p + "uq", q[:, :dim], H * (dim + rot), qr, seen_as=heads, index=(slice(None), slice(0, dim)))
        w.place(p + "uq", pairs(q[:, np_:np_ + rot]), H * (dim + rot), qr, seen_as=heads, index=(slice(None), slice(dim, None)))
        self.w_ukv = w.matrix(H * (np_ + vp), kp)
        w.place(p + "uk", self.w_ukv[:H * np_].view(H, np_, kp)[:, :dim, :kr], H * dim, kr)
        w.place(p + "uv", self.w_ukv[H * np_:].view(H, vp, kp)[:, :vdim, :kr], H * vdim, kr)
        self.w_uk_t = w.matrix(H, kp, np_)
        w.derive(p + "uk", self.w_uk_t[:, :kr, :dim], lambda t: t.view(H, dim, kr).transpose(1, 2))
        self.w_out = w.matrix(Dp, H * vp)
        w.place(p + "o", self.w_out[:D].view(D, H, vp)[:, :, :vdim], D, H * vdim)
        window = (m.get("mask") or {}).get("size") or 0
        self.latent = hip.Latent(self.w_uq.data_ptr(), self.w_uk_t.data_ptr(), self.w_ukv.data_ptr(), self.q_norm.data_ptr(),
                                 self.kv_norm.data_ptr() if own else None, m["scale"], eps, H, qr, qp, kr, kp, np_, rp, vp, window, int(own))
        n = self.native
        n.mixer, n.heads, n.dim, n.head_dim, n.latent = hip.MIXER_LATENT, H, vdim, vp, ctypes.pointer(self.latent)
        self.plan = {"latent": (kp, rp), "angles": (m["rot"]["base"], rot)} if own else {"latent_from": m["kv_from"]}

    def _rglru(self, m: dict) -> None:
        w, p, D, Dp = self.w, self.p + "mix.", self.D, self.Dp
        n_blocks, width, taps = m["blocks"], m["width"], m["conv"]
        size = width // n_blocks
        sp = pad8(size)
        W = n_blocks * sp
        blocks = lambda t: t.unflatten(-1, (n_blocks, sp))[..., :size]  # [..., blocks, size] of a channel vector
        self.w_in, self.in_bias = w.matrix(2 * W, Dp), w.vector(2 * W)
        for i, name in enumerate(("y", "x")):
            w.place(p + name, self.w_in[i * W:(i + 1) * W].view(n_blocks, sp, Dp)[:, :size, :D], width, D)
            w.place(p + name + ".b", blocks(self.in_bias[i * W:(i + 1) * W]), width)
        self.conv, self.conv_bias = w.vector(taps, W), w.vector(W)
        w.place(p + "conv", blocks(self.conv).permute(1, 2, 0), width, taps)
        w.place(p + "conv.b", blocks(self.conv_bias), width)
        self.gates, self.gate_bias = w.matrix(n_blocks, 2, sp, sp), w.vector(2, W)
        for i, name in enumerate(("ra", "ri")):
            w.place(p + name, self.gates[:, i, :size, :size], n_blocks, size, size)
            w.place(p + name + ".b", blocks(self.gate_bias[i]), n_blocks, size)
        self.lam, self.softplus = w.vector(W), w.vector(W)
        w.place(p + "lam", blocks(self.lam), width)
        w.derive(p + "lam", blocks(self.softplus), torch.nn.functional.softplus)
        self.w_out = w.matrix(Dp, W)
        w.place(p + "o", blocks(self.w_out[:D]), D, width)
        self.rglru = hip.Rglru(self.conv.data_ptr(), self.conv_bias.data_ptr(), self.gates.data_ptr(), self.gate_bias.data_ptr(),
                               self.softplus.data_ptr(), n_blocks, sp, taps, W)
        n = self.native
        n.mixer, n.heads, n.dim, n.head_dim = hip.MIXER_RGLRU, n_blocks, size, sp
        n.rglru, n.in_bias = ctypes.pointer(self.rglru), self.in_bias.data_ptr()
        self.plan = {"taps": taps, "ld": W, "state": (W,)}

    def _gated(self, name: str, ff: int, up=None, down=None):
        """Places a gated feed-forward: gate rows and up rows in one matrix."""
        w, D, Dp, fp = self.w, self.D, self.Dp, pad8(ff)
        up = w.matrix(2 * fp, Dp) if up is None else up
        down = w.matrix(Dp, fp) if down is None else down
        self._rows(name + "gate", up, 0, ff)
        self._rows(name + "up", up, fp, ff)
        w.place(self.p + name + "down", down[:D, :ff], D, ff)
        return up, down

    def _mixture(self, mlp: dict) -> None:
        w, Dp = self.w, self.Dp
        E, ff, shared = mlp["router"]["experts"], mlp["expert"]["ff"], mlp.get("shared")
        fp = pad8(ff)
        self.up, self.down = w.matrix(E, 2 * fp, Dp), w.matrix(E, Dp, fp)
        for e in range(E):
            self._gated(f"mlp.e{e}.", ff, self.up[e], self.down[e])
        logit_ld = (E + 1 + 15) // 16 * 16  # whole matrix-core tiles of router rows
        self.router = w.matrix(logit_ld, Dp)
        self._rows("mlp.router", self.router, 0, E)
        self.shared_up = self.shared_down = None
        if shared is not None:
            self.shared_up, self.shared_down = self._gated("mlp.shared.", shared["ff"])
            self._rows("mlp.shared.sg", self.router, E, 1)
        self.moe = hip.Moe(self.router.data_ptr(), self.up.data_ptr(), self.down.data_ptr(), _ptr(self.shared_up), _ptr(self.shared_down), E,
                           mlp["router"]["top"], fp, pad8(shared["ff"]) if shared is not None else 0, logit_ld)
        self.native.ff_kind, self.native.moe = hip.FF_MOE, ctypes.pointer(self.moe)


class GupitarForCausalLM(StreamDecoderForCausalLM):
    config_class = GupitarConfig
    KERNEL_SOURCES = ("gemm_skinny.hip", "gemm_splitk.hip", "gemm_tiled.hip", "gemv_decode.hip", "norm_conv.hip", "latent_attention.hip", "rglru.hip",
                      "moe.hip", "compose_mixer.hip", "misc.hip")

    def build(self, w: Weights) -> None:
        cfg = self.config
        V, D, Dp = cfg.vocab, cfg.width, pad8(cfg.width)
        self.embed = w.matrix(V, Dp)
        w.place("embed", self.embed[:, :D], V, D)
        self.layers = [GupitarLayer(w, cfg, i) for i in range(len(cfg.layers))]
        stored, self.final_norm = w.vector(Dp), w.vector(Dp)
        w.place("final.norm", stored[:D], D)
        w.derive("final.norm", self.final_norm[:D], lambda t: 1.0 + t)
        self.head = w.matrix(V, Dp)
        w.place("head", self.head[:, :D], V, D)

    def initial_mean(self, name: str) -> float:
        return 1.0 if name.endswith(("dq.norm", "dkv.norm")) else -5.0 if name.endswith("mix.lam") else 0.0


AutoConfig.register("gupitar", GupitarConfig, exist_ok=True)
AutoModelForCausalLM.register(GupitarConfig, GupitarForCausalLM, exist_ok=True)
