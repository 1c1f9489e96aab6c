"""Small Gupitar configurations and comparison helpers shared by the tests."""

import torch

from oracle import gupitar_oracle as O


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Gupitar", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": None if shared is None else {"ff": shared}}


def latent(heads, dim, rot, vdim, q_rank, kv_rank, window, mlp=None, kv_from=None, base=10000.0, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot},
         "scale": (dim + rot) ** -0.5 if scale is None else scale, "mask": None if window is None else {"size": window}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def rglru(width, blocks, taps, mlp=None):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": taps}, "mlp": mlp}


CASES = {
    "both mixers, latents read by later layers under other windows": config(72, 211, [
        latent(3, 24, 8, 40, 40, 56, 19, dense(88)), rglru(96, 3, 3, moe(5, 2, 24, 40)), latent(5, 16, 8, 24, 32, 56, 7, moe(6, 6, 16), kv_from=0),
        latent(2, 32, 16, 32, 24, 48, 64), latent(4, 8, 16, 16, 48, 48, 33, moe(9, 3, 8, 16), kv_from=3), latent(3, 8, 8, 8, 16, 56, 90, kv_from=0)]),
    "sizes that are no multiple of eight": config(50, 77, [
        latent(3, 10, 6, 13, 21, 27, 5, moe(3, 1, 11, 9), base=500.0), rglru(39, 3, 2, dense(27)), latent(1, 7, 6, 5, 19, 27, 18, moe(4, 2, 13), kv_from=0, base=500.0)],
        eps=1e-3),
    "recurrent layers alone, one tap, blocks of one channel": config(64, 128, [
        rglru(40, 1, 1, dense(40)), rglru(24, 24, 5), rglru(64, 2, 4, moe(2, 1, 32, 24))], eps=1e-6),
    "a window of one, wide heads, many experts, no window": config(136, 301, [
        latent(1, 16, 16, 24, 40, 64, 1, dense(72), scale=0.3), latent(16, 64, 32, 128, 96, 256, 70, moe(70, 8, 16, 48)), rglru(160, 4, 4),
        latent(2, 128, 64, 72, 64, 136, None, moe(2, 2, 40))]),
}


def rel(got, want):
    """Root mean square of the difference over that of the reference, per last dimension, worst row."""
    return rows(got, want).max().item()


def rows(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp(min=1e-6)


def build(pkg, name, dtype, seed=0, device="cuda"):
    cfg = CASES[name]
    w = O.random_weights(cfg, seed)
    model = pkg.GupitarForCausalLM(pkg.GupitarConfig(**cfg), device=device, dtype=dtype)
    model.load_state_dict(w)
    return cfg, w, model


def tokens(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed))
