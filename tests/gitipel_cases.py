"""Small Gitipel configurations and comparison helpers shared by the tests."""

import torch

from oracle import gitipel_oracle as O


def config(width, vocab, layers, taps=3, loop=None, eps=1e-5, emb=3.0, logit_scale=1.7):
    return {"architecture": "Gitipel", "vocab": vocab, "width": width, "layers": layers, "canon": {"taps": taps}, "loop": loop,
            "norm": {"eps": eps}, "embedding": {"scale": emb}, "logit_scale": logit_scale}


def attn(heads, kv, dim, ff=None, cap=7.0, scale=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "softcap": cap,
                                           "scale": dim ** -0.5 if scale is None else scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def delta(heads, dim, ff=None):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


# name -> (configuration, rank of the decay projection)
CASES = {
    "looped middle, grouped heads, a layer without feed-forward": (
        config(72, 211, [delta(2, 24, 88), attn(6, 2, 24), delta(3, 16, 56), attn(3, 1, 40, 64)], taps=4,
               loop={"start": 1, "stop": 3, "times": 3}), 8),
    "sizes that are no multiple of eight": (
        config(50, 77, [attn(4, 2, 10, 30, cap=2.5), delta(3, 13, 27)], taps=2, loop={"start": 0, "stop": 1, "times": 2}, eps=1e-3), 5),
    "no loop, one tap, single head": (config(64, 128, [delta(1, 40, 96), attn(1, 1, 72, 40, scale=0.3)], taps=1, emb=1.0, logit_scale=1.0), 16),
    "one pass over the last layer, wide heads": (
        config(136, 301, [attn(2, 2, 136, 72, cap=30.0), delta(2, 72, 104)], taps=5, loop={"start": 1, "stop": 2, "times": 1}), 24),
}


def rel(got, want):
    """Root mean square of the difference over that of the reference, per last dimension, worst row."""
    got, want = got.double().cpu(), want.double().cpu()
    return ((got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp(min=1e-6)).max().item()


def build(pkg, name, dtype, seed=0, device="cuda"):
    cfg, rank = CASES[name]
    w = O.random_weights(cfg, rank, seed)
    raw = {**cfg, "layers": [{**x, "mixer": {**x["mixer"], **({"rank": rank} if x["type"] == "general_delta" else {})}} for x in cfg["layers"]]}
    model = pkg.GitipelForCausalLM(pkg.GitipelConfig(**raw), device=device, dtype=dtype)
    model.load_state_dict(w)
    return cfg, w, model


def tokens(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed))
