"""Gupitar on the GPU against the CPU oracle: every mechanism alone, then whole models -- prompts, portions, decoding, batches,
caches used again, greedy generation."""

import io
import json
import math

import pytest
import torch

import gupitar_cases as G
from oracle import gupitar_oracle as O

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DT = pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])
BOTH = "both mixers, latents read by later layers under other windows"
ODD = "sizes that are no multiple of eight"
WIDE = "a window of one, wide heads, many experts, no window"


def pad8(n):
    return (n + 7) // 8 * 8


# ---- latent attention alone ----------------------------------------------------------------------------
class Latent:
    """A latent-attention mixer of one layer without its projections of the stream: rows z and queries in, gated heads out."""

    def __init__(self, pkg, H, dim, rot, vdim, kr, window, dtype, seed=0, scale=None, t_max=256, own=True, batch=1):
        self.pkg, self.hip, self.dtype = pkg, pkg.hip, dtype
        layers = [G.latent(H, dim, rot, vdim, 16, kr, window, scale=scale)] + ([] if own else [G.latent(H, dim, rot, vdim, 16, kr, window, kv_from=0)])
        self.cfg = G.config(24, 8, layers)
        self.w = O.random_weights(self.cfg, seed)
        self.model = pkg.GupitarForCausalLM(pkg.GupitarConfig(**self.cfg), device="cuda", dtype=dtype)
        self.model.load_state_dict(self.w)
        self.layer = self.model.layers[-1]
        self.desc, self.m = self.layer.latent, self.cfg["layers"][0]["mixer"]
        self.cache = self.model.new_cache(t_max)
        self.cache.ensure(batch, t_max, dtype, "cuda")
        self.native = self.cache.native(0).latent
        self.p = f"l{len(layers) - 1}.mix."

    def rows(self, latent, rotated, gate, q):
        """z and q rows in the kernels' layout: key latent [T, kr] (not normed), rotated part [T, rot] and queries [T, H, dim + rot] not rotated."""
        m, d = self.m, self.desc
        T, H, rot = q.shape[0], m["heads"], m["rot_dim"]
        pairs = torch.arange(rot).view(2, rot // 2).t().reshape(-1)
        z = torch.zeros(T, d.q_rank + (d.kv_rank + d.rot if d.own_kv else 0) + H * d.vdim)
        if d.own_kv:
            z[:, d.q_rank:d.q_rank + m["kv_rank"]] = latent
            z[:, d.q_rank + d.kv_rank:d.q_rank + d.kv_rank + rot] = rotated[:, pairs]
        z[:, z.shape[1] - H * d.vdim:].view(T, H, d.vdim)[:, :, :m["vdim"]] = gate
        qq = torch.zeros(T, H, d.nope + d.rot)
        qq[:, :, :m["dim"]] = q[:, :, :m["dim"]]
        qq[:, :, d.nope:d.nope + rot] = q[:, :, m["dim"]:][:, :, pairs]
        return z.to(self.dtype).cuda(), qq.view(T, -1).to(self.dtype).cuda()

    def run(self, z, q, cuts, pos0=0, device_position=False, bound=None):
        out, pos = [], pos0
        for n in cuts:
            i = pos - pos0
            zz, qq = z[i:i + n].contiguous(), q[i:i + n].contiguous()
            at = dict(pos_dev=torch.tensor([pos], dtype=torch.int32, device="cuda")) if device_position else {}
            by_value = bound if device_position and bound is not None else pos
            if self.desc.own_kv:
                self.hip.latent_rows(self.desc, zz, self.native, 1, n, by_value, self.dtype, want_cq=False, **at)
            out.append(self.hip.latent_attention(self.desc, qq, zz, self.native, 1, n, by_value, **at))
            pos += n
        T = q.shape[0]
        return torch.cat(out).float().cpu().view(T, self.m["heads"], self.desc.vdim)[:, :, :self.m["vdim"]]

    def want(self, latent, rotated, gate, q, eps=1e-5):
        """The same in float64 from the operands as the kernels get them."""
        r = lambda t: t.to(self.dtype).double()
        m, w = self.m, {k: t.double() for k, t in self.w.items()}
        T, H = q.shape[0], m["heads"]
        c = O.plain_norm(r(latent), w["l0.mix.dkv.norm"], eps)
        kr = O.rotate(r(rotated), torch.arange(T), m["rot"]["base"], m["rot"]["dims"])
        if self.dtype == BF16:
            c, kr = c.to(BF16).double(), kr.to(BF16).double()
        q = torch.cat([r(q)[..., :m["dim"]], O.rotate(r(q)[..., m["dim"]:], torch.arange(T), m["rot"]["base"], m["rot"]["dims"])], -1)
        k = torch.cat([(c @ w[self.p + "uk"].T).view(T, H, -1), kr[:, None].expand(T, H, -1)], -1)
        v = (c @ w[self.p + "uv"].T).view(T, H, -1)
        return O.windowed_attention(q, k, v, m["scale"], m["mask"]["size"] if m["mask"] else T) * torch.sigmoid(r(gate).double())


def inputs(T, H, dim, rot, vdim, kr, seed=0, q_scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(T, kr, generator=g) * 3, torch.randn(T, rot, generator=g), torch.randn(T, H, vdim, generator=g),
            torch.randn(T, H, dim + rot, generator=g) * q_scale)


SHAPES = [(2, 16, 8, 16, 24, 20), (3, 10, 6, 13, 27, 33), (6, 64, 32, 56, 120, 100), (5, 32, 64, 72, 136, 64), (16, 128, 64, 128, 512, 70),
          (1, 24, 2, 40, 1016, 1), (4, 200, 40, 120, 64, 5), (2, 56, 8, 136, 40, 500)]


@DT
@pytest.mark.parametrize("H,dim,rot,vdim,kr,window", SHAPES)
def test_attention_prompts_portions_and_decoding(pkg, dtype, H, dim, rot, vdim, kr, window):
    T = 170
    ins = inputs(T, H, dim, rot, vdim, kr, seed=H)
    a = Latent(pkg, H, dim, rot, vdim, kr, window, dtype, t_max=T)
    z, q = a.rows(*ins)
    want = a.want(*ins)
    for cuts in ([T], [2, 61, 1, 64, 17, 3, 22], [100] + [1] * 70, [1] * 20 + [150], [16, 15, 33, 106]):
        a.cache.latents[0][0].fill_(float("nan"))  # what an earlier sequence left must not matter
        a.cache.latents[0][1].fill_(float("nan"))
        got = a.run(z, q, cuts)
        err = G.rows(got.flatten(1), want.flatten(1)).max().item()
        assert err < (2e-5 if dtype == F32 else 3e-2), cuts


@DT
@pytest.mark.parametrize("how", ["prompt", "decoded", "portions", "short portions"])
@pytest.mark.parametrize("window", [64, 90, 130])
def test_attention_keys_at_the_edges_of_a_window(pkg, dtype, window, how):
    """Single keys that dominate their query: just inside the window, just outside, and at tile borders."""
    T, H, dim, rot, vdim, kr = 420, 2, 32, 8, 32, 32
    lat, rotated, gate, q = inputs(T, H, dim, rot, vdim, kr, seed=7, q_scale=0.3)
    a = Latent(pkg, H, dim, rot, vdim, kr, window, dtype, t_max=T, scale=0.5)
    uk = a.w["l0.mix.uk"].view(H, dim, kr)
    spots = []
    for n, at in enumerate([window, window + 2, 191, 193, 255, 257, 300, 319, 320, 337, 383, 385, 411, 419]):
        src = at - window + (1 if n % 2 == 0 else 0)  # the first key inside, or the last one outside
        lat[src] = torch.randn(kr, generator=torch.Generator().manual_seed(n)) * 3
        c = O.rms(lat[src], 1e-5) * a.w["l0.mix.dkv.norm"]
        k = uk @ c
        q[at, :, :dim] = 14 * k / k.norm(dim=-1, keepdim=True)
        spots.append((at, n % 2 == 0))
    ins = (lat, rotated, gate, q)
    z, qq = a.rows(*ins)
    want = a.want(*ins)
    cuts = {"prompt": [T], "decoded": [60] + [1] * (T - 60), "portions": [63, 2, 64, 31, 33, 178, 20, 29], "short portions": [7] * 60}[how]
    got = a.run(z, qq, cuts)
    rows = [at for at, _ in spots]
    assert G.rows(got[rows].flatten(1), want[rows].flatten(1)).max() < (2e-5 if dtype == F32 else 3e-2)
    b = Latent(pkg, H, dim, rot, vdim, kr, window, dtype, t_max=T, scale=0.5)
    for wrong in (window - 1, window + 1):  # the test sees a window that is one off
        b.m["mask"] = {"size": wrong}
        off = G.rows(b.want(*ins)[rows].flatten(1), want[rows].flatten(1))
        assert all(off[i] > 0.2 for i, (_, inside) in enumerate(spots) if inside == (wrong < window))


@DT
def test_attention_reference_follows_every_lane(pkg, dtype):
    """Scores hundreds apart inside one tile, the largest at each of its places in turn."""
    T, H, dim, rot, vdim, kr = 128, 1, 16, 8, 16, 16
    lat, rotated, gate, q = inputs(T, H, dim, rot, vdim, kr, seed=3)
    a = Latent(pkg, H, dim, rot, vdim, kr, T, dtype, t_max=T, scale=1.0)
    uk = a.w["l0.mix.uk"].view(H, dim, kr)
    c = O.rms(lat, 1e-5) * a.w["l0.mix.dkv.norm"]
    for i in range(64, T):
        k = uk[0] @ c[i - 64]
        q[i, 0, :dim] = 150 * k / k.norm()
    ins = (lat, rotated, gate, q)
    z, qq = a.rows(*ins)
    want = a.want(*ins)
    for cuts in ([T], [64] + [1] * 64):
        got = a.run(z, qq, cuts)
        assert torch.isfinite(got).all()
        assert G.rows(got[64:].flatten(1), want[64:].flatten(1)).max() < (1e-3 if dtype == F32 else 0.25), cuts  # scores of 150 carry an error of 1


@DT
def test_attention_long_cache_with_the_position_on_the_device(pkg, dtype):
    """Decode rows far into a long window, ranges over several workgroups, the bound by value larger than the position."""
    T, H, dim, rot, vdim, kr, window = 1500, 6, 16, 8, 24, 40, 1100
    ins = inputs(T, H, dim, rot, vdim, kr, seed=5)
    a = Latent(pkg, H, dim, rot, vdim, kr, window, dtype, t_max=T)
    z, q = a.rows(*ins)
    a.hip.latent_rows(a.desc, z, a.native, 1, T, 0, dtype, want_cq=False)
    rows = [0, 1, 2, 63, 64, 1000, 1098, 1099, 1100, 1101, 1499]
    want = a.want(*ins)
    for r in rows:
        got = a.hip.latent_attention(a.desc, q[r:r + 1].contiguous(), z[r:r + 1].contiguous(), a.native, 1, 1, T - 1,
                                     pos_dev=torch.tensor([r], dtype=torch.int32, device="cuda"))
        got = got.float().cpu().view(1, H, a.desc.vdim)[:, :, :vdim]
        assert G.rel(got.flatten(1), want[r:r + 1].flatten(1)) < (2e-5 if dtype == F32 else 3e-2), r


@DT
def test_attention_of_a_batch_and_of_a_reading_layer(pkg, dtype):
    """Several sequences in one call; a layer without latents of its own under the same cache."""
    B, T, H, dim, rot, vdim, kr, window = 3, 90, 3, 16, 8, 16, 32, 21
    ins = [inputs(T, H, dim, rot, vdim, kr, seed=b) for b in range(B)]
    a = Latent(pkg, H, dim, rot, vdim, kr, window, dtype, t_max=T, batch=B)
    b = Latent(pkg, H, dim, rot, vdim, kr, window, dtype, t_max=T, own=False)
    za = [a.rows(*i) for i in ins]
    stack = lambda k, lo, n: torch.cat([r[k][lo:lo + n] for r in za]).contiguous()
    for cuts in ([T], [50, 40], [40] + [1] * 50, [9] * 10):
        pos, out = 0, []
        for n in cuts:
            a.hip.latent_rows(a.desc, stack(0, pos, n), a.native, B, n, pos, dtype, want_cq=False)
            out.append(a.hip.latent_attention(a.desc, stack(1, pos, n), stack(0, pos, n), a.native, B, n, pos).view(B, n, -1))
            pos += n
        got = torch.cat(out, 1).float().cpu().view(B, T, H, a.desc.vdim)[..., :vdim]
        for s in range(B):
            assert G.rel(got[s].flatten(1), a.want(*ins[s]).flatten(1)) < (2e-5 if dtype == F32 else 3e-2), cuts
    z, q = b.rows(*ins[0])
    b.native = pkg.hip.LatentCache(a.native.latent, a.native.rotated, a.native.angles, 1, T)
    for cuts in ([T], [40] + [1] * 50):
        got = b.run(z, q, cuts)
        assert G.rel(got.flatten(1), b.want(*ins[0]).flatten(1)) < (2e-5 if dtype == F32 else 3e-2)


# ---- recurrent unit alone ------------------------------------------------------------------------------
class Unit:
    def __init__(self, pkg, width, blocks, taps, dtype, lam_mean=-4.0, seed=0):
        self.hip, self.dtype = pkg.hip, dtype
        cfg = G.config(24, 8, [G.rglru(width, blocks, taps)])
        self.w = O.random_weights(cfg, seed)
        self.w["l0.mix.lam"] = (self.w["l0.mix.lam"] + 4.0 + lam_mean).bfloat16().float()
        model = pkg.GupitarForCausalLM(pkg.GupitarConfig(**cfg), device="cuda", dtype=dtype)
        model.load_state_dict(self.w)
        self.layer, self.desc = model.layers[0], model.layers[0].rglru
        self.width, self.blocks, self.size, self.sp, self.taps = width, blocks, width // blocks, pad8(width // blocks), taps

    def pad(self, x):
        return torch.nn.functional.pad(x.unflatten(-1, (self.blocks, self.size)), (0, self.sp - self.size)).flatten(-2)

    def unpad(self, x):
        return x.unflatten(-1, (self.blocks, self.sp))[..., :self.size].flatten(-2)

    def run(self, v, x, cuts, B=1):
        """v, x [B, T, width]."""
        W = self.blocks * self.sp
        z = torch.cat([self.pad(v), self.pad(x)], -1).to(self.dtype).cuda()
        ring = torch.full((B, self.taps, W), float("nan"), device="cuda")  # an earlier sequence's
        state = torch.full((B, W), float("nan"), device="cuda")
        pos, out = 0, []
        for n in cuts:
            out.append(self.hip.rglru(self.desc, z[:, pos:pos + n].reshape(B * n, -1).contiguous(), ring, state, B, n, pos).view(B, n, -1))
            pos += n
        return self.unpad(torch.cat(out, 1).float().cpu()), self.unpad(state.cpu())

    def want(self, v, x):
        w = {k: t.double() for k, t in self.w.items()}
        v, x = v.to(self.dtype).double(), x.to(self.dtype).double()
        u = O.causal_conv(x, w["l0.mix.conv"], w["l0.mix.conv.b"])
        if self.dtype == BF16:
            u = u.to(BF16).double()
        r, i = (O.block_gate(u, w["l0.mix." + n], w["l0.mix." + n + ".b"]) for n in ("ra", "ri"))
        S, last = O.gated_recurrence(u, r, i, w["l0.mix.lam"])
        return S * O.gelu_tanh(v), last


@DT
@pytest.mark.parametrize("width,blocks,taps", [(16, 2, 4), (39, 3, 2), (40, 1, 1), (24, 24, 5), (96, 3, 3), (256, 2, 4), (1032, 4, 3)])
def test_recurrent_unit_prompts_portions_and_decoding(pkg, dtype, width, blocks, taps):
    T = 150
    g = torch.Generator().manual_seed(width)
    v, x = (torch.randn(T, width, generator=g) for _ in range(2))
    unit = Unit(pkg, width, blocks, taps, dtype)
    want, last = unit.want(v, x)
    for cuts in ([T], [2, 3, 1, 2, 32, 33, 1, 64, 12], [100] + [1] * 50, [1] * 30 + [120], [31, 65, 54]):
        got, state = unit.run(v[None], x[None], cuts)
        # bf16: u on a tie of the bf16 grid may round the other way, and then enters the state
        tol = 2e-5 if dtype == F32 else 1e-2
        assert (got[0] - want).abs().max() < tol * max(1.0, want.abs().max().item()), cuts
        assert (state[0] - last).norm() / last.norm() < (1e-5 if dtype == F32 else 5e-3), cuts


@DT
@pytest.mark.parametrize("lam", [-12.0, 6.0])
def test_recurrent_unit_keeps_slow_and_drops_fast_states(pkg, dtype, lam):
    """1000 tokens at decays of one part in ten thousand and at decays that leave nothing."""
    T, width = 1000, 32
    g = torch.Generator().manual_seed(1)
    v, x = (torch.randn(T, width, generator=g) for _ in range(2))
    x[:5] *= 20
    unit = Unit(pkg, width, 2, 3, dtype, lam_mean=lam)
    want, last = unit.want(v, x)
    for cuts in ([T], [700] + [1] * 20 + [280]):
        got, state = unit.run(v[None], x[None], cuts)
        assert (got[0] - want).norm() / want.norm() < (2e-5 if dtype == F32 else 6e-3)
        assert (state[0] - last).norm() / last.norm() < (2e-5 if dtype == F32 else 6e-3)


@DT
def test_recurrent_unit_of_several_sequences(pkg, dtype):
    B, T, width = 3, 70, 48
    g = torch.Generator().manual_seed(2)
    v, x = (torch.randn(B, T, width, generator=g) for _ in range(2))
    unit = Unit(pkg, width, 3, 4, dtype)
    for cuts in ([T], [33, 2, 1, 1, 33]):
        got, state = unit.run(v, x, cuts, B=B)
        for b in range(B):
            want, last = unit.want(v[b], x[b])
            assert (got[b] - want).abs().max() < (2e-5 if dtype == F32 else 1e-2) * max(1.0, want.abs().max().item())


# ---- mixture of experts alone --------------------------------------------------------------------------
@DT
@pytest.mark.parametrize("M", [1, 2, 9, 40, 300])
@pytest.mark.parametrize("D,E,top,ff,shared", [(50, 5, 2, 11, 9), (64, 3, 3, 24, None), (96, 70, 8, 40, 56), (136, 11, 1, 200, 64), (72, 300, 4, 16, 8)])
def test_mixture(pkg, dtype, M, D, E, top, ff, shared):
    cfg = G.config(D, 8, [G.rglru(8, 1, 1, G.moe(E, top, ff, shared))])
    w = O.random_weights(cfg, E)
    model = pkg.GupitarForCausalLM(pkg.GupitarConfig(**cfg), device="cuda", dtype=dtype)
    model.load_state_dict(w)
    desc, Dp = model.layers[0].moe, pad8(D)
    g = torch.Generator().manual_seed(M)
    h = torch.randn(M, D, generator=g).to(dtype).float()
    if M > 100:
        h[100:] = h[100:] * 0.02 + h[0]  # most rows choose the same experts
        h = h.to(dtype).float()
    x = torch.randn(M, D, generator=g) * 30
    pad = lambda t: torch.nn.functional.pad(t, (0, Dp - D))
    logits = torch.zeros(M, desc.logit_ld)
    logits[:, :E] = h @ w["l0.mlp.router"].T
    logits[:, E + 1:] = 1e9  # pads are never chosen
    if shared is not None:
        logits[:, E] = (h @ w["l0.mlp.shared.sg"].T)[:, 0]
    stream = pad(x).cuda()
    pkg.hip.moe(desc, pad(h).to(dtype).cuda(), logits.cuda(), stream)
    want = O.mixture(h.double(), {k: t.double() for k, t in w.items()}, "l0.mlp.", cfg["layers"][0]["mlp"])
    got = stream.cpu()[:, :D].double() - x.double()
    assert (got - want).abs().max() < (3e-5 if dtype == F32 else 2e-2) * max(1.0, want.abs().max().item())
    assert Dp == D or stream[:, D:].abs().max() == 0


@pytest.mark.parametrize("M,D,E,top,ff", [(900, 96, 2, 1, 136), (700, 64, 3, 3, 264), (1100, 264, 1, 1, 72)])
def test_mixture_in_large_tiles(pkg, M, D, E, top, ff):
    """Enough rows per expert for the 256-row tiles, a last tile cut short, experts of unequal share; every row against a dense sum."""
    cfg = G.config(D, 8, [G.rglru(8, 1, 1, G.moe(E, top, ff))])
    w = O.random_weights(cfg, E)
    model = pkg.GupitarForCausalLM(pkg.GupitarConfig(**cfg), device="cuda", dtype=BF16)
    model.load_state_dict(w)
    g = torch.Generator().manual_seed(M)
    h = torch.randn(M, D, generator=g).to(BF16)
    logits = torch.full((M, model.layers[0].moe.logit_ld), 1e9)
    logits[:, :E] = torch.randn(M, E, generator=g) + torch.arange(E) * 0.5
    x = torch.randn(M, D, generator=g) * 10
    stream = x.clone().cuda()
    pkg.hip.moe(model.layers[0].moe, h.cuda(), logits.cuda(), stream)
    s, want = torch.sigmoid(logits[:, :E].double()), torch.zeros(M, D).double()
    chosen = torch.zeros(M, E).scatter(1, s.topk(top, 1).indices, 1.0)
    for e in range(E):
        want += chosen[:, e:e + 1] * O.gated_mlp(s[:, e:e + 1] * h.double(), {k: t.double() for k, t in w.items()}, f"l0.mlp.e{e}.")
    assert (stream.cpu().double() - x - want).abs().max() < 2e-2 * max(1.0, want.abs().max().item())


@DT
@pytest.mark.parametrize("M", [1, 20])
def test_mixture_prefers_the_lower_index_among_equals(pkg, dtype, M):
    D, E, top = 32, 6, 2
    cfg = G.config(D, 8, [G.rglru(8, 1, 1, G.moe(E, top, 16))])
    w = O.random_weights(cfg, 5)
    model = pkg.GupitarForCausalLM(pkg.GupitarConfig(**cfg), device="cuda", dtype=dtype)
    model.load_state_dict(w)
    h = torch.randn(M, D, generator=torch.Generator().manual_seed(0)).to(dtype)
    logits = torch.full((M, 16), -3.0)
    logits[:, 4] = logits[:, 1] = logits[:, 2] = 0.5
    x = torch.zeros(M, D, device="cuda")
    pkg.hip.moe(model.layers[0].moe, h.cuda(), logits.cuda(), x)
    s = torch.sigmoid(torch.tensor(0.5))
    want = sum(O.gated_mlp(s * h.float(), w, f"l0.mlp.e{e}.") for e in (1, 2))
    assert (x.cpu() - want).abs().max() < (1e-5 if dtype == F32 else 2e-2)


# ---- whole models ------------------------------------------------------------------------------------
def feed(model, ids, cuts, cache=None, runner=None):
    """Portions of a prompt through forward(), single tokens through the decode runner; logits of every position."""
    cache = cache or model.new_cache()
    pos, out = 0, []
    for n in cuts:
        part = ids[pos:pos + n][None].cuda()
        if n == 1:
            runner = runner or model.decode_runner(cache, 1)
            out.append(runner.step(part.view(-1))[0].clone())
        else:
            out.append(model.forward(part, past_key_values=cache).logits[0])
        pos += n
    return torch.cat(out).cpu(), runner


@pytest.mark.parametrize("name", G.CASES)
def test_model_against_the_oracle(pkg, name):
    cfg, w, model = G.build(pkg, name, F32)
    ids = G.tokens(cfg, 110)
    want, trail = O.forward(cfg, w, ids)
    out = model.forward(ids[None], output_hidden_states=True)
    for layer, (got, ref) in enumerate(zip(out.hidden_states[:, 0], trail)):
        assert G.rel(got, ref) < 5e-5, layer
    assert G.rel(out.logits[0], want) < 5e-5
    cache, runner = model.new_cache(), None
    for cuts in ([110], [2, 3, 1, 2, 40, 1, 1, 33, 27], [60] + [1] * 50, [1] * 30 + [80]):
        cache.reset()  # the same storage again: nothing of the earlier sequence may show
        got, runner = feed(model, ids, cuts, cache, runner)
        assert G.rel(got, want) < 5e-5, cuts
    for places in ([3, 109], [109, 3, 3], [7]):
        assert G.rel(model.forward(ids[None], logit_positions=places).logits[0], want[places]) < 5e-5


@pytest.mark.parametrize("name", G.CASES)
def test_model_in_bf16(pkg, name):
    cfg, w, model = G.build(pkg, name, BF16)
    ids = G.tokens(cfg, 110)
    want, _ = O.forward(cfg, w, ids)
    for cuts in ([110], [2, 3, 1, 2, 40, 1, 1, 33, 27], [60] + [1] * 50):
        err = G.rows(feed(model, ids, cuts)[0], want)
        # a row whose choice of experts is a close call may take another expert than the oracle's
        assert err.quantile(0.9) < 6e-2 and err.median() < 3e-2, cuts


def test_long_prompt_runs_in_portions_of_its_own(pkg):
    cfg, w, model = G.build(pkg, BOTH, F32)
    ids = G.tokens(cfg, 150)
    want = model.forward(ids[None]).logits
    model.ROWS_PER_CALL = 64
    assert G.rel(model.forward(ids[None]).logits, want) < 1e-5
    assert G.rel(model.forward(ids[None], logit_positions=[63, 64, 149]).logits, want[:, [63, 64, 149]]) < 1e-5


@pytest.mark.parametrize("name", [BOTH, ODD])
def test_batch_of_equal_lengths_against_each_alone(pkg, name):
    cfg, w, model = G.build(pkg, name, F32)
    ids = torch.stack([G.tokens(cfg, 50, seed=s) for s in range(3)])
    cache = model.new_cache()
    got = [model.forward(ids[:, :23], past_key_values=cache).logits, model.forward(ids[:, 23:40], past_key_values=cache).logits]
    runner = model.decode_runner(cache, 3)
    got += [runner.step(ids[:, t].cuda())[0].clone()[:, None] for t in range(40, 50)]
    got = torch.cat(got, 1)
    for b in range(3):
        assert G.rel(got[b], O.forward(cfg, w, ids[b])[0]) < 5e-5


def test_interleaved_requests_of_unequal_length(pkg):
    """Requests that live at the same time, end, and hand their caches on."""
    from recurrent_pretraining_amd.trace import TraceReplay

    cfg, w, model = G.build(pkg, ODD, F32)
    want = {n: O.forward(cfg, w, G.tokens(cfg, n, seed=n))[0] for n in (60, 35, 20, 44)}
    trace, at, got = TraceReplay(model, 64), {}, {}

    def go(n, count):
        lo = at.get(n, 0)
        rows = trace.feed(f"req{n}", G.tokens(cfg, n, seed=n)[lo:lo + count].tolist(), list(range(count)))
        got.setdefault(n, []).append(rows.cpu().clone())
        at[n] = lo + count

    go(60, 30), go(35, 2), go(60, 1), go(35, 30), go(60, 2), go(35, 1), go(35, 1), go(35, 1)
    trace.end("req35")
    go(20, 1), go(60, 25), go(20, 18), go(44, 43), go(20, 1), go(60, 1), go(60, 1), go(44, 1)
    for n in want:
        assert G.rel(torch.cat(got[n]), want[n]) < 5e-5, n
    assert len(trace.caches) == 3


def test_trace_replay_writes_what_was_asked_for(pkg, tmp_path):
    from recurrent_pretraining_amd import trace

    cfg, w, model = G.build(pkg, BOTH, F32)
    ids = G.tokens(cfg, 12)
    want = O.forward(cfg, w, ids)[0]
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": ids[:9].tolist(), "want": [2, 8]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": ids[9:11].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": ids[11:].tolist(), "want": [0]}], "end": ["x"]}]
    done = io.StringIO()
    trace.replay(model, io.StringIO("\n".join(json.dumps(s) for s in steps)), str(tmp_path), done, max_tokens=12)
    assert done.getvalue().split() == ["done", "0", "done", "1", "done", "2"] and not (tmp_path / "1.f32").exists()
    got = torch.frombuffer(bytearray((tmp_path / "0.f32").read_bytes()), dtype=F32).view(2, -1)
    assert G.rel(got, want[[2, 8]]) < 5e-5
    assert G.rel(torch.frombuffer(bytearray((tmp_path / "2.f32").read_bytes()), dtype=F32).view(1, -1), want[[11]]) < 5e-5


@pytest.mark.parametrize("name", [BOTH, WIDE])
def test_greedy_generation(pkg, name):
    cfg, w, model = G.build(pkg, name, F32)
    prompt = G.tokens(cfg, 17)
    want = O.greedy(cfg, w, prompt.tolist(), 20)
    for graph in (True, False):
        got = model.generate(prompt[None].cuda(), pkg.GenerationSettings(max_new_tokens=20), use_graph=graph)
        assert got[0, 17:].tolist() == want
    assert model.generate(prompt[None].cuda(), max_new_tokens=20, do_sample=False)[0, 17:].tolist() == want  # transformers' own loop
    stop = model.generate(prompt[None].cuda(), pkg.GenerationSettings(max_new_tokens=20, eos_token_id=want[3]))
    assert stop[0, 17:].tolist() == want[:want.index(want[3]) + 1]
    torch.manual_seed(0)
    s = model.generate(prompt[None].cuda(), pkg.GenerationSettings(max_new_tokens=6, do_sample=True, top_k=1))
    assert s[0, 17:].tolist() == want[:6]
    two = torch.stack([prompt, G.tokens(cfg, 17, seed=8)])
    both = model.generate(two.cuda(), pkg.GenerationSettings(max_new_tokens=8))
    assert both[0, 17:].tolist() == want[:8] and both[1, 17:].tolist() == O.greedy(cfg, w, two[1].tolist(), 8)


@pytest.mark.parametrize("name", [BOTH, WIDE])
def test_long_decoding_across_captures_and_growing_caches(pkg, name):
    """Past the bound a captured step was sized for and past the cache's first capacity, replayed steps against one prompt pass."""
    cfg, w, model = G.build(pkg, name, F32)
    ids = G.tokens(cfg, 1040)
    want = model.forward(ids[None]).logits[0].cpu()
    cache = model.new_cache()
    model.forward(ids[None, :1000], past_key_values=cache)
    runner = model.decode_runner(cache, 1)
    got = torch.cat([runner.step(ids[t:t + 1].cuda())[0].clone() for t in range(1000, 1040)]).cpu()
    assert G.rel(got, want[1000:]) < 2e-5


@DT
@pytest.mark.parametrize("N,D,dim", [(40, 56, 50), (1408, 2048, 2044)])
def test_gated_product_behind_a_norm(pkg, dtype, N, D, dim):
    """A dense feed-forward's first half at one row, through a layer: its norm rides in the product."""
    cfg = G.config(dim, 16, [G.rglru(8, 1, 1, G.dense(N))])
    w = O.random_weights(cfg, 1)
    model = pkg.GupitarForCausalLM(pkg.GupitarConfig(**cfg), device="cuda", dtype=dtype)
    model.load_state_dict(w)
    ids = torch.tensor([3])
    want, trail = O.forward(cfg, {k: t.double() for k, t in w.items()}, ids)
    out = model.forward(ids[None], output_hidden_states=True)
    assert G.rel(out.hidden_states[0, 0], trail[0]) < (1e-5 if dtype == F32 else 2e-2)
    assert G.rel(out.logits[0], want) < (1e-5 if dtype == F32 else 3e-2)


def test_invalid_arguments_are_refused(pkg):
    hip = pkg.hip
    a = Latent(pkg, 2, 16, 8, 16, 24, 20, F32, t_max=32)
    z, q = a.rows(*inputs(4, 2, 16, 8, 16, 24))
    with pytest.raises(hip.RavenHipError):
        hip.latent_attention(a.desc, q, z, a.native, 1, 4, 30)           # positions past the cache
    with pytest.raises(hip.RavenHipError):
        hip.latent_attention(a.desc, q, z, a.native, 2, 2, 0)            # two sequences in a cache of one
    with pytest.raises(hip.RavenHipError):
        hip.rglru(hip.Rglru(None, None, None, None, None, 2, 12, 2, 24), torch.zeros(1, 48, device="cuda"), torch.zeros(1, 2, 24, device="cuda"),
                  torch.zeros(1, 24, device="cuda"), 1, 1, 0)            # a block that is no multiple of 8
    with pytest.raises(hip.RavenHipError):
        hip.moe(hip.Moe(None, None, None, None, None, 4, 5, 8, 0, 16), torch.zeros(1, 8, device="cuda"), torch.zeros(1, 16, device="cuda"),
                torch.zeros(1, 8, device="cuda"))                        # more experts than there are
