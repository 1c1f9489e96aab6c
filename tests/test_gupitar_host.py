"""Gupitar on the host: configuration, registry, checkpoint loading into the kernels' padded buffers, cache bookkeeping, and the closed
forms that pin the CPU oracle."""

import math

import pytest
import torch

import gupitar_cases as G
from oracle import gupitar_oracle as O

ODD = "sizes that are no multiple of eight"
BOTH = "both mixers, latents read by later layers under other windows"


@pytest.mark.parametrize("name", G.CASES)
def test_checkpoint_round_trip_through_the_padded_buffers(pkg, tmp_path, name):
    cfg, w, model = G.build(pkg, name, torch.bfloat16, device="cpu")
    assert set(model.state_dict()) == set(w)
    for k, t in model.state_dict().items():
        assert torch.equal(t.float(), w[k]), k
    model.save_pretrained(tmp_path)
    again = pkg.load_model(str(tmp_path), device="cpu", dtype=torch.float32)
    assert type(again) is pkg.GupitarForCausalLM
    for k, t in again.state_dict().items():
        assert torch.equal(t.float(), w[k]), k


def test_layout_of_a_latent_layer(pkg):
    """Heads, ranks and rotated parts padded one by one, rotation pairs side by side, W_uk a second time transposed."""
    cfg, w, model = G.build(pkg, ODD, torch.float32, device="cpu")
    layer = model.layers[0]
    assert layer.w_in.shape == (24 + 32 + 8 + 3 * 16, 56)
    rot = layer.w_in[24 + 32:24 + 32 + 8]
    stored = w["l0.mix.dkv"][27:]
    assert torch.equal(rot[:6, :50], stored[[0, 3, 1, 4, 2, 5]]) and rot[6:].abs().max() == 0
    q = layer.w_uq.view(3, 16 + 8, 24)
    assert torch.equal(q[1, :10, :21], w["l0.mix.uq"].view(3, 16, 21)[1, :10])
    assert torch.equal(q[2, 16:22, :21], w["l0.mix.uq"].view(3, 16, 21)[2, [10, 13, 11, 14, 12, 15]])
    assert q[:, 10:16].abs().max() == 0 and q[:, 22:].abs().max() == 0 and q[:, :, 21:].abs().max() == 0
    uk = w["l0.mix.uk"].view(3, 10, 27)
    assert torch.equal(layer.w_uk_t[:, :27, :10], uk.transpose(1, 2)) and layer.w_uk_t[:, 27:].abs().max() == 0
    assert torch.equal(layer.norm1[:50], 1 + w["l0.norm1"]) and layer.norm1[50:].abs().max() == 0
    assert model.layers[2].w_in.shape == (24 + 8, 56) and model.layers[2].latent.own_kv == 0


def test_layout_of_a_recurrent_layer(pkg):
    cfg, w, model = G.build(pkg, ODD, torch.float32, device="cpu")
    layer = model.layers[1]
    assert layer.conv.shape == (2, 48)
    assert torch.equal(layer.conv.view(2, 3, 16)[:, :, :13].permute(1, 2, 0).reshape(39, 2), w["l1.mix.conv"])
    assert torch.equal(layer.gates[2, 1, :13, :13], w["l1.mix.ri"][2]) and layer.gates[:, :, 13:].abs().max() == 0
    assert torch.allclose(layer.softplus.view(3, 16)[:, :13].reshape(39), torch.nn.functional.softplus(w["l1.mix.lam"]))
    assert layer.softplus.view(3, 16)[:, 13:].abs().max() == 0


def test_loading_refuses_what_does_not_fit(pkg):
    cfg, w, model = G.build(pkg, ODD, torch.float32, device="cpu")
    with pytest.raises(KeyError):
        model.load_state_dict({k: v for k, v in w.items() if k != "l0.mix.dq.norm"})
    with pytest.raises(ValueError):
        model.load_state_dict({**w, "l0.mix.uq": w["l0.mix.uq"][:-1]})
    with pytest.raises(pkg.hip.RavenHipError):
        model.forward(torch.zeros(1, 3, dtype=torch.long))  # no CPU path


def test_registry_resolves_the_family(pkg):
    assert pkg.family_of({"architecture": "Gupitar"}) == (pkg.GupitarConfig, pkg.GupitarForCausalLM)
    assert pkg.family_of({"model_type": "gupitar"})[1] is pkg.GupitarForCausalLM


@pytest.mark.parametrize("layers", [
    [G.latent(2, 8, 4, 8, 16, 16, 4, kv_from=0)],                                                            # of itself
    [G.rglru(16, 2, 2), G.latent(2, 8, 4, 8, 16, 16, 4, kv_from=0)],                                         # of a recurrent layer
    [G.latent(2, 8, 4, 8, 16, 16, 4), G.latent(2, 8, 4, 8, 16, 24, 4, kv_from=0)],                           # another rank
    [G.latent(2, 8, 4, 8, 16, 16, 4), G.latent(2, 8, 4, 8, 16, 16, 4, kv_from=0, base=7.0)],                 # another rotation
    [G.latent(2, 8, 4, 8, 16, 16, 4), G.latent(2, 8, 4, 8, 16, 16, 4, kv_from=0), G.latent(2, 8, 4, 8, 16, 16, 4, kv_from=1)],
    [G.latent(2, 8, 5, 8, 16, 16, 4)], [G.latent(2, 8, 4, 8, 16, 16, 0)], [G.rglru(15, 2, 2)], [G.rglru(16, 2, 2, G.moe(3, 4, 8))],
    [{"type": "attention", "mixer": {}, "mlp": None}], [{**G.rglru(16, 2, 2), "mlp": {"kind": "sparse"}}]])
def test_configuration_errors_are_named(pkg, layers):
    with pytest.raises(ValueError):
        pkg.GupitarConfig(**G.config(32, 64, layers))


def test_cache_of_latents_grows_and_is_shared(pkg):
    plan = [{"latent": (16, 8), "angles": (100.0, 6)}, {"taps": 2, "ld": 24, "state": (24,)}, {"latent_from": 0}]
    c = pkg.MixerStateCache(plan)
    c.ensure(2, 10, torch.float32, "cpu")
    c.latents[0][0].normal_()
    c.latents[0][1].normal_()
    before, state, ring = [t.clone() for t in c.latents[0]], c.states[1], c.rings[1]
    assert c.native(2).latent.latent == c.native(0).latent.latent == c.latents[0][0].data_ptr() and c.latents[2] is None
    assert state.shape == (2, 24) and ring.shape == (2, 2, 24) and c.rings[0] is None and c.states[2] is None
    c.advance(10)
    c.ensure(2, 700, torch.float32, "cpu")
    assert c.t_max >= 700 and all(torch.equal(n[:, :o.shape[1]], o) for n, o in zip(c.latents[0], before)) and c.states[1] is state
    assert c.native(2).latent.latent == c.latents[0][0].data_ptr() and c.generation == 2
    table = c.angles[(100.0, 6, 8)]
    assert table.shape == (c.t_max, 8)
    for pos, pair in ((0, 1), (5, 0), (699, 2)):
        a = pos * 100.0 ** (-2 * pair / 6)
        assert abs(table[pos, 2 * pair].item() - math.cos(a)) < 1e-6 and abs(table[pos, 2 * pair + 1].item() - math.sin(a)) < 1e-6
    assert table[:, 6].eq(1).all() and table[:, 7].eq(0).all()
    assert c.get_memory_usage() > 0


# ---- the oracle's own pins ------------------------------------------------------------------------
def test_oracle_rotation():
    x = torch.randn(5, 2, 10, dtype=torch.float64)
    pos = torch.arange(5)
    y = O.rotate(x, pos, 100.0, 6)
    assert torch.equal(y[..., 6:], x[..., 6:]) and torch.equal(y[0], x[0])
    z = torch.complex(x[..., :3], x[..., 3:6]) * torch.exp(1j * pos[:, None, None] * 100.0 ** (-torch.arange(3) / 3.0))
    assert torch.allclose(y[..., :6], torch.cat([z.real, z.imag], -1))


def test_oracle_attention_with_a_window_of_everything_is_causal_attention():
    q, k, v = torch.randn(9, 3, 6), torch.randn(9, 3, 6), torch.randn(9, 3, 4)
    got = O.windowed_attention(q, k, v, 0.4, 9)
    want = torch.nn.functional.scaled_dot_product_attention(*(t.transpose(0, 1) for t in (q, k, v)), is_causal=True, scale=0.4).transpose(0, 1)
    assert torch.allclose(got, want, atol=1e-5)
    assert torch.allclose(O.windowed_attention(q, k, v, 0.4, 1), v)
    two = O.windowed_attention(q, k, v, 0.4, 2)
    moved = v.clone()
    moved[3] += 1
    changed = (O.windowed_attention(q, k, moved, 0.4, 2) != two).flatten(1).any(1)
    assert changed.tolist() == [i in (3, 4) for i in range(9)]


def test_oracle_recurrence_closed_forms():
    u, ones = torch.randn(6, 3, dtype=torch.float64), torch.ones(6, 3, dtype=torch.float64)
    out, _ = O.gated_recurrence(u, ones, ones, torch.full((3,), 50.0, dtype=torch.float64))   # full decay: the input alone
    assert torch.allclose(out, u)
    out, _ = O.gated_recurrence(u, 0 * ones, ones, torch.zeros(3, dtype=torch.float64))        # no decay: nothing ever enters
    assert out.abs().max() == 0
    lam = torch.zeros(3, dtype=torch.float64)
    r = ones * 0.1
    a = math.exp(-8 * 0.1 * math.log(2.0))
    out, S = O.gated_recurrence(u, r, ones, lam)
    want = sum(a ** (5 - t) * math.sqrt(1 - a * a) * u[t] for t in range(6))
    assert torch.allclose(out[-1], want) and torch.equal(S, out[-1])


def test_oracle_convolution_and_gates():
    u, w, b = torch.randn(9, 5), torch.randn(5, 3), torch.randn(5)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(u.t()[None], (2, 0)), w[:, None], b, groups=5)[0].t()
    assert torch.allclose(O.causal_conv(u, w, b), want, atol=1e-5)
    x, m, bias = torch.randn(4, 6), torch.randn(2, 3, 3), torch.randn(2, 3)
    assert torch.allclose(O.block_gate(x, m, bias), torch.sigmoid(x @ torch.block_diag(*m).T + bias.view(-1)), atol=1e-6)


def test_oracle_mixture_scales_the_experts_input():
    """Against the same sum written the other way; the scores are neither normalised nor applied to the outputs."""
    D, ff = 6, 5
    g = torch.Generator().manual_seed(0)
    cfg = G.config(D, 8, [G.rglru(8, 1, 1, G.moe(4, 2, ff, 3))])
    w = O.random_weights(cfg, 1)
    h = torch.randn(7, D, generator=g)
    out = O.mixture(h, w, "l0.mlp.", cfg["layers"][0]["mlp"])
    s = torch.sigmoid(h @ w["l0.mlp.router"].T)
    for t in range(7):
        want = torch.sigmoid(h[t] @ w["l0.mlp.shared.sg"][0]) * O.gated_mlp(h[t], w, "l0.mlp.shared.")
        for e in sorted(range(4), key=lambda e: -s[t, e])[:2]:
            want = want + O.gated_mlp(s[t, e] * h[t], w, f"l0.mlp.e{e}.")
        assert torch.allclose(out[t], want, atol=1e-5)
    assert torch.allclose(O.gelu_tanh(h), torch.nn.functional.gelu(h, approximate="tanh"), atol=1e-6)
    assert torch.allclose(O.centred_norm(h, torch.zeros(D), 0.0).pow(2).mean(-1), torch.ones(7), atol=1e-5)
