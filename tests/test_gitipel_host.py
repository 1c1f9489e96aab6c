"""Gitipel on the host: configuration, registry, checkpoint loading into the kernels' padded buffers, cache bookkeeping, and the
closed forms that pin the CPU oracle."""

import json
import math
import os
import subprocess
import sys

import pytest
import torch

import gitipel_cases as G
from oracle import gitipel_oracle as O


@pytest.mark.parametrize("name", G.CASES)
def test_checkpoint_round_trip_through_the_padded_buffers(pkg, tmp_path, name):
    cfg, w, model = G.build(pkg, name, torch.bfloat16, device="cpu")
    assert set(model.state_dict()) == set(w)
    for k, t in model.state_dict().items():
        assert torch.equal(t.float(), w[k]), k
    model.save_pretrained(tmp_path)
    again = pkg.load_model(str(tmp_path), device="cpu", dtype=torch.float32)
    assert type(again) is pkg.GitipelForCausalLM and again.runs == O.layer_runs(cfg)
    for k, t in again.state_dict().items():
        assert torch.equal(t.float(), w[k]), k


def test_padding_stays_zero_and_heads_are_padded_one_by_one(pkg):
    cfg, w, model = G.build(pkg, "sizes that are no multiple of eight", torch.float32, device="cpu")
    q = model.layers[0].w_in[:4 * 16].view(4, 16, 56)
    assert torch.equal(q[:, :10, :50].reshape(40, 50), w["l0.mix.q"]) and q[:, 10:].abs().max() == 0 and q[:, :, 50:].abs().max() == 0
    o = model.layers[0].w_out.view(56, 4, 16)
    assert torch.equal(o[:50, :, :10].reshape(50, 40), w["l0.mix.o"]) and o[50:].abs().max() == 0 and o[:, :, 10:].abs().max() == 0
    assert torch.equal(model.layers[1].conv[:, :50], w["l1.canon1"].t()) and model.layers[1].conv[:, 50:].abs().max() == 0


def test_loading_refuses_what_does_not_fit(pkg):
    cfg, w, model = G.build(pkg, "no loop, one tap, single head", torch.float32, device="cpu")
    with pytest.raises(KeyError):
        model.load_state_dict({k: v for k, v in w.items() if k != "head"})
    with pytest.raises(ValueError):
        model.load_state_dict({**w, "head": w["head"][:-1]})
    with pytest.raises(pkg.hip.RavenHipError):
        model.forward(torch.zeros(1, 3, dtype=torch.long))  # no CPU path


def test_registry_resolves_families_by_config(pkg):
    assert pkg.family_of({"architecture": "Gitipel"})[1] is pkg.GitipelForCausalLM
    assert pkg.family_of({"model_type": "huginn_raven"})[1] is pkg.RavenForCausalLM
    with pytest.raises(ValueError):
        pkg.family_of({"architecture": "Unheard-of"})


@pytest.mark.parametrize("change", [dict(layers=[{"type": "attention", "mixer": {"heads": 5, "kv_heads": 2, "dim": 8, "vdim": 8}, "mlp": None}]),
                                    dict(layers=[{"type": "convolution", "mixer": {}, "mlp": None}]),
                                    dict(loop={"start": 2, "stop": 2, "times": 2}),
                                    dict(layers=[{"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 16}, "mlp": None}])])
def test_configuration_errors_are_named(pkg, change):
    cfg, _ = G.CASES["no loop, one tap, single head"]
    with pytest.raises(ValueError):
        pkg.GitipelConfig(**{**cfg, **change})


def test_order_of_runs(pkg):
    cfg, _ = G.CASES["looped middle, grouped heads, a layer without feed-forward"]
    assert pkg.GitipelConfig(**cfg).runs() == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (1, 2), (2, 2), (3, None)]


def test_mixer_cache_grows_and_is_given_back(pkg):
    plan = [{"taps": 3, "ld": 16, "heads": 2, "head_dim": 8, "kv_heads": 1}, {"taps": 3, "ld": 16, "heads": 2, "head_dim": 8, "kv_heads": 0}]
    c = pkg.MixerStateCache(plan)
    c.ensure(1, 10, torch.float32, "cpu")
    c.keys[0].normal_()
    c.states[1].normal_()
    before, state = c.keys[0].clone(), c.states[1]
    c.advance(10)
    c.ensure(1, 300, torch.float32, "cpu")
    assert c.t_max >= 300 and torch.equal(c.keys[0][:, :, :before.shape[2]], before) and c.states[1] is state and c.generation == 2
    with pytest.raises(ValueError):
        c.ensure(2, 11, torch.float32, "cpu")
    c.reset()
    c.ensure(2, 11, torch.float32, "cpu")
    assert c.keys[0].shape[0] == 2 and c.get_seq_length() == 0
    fixed = pkg.MixerStateCache(plan, max_length=20)
    with pytest.raises(ValueError):
        fixed.ensure(1, 21, torch.float32, "cpu")


def test_requests_share_a_pool_of_caches(pkg):
    made = []

    def make():
        made.append(pkg.MixerStateCache([]))
        return made[-1]

    pool = pkg.RequestCaches(make)
    a, b = pool.get("a"), pool.get("b")
    assert a is not b and pool.get("a") is a and len(pool) == 2
    a.advance(5)
    pool.release("a")
    assert pool.get("c") is a and a.get_seq_length() == 0 and len(made) == 2


# ---- the oracle's own pins ------------------------------------------------------------------------
def test_oracle_convolution_is_a_causal_depthwise_convolution():
    h, w = torch.randn(9, 5), torch.randn(5, 3)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(h.t()[None], (2, 0)), w[:, None], groups=5)[0].t()
    assert torch.allclose(O.causal_conv(h, w), want, atol=1e-5)


def test_oracle_attention_without_cap_and_bias_is_plain_attention():
    q, k = torch.randn(7, 4, 6), torch.randn(7, 2, 6)
    got = O.attention(q, k, 0.4, 1e6, torch.zeros(4), torch.zeros(4))
    kk = k.repeat_interleave(2, 1).transpose(0, 1)
    want = torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1), kk, kk, is_causal=True, scale=0.4).transpose(0, 1)
    assert torch.allclose(got, want, atol=2e-3)  # tanh at 1e-6 of its range is not exactly linear in float32


def test_oracle_distance_bias_and_cap_by_hand():
    assert math.isclose(O.distance_bias(1.5, 0.25, 9, 1), 1.5 * math.log(3.0), rel_tol=1e-6)
    assert abs(float(O.softcap(torch.tensor(1e4), 5.0)) - 5.0) < 1e-6
    # two keys, equal scores: the nearer one wins by exactly the bias
    k = torch.ones(2, 1, 1)
    out = O.attention(torch.zeros(2, 1, 1), k * torch.tensor([0.0, 1.0]).view(2, 1, 1), 1.0, 3.0, torch.tensor([2.0]), torch.tensor([1.0]))
    assert abs(float(out[1, 0, 0]) - 1 / (1 + math.exp(-2 * math.log(2.0)))) < 1e-6


def test_oracle_delta_rule_closed_forms():
    T, H, d = 6, 1, 4
    r, k, v = (torch.randn(T, H, d, dtype=torch.float64) for _ in range(3))
    ones, zeros = torch.ones(T, H, d, dtype=torch.float64), torch.zeros(T, H, d, dtype=torch.float64)
    out, S = O.delta_rule(r, k, v, ones, zeros)                         # no decay, no removal: linear attention
    assert torch.allclose(S[0], torch.einsum("thk,thv->kv", k, v))
    assert torch.allclose(out[-1, 0], S[0].T @ r[-1, 0])
    # full removal of a repeated unit key: only the last value stays
    key = torch.nn.functional.normalize(torch.randn(d, dtype=torch.float64), dim=0).expand(T, H, d)
    _, S = O.delta_rule(r, key, v, ones, ones)
    assert torch.allclose(key[0, 0] @ S[0], v[-1, 0], atol=1e-5)
    w = O.delta_decay(torch.zeros(1, 3), torch.zeros(2, 3), torch.zeros(4, 2), torch.tensor([-50.0, 0.0, 50.0, 1.0]))
    assert abs(float(w[0, 0]) - 1.0) < 1e-6 and abs(float(w[0, 2]) - math.exp(-math.exp(-0.5))) < 1e-6


def test_trace_command_refuses_an_unknown_model(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Unheard-of"}))
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out",
                        str(tmp_path)], input="", capture_output=True, text=True)
    assert r.returncode == 1 and "Unheard-of" in r.stderr
