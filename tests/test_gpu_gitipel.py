"""Gitipel on the GPU against the CPU oracle: every mechanism alone, then whole models -- prompts, portions, decoding, batches,
caches used again, greedy generation."""

import io
import json
import math

import pytest
import torch

import gitipel_cases as G
from oracle import gitipel_oracle as O

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DT = pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])


def pad8(n):
    return (n + 7) // 8 * 8


def pad_heads(x, dp):
    """[T, H, d] -> [T, H * dp], zeros behind each head."""
    T, H, d = x.shape
    out = torch.zeros(T, H, dp)
    out[:, :, :d] = x
    return out.view(T, H * dp)


# ---- products ----------------------------------------------------------------------------------------
@DT
@pytest.mark.parametrize("M", [1, 2, 7, 32, 33, 70, 300])
@pytest.mark.parametrize("N,K0,K1", [(72, 56, 0), (80, 64, 64), (24, 16, 0), (211, 40, 0), (320, 2048, 0)])
def test_linear_epilogue(pkg, dtype, M, N, K0, K1):
    g = torch.Generator().manual_seed(M * 1000 + N)
    x0, w = torch.randn(M, K0, generator=g).to(dtype), (torch.randn(N, K0 + K1, generator=g) / math.sqrt(K0 + K1)).to(dtype)
    x1 = torch.randn(M, K1, generator=g).to(dtype) if K1 else None
    bias, res = torch.randn(N, generator=g), torch.randn(M, N, generator=g) * 30
    x = x0 if x1 is None else torch.cat([x0, x1], 1)
    z = x.double() @ w.double().T
    dev = lambda t: None if t is None else t.cuda()
    ws = pkg.hip.linear_workspace(M, N, "cuda")
    run = lambda **kw: pkg.hip.linear_epilogue(dev(x0), dev(w), x1=dev(x1), workspace=ws, **kw).double().cpu()
    tol = 2e-5 if dtype == F32 else 3e-5  # bf16 operands are exact in float: only the order of the sums differs
    assert (run(bias=dev(bias), scale=0.5, residual=dev(res)) - (0.5 * z + bias + res)).abs().max() < tol
    stream = dev(res).clone()
    pkg.hip.linear_epilogue(dev(x0), dev(w), x1=dev(x1), residual=stream, out=stream, workspace=ws)  # in place
    assert (stream.double().cpu() - (z + res)).abs().max() < tol
    for act, fn in ((pkg.hip.ACT_GELU, O.gelu_erf), (pkg.hip.ACT_TANH, torch.tanh)):
        want = fn(z + bias)
        assert (run(bias=dev(bias), act=act) - want).abs().max() < tol
        got = run(bias=dev(bias), act=act, out_f32=False)
        assert ((got - want).abs() <= (2e-5 if dtype == F32 else want.abs() * 2 ** -8 + 1e-4)).all()


@pytest.mark.parametrize("M,N,K", [(129, 16, 256), (700, 80, 2048), (1000, 128, 288), (333, 64, 1056), (8192, 96, 512)])
def test_linear_epilogue_of_narrow_matrices(pkg, M, N, K):
    """Many rows against a few matrix rows; K with and without whole cache lines per row."""
    g = torch.Generator(device="cuda").manual_seed(N)
    x, w = torch.randn(M, K, generator=g, device="cuda").to(BF16), (torch.randn(N, K, generator=g, device="cuda") / K ** 0.5).to(BF16)
    bias, res = torch.randn(N, generator=g, device="cuda"), torch.randn(M, N, generator=g, device="cuda")
    want = torch.nn.functional.linear(x.float(), w.float())
    assert (pkg.hip.linear_epilogue(x, w, bias=bias, residual=res, scale=0.5) - (0.5 * want + bias + res)).abs().max() < 1e-4
    got = pkg.hip.linear_epilogue(x, w, bias=bias, act=pkg.hip.ACT_TANH, out_f32=False).float()
    assert ((got - torch.tanh(want + bias)).abs() <= 2 ** -8 + 1e-4).all()


def test_linear_epilogue_narrow_rest_behind_large_tiles(pkg):
    """4096 x 4160: a round of 256 x 256 tiles and 64 columns more, which write into the same rows."""
    g = torch.Generator(device="cuda").manual_seed(5)
    M, N, K = 4096, 4160, 256
    x, w = torch.randn(M, K, generator=g, device="cuda").to(BF16), (torch.randn(N, K, generator=g, device="cuda") / K ** 0.5).to(BF16)
    bias, res = torch.randn(N, generator=g, device="cuda"), torch.randn(M, N, generator=g, device="cuda")
    want = torch.nn.functional.linear(x.float(), w.float())
    assert (pkg.hip.linear_epilogue(x, w, bias=bias, residual=res) - (want + bias + res)).abs().max() < 1e-4
    got, ref = pkg.hip.linear_epilogue(x, w, bias=bias, out_f32=False).float(), want + bias
    assert ((got - ref).abs() <= ref.abs() * 2 ** -8 + 1e-4).all()


@pytest.mark.parametrize("M,N,K", [(4096, 2048, 96), (4200, 4096, 64), (16384, 1160, 128)])
def test_linear_epilogue_large_tiles(pkg, M, N, K):
    """Shapes that take the 256 x 256 tiles, also with the last tile columns handed to small tiles."""
    g = torch.Generator(device="cuda").manual_seed(3)
    x, w = torch.randn(M, K, generator=g, device="cuda").to(BF16), (torch.randn(N, K, generator=g, device="cuda") / K ** 0.5).to(BF16)
    bias, res = torch.randn(N, generator=g, device="cuda"), torch.randn(M, N, generator=g, device="cuda")
    want = torch.nn.functional.linear(x.float(), w.float())
    assert (pkg.hip.linear_epilogue(x, w, bias=bias, residual=res, scale=1.5) - (1.5 * want + bias + res)).abs().max() < 1e-4
    got, ref = pkg.hip.linear_epilogue(x, w, bias=bias, act=pkg.hip.ACT_GELU, out_f32=False).float(), torch.nn.functional.gelu(want + bias)
    assert ((got - ref).abs() <= ref.abs() * 2 ** -8 + 1e-4).all()


@DT
@pytest.mark.parametrize("N,D,dim", [(77, 56, 50), (128, 320, 320), (4100, 2048, 2044)])
def test_gemv_behind_a_norm(pkg, dtype, N, D, dim):
    g = torch.Generator().manual_seed(D)
    x, norm, w = torch.randn(D, generator=g) * 20, torch.rand(D, generator=g) + 0.5, (torch.randn(N, D, generator=g) / D ** 0.5).to(dtype)
    x[dim:] = 0
    bias, res = torch.randn(N, generator=g), torch.randn(N, generator=g)
    h = (x / torch.sqrt((x * x).sum() / dim + 1e-3) * norm).to(dtype).double()
    z = w.double() @ h + bias
    run = lambda **kw: pkg.hip.gemv_stream(x.cuda(), norm.cuda(), dim, 1e-3, w.cuda(), dtype, bias=bias.cuda(), **kw).double().cpu()
    tol = 3e-5 if dtype == F32 else 6e-3  # a row element on a tie of the bf16 grid may round the other way
    assert (run(residual=res.cuda()) - (z + res)).abs().max() < tol
    assert (run(act=pkg.hip.ACT_GELU, out_f32=False) - O.gelu_erf(z)).abs().max() < (3e-5 if dtype == F32 else 4e-2)


def test_gelu_over_its_whole_range(pkg):
    """bf16 results use an approximation of erf: every magnitude against the float64 function."""
    z = torch.cat([torch.linspace(-12, 12, 4001), torch.tensor([0.0, -0.0, 1e-30, -1e-6, 100.0, -100.0])]).bfloat16()
    eye = torch.zeros(z.numel(), 8).bfloat16()
    eye[:, 0] = z
    w = torch.zeros(8, 8).bfloat16()
    w[0, 0] = 1
    got = pkg.hip.linear_epilogue(eye.cuda(), w.cuda(), act=pkg.hip.ACT_GELU, out_f32=False)[:, 0].double().cpu()
    want = O.gelu_erf(z.double())
    assert ((got - want).abs() <= want.abs() * 2 ** -8 + 2e-6).all()


# ---- norm and convolution ----------------------------------------------------------------------------
@DT
@pytest.mark.parametrize("D,taps", [(50, 3), (320, 2), (72, 1), (1032, 5), (4104, 4)])
def test_norm_conv_in_portions(pkg, dtype, D, taps):
    T, B, eps = 37, 2, 1e-3
    g = torch.Generator().manual_seed(D)
    x, w, c = torch.randn(B, T, D, generator=g) * 5, torch.rand(D, generator=g) + 0.5, torch.randn(D, taps, generator=g)
    want = torch.stack([(lambda h: h + O.causal_conv(h, c))(O.rms_norm(x[b], w, eps)) for b in range(B)])
    ld = pad8(D)
    row = lambda t: torch.nn.functional.pad(t, (0, ld - D)).cuda().contiguous()
    conv, weight = row(c.t()), row(w)
    for cuts in ([T], [1] * T, [2, 3, 1, 1, 7, 2, 2, 19], [1, 16, 20]):
        ring = torch.full((B, taps, ld), float("nan"), device="cuda")  # what an earlier sequence left must not matter
        pos, parts = 0, []
        for n in cuts:
            rows = row(x[:, pos:pos + n].reshape(B * n, D))
            parts.append(pkg.hip.norm_conv(rows, weight, D, eps, B, n, dtype, conv=conv, ring=ring, pos0=pos).view(B, n, ld))
            pos += n
        got = torch.cat(parts, 1).float().cpu()
        assert got[:, :, D:].abs().max() == 0 if ld > D else True
        assert ((got[:, :, :D] - want).abs() <= (2e-5 if dtype == F32 else 2 ** -8 * want.abs() + 1e-4)).all(), cuts
    plain = pkg.hip.norm_conv(row(x.reshape(B * T, D)), weight, D, eps, B, T, dtype)[:, :D].float().cpu().view(B, T, D)
    want = O.rms_norm(x, w, eps)
    assert ((plain - want).abs() <= (2e-5 if dtype == F32 else 2 ** -8 * want.abs() + 1e-4)).all()


# ---- attention ---------------------------------------------------------------------------------------
def run_attention(pkg, q, k, score, cuts, dtype, t_max=None, dp=None):
    """q [T, H, d], k [T, G, d] in portions; returns [T, H, d] float."""
    T, H, d = q.shape
    dp = dp or pad8(d)
    rows = torch.cat([pad_heads(q, dp), pad_heads(k, dp)], 1).to(dtype).cuda().contiguous()
    keys = torch.full((1, k.shape[1], t_max or T, dp), float("nan"), dtype=dtype, device="cuda")
    pos, out = 0, []
    for n in cuts:
        out.append(pkg.hip.capped_attention(rows[pos:pos + n].contiguous(), keys, score, 1, n, pos, H))
        pos += n
    assert torch.equal(keys[0, :, :T].cpu(), rows[:, H * dp:].view(T, -1, dp).transpose(0, 1).cpu())
    return torch.cat(out).float().cpu().view(T, H, dp)[:, :, :d]


@DT
@pytest.mark.parametrize("H,Gk,d", [(2, 2, 16), (3, 1, 20), (8, 2, 48), (4, 2, 64), (5, 1, 96), (2, 1, 128), (2, 2, 200)])
def test_attention_prompts_portions_and_decoding(pkg, dtype, H, Gk, d):
    T = 150
    g = torch.Generator().manual_seed(H * 100 + d)
    q, k = (torch.randn(T, n, d, generator=g).to(dtype).float() for n in (H, Gk))
    r1, r2 = torch.randn(H, generator=g) * 0.5 + 0.7, torch.rand(H, generator=g)
    score = lambda: pkg.hip.make_score(1.3 / math.sqrt(d), 4.0, r1.cuda(), r2.cuda())
    r1c, r2c = r1.cuda(), r2.cuda()
    sc = pkg.hip.make_score(1.3 / math.sqrt(d), 4.0, r1c, r2c)
    want = O.attention(q, k, 1.3 / math.sqrt(d), 4.0, r1, r2)
    for cuts in ([T], [2, 61, 1, 64, 17, 3, 2], [100] + [1] * 50, [1] * 20 + [130]):
        got = run_attention(pkg, q, k, sc, cuts, dtype, t_max=T + 13)
        assert G.rel(got, want) < (1e-5 if dtype == F32 else 1.2e-2), cuts


@DT
@pytest.mark.parametrize("cap", [0.0, 1.5, 35.0, 60.0])
@pytest.mark.parametrize("bias", [False, True])
def test_attention_caps_and_bias(pkg, dtype, cap, bias):
    """No cap, caps on either side of the bound up to which weights are taken relative to the cap itself, with scores that
    reach it on both sides; without a bias."""
    T, H, Gk, d = 170, 4, 2, 32
    g = torch.Generator().manual_seed(int(cap))
    q, k = (torch.randn(T, n, d, generator=g) for n in (H, Gk))
    q[100:] *= 6
    k[0] = -3 * k[0].abs()
    q[160] = q[160].abs() * 3   # sees scores far below zero only at key 0
    q, k = q.to(dtype).float(), k.to(dtype).float()
    r1, r2 = torch.tensor([0.0, 3.0, 0.4, 1.0]), torch.tensor([1.0, 0.5, 0.01, 0.0])
    if not bias:
        r1, r2 = torch.zeros(H), torch.zeros(H)
    r1c, r2c = r1.cuda(), r2.cuda()
    sc = pkg.hip.make_score(0.5, cap, r1c, r2c) if bias else pkg.hip.make_score(0.5, cap)
    want = O.attention(q.double(), k.double(), 0.5, cap if cap else 1e9, r1.double(), r2.double())
    for cuts in ([T], [20, 2, 100, 1, 1, 46]):
        assert G.rel(run_attention(pkg, q, k, sc, cuts, dtype), want) < (2e-5 if dtype == F32 else 1.5e-2), cuts


@DT
@pytest.mark.parametrize("how", ["prompt", "decoded", "portions"])
def test_attention_far_key_stands_out(pkg, dtype, how):
    """One key aligned with one late query, far back and next to tile borders: it must carry its weight exactly."""
    T, H, d, cap = 700, 2, 64, 20.0
    g = torch.Generator().manual_seed(5)
    q, k = torch.randn(T, H, d, generator=g) * 0.3, torch.randn(T, 1, d, generator=g) * 0.3
    spots = [(0, 699), (63, 640), (64, 641), (127, 650), (128, 655), (511, 690), (512, 691), (1, 64), (2, 63)]
    for i, (src, at) in enumerate(spots):
        axis = torch.zeros(d)
        axis[i] = 1.0
        k[src, 0] = 9.0 * axis
        q[at] = 9.0 * axis
    q, k = q.to(dtype).float(), k.to(dtype).float()
    r1, r2 = torch.tensor([0.5, 1.2]), torch.tensor([0.3, 0.02])
    r1c, r2c = r1.cuda(), r2.cuda()
    sc = pkg.hip.make_score(1 / 8, cap, r1c, r2c)
    cuts = {"prompt": [T], "decoded": [60] + [1] * 10 + [565] + [1] * 65, "portions": [63, 2, 64, 300, 33, 178, 60]}[how]
    got = run_attention(pkg, q, k, sc, cuts, dtype)
    rows = [at for _, at in spots]
    want = O.attention(q[:, :, :].double(), k.double(), 1 / 8, cap, r1.double(), r2.double())
    assert G.rel(got[rows], want[rows]) < (1e-5 if dtype == F32 else 1e-2)
    without = k.clone()
    without[0, 0] = 0
    lost = O.attention(q.double(), without.double(), 1 / 8, cap, r1.double(), r2.double())
    assert G.rel(lost[[699]], want[[699]]) > 0.3  # the test sees a lost far key


@DT
@pytest.mark.parametrize("cap", [0.0, 300.0])
def test_attention_reference_follows_every_lane(pkg, dtype, cap):
    """Without a small cap, scores far apart inside a tile, the largest at each of its places in turn."""
    T, H, d = 128, 2, 32
    g = torch.Generator().manual_seed(4)
    q, k = torch.randn(T, H, d, generator=g), torch.randn(T, 1, d, generator=g)
    for i in range(64, T):
        q[i] = 40 * k[i - 64]
    q, k = q.to(dtype).float(), k.to(dtype).float()
    want = O.attention(q.double(), k.double(), 0.2, cap if cap else 1e9, torch.zeros(H).double(), torch.zeros(H).double())
    for cuts in ([T], [64] + [1] * 64):
        got = run_attention(pkg, q, k, pkg.hip.make_score(0.2, cap), cuts, dtype)
        assert torch.isfinite(got).all() and G.rel(got, want) < (1e-4 if dtype == F32 else 2e-2), cuts


@DT
def test_attention_long_cache_split_over_workgroups(pkg, dtype):
    """Decode rows over a few thousand positions, with the position on the device and a larger bound by value."""
    T, H, Gk, d = 3000, 4, 2, 48
    g = torch.Generator().manual_seed(9)
    q, k = torch.randn(1, H, d, generator=g).to(dtype).float(), torch.randn(T, Gk, d, generator=g).to(dtype).float()
    r1, r2 = torch.tensor([0.1, 2.0, 0.7, 0.0]), torch.tensor([0.3, 0.01, 1.0, 0.5])
    r1c, r2c = r1.cuda(), r2.cuda()
    sc = pkg.hip.make_score(0.4, 9.0, r1c, r2c)
    for t in (1, 2, 127, 128, 129, 1000, 3000):
        keys = torch.full((1, Gk, 4096, d), float("nan"), dtype=dtype, device="cuda")
        keys[0, :, :t - 1] = k[:t - 1].transpose(0, 1).to(dtype)
        row = torch.cat([q.reshape(1, -1), k[t - 1].reshape(1, -1)], 1).to(dtype).cuda()
        got = pkg.hip.capped_attention(row, keys, sc, 1, 1, 4000, H, pos_dev=torch.tensor([t - 1], dtype=torch.int32, device="cuda"))
        s = O.softcap((q[0].view(Gk, 2, d) @ k[:t].permute(1, 2, 0)).view(H, t) * 0.4, 9.0)
        s = s - r1[:, None] * torch.log1p(r2[:, None] * (t - 1 - torch.arange(t)))
        want = (torch.softmax(s.double(), -1).view(Gk, 2, t) @ k[:t].permute(1, 0, 2).double()).view(H, d)
        assert G.rel(got.float().cpu().view(H, d), want) < (1e-5 if dtype == F32 else 6e-3), t


# ---- delta rule --------------------------------------------------------------------------------------
def delta_inputs(T, H, d, seed, decay_shift=-2.0, repeat=False):
    g = torch.Generator().manual_seed(seed)
    r, k, v, gate, a = (torch.randn(T, H, d, generator=g) for _ in range(5))
    decay = torch.randn(T, H, d, generator=g) * 2 + decay_shift
    if repeat:  # the same key again and again, almost fully removed each time: the hardest case for a blocked solve
        k = k[:1].expand(T, H, d) + 0.01 * torch.randn(T, H, d, generator=g)
        a = a + 6.0
    return r, k, v, gate, a, decay, torch.randn(H, d, generator=g) * 0.5, torch.rand(H, d, generator=g) + 0.5


def delta_want(r, k, v, gate, a, decay, a_bias, norm, eps, state=None):
    D = lambda t: t.double()
    w = torch.exp(-math.exp(-0.5) * torch.sigmoid(D(decay)))
    o, S = O.delta_rule(D(r), D(k), D(v), w, torch.sigmoid(D(a) + D(a_bias)), state)
    return O.rms(o, eps) * D(norm) * torch.sigmoid(D(gate)), S


def run_delta(pkg, ins, cuts, eps, dtype, parallel=True, state=None):
    r, k, v, gate, a, decay, a_bias, norm = ins
    T, H, d = r.shape
    dp = pad8(d)
    z = torch.cat([pad_heads(t, dp) for t in (r, k, v, gate, a)], 1).cuda()
    z = torch.nn.functional.pad(z, (0, 24))  # a row pitch beyond the five sections
    dec = pad_heads(decay, dp).cuda()
    ab, nm = pad_heads(a_bias[None], dp)[0].cuda(), pad_heads(norm[None], dp)[0].cuda()
    S = torch.full((1, H, dp, dp), float("nan"), device="cuda") if state is None else state
    pos, out = 0, []
    for n in cuts:
        out.append(pkg.hip.delta_rule(z[pos:pos + n].contiguous(), dec[pos:pos + n].contiguous(), ab, nm, S, 1, n, pos, d, eps, dtype, parallel=parallel))
        pos += n
    return torch.cat(out).float().cpu().view(T, H, dp)[:, :, :d], S[0, :, :d, :d].transpose(1, 2).cpu()  # stored value channel first


@pytest.mark.parametrize("H,d", [(3, 13), (2, 24), (2, 40), (4, 48), (2, 64), (1, 96), (2, 128), (1, 200)])
@pytest.mark.parametrize("kind", ["usual", "strong decay", "repeated keys"])
def test_delta_rule_prompts_portions_and_decoding(pkg, H, d, kind):
    T, eps = 75, 1e-4
    ins = delta_inputs(T, H, d, H * 7 + d, decay_shift=60.0 if kind == "strong decay" else -2.0, repeat=kind == "repeated keys")
    want, S = delta_want(*ins, eps)
    for parallel in (False, True):
        for cuts in ([T], [2, 3, 1, 1, 16, 17, 35], [60] + [1] * 15, [33, 42]):
            got, state = run_delta(pkg, ins, cuts, eps, F32, parallel=parallel)
            assert G.rel(got, want) < 1e-4, (parallel, cuts)
            assert ((state - S).norm() / S.norm()) < 2e-5, (parallel, cuts)
    got, _ = run_delta(pkg, ins, [T], eps, BF16)
    assert ((got - want).abs() <= 2 ** -8 * want.abs() + 1e-3).all()


@DT
@pytest.mark.parametrize("rank", [8, 64, 120])
def test_delta_rule_forms_its_decay_logits(pkg, dtype, rank):
    T, H, d, eps = 21, 3, 40, 1e-4
    r, k, v, gate, a, _, a_bias, norm = delta_inputs(T, H, d, rank)
    g = torch.Generator().manual_seed(rank)
    low, w0 = torch.randn(T, rank, generator=g), torch.randn(H * d, generator=g) - 2
    w2 = (torch.randn(H * d, rank, generator=g) * 2 / rank ** 0.5).to(dtype)
    decay = (torch.tanh(low) @ w2.float().T + w0).view(T, H, d)
    want, _ = delta_want(r, k, v, gate, a, decay, a_bias, norm, eps)
    z = torch.cat([t.reshape(T, -1) for t in (r, k, v, gate, a)] + [low], 1).cuda()
    S = torch.zeros(1, H, d, d, device="cuda")
    pos, out = 0, []
    for n in (1, 8, 1, 5, 2, 4):
        out.append(pkg.hip.delta_rule(z[pos:pos + n].contiguous(), None, a_bias.reshape(-1).cuda(), norm.reshape(-1).cuda(), S, 1, n, pos, d, eps, dtype,
                                      w_decay=w2.cuda(), decay_bias=w0.cuda()))
        pos += n
    assert G.rel(torch.cat(out).float().view(T, H, d), want) < (1e-4 if dtype == F32 else 5e-3)
    with pytest.raises(pkg.hip.RavenHipError):
        pkg.hip.delta_rule(z[:9].contiguous(), None, a_bias.reshape(-1).cuda(), norm.reshape(-1).cuda(), S, 1, 9, 0, d, eps, dtype, w_decay=w2.cuda(),
                           decay_bias=w0.cuda())


def test_delta_rule_long_sequences(pkg):
    """Far more tokens than a chunk: what the first tokens left must survive slow decays."""
    T, H, d, eps = 1500, 1, 64, 1e-5
    ins = delta_inputs(T, H, d, 3, decay_shift=-9.0)
    want, S = delta_want(*ins, eps)
    for cuts in ([T], [1000] + [1] * 20 + [480]):
        got, state = run_delta(pkg, ins, cuts, eps, F32)
        assert G.rel(got, want) < 3e-4 and ((state - S).norm() / S.norm()) < 5e-5


def test_delta_rule_of_several_sequences(pkg):
    B, T, H, d, eps = 3, 50, 2, 24, 1e-5
    ins = [delta_inputs(T, H, d, 100 + b) for b in range(B)]
    ab, nm = ins[0][6], ins[0][7]
    z = torch.cat([torch.cat([pad_heads(t, d) for t in i[:5]], 1) for i in ins]).cuda()
    dec = torch.cat([pad_heads(i[5], d) for i in ins]).cuda()
    S = torch.zeros(B, H, d, d, device="cuda")
    got = pkg.hip.delta_rule(z, dec, ab.reshape(-1).cuda(), nm.reshape(-1).cuda(), S, B, T, 0, d, eps, F32).cpu().view(B, T, H, d)
    for b in range(B):
        want, _ = delta_want(*ins[b][:6], ab, nm, eps)
        assert G.rel(got[b], want) < 1e-4


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
    ids = G.tokens(cfg, 90)
    want, trail = O.forward(cfg, w, ids)
    out = model.forward(ids[None], output_hidden_states=True)
    for run, (got, ref) in enumerate(zip(out.hidden_states[:, 0], trail)):
        assert G.rel(got, ref) < 3e-5, run
    assert G.rel(out.logits[0], want) < 3e-5
    cache, runner = model.new_cache(), None
    for cuts in ([90], [2, 3, 1, 2, 40, 1, 1, 33, 7], [50] + [1] * 40, [1] * 30 + [60]):
        cache.reset()  # the same storage again: nothing of the earlier sequence may show
        got, runner = feed(model, ids, cuts, cache, runner)
        assert G.rel(got, want) < 3e-5, cuts
    for places in ([3, 89], [89, 3, 3], list(range(89, -1, -1)), [7]):
        assert G.rel(model.forward(ids[None], logit_positions=places).logits[0], want[places]) < 3e-5


@pytest.mark.parametrize("name", G.CASES)
def test_model_in_bf16(pkg, name):
    cfg, w, model = G.build(pkg, name, BF16)
    ids = G.tokens(cfg, 90)
    want, _ = O.forward(cfg, w, ids)
    whole = model.forward(ids[None]).logits[0]
    assert G.rel(whole, want) < 6e-2
    for cuts in ([2, 3, 1, 2, 40, 1, 1, 33, 7], [50] + [1] * 40):
        got, _ = feed(model, ids, cuts)
        assert G.rel(got, want) < 6e-2, cuts


def test_long_prompt_runs_in_portions_of_its_own(pkg):
    cfg, w, model = G.build(pkg, "looped middle, grouped heads, a layer without feed-forward", F32)
    ids = G.tokens(cfg, 150)
    want = model.forward(ids[None]).logits
    model.ROWS_PER_CALL = 64
    assert G.rel(model.forward(ids[None]).logits, want) < 1e-5
    assert G.rel(model.forward(ids[None], logit_positions=[63, 64, 149]).logits, want[:, [63, 64, 149]]) < 1e-5


def test_batch_of_equal_lengths_against_each_alone(pkg):
    cfg, w, model = G.build(pkg, "looped middle, grouped heads, a layer without feed-forward", F32)
    ids = torch.stack([G.tokens(cfg, 40, seed=s) for s in range(3)])
    cache = model.new_cache()
    got = [model.forward(ids[:, :23], past_key_values=cache).logits, model.forward(ids[:, 23:30], past_key_values=cache).logits]
    runner = model.decode_runner(cache, 3)
    got += [runner.step(ids[:, t].cuda())[0].clone()[:, None] for t in range(30, 40)]
    got = torch.cat(got, 1)
    for b in range(3):
        assert G.rel(got[b], O.forward(cfg, w, ids[b])[0]) < 3e-5


def test_interleaved_requests_of_unequal_length(pkg):
    """Requests that live at the same time, end, and hand their caches on."""
    from recurrent_pretraining_amd.trace import TraceReplay

    cfg, w, model = G.build(pkg, "sizes that are no multiple of eight", F32)
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
        assert G.rel(torch.cat(got[n]), want[n]) < 3e-5, n
    assert len(trace.caches) == 3


def test_trace_replay_writes_what_was_asked_for(pkg, tmp_path):
    from recurrent_pretraining_amd import trace

    cfg, w, model = G.build(pkg, "no loop, one tap, single head", F32)
    ids = G.tokens(cfg, 12)
    want = O.forward(cfg, w, ids)[0]
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": ids[:9].tolist(), "want": [2, 8]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": ids[9:11].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": ids[11:].tolist(), "want": [0]}], "end": ["x"]}]
    done = io.StringIO()
    trace.replay(model, io.StringIO("\n".join(json.dumps(s) for s in steps)), str(tmp_path), done, max_tokens=12)
    assert done.getvalue().split() == ["done", "0", "done", "1", "done", "2"] and not (tmp_path / "1.f32").exists()
    got = torch.frombuffer(bytearray((tmp_path / "0.f32").read_bytes()), dtype=F32).view(2, -1)
    assert G.rel(got, want[[2, 8]]) < 3e-5
    assert G.rel(torch.frombuffer(bytearray((tmp_path / "2.f32").read_bytes()), dtype=F32).view(1, -1), want[[11]]) < 3e-5


def test_greedy_generation(pkg):
    cfg, w, model = G.build(pkg, "looped middle, grouped heads, a layer without feed-forward", F32)
    prompt = G.tokens(cfg, 17)
    want = O.greedy(cfg, w, prompt.tolist(), 24)
    for graph in (True, False):
        got = model.generate(prompt[None].cuda(), pkg.GenerationSettings(max_new_tokens=24), use_graph=graph)
        assert got[0, 17:].tolist() == want
    assert model.generate(prompt[None].cuda(), max_new_tokens=24, do_sample=False)[0, 17:].tolist() == want  # transformers' own loop
    stop = model.generate(prompt[None].cuda(), pkg.GenerationSettings(max_new_tokens=24, eos_token_id=want[3]))
    assert stop[0, 17:].tolist() == want[:want.index(want[3]) + 1]
    torch.manual_seed(0)
    s = model.generate(prompt[None].cuda(), pkg.GenerationSettings(max_new_tokens=6, do_sample=True, top_k=1))
    assert s[0, 17:].tolist() == want[:6]
    two = torch.stack([prompt, G.tokens(cfg, 17, seed=8)])
    both = model.generate(two.cuda(), pkg.GenerationSettings(max_new_tokens=8))
    assert both[0, 17:].tolist() == want[:8] and both[1, 17:].tolist() == O.greedy(cfg, w, two[1].tolist(), 8)


def test_long_decoding_across_captures(pkg):
    """Past the bound a captured step was sized for, replayed steps against one prompt pass."""
    cfg, w, model = G.build(pkg, "no loop, one tap, single head", F32)
    ids = G.tokens(cfg, 1040)
    want = model.forward(ids[None]).logits[0].cpu()
    cache = model.new_cache()
    model.forward(ids[None, :1000], past_key_values=cache)
    runner = model.decode_runner(cache, 1)
    got = torch.cat([runner.step(ids[t:t + 1].cuda())[0].clone() for t in range(1000, 1040)]).cpu()
    assert G.rel(got, want[1000:]) < 1e-5


def test_invalid_arguments_are_refused(pkg):
    hip = pkg.hip
    keys = torch.zeros(1, 2, 16, 24, device="cuda")
    sc = hip.make_score(1.0, 5.0)
    with pytest.raises(hip.RavenHipError):
        hip.capped_attention(torch.zeros(1, 5 * 24, device="cuda"), keys, sc, 1, 1, 16, 3)   # 3 query heads over 2 key heads
    with pytest.raises(hip.RavenHipError):
        hip.capped_attention(torch.zeros(1, 6 * 24, device="cuda"), keys, sc, 1, 1, 16, 4)   # position 16 of 16
    with pytest.raises(hip.RavenHipError):
        hip.norm_conv(torch.zeros(2, 20, device="cuda"), torch.zeros(20, device="cuda"), 20, 1e-5, 1, 2, F32)  # pitch not a multiple of 8
    with pytest.raises(hip.RavenHipError):
        hip.linear_epilogue(torch.zeros(1, 12, device="cuda"), torch.zeros(8, 16, device="cuda"))
