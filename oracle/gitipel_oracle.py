"""CPU restatement of the Gitipel decoder, for the tests only (nothing of the product path imports it, and it imports
nothing of the product path).  One plain function per mechanism, token by token where the mechanism is a
recurrence, in the dtype of its inputs (float32 or float64).  Sequences are processed whole, from position 0.

`cfg` is the dictionary of a config.json; `w` maps tensor names to floating-point tensors.
"""

import math

import torch


def rms(x, eps):
    """x divided by its root mean square over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


def causal_conv(h, weight):
    """Depthwise convolution over time of h [T, C] with weight [C, taps]; the last tap sees the current token, tokens before
    the first are zero."""
    taps = weight.shape[1]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                out[t] += weight[:, j] * h[src]
    return out


def softcap(s, cap):
    return cap * torch.tanh(s / cap)


def distance_bias(r1, r2, i, j):
    """What a head takes off the score of query position i and key position j <= i."""
    return r1 * math.log1p(float(r2) * (i - j))


def attention(q, k, scale, cap, r1, r2):
    """q [T, H, d], k [T, G, d]; the keys are the values too.  Returns [T, H, d]."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = torch.zeros_like(q)
    dist = torch.arange(T, dtype=q.dtype)
    for h in range(H):
        kh = k[:, h // group]
        for i in range(T):
            s = softcap((kh[:i + 1] @ q[i, h]) * scale, cap)
            s = s - r1[h] * torch.log1p(r2[h] * (i - dist[:i + 1]))
            out[i, h] = torch.softmax(s, 0) @ kh[:i + 1]
    return out


def attention_mixer(h, w, p, m):
    T = h.shape[0]
    q = (h @ w[p + "q"].T).view(T, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T).view(T, m["kv_heads"], m["dim"])
    o = attention(q, k, m["scale"], m["softcap"], w[p + "r1"], w[p + "r2"])
    return o.reshape(T, -1) @ w[p + "o"].T


def delta_decay(h, w1, w2, w0):
    """Per-channel decay of the state in (exp(-exp(-1/2)), 1)."""
    z = torch.tanh(h @ w1.T) @ w2.T + w0
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(z))


def delta_rule(r, k, v, decay, a, state=None):
    """All [T, H, d].  Row index of the state [H, d, d]: key channel; column index: value channel."""
    T, H, d = r.shape
    S = torch.zeros(H, d, d, dtype=r.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            u = k[t, h] / torch.sqrt((k[t, h] ** 2).sum() + 1e-6)
            old = S[h]
            S[h] = decay[t, h][:, None] * old - torch.outer(a[t, h] * u, u @ old) + torch.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ r[t, h]
    return out, S


def delta_output(o, h, norm, wg, wo, eps):
    """Heads to unit root mean square, weight, gate, projection; o [T, H, d]."""
    T = o.shape[0]
    y = rms(o, eps).reshape(T, -1) * norm
    return (y * torch.sigmoid(h @ wg.T)) @ wo.T


def delta_mixer(h, w, p, m, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    heads = lambda x: x.view(T, H, d)
    r, k, v = (heads(h @ w[p + n].T) for n in "rkv")
    decay = heads(delta_decay(h, w[p + "w1"], w[p + "w2"], w[p + "w0"]))
    a = heads(torch.sigmoid(h @ w[p + "a"].T + w[p + "a.b"]))
    o, _ = delta_rule(r, k, v, decay, a)
    return delta_output(o, h, w[p + "norm"], w[p + "g"], w[p + "o"], eps)


def gelu_erf(x):
    return 0.5 * x * (1 + torch.erf(x / math.sqrt(2.0)))


def mlp(h, up, down):
    return gelu_erf(h @ up.T) @ down.T


def layer(x, w, i, spec, eps):
    p = f"l{i}."
    h = rms_norm(x, w[p + "norm1"], eps)
    h = h + causal_conv(h, w[p + "canon1"])
    mix = {"attention": lambda: attention_mixer(h, w, p + "mix.", spec["mixer"]),
           "general_delta": lambda: delta_mixer(h, w, p + "mix.", spec["mixer"], eps)}[spec["type"]]
    x = x + mix()
    if spec.get("mlp") is not None:
        x = x + mlp(rms_norm(x, w[p + "norm2"], eps), w[p + "mlp.up"], w[p + "mlp.down"])
    return x


def layer_runs(cfg):
    """(layer, pass) in the order they run; pass is None outside the loop."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    inside = [(i, t) for t in range(loop["times"]) for i in range(loop["start"], loop["stop"])]
    return [(i, None) for i in range(loop["start"])] + inside + [(i, None) for i in range(loop["stop"], n)]


def enter_pass(x, x0, w, t):
    return torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][t]


def forward(cfg, w, tokens):
    """Logits [T, vocab] and the residual after every layer run [runs, T, width] of one sequence."""
    eps = cfg["norm"]["eps"]
    x0 = w["embed"][tokens] * cfg["embedding"]["scale"]
    x, trail = x0, []
    for i, t in layer_runs(cfg):
        if t is not None and i == cfg["loop"]["start"]:
            x = enter_pass(x, x0, w, t)
        x = layer(x, w, i, cfg["layers"][i], eps)
        trail.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]
    return logits, torch.stack(trail)


def greedy(cfg, w, prompt, n_new):
    """prompt: list of ids; returns the n_new ids picked one by one, each from a forward over everything before it."""
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(forward(cfg, w, torch.tensor(ids))[0][-1].argmax()))
    return ids[len(prompt):]


def random_weights(cfg, rank, seed, dtype=torch.float32, round_bf16=True):
    """Weights of every tensor a configuration needs, scaled so that activations stay of order one; with round_bf16 the
    values are representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    D, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    w = {}

    def normal(name, *shape, std=None, mean=0.0):
        std = (1.0 / math.sqrt(shape[-1])) if std is None else std
        t = torch.randn(*shape, generator=g) * std + mean
        w[name] = (t.bfloat16().float() if round_bf16 else t).to(dtype)

    normal("embed", V, D, std=1.0 / cfg["embedding"]["scale"])
    if cfg.get("loop"):
        normal("loop.in", D, 2 * D)
        normal("loop.step", cfg["loop"]["times"], D, std=0.3)
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        normal(p + "norm1", D, std=0.1, mean=1.0)
        normal(p + "canon1", D, taps, std=0.4)
        mp = p + "mix."
        if spec["type"] == "attention":
            normal(mp + "q", m["heads"] * m["dim"], D)
            normal(mp + "k", m["kv_heads"] * m["dim"], D)
            normal(mp + "r1", m["heads"], std=0.2, mean=0.6)
            w[mp + "r2"] = (0.05 + 0.5 * torch.rand(m["heads"], generator=g)).bfloat16().to(dtype)
            normal(mp + "o", D, m["heads"] * m["vdim"])
        else:
            n = m["heads"] * m["dim"]
            for t in "rkvga":
                normal(mp + t, n, D)
            normal(mp + "a.b", n, std=0.5)
            normal(mp + "w1", rank, D)
            normal(mp + "w2", n, rank)
            normal(mp + "w0", n, std=1.5, mean=-2.0)
            normal(mp + "norm", n, std=0.1, mean=1.0)
            normal(mp + "o", D, n)
        if spec.get("mlp") is not None:
            normal(p + "norm2", D, std=0.1, mean=1.0)
            normal(p + "mlp.up", spec["mlp"]["ff"], D)
            normal(p + "mlp.down", D, spec["mlp"]["ff"])
    normal("final.norm", D, std=0.1, mean=1.0)
    normal("head", V, D)
    return w
