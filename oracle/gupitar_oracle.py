"""CPU restatement of the Gupitar decoder, for the tests only (nothing of the product path imports it, and it imports
nothing of the product path).  One plain function per mechanism, token by token where the mechanism is a recurrence, in the
dtype of its inputs (float32 or float64).  Sequences are processed whole, from position 0.

`cfg` is the dictionary of a config.json; `w` maps tensor names to floating-point tensors.
"""

import math

import torch


# ---- norms and activations ---------------------------------------------------------------------------
def rms(x, eps):
    """x divided by its root mean square over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def plain_norm(x, weight, eps):
    return rms(x, eps) * weight


def centred_norm(x, weight, eps):
    """A norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1 + weight)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- latent attention ----------------------------------------------------------------------------------
def rotate(x, positions, base, dims):
    """x [T, ..., n]: the first `dims` entries of the last dimension, entry i turned together with entry i + dims / 2."""
    half = dims // 2
    freq = base ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims)
    angle = (positions.double()[:, None] * freq).to(x.dtype)
    angle = angle.view(len(positions), *([1] * (x.dim() - 2)), half)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(angle) - v * torch.sin(angle), v * torch.cos(angle) + u * torch.sin(angle), x[..., dims:]], -1)


def visible(i, j, window):
    return 0 <= i - j < window


def windowed_attention(q, k, v, scale, window):
    """q, k [T, H, n], v [T, H, m]; every query one by one.  Returns [T, H, m]."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        seen = [j for j in range(T) if visible(i, j, window)] if T <= 64 else list(range(max(0, i - window + 1), i + 1))
        for h in range(H):
            s = (k[seen, h] @ q[i, h]) * scale
            out[i, h] = torch.softmax(s, 0) @ v[seen, h]
    return out


def latent_queries(h, w, p, m, eps):
    c = plain_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (c @ w[p + "uq"].T).view(h.shape[0], m["heads"], m["dim"] + m["rot_dim"])
    q_rot = rotate(q[..., m["dim"]:], torch.arange(h.shape[0]), m["rot"]["base"], m["rot"]["dims"])
    return torch.cat([q[..., :m["dim"]], q_rot], -1)


def latent_keys(h, w, p, m, eps):
    """What a layer with a down projection leaves for itself and for the layers that read from it: the normed latent [T, kv_rank] and
    the rotated part [T, rot_dim]."""
    z = h @ w[p + "dkv"].T
    c = plain_norm(z[:, :m["kv_rank"]], w[p + "dkv.norm"], eps)
    return c, rotate(z[:, m["kv_rank"]:], torch.arange(h.shape[0]), m["rot"]["base"], m["rot"]["dims"])


def latent_attention_mixer(h, w, p, m, eps, kept):
    """kept: (latent, rotated part) of the layer the keys come from."""
    T, H = h.shape[0], m["heads"]
    c, k_rot = kept
    q = latent_queries(h, w, p, m, eps)
    k = torch.cat([(c @ w[p + "uk"].T).view(T, H, m["dim"]), k_rot[:, None].expand(T, H, m["rot_dim"])], -1)
    v = (c @ w[p + "uv"].T).view(T, H, m["vdim"])
    window = m["mask"]["size"] if m.get("mask") else T
    o = windowed_attention(q, k, v, m["scale"], window).reshape(T, -1)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- real-gated linear recurrent unit ------------------------------------------------------------------
def causal_conv(u, weight, bias):
    """Depthwise convolution over time of u [T, C] with weight [C, taps]; the last tap sees the current token, tokens before the
    first are zero."""
    taps = weight.shape[1]
    out = bias.expand(u.shape).clone()
    for t in range(u.shape[0]):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                out[t] = out[t] + weight[:, j] * u[src]
    return out


def block_gate(u, matrices, bias):
    """sigmoid of a product with a block-diagonal matrix [blocks, out, in]; bias [blocks, out] or flat."""
    n, size, _ = matrices.shape
    parts = u.view(u.shape[0], n, size)
    z = torch.stack([parts[:, b] @ matrices[b].T for b in range(n)], 1).reshape(u.shape)
    return torch.sigmoid(z + bias.reshape(-1))


def decay_logarithm(r, lam):
    return -8.0 * r * torch.nn.functional.softplus(lam)


def gated_recurrence(u, r, i, lam, state=None):
    """S <- a S + sqrt(1 - a^2) i u, token by token; returns every S and the last one."""
    log_a = decay_logarithm(r, lam)
    a = torch.exp(log_a)
    gain = torch.sqrt(-torch.expm1(2 * log_a))
    S = torch.zeros(u.shape[1], dtype=u.dtype) if state is None else state.clone()
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + gain[t] * i[t] * u[t]
        out[t] = S
    return out, S


def rglru_mixer(h, w, p):
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"])
    r = block_gate(u, w[p + "ra"], w[p + "ra.b"])
    i = block_gate(u, w[p + "ri"], w[p + "ri.b"])
    S, _ = gated_recurrence(u, r, i, w[p + "lam"])
    return (S * y) @ w[p + "o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------
def gated_mlp(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, router, top):
    """(expert indices, weights) [T, top]: the largest sigmoid scores, as they are."""
    s = torch.sigmoid(h @ router.T)
    weight, index = torch.topk(s, top, dim=-1)
    return index, weight


def mixture(h, w, p, mlp):
    index, weight = route(h, w[p + "router"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(index[t].tolist(), weight[t]):
            out[t] += gated_mlp((s * h[t])[None], w, f"{p}e{e}.")[0]
    if mlp.get("shared") is not None:
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * gated_mlp(h, w, p + "shared.")
    return out


def feed_forward(h, w, p, mlp):
    return gated_mlp(h, w, p) if mlp["kind"] == "dense" else mixture(h, w, p, mlp)


# ---- the model ------------------------------------------------------------------------------------------
def forward(cfg, w, tokens):
    """Logits [T, vocab] and the residual after every layer [layers, T, width] of one sequence."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][tokens]
    trail, kept = [], {}
    for n, spec in enumerate(cfg["layers"]):
        p, m = f"l{n}.", spec["mixer"]
        h = centred_norm(x, w[p + "norm1"], eps)
        if spec["type"] == "latent_attention":
            source = m.get("kv_from")
            if source is None:
                kept[n] = latent_keys(h, w, p + "mix.", m, eps)
            x = x + latent_attention_mixer(h, w, p + "mix.", m, eps, kept[n if source is None else source])
        else:
            x = x + rglru_mixer(h, w, p + "mix.")
        if spec.get("mlp") is not None:
            x = x + feed_forward(centred_norm(x, w[p + "norm2"], eps), w, p + "mlp.", spec["mlp"])
        trail.append(x)
    return centred_norm(x, w["final.norm"], eps) @ w["head"].T, torch.stack(trail)


def greedy(cfg, w, prompt, n_new):
    """prompt: list of ids; returns the n_new ids picked one by one, each from a forward over everything before it."""
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(forward(cfg, w, torch.tensor(ids))[0][-1].argmax()))
    return ids[len(prompt):]


def random_weights(cfg, seed, dtype=torch.float32, round_bf16=True):
    """Weights of every tensor a configuration needs, scaled so that activations stay of order one; with round_bf16 the
    values are representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]
    w = {}

    def normal(name, *shape, std=None, mean=0.0):
        std = (1.0 / math.sqrt(shape[-1])) if std is None else std
        t = torch.randn(*shape, generator=g) * std + mean
        w[name] = (t.bfloat16().float() if round_bf16 else t).to(dtype)

    def gated(p, ff):
        normal(p + "gate", ff, D)
        normal(p + "up", ff, D)
        normal(p + "down", D, ff)

    normal("embed", V, D, std=1.0)
    for n, spec in enumerate(cfg["layers"]):
        p, m, mp = f"l{n}.", spec["mixer"], f"l{n}.mix."
        normal(p + "norm1", D, std=0.2)
        if spec["type"] == "latent_attention":
            H = m["heads"]
            normal(mp + "dq", m["q_rank"], D)
            normal(mp + "dq.norm", m["q_rank"], std=0.2, mean=1.0)
            normal(mp + "uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"], std=1.5 / math.sqrt(m["q_rank"]))
            if m.get("kv_from") is None:
                normal(mp + "dkv", m["kv_rank"] + m["rot_dim"], D)
                normal(mp + "dkv.norm", m["kv_rank"], std=0.2, mean=1.0)
            normal(mp + "uk", H * m["dim"], m["kv_rank"])
            normal(mp + "uv", H * m["vdim"], m["kv_rank"])
            normal(mp + "g", H * m["vdim"], D)
            normal(mp + "o", D, H * m["vdim"], std=2.0 / math.sqrt(H * m["vdim"]))
        else:
            W, n_blocks = m["width"], m["blocks"]
            size = W // n_blocks
            for t in "yx":
                normal(mp + t, W, D)
                normal(mp + t + ".b", W, std=0.3)
            normal(mp + "conv", W, m["conv"], std=0.6)
            normal(mp + "conv.b", W, std=0.3)
            for t in ("ra", "ri"):
                normal(mp + t, n_blocks, size, size)
                normal(mp + t + ".b", n_blocks, size, std=0.5)
            normal(mp + "lam", W, std=2.0, mean=-4.0)  # decays from almost none to strong
            normal(mp + "o", D, W, std=2.0 / math.sqrt(W))
        mlp = spec.get("mlp")
        if mlp is None:
            continue
        normal(p + "norm2", D, std=0.2)
        if mlp["kind"] == "dense":
            gated(p + "mlp.", mlp["ff"])
            continue
        normal(p + "mlp.router", mlp["router"]["experts"], D, std=1.5 / math.sqrt(D))
        for e in range(mlp["router"]["experts"]):
            gated(f"{p}mlp.e{e}.", mlp["expert"]["ff"])
        if mlp.get("shared") is not None:
            gated(p + "mlp.shared.", mlp["shared"]["ff"])
            normal(p + "mlp.shared.sg", 1, D)
    normal("final.norm", D, std=0.2)
    normal("head", V, D)
    return w
