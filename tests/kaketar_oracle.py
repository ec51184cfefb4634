"""A plain, slow Kaketar in float64, one function per mechanism.

Written from the design's equations only; shares no code with
gllm_amd. ``forward`` runs one whole sequence from position 0 and
returns the logits of every position (and, on request, the residual
stream after every layer).

cfg: the parsed config.json (a dict); W: name -> float64 tensor.
"""

import math

import torch

F64 = torch.float64


def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_norm(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return over_rms(x, eps) * (1.0 + w)


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp_min(0.0)


def embed(tokens, cfg, W):
    ids = torch.as_tensor(tokens)
    x = W["embed"][ids] * float(cfg["embedding"]["scale"]) \
        + W["pos"][:len(ids)]
    return centred_norm(x, W["embed.norm"], float(cfg["norm"]["eps"]))


# ---------------------------------------------------------------- delta rule
def conv_silu(u, w):
    """u [T, C] over time with w [C, taps]; the last tap sits on the
    current token, zeros ahead of the first; then silu."""
    T, C = u.shape
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y * torch.sigmoid(y)


def channel_decay(h, W, pre, heads):
    """[T, heads, dim]: exp(-exp(A) softplus(W_a2 W_a1 h + dt))."""
    z = (h @ W[pre + "a1"].T) @ W[pre + "a2"].T + W[pre + "dt_bias"]
    rate = torch.exp(W[pre + "A_log"])
    return torch.exp(-rate[:, None] * softplus(z).view(len(h), heads, -1))


def delta_recurrence(q, k, v, g, beta):
    """q, k [T, G, D]; v [T, H, Dv]; g [T, H, D]; beta [T, H]. One state
    [D, Dv] per head, from zero: decay the rows, write the correction,
    read."""
    T, H, Dv = v.shape
    G, D = q.shape[1:]
    out = torch.zeros(T, H, Dv, dtype=F64)
    for h in range(H):
        kv = h // (H // G)
        S = torch.zeros(D, Dv, dtype=F64)
        for t in range(T):
            S = g[t, h][:, None] * S
            u = beta[t, h] * (v[t, h] - k[t, kv] @ S)
            S = S + torch.outer(k[t, kv], u)
            out[t, h] = q[t, kv] @ S
    return out


def channel_delta(h, m, W, pre, eps):
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = len(h)

    def branch(name, heads, size):
        return conv_silu(h @ W[pre + name].T,
                         W[pre + name + ".conv"]).view(T, heads, size)

    def unit(x):
        return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)

    q = unit(branch("q", G, D)) * D ** -0.5
    k = unit(branch("k", G, D))
    v = branch("v", H, Dv)
    beta = torch.sigmoid(h @ W[pre + "b"].T)
    o = delta_recurrence(q, k, v, channel_decay(h, W, pre, H), beta)
    o = over_rms(o, eps) * W[pre + "norm"]
    gate = torch.sigmoid((h @ W[pre + "g1"].T) @ W[pre + "g2"].T)
    return (o.reshape(T, H * Dv) * gate) @ W[pre + "o"].T


# ---------------------------------------------------------------- attention
def yarn(rot):
    """(frequencies [dims/2], magnitude of cos and sin)."""
    dims, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F64), 1.0

    def turning_dim(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(turning_dim(sc["fast"])), 0)
    hi = min(math.ceil(turning_dim(sc["slow"])), dims - 1)
    for i in range(dims // 2):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        f[i] = f[i] / sc["factor"] * r + f[i] * (1.0 - r)
    return torch.tensor(f, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, rot):
    """x [T, ..., dims]: dims 2i and 2i+1 turn by position * f_i."""
    f, mag = yarn(rot)
    ang = torch.arange(len(x), dtype=F64)[:, None] * f
    c, s = mag * ang.cos(), mag * ang.sin()
    while c.dim() < x.dim():
        c, s = c.unsqueeze(1), s.unsqueeze(1)
    u, v = x[..., 0::2], x[..., 1::2]
    out = torch.empty_like(x)
    out[..., 0::2] = u * c - v * s
    out[..., 1::2] = v * c + u * s
    return out


def sink_softmax(s, sink):
    """Softmax weights with exp(sink) joining the denominator."""
    top = max(float(s.max()), float(sink))
    e = torch.exp(s - top)
    return e / (e.sum() + math.exp(float(sink) - top))


def window_sink_attention(q, k, v, scale, window, sink):
    """q, k [T, H, D], v [T, H, Dv]; i sees j with 0 <= i - j < window
    (window None: every j <= i)."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        for i in range(T):
            lo = 0 if not window else max(0, i - window + 1)
            s = (k[lo:i + 1, h] @ q[i, h]) * scale
            out[i, h] = sink_softmax(s, sink[h]) @ v[lo:i + 1, h]
    return out


def latent_attention(h, m, W, pre, eps):
    H, D, Dr, Dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    R, T = m["kv_rank"], len(h)
    cq = over_rms(h @ W[pre + "dq"].T, eps) * W[pre + "dq.norm"]
    q = (cq @ W[pre + "uq"].T).view(T, H, D + Dr)
    kv = h @ W[pre + "dkv"].T
    c = over_rms(kv[:, :R], eps) * W[pre + "dkv.norm"]
    k_rot = rotate_pairs(kv[:, R:], m["rot"])
    k = torch.cat([(c @ W[pre + "uk"].T).view(T, H, D),
                   k_rot[:, None].expand(T, H, Dr)], -1)
    v = (c @ W[pre + "uv"].T).view(T, H, Dv)
    q = torch.cat([q[..., :D], rotate_pairs(q[..., D:], m["rot"])], -1)
    window = (m.get("mask") or {}).get("size")
    o = window_sink_attention(q, k, v, float(m["scale"]), window,
                              W[pre + "sink"])
    gate = torch.sigmoid(h @ W[pre + "g"].T)
    return (o.reshape(T, H * Dv) * gate) @ W[pre + "o"].T


# ---------------------------------------------------------------- the rest
def feed_forward(h, W, pre):
    return gelu_erf(h @ W[pre + "up"].T) @ W[pre + "down"].T


def token_side(x, tokens, i, cfg, W):
    """What the layer adds per token: gated by its own slice of the
    side table."""
    n = cfg["token_side"]["dim"]
    p = f"l{i}.side."
    e = W["side.embed"][torch.as_tensor(tokens)][:, i * n:(i + 1) * n]
    y = (gelu_tanh(x @ W[p + "gate"].T) * e) @ W[p + "proj"].T
    return over_rms(y, float(cfg["norm"]["eps"])) * W[p + "norm"]


MIXERS = {"latent_attention": latent_attention,
          "channel_delta": channel_delta}


def layer(x, tokens, i, cfg, W):
    lay, eps, p = cfg["layers"][i], float(cfg["norm"]["eps"]), f"l{i}."
    y = MIXERS[lay["type"]](x, lay["mixer"], W, p + "mix.", eps)
    x = x + centred_norm(y, W[p + "norm1"], eps)
    if lay.get("mlp"):
        y = feed_forward(x, W, p + "mlp.")
        x = x + centred_norm(y, W[p + "norm2"], eps)
    return x + token_side(x, tokens, i, cfg, W)


def forward(cfg, W, tokens, probe=None):
    x = embed(tokens, cfg, W)
    for i in range(len(cfg["layers"])):
        x = layer(x, tokens, i, cfg, W)
        if probe is not None:
            probe.append(x.clone())
    x = centred_norm(x, W["final.norm"], float(cfg["norm"]["eps"]))
    logits = x @ W["head"].T
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
