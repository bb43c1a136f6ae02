"""A slow float64 implementation of Minerax written from its equations, one function per
mechanism.  It shares no code with the package: the configuration comes as the dictionary of a
checkpoint's config.json, tensors by their checkpoint names, and whole sequences are computed at
once with dense masks and token-by-token recurrences."""
import math

import torch

D64 = torch.float64


# ------------------------------------------------------------------ norms and units
def over_rms(x, eps):
    """x over its root mean square (last axis)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    """Centred and divided by the deviation (last axis), times w; no bias."""
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def unit_vectors(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def feed_forward(h, gate, up, down):
    return (gelu_tanh(h @ gate.T) * (h @ up.T)) @ down.T


# ------------------------------------------------------------------ residual streams
def streams_in(streams, w_in):
    """streams [S, T, d] -> the sublayer's input row: their weighted sum."""
    return sum(float(w_in[s]) * streams[s] for s in range(len(w_in)))


def streams_update(streams, mix, w_out, y):
    """Every new stream t is a mixture of the previous streams plus its share of y; row s of mix holds
    what stream s gives."""
    S = streams.shape[0]
    return torch.stack([sum(float(mix[s, t]) * streams[s] for s in range(S)) + float(w_out[t]) * y
                        for t in range(S)])


# ------------------------------------------------------------------ rotation
def frequencies(rot):
    """(f_i, factor of cos and sin) of a mixer's ``rot`` entry, with YaRN scaling if it has one."""
    dims, base = rot["dims"], rot["base"]
    i = torch.arange(dims // 2, dtype=D64)
    f = base ** (-2.0 * i / max(dims, 1))
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def dim_of(t):
        return dims * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), dims - 1)
    ramp = torch.clamp((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, pos, freq, mult, neighbours):
    """x [T, heads, n]: the leading 2 len(freq) entries turn in pairs (2i, 2i + 1)
    (``neighbours``) or (i, i + len(freq))."""
    n = freq.numel()
    y = x.clone()
    for i in range(n):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + n)
        ang = pos.to(D64) * freq[i]
        c, s = (torch.cos(ang) * mult)[:, None], (torch.sin(ang) * mult)[:, None]
        y[..., a] = x[..., a] * c - x[..., b] * s
        y[..., b] = x[..., b] * c + x[..., a] * s
    return y


# ------------------------------------------------------------------ attention
def visible(T, window=0):
    """[i, j]: j <= i, and i - j < window (0: no window)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & (d < window) if window > 0 else d >= 0


def cap(scores, c):
    return c * torch.tanh(scores / c) if c else scores


def weights(scores, ok, sink=None):
    """Softmax over the visible keys; exp(sink) joins the denominator."""
    s = scores.masked_fill(~ok, -math.inf)
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.clamp(top, min=float(sink))
    e = torch.exp(s - top)
    den = e.sum(-1, keepdim=True)
    return e / (den if sink is None else den + torch.exp(float(sink) - top))


# ------------------------------------------------------------------ short convolution
def causal_conv(u, w, before=None):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j); ``before`` [taps - 1, C]:
    the inputs ahead of u (zeros at a sequence's start)."""
    T, C = u.shape
    taps = w.shape[1]
    lead = torch.zeros(taps - 1, C, dtype=D64) if before is None else before
    full = torch.cat([lead, u], 0)
    y = torch.zeros(T, C, dtype=D64)
    for t in range(T):
        for j in range(taps):
            y[t] += w[:, j] * full[t + j]
    return y


# ------------------------------------------------------------------ gated delta rule
def channel_decay(z, a_log):
    """z [T, H, dim] (bias added), a_log [H] -> exp(-exp(a_log) softplus(z))."""
    return torch.exp(-torch.exp(a_log)[None, :, None] * softplus(z))


def delta_scan(q, k, v, g, beta, S=None):
    """One head: q, k, g [T, dim], v [T, vdim], beta [T].  Returns (o [T, vdim], S)."""
    T = q.shape[0]
    S = torch.zeros(q.shape[1], v.shape[1], dtype=D64) if S is None else S.clone()
    o = torch.zeros(T, v.shape[1], dtype=D64)
    for t in range(T):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + k[t][:, None] * u[None, :]
        o[t] = S.T @ q[t]
    return o, S


# ------------------------------------------------------------------ mixers
def left_attention(m, w, p, h, eps):
    T = h.shape[0]
    H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q, k, v = (causal_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    q = (over_rms(q, eps) * w[p + "q.norm"]).view(T, H, dim)
    k = (over_rms(k, eps) * w[p + "k.norm"]).view(T, G, dim)
    v = v.view(T, G, vd)
    f, mult = frequencies(m["rot"])
    q, k = rotate(q, pos, f, mult, False), rotate(k, pos, f, mult, False)
    ok = visible(T)
    out = torch.zeros(T, H, vd, dtype=D64)
    for a in range(H):
        b = a // (H // G)
        out[:, a] = weights(cap((q[:, a] @ k[:, b].T) * m["scale"], m.get("softcap")), ok) @ v[:, b]
    return out.reshape(T, H * vd) @ w[p + "o"].T


def right_delta(m, w, p, h, eps):
    T = h.shape[0]
    H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = unit_vectors(q.view(T, G, dim)) * dim ** -0.5
    k = unit_vectors(k.view(T, G, dim))
    v = v.view(T, H, vd)
    beta = sigmoid(h @ w[p + "b"].T)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = channel_decay(z.view(T, H, dim), w[p + "A_log"])
    o = torch.zeros(T, H, vd, dtype=D64)
    for a in range(H):
        b = a // (H // G)
        o[:, a], _ = delta_scan(q[:, b], k[:, b], v[:, a], g[:, a], beta[:, a])
    o = (over_rms(o, eps) * w[p + "norm"]).reshape(T, H * vd)
    return (o * sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)) @ w[p + "o"].T


def parallel(m, w, p, h, eps):
    return m["left_scale"] * left_attention(m["left"], w, p + "left.", h, eps) \
        + m["right_scale"] * right_delta(m["right"], w, p + "right.", h, eps)


def latent_attention(m, w, p, h, eps):
    T = h.shape[0]
    H, dim, rd, vd, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    f, mult = frequencies(m["rot"])
    q = (h @ w[p + "q"].T).view(T, H, dim + rd)
    kv = h @ w[p + "dkv"].T
    c = over_rms(kv[:, :R], eps) * w[p + "dkv.norm"]
    kr = rotate(kv[:, None, R:], pos, f, mult, True)[:, 0]
    k = (c @ w[p + "uk"].T).view(T, H, dim)
    v = (c @ w[p + "uv"].T).view(T, H, vd)
    qr = rotate(q[..., dim:], pos, f, mult, True)
    ok = visible(T, (m.get("mask") or {}).get("size", 0))
    out = torch.zeros(T, H, vd, dtype=D64)
    for a in range(H):
        s = (q[:, a, :dim] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        out[:, a] = weights(s, ok, w[p + "sink"][a]) @ v[:, a]
    return (out.reshape(T, H * vd) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------ whole model
def forward(cfg, tensors, tokens, layers=None):
    """Logits [T, vocab] of one sequence; ``layers`` (a list) receives the sum of the residual
    streams after every layer."""
    w = {k: v.to(D64) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    e = w["embed"][torch.as_tensor(tokens)]
    x = torch.stack([e] * cfg["streams"])
    for i, ly in enumerate(cfg["layers"]):
        L = f"l{i}."
        mix = {"parallel": parallel, "latent_attention": latent_attention}[ly["type"]]
        u = layer_norm(streams_in(x, w[L + "hc1.in"]), w[L + "norm1"], eps)
        x = streams_update(x, w[L + "hc1.mix"], w[L + "hc1.out"], mix(ly["mixer"], w, L + "mix.", u, eps))
        if ly["mlp"] is not None:
            u = layer_norm(streams_in(x, w[L + "hc2.in"]), w[L + "norm2"], eps)
            y = feed_forward(u, w[L + "mlp.gate"], w[L + "mlp.up"], w[L + "mlp.down"])
            x = streams_update(x, w[L + "hc2.mix"], w[L + "hc2.out"], y)
        if layers is not None:
            layers.append(x.sum(0))
    return layer_norm(x.sum(0), w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]


def greedy(cfg, tensors, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, tensors, toks)[-1].argmax()))
    return toks[len(prompt):]
