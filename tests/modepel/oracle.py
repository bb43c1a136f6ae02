"""A slow float64 implementation of Modepel written from its equations, one function per
mechanism.  It shares no code with the package: the configuration comes as the dictionary of a
checkpoint's config.json, tensors by their checkpoint names, and whole sequences are computed at
once with dense masks and token-by-token recurrences."""
import math

import torch

D64 = torch.float64


# ------------------------------------------------------------------ norms and units
def rms_unit(x, eps):
    """x over its root mean square (last axis)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gain_norm(x, g, eps):
    """RMS norm with one number for all coordinates."""
    return rms_unit(x, eps) * g


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def logsigmoid(x):
    return -(torch.clamp(-x, min=0.0) + torch.log1p(torch.exp(-x.abs())))


def poly_norm(z, coef, eps):
    """a N(z) + b N(z^2) + c N(z^3) + e with powers per element and N(u) = u / rms(u) over the
    last axis; coef = (a, b, c, e)."""
    a, b, c, e = (float(x) for x in coef)
    return a * rms_unit(z, eps) + b * rms_unit(z * z, eps) + c * rms_unit(z * z * z, eps) + e


def swiglu_expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


# ------------------------------------------------------------------ rotation
def rotate_half(x, positions, dims, base):
    """x [T, heads, n]: entry i turns with entry i + dims/2 by position * base^(-2i/dims)."""
    half = dims // 2
    if half == 0:
        return x
    f = base ** (-2.0 * torch.arange(half, dtype=D64) / dims)
    ang = positions.to(D64)[:, None] * f[None]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    y = x.clone()
    u, v = x[..., :half], x[..., half:2 * half]
    y[..., :half] = u * c - v * s
    y[..., half:2 * half] = v * c + u * s
    return y


# ------------------------------------------------------------------ attention
def softmax_plus_one(scores, ok):
    """exp(s_j) / (1 + sum_j exp(s_j)) over the visible keys."""
    s = scores.masked_fill(~ok, -math.inf)
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def mixed_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def attention(m, w, pre, h, pos, v_first=None):
    """Returns (output [T, d], this layer's values as projected [T, G, vdim])."""
    T = h.shape[0]
    H, G, dim, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T + w[pre + "q.b"]).view(T, H, dim)
    k = (h @ w[pre + "k"].T + w[pre + "k.b"]).view(T, G, dim)
    v0 = (h @ w[pre + "v"].T + w[pre + "v.b"]).view(T, G, vd)
    v = v0 if v_first is None else mixed_values(v0, v_first, float(w[pre + "vmix"]))
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    q = rotate_half(q, pos, rot["dims"], rot["base"])
    k = rotate_half(k, pos, rot["dims"], rot["base"])
    ok = pos[None, :] <= pos[:, None]
    out = torch.zeros(T, H, vd, dtype=D64)
    for hh in range(H):
        g = hh // (H // G)
        out[:, hh] = softmax_plus_one((q[:, hh] @ k[:, g].T) * m["scale"], ok) @ v[:, g]
    out = out.reshape(T, H * vd) * sigmoid(h @ w[pre + "g"].T)
    return out @ w[pre + "o"].T, v0


# ------------------------------------------------------------------ matrix memory
def memory_gates(zi, zf, cap):
    """Capped log gates of raw logits: (log input gate, log forget gate)."""
    return cap * torch.tanh(zi / cap), logsigmoid(cap * torch.tanh(zf / cap))


def matrix_memory(q, k, v, li, lf, state=None):
    """One head, token by token.  q, k [T, dim], v [T, vdim], log gates li, lf [T]; q already
    scaled.  state = (S [dim, vdim], n [dim], m) to start from.  Returns (o [T, vdim], state)."""
    T, dim = q.shape
    if state is None:
        S, n, m = torch.zeros(dim, v.shape[1], dtype=D64), torch.zeros(dim, dtype=D64), 0.0
    else:
        S, n, m = state
    out = torch.zeros(T, v.shape[1], dtype=D64)
    for t in range(T):
        mn = max(float(lf[t]) + m, float(li[t]))
        keep, add = math.exp(float(lf[t]) + m - mn), math.exp(float(li[t]) - mn)
        S = keep * S + add * k[t][:, None] * v[t][None, :]
        n = keep * n + add * k[t]
        m = mn
        den = max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6
        out[t] = (S.T @ q[t]) / den
    return out, (S, n, m)


def mlstm(m, w, pre, h, eps):
    T = h.shape[0]
    H, dim, vd = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T).view(T, H, dim) * dim ** -0.5
    k = (h @ w[pre + "k"].T).view(T, H, dim)
    v = (h @ w[pre + "v"].T).view(T, H, vd)
    li, lf = memory_gates(h @ w[pre + "i"].T + w[pre + "i.b"], h @ w[pre + "f"].T + w[pre + "f.b"],
                          m["gate_cap"])
    o = torch.stack([matrix_memory(q[:, a], k[:, a], v[:, a], li[:, a], lf[:, a])[0]
                     for a in range(H)], 1)
    o = rms_unit(o, eps).reshape(T, H * vd) * w[pre + "norm"]
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# ------------------------------------------------------------------ feed-forward
def dense(w, pre, h, eps):
    return poly_norm(h @ w[pre + "up"].T, w[pre + "act"], eps) @ w[pre + "down"].T


def route(z, correction, r):
    """z [T, n] router logits -> (chosen [T, top], weights [T, top]); ties to the lower index."""
    T, n = z.shape
    e = torch.exp(z - z.max(-1, keepdim=True).values)
    s = e / e.sum(-1, keepdim=True)
    groups = r.get("groups") or {"count": 1, "keep": 1}
    per = n // groups["count"]
    ids = torch.zeros(T, r["top"], dtype=torch.long)
    wts = torch.zeros(T, r["top"], dtype=D64)
    for t in range(T):
        c = (s[t] + correction).tolist()
        best = [max(c[g * per:(g + 1) * per]) for g in range(groups["count"])]
        kept = sorted(range(groups["count"]), key=lambda g: (-best[g], g))[:groups["keep"]]
        allowed = [j for j in range(n) if j // per in kept]
        order = sorted(allowed, key=lambda j: (-c[j], j))[:r["top"]]
        ids[t] = torch.tensor(order)
        wts[t] = s[t][order] * r.get("scale", 1.0)
    return ids, wts


def mixture(f, w, pre, h):
    r = f["router"]
    E = r["experts"]
    ids, wts = route(h @ w[pre + "router"].T, w[pre + "correction"], r)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j, p in zip(ids[t].tolist(), wts[t]):
            if j >= E:                                   # an identity expert
                out[t] += p * h[t]
            else:
                e = f"{pre}e{j}."
                out[t] += p * swiglu_expert(h[t], w[e + "gate"], w[e + "up"], w[e + "down"])
    if f.get("shared"):
        y = swiglu_expert(h, w[pre + "shared.gate"], w[pre + "shared.up"], w[pre + "shared.down"])
        out = out + y * sigmoid(h @ w[pre + "shared.sg"].T)
    return out


# ------------------------------------------------------------------ model
def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence; ``layers_out`` receives the stream after every
    layer."""
    w = {k: v.to(D64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.as_tensor(tokens, dtype=torch.long)
    pos = torch.arange(ids.numel())
    x = w["embed"][ids]
    v_first = None
    for i, ly in enumerate(cfg["layers"]):
        L, m, f = "l%d." % i, ly["mixer"], ly.get("mlp")
        h = gain_norm(x, w[L + "norm1"], eps)
        if ly["type"] == "attention":
            mixing = bool(m.get("v_mix"))
            y, v = attention(m, w, L + "mix.", h, pos, v_first if mixing else None)
            if mixing and v_first is None:
                v_first = v
        elif ly["type"] == "mlstm":
            y = mlstm(m, w, L + "mix.", h, eps)
        else:
            raise ValueError(ly["type"])
        x = x + gain_norm(y, w[L + "norm1b"], eps)
        if f is not None:
            h = gain_norm(x, w[L + "norm2"], eps)
            y = dense(w, L + "mlp.", h, eps) if f["kind"] == "dense" else mixture(f, w, L + "mlp.", h)
            x = x + gain_norm(y, w[L + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return gain_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(cfg, weights, prompt, n):
    """n tokens after the prompt, each the largest logit of the sequence so far."""
    toks, out = list(prompt), []
    for _ in range(n):
        nxt = int(forward(cfg, weights, toks)[-1].argmax())
        out.append(nxt)
        toks.append(nxt)
    return out
