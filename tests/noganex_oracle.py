"""Plain, slow Noganex oracle: whole sequences, no cache, no state slots, no batching.

One function per mechanism, written from the equations in double precision.  It
imports nothing from the package, so agreement with the engine means two
independent readings of the design agree.

Notation: a config is the decoded config.json dict, ``W`` maps tensor names to
float64 tensors, ``T`` is the number of tokens of one sequence.
"""
import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------ positions


def yarn(rot):
    """Angles per position of the pairs, slowed along a ramp; the factor on cos and sin."""
    dims, base, s = rot["dims"], rot["base"], rot["scaling"]

    def pair_with(turns):
        """The (fractional) pair that makes so many turns over the original length."""
        return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(pair_with(s["fast"])), 0)
    hi = min(math.ceil(pair_with(s["slow"])), dims - 1)
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * r + f * (1 - r))
    return out, 0.1 * math.log(s["factor"]) + 1


def rotate(x, freqs, mult=1.0):
    """x [T, heads, size]: dimension i turns with i + n, n = len(freqs), the rest stays."""
    n = len(freqs)
    a = torch.arange(x.shape[0], dtype=torch.float64).view(-1, 1, 1) * torch.tensor(
        freqs, dtype=torch.float64)
    c, s = mult * torch.cos(a), mult * torch.sin(a)
    u, v = x[..., :n], x[..., n : 2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n :]], -1)


# ------------------------------------------------------------------ attention


def visible(T, size):
    """[T, T] bool: position i (row) sees the keys of its own chunk up to itself."""
    i = torch.arange(T).view(-1, 1)
    j = torch.arange(T).view(1, -1)
    return (j <= i) & (i // size == j // size)


def mixed_scores(s, talk):
    """s [heads, T, T]: every head's scores become a mix of all heads' scores."""
    return torch.einsum("hg,gij->hij", talk, s)


def softmax(s):
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def attention(h, W, p, mix, eps):
    """h: [T, width] -> [T, width]."""
    T, H, G, D, E = h.shape[0], *(mix[n] for n in ("heads", "kv_heads", "dim", "vdim"))
    freqs, mult = yarn(mix["rot"])
    q = rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"]
    k = rms(h @ W[p + "k"].T, eps) * W[p + "k.norm"]
    q, k = rotate(q.view(T, H, D), freqs, mult), rotate(k.view(T, G, D), freqs, mult)
    v = (h @ W[p + "v"].T).view(T, G, E)
    s = torch.stack([q[:, n] @ k[:, n // (H // G)].T * mix["scale"] for n in range(H)])
    s = mixed_scores(s, W[p + "talk"])
    a = softmax(s.masked_fill(~visible(T, mix["mask"]["size"]), -math.inf))
    heads = [a[n] @ v[:, n // (H // G)] for n in range(H)]
    return torch.stack(heads, 1).reshape(T, -1) @ W[p + "o"].T


# ----------------------------------------------------------------- delta rule


def short_conv(x, w):
    """Causal per-channel convolution then silu; x [T, C], w [C, taps]."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for n in range(taps):
        ago = taps - 1 - n
        if ago < T:
            out[ago:] += w[:, n] * x[: T - ago]
    return silu(out)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k [T, D] (unit, q scaled), v [T, V], g, beta [T] of one head."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=torch.float64)
    out = []
    for t in range(q.shape[0]):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out.append(S.T @ q[t])
    return torch.stack(out)


def decay(z, A_log):
    """z [T, heads] before softplus -> one factor per head."""
    return torch.exp(-torch.exp(A_log) * softplus(z))


def delta(h, W, p, mix, eps):
    """h: [T, width] -> [T, width]."""
    T = h.shape[0]
    H, G, D, V = (mix[n] for n in ("heads", "kv_heads", "dim", "vdim"))
    q = unit(short_conv(h @ W[p + "q"].T, W[p + "q.conv"]).view(T, G, D)) * D ** -0.5
    k = unit(short_conv(h @ W[p + "k"].T, W[p + "k.conv"]).view(T, G, D))
    v = short_conv(h @ W[p + "v"].T, W[p + "v.conv"]).view(T, H, V)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    g = decay(h @ W[p + "a"].T + W[p + "dt_bias"], W[p + "A_log"])
    gate = silu(h @ W[p + "g"].T).view(T, H, V)
    heads = []
    for n in range(H):
        j = n // (H // G)
        o = delta_rule(q[:, j], k[:, j], v[:, n], g[:, n], beta[:, n])
        heads.append(rms(o, eps) * W[p + "norm"] * gate[:, n])
    return torch.stack(heads, 1).reshape(T, H * V) @ W[p + "o"].T


# --------------------------------------------------------------- feed-forward


def dense(h, W, p):
    gate = gelu_tanh(h @ W[p + "gate"].T + W[p + "gate.b"])
    return (gate * (h @ W[p + "up"].T + W[p + "up.b"])) @ W[p + "down"].T + W[p + "down.b"]


def silu_glu(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(h, W, p, router):
    """Chosen experts [T, top] and their weights: the correction joins the choice only."""
    s = torch.sigmoid(h @ W[p + "router"].T)
    ids = torch.topk(s + W[p + "correction"], router["top"], -1).indices
    w = s.gather(-1, ids)
    return ids, w / (w.sum(-1, keepdim=True) + 1e-20) * router["scale"]


def experts(h, W, p, mlp):
    ids, weights = route(h, W, p, mlp["router"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        w = (weights * (ids == e)).sum(-1, keepdim=True)
        rows = (ids == e).any(-1).nonzero()[:, 0]
        out[rows] += w[rows] * silu_glu(h[rows], W, f"{p}e{e}.")
    if mlp.get("shared"):
        out = out + silu_glu(h, W, p + "shared.")
    return out


def gated(y, h, W, name):
    """A sublayer's result times the gate that its input opens."""
    return y * torch.sigmoid(h @ W[name].T + W[name + ".b"])


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab]; appends the residual after every layer to trace."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens)]
    for i, spec in enumerate(cfg["layers"]):
        j = spec.get("weights_of")
        p, mix, mlp = f"l{i if j is None else j}.", spec["mixer"], spec.get("mlp")
        mixer = attention if spec["type"] == "attention" else delta
        y = gated(mixer(x, W, p + "mix.", mix, eps), x, W, p + "rg1")
        x = x + rms(y, eps) * W[p + "norm1"]
        if mlp:
            y = dense(x, W, p + "mlp.") if mlp["kind"] == "dense" else experts(x, W, p + "mlp.", mlp)
            x = x + rms(gated(y, x, W, p + "rg2"), eps) * W[p + "norm2"]
        if trace is not None:
            trace.append(x)
    return rms(x, eps) * W["final.norm"] @ W["head"].T * cfg["logit_scale"]
