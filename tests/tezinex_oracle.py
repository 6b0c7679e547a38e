"""Plain, slow Tezinex oracle: whole sequences, no cache, no state slots, no batching.

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


def norm(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1 + w)


def silu(z):
    return z / (1 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def cap(z, limit):
    return limit * torch.tanh(z / limit)


def positions(T, width):
    """[T, width]: sin and cos of p / 10000^(2i/width) in turn."""
    out = torch.zeros(T, width, dtype=torch.float64)
    p = torch.arange(T, dtype=torch.float64)
    for c in range(width):
        a = p * 10000.0 ** (-2.0 * (c // 2) / width)
        out[:, c] = torch.cos(a) if c % 2 else torch.sin(a)
    return out


def short_conv(x, w):
    """Causal per-channel convolution then silu; x [T, C], w [C, taps]."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for n in range(taps):
            s = t - (taps - 1) + n
            if s >= 0:
                out[t] += w[:, n] * x[s]
    return silu(out)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k [T, D] (unit, q scaled), v [T, V], g [T, D], beta [T] of one head."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=torch.float64)
    out = []
    for t in range(q.shape[0]):
        S = g[t].unsqueeze(1) * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out.append(S.T @ q[t])
    return torch.stack(out)


def decay(z, A_log):
    """z [T, heads, D] before softplus -> per-channel factors."""
    return torch.exp(-torch.exp(A_log).view(1, -1, 1) * softplus(z))


def channel_delta(h, W, p, mix, eps):
    """h: [T, width] -> [T, width]."""
    T = h.shape[0]
    H, G, D, V = (mix[n] for n in ("heads", "kv_heads", "dim", "vdim"))
    q = unit(short_conv(h @ W[p + "q"].T, W[p + "q.conv"]).view(T, G, D)) * D ** -0.5
    k = unit(short_conv(h @ W[p + "k"].T, W[p + "k.conv"]).view(T, G, D))
    v = short_conv(h @ W[p + "v"].T, W[p + "v.conv"]).view(T, H, V)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]
    g = decay(z.view(T, H, D), W[p + "A_log"])
    gate = torch.sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T).view(T, H, V)
    heads = []
    for n in range(H):
        j = n // (H // G)
        o = delta_rule(q[:, j], k[:, j], v[:, n], g[:, n], beta[:, n])
        heads.append(rms(o, eps) * W[p + "norm"] * gate[:, n])
    return torch.stack(heads, 1).reshape(T, H * V) @ W[p + "o"].T


def visible(T, size, keep):
    """[T, T] bool: may position i (row) see position j (column)?"""
    i = torch.arange(T).view(-1, 1)
    j = torch.arange(T).view(1, -1)
    return (j <= i) & ((i - j < size) | (j < keep))


def sink_softmax(s, sink):
    """Weights of scores s [.., keys]; exp(sink) joins the denominator only."""
    m = torch.clamp(s.max(-1, keepdim=True).values, min=sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def keys_values(h, W, p, mix):
    T, G = h.shape[0], mix["kv_heads"]
    k = (h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, mix["dim"])
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(T, G, mix["vdim"])
    return k, v


def attention(h, W, p, mix, kv):
    """h: [T, width], kv: keys and values of this layer or the one it borrows from."""
    T, H, G, D = h.shape[0], mix["heads"], mix["kv_heads"], mix["dim"]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, D)
    k, v = kv
    ok = visible(T, mix["mask"]["size"], mix["mask"]["keep_first"])
    heads = []
    for n in range(H):
        j = n // (H // G)
        s = cap(q[:, n] @ k[:, j].T * mix["scale"], mix["softcap"])
        a = sink_softmax(s.masked_fill(~ok, -math.inf), W[p + "sink"][n])
        heads.append(a @ v[:, j])
    return torch.stack(heads, 1).reshape(T, -1) @ W[p + "o"].T


def feed_forward(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def depth_average(states, c):
    return sum(c[j] * x for j, x in enumerate(states))


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab]; appends what every layer hands on to trace."""
    tokens = torch.as_tensor(tokens)
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = W["embed"][tokens] + positions(len(tokens), cfg["width"])
    states, kv = [x], {}
    for i, spec in enumerate(cfg["layers"]):
        p, mix = f"l{i}.", spec["mixer"]
        h = norm(x, W[p + "norm1"], eps)
        if spec["type"] == "channel_delta":
            y = channel_delta(h, W, p + "mix.", mix, eps)
        else:
            j = mix.get("kv_from")
            if j is None:
                kv[i] = keys_values(h, W, p + "mix.", mix)
            y = attention(h, W, p + "mix.", mix, kv[i if j is None else j])
        x = x + m * norm(y, W[p + "norm1b"], eps)
        if spec.get("mlp"):
            y = feed_forward(norm(x, W[p + "norm2"], eps), W, p + "mlp.")
            x = x + m * norm(y, W[p + "norm2b"], eps)
        states.append(x)
        x = depth_average(states, W[p + "dwa"])
        if trace is not None:
            trace.append(x)
    return cap(norm(x, W["final.norm"], eps) @ W["embed"].T, cfg["logit_softcap"])
