"""Plain, slow Lobuvik oracle: whole sequences, no cache, no state slots, no batching.

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


def layer_norm(x, w, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def cap(z, limit):
    return limit * torch.tanh(z / limit)


# ------------------------------------------------------------------ positions


def frequencies(rot):
    dims, base = rot["dims"], rot["base"]
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def smoothed(f, s):
    """Low frequencies slowed by a factor, the ones between two wavelengths blended."""
    out = []
    for x in f:
        turns = s["original"] * x / (2 * math.pi)  # over the original context
        if turns > s["high"]:
            out.append(x)
        elif turns < s["low"]:
            out.append(x / s["factor"])
        else:
            m = (turns - s["low"]) / (s["high"] - s["low"])
            out.append((1 - m) * x / s["factor"] + m * x)
    return out


def yarn(f, rot):
    """Frequencies slowed along a ramp over the dimensions; factor on cos and sin."""
    s, dims = rot["scaling"], rot["dims"]

    def where(turns):
        return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(rot["base"]))

    lo = max(math.floor(where(s["fast"])), 0)
    hi = min(math.ceil(where(s["slow"])), dims - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / s["factor"] * r + x * (1 - r))
    return out, 0.1 * math.log(s["factor"]) + 1


def rotate(x, freqs, mult=1.0):
    """x [T, heads, size]: dimension i turns with i + n, n = len(freqs), the rest stays."""
    n = len(freqs)
    a = torch.arange(x.shape[0], dtype=torch.float64).view(-1, 1, 1) * torch.tensor(
        freqs, dtype=torch.float64)
    c, s = mult * torch.cos(a), mult * torch.sin(a)
    u, v = x[..., :n], x[..., n : 2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n :]], -1)


def bucket(n, B, D):
    """Bucket of distance n: single distances, then widths that grow by a constant factor."""
    half = B // 2
    if n < half:
        return n
    grow = math.log(n / half) / math.log(D / half)
    return min(B - 1, half + math.floor(grow * (B - half) + 1e-9))


def distance_bias(rel, D, T):
    """[heads, T, T] for query i and key j <= i."""
    b = torch.tensor([bucket(n, rel.shape[0], D) for n in range(T)])
    i = torch.arange(T)
    return rel[b[(i.view(-1, 1) - i.view(1, -1)).clamp(min=0)]].permute(2, 0, 1)


def query_temperature(T, coef, every):
    p = torch.arange(T, dtype=torch.float64)
    return 1 + coef * torch.log(torch.floor((p + 1) / every) + 1)


def visible(T, size=None):
    """[T, T] bool: may position i (row) see position j (column)?"""
    i = torch.arange(T).view(-1, 1)
    j = torch.arange(T).view(1, -1)
    return (j <= i) if size is None else (j <= i) & (i - j < size)


# --------------------------------------------------------------------- mixers


def short_conv(x, w):
    """Causal per-channel convolution; x [T, C], w [C, taps]."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for n in range(taps):
        ago = taps - 1 - n
        if ago < T:
            out[ago:] += w[:, n] * x[: T - ago]
    return out


def sigmoid_weights(s, ok):
    return torch.sigmoid(s) * ok


def sink_softmax(s, sink=None):
    """Weights of scores s [.., keys]; exp(sink) joins the denominator only."""
    m = s.max(-1, keepdim=True).values
    if sink is not None:
        m = torch.clamp(m, min=float(sink))
    e = torch.exp(s - m)
    z = e.sum(-1, keepdim=True)
    return e / (z if sink is None else z + torch.exp(sink - m))


def attention(h, W, p, mix, eps):
    """Unnormalized sigmoid attention with distance biases.  h: [T, width]."""
    T, H, G, D, E = h.shape[0], *(mix[n] for n in ("heads", "kv_heads", "dim", "vdim"))

    def project(n, heads, size):
        u = short_conv(h @ W[p + n].T + W[p + n + ".b"], W[p + n + ".conv"])
        return u.view(T, heads, size)

    q = rms(project("q", H, D), eps) * W[p + "q.norm"]
    k = rms(project("k", G, D), eps) * W[p + "k.norm"]
    v = rms(project("v", G, E), eps)
    q = q * query_temperature(T, mix["q_temp"]["coef"], mix["q_temp"]["every"]).view(T, 1, 1)
    bias, ok = distance_bias(W[p + "rel"], mix["bias_max"], T), visible(T)
    heads = []
    for n in range(H):
        j = n // (H // G)
        s = q[:, n] @ k[:, j].T * mix["scale"] + bias[n] + W[p + "pb"][n]
        heads.append(sigmoid_weights(s, ok) @ v[:, j])
    return torch.stack(heads, 1).reshape(T, -1) @ W[p + "o"].T + W[p + "o.b"]


def latent_attention(h, W, p, mix, eps):
    T, H, D, R, E = h.shape[0], *(mix[n] for n in ("heads", "dim", "rot_dim", "vdim"))
    rank = mix["kv_rank"]
    freqs, mult = yarn(frequencies(mix["rot"]), mix["rot"])
    q = (h @ W[p + "q"].T).view(T, H, D + R)
    down = h @ W[p + "dkv"].T
    c = rms(down[:, :rank], eps) * W[p + "dkv.norm"]
    qr = rotate(q[..., D:], freqs, mult)
    kr = rotate(down[:, rank:].view(T, 1, R), freqs, mult)[:, 0]
    k = (c @ W[p + "uk"].T).view(T, H, D)
    v = (c @ W[p + "uv"].T).view(T, H, E)
    ok = visible(T, mix["mask"]["size"])
    heads = []
    for n in range(H):
        s = (q[:, n, :D] @ k[:, n].T + qr[:, n] @ kr.T) * mix["scale"]
        heads.append(sink_softmax(s.masked_fill(~ok, -math.inf), W[p + "sink"][n]) @ v[:, n])
    return torch.stack(heads, 1).reshape(T, -1) @ W[p + "o"].T


def rotated_attention(h, W, p, mix):
    T, H, G, D, E = h.shape[0], *(mix[n] for n in ("heads", "kv_heads", "dim", "vdim"))
    freqs = smoothed(frequencies(mix["rot"]), mix["rot"]["scaling"])
    q = rotate((h @ W[p + "q"].T).view(T, H, D), freqs)
    k = rotate((h @ W[p + "k"].T).view(T, G, D), freqs)
    v = (h @ W[p + "v"].T).view(T, G, E)
    gate = torch.sigmoid(h @ W[p + "g"].T)
    ok = visible(T, mix["mask"]["size"])
    heads = []
    for n in range(H):
        j = n // (H // G)
        s = cap(q[:, n] @ k[:, j].T * mix["scale"] * W[p + "temp"][n], mix["softcap"])
        heads.append(sink_softmax(s.masked_fill(~ok, -math.inf)) @ v[:, j] * gate[:, n : n + 1])
    return torch.stack(heads, 1).reshape(T, -1) @ W[p + "o"].T


# --------------------------------------------------------------- feed-forward


def gelu_glu(h, W, p):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def clamped_glu(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ W[p + "down"].T


def route(h, W, p, top):
    """Chosen experts [T, top] and their weights."""
    z = h @ W[p + "router"].T + W[p + "router.b"]
    best = torch.topk(z, top, -1)
    return best.indices, torch.softmax(best.values, -1)


def experts(h, W, p, mlp):
    ids, weights = route(h, W, p, mlp["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        w = (weights * (ids == e)).sum(-1, keepdim=True)
        rows = (w[:, 0] > 0).nonzero()[:, 0]
        out[rows] += w[rows] * clamped_glu(h[rows], W, f"{p}e{e}.", mlp["expert"]["limit"])
    if mlp.get("shared"):
        out = out + clamped_glu(h, W, p + "shared.", mlp["shared"]["limit"])
    return out


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab]; appends the residual after every layer to trace."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, spec in enumerate(cfg["layers"]):
        p, mix = f"l{i}.", spec["mixer"]
        h = layer_norm(x, W[p + "norm1"], eps)
        if spec["type"] == "attention":
            y = attention(h, W, p + "mix.", mix, eps)
        elif spec["type"] == "latent_attention":
            y = latent_attention(h, W, p + "mix.", mix, eps)
        else:
            y = rotated_attention(h, W, p + "mix.", mix)
        mlp = spec.get("mlp")
        if mlp:
            h = layer_norm(x, W[p + "norm2"], eps)
            if mlp["kind"] == "dense":
                y = y + gelu_glu(h, W, p + "mlp.")
            else:
                y = y + experts(h, W, p + "mlp.", mlp)
        x = x + y
        if trace is not None:
            trace.append(x)
    return layer_norm(x, W["final.norm"], eps) @ W["head"].T
