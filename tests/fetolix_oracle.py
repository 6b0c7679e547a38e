"""Plain, slow Fetolix oracle: whole sequences, no cache, no batching.

One function per mechanism, written from the equations in double precision.
It imports nothing from the package, so agreement with the engine means two
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
    mu = x.mean(-1, keepdim=True)
    var = ((x - mu) ** 2).mean(-1, keepdim=True)
    return (x - mu) / torch.sqrt(var + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate_pairs(x, positions, base):
    """Rotate (x[2i], x[2i+1]) by positions * base^(-2i/n); x: [T, ..., n]."""
    n = x.shape[-1]
    out = torch.empty_like(x)
    for i in range(n // 2):
        a = positions.double() * base ** (-2.0 * i / n)
        shape = [-1] + [1] * (x.dim() - 2)
        c, s = torch.cos(a).view(shape), torch.sin(a).view(shape)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def visible(T, window=None):
    """[T, T] bool: may position i (row) see position j (column)?"""
    i = torch.arange(T).view(-1, 1)
    j = torch.arange(T).view(1, -1)
    ok = j <= i
    if window is not None:
        ok &= (i - j) < window
    return ok


def latent_attention(h, W, p, mix, eps, positions=None):
    """h: [T, width] -> [T, width].  A low-rank query when the config has
    q_rank, a sliding window when it has a mask."""
    T = h.shape[0]
    H, d, r, dv, rank = (mix[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    pos = torch.arange(T) if positions is None else positions
    if "q_rank" in mix:
        cq = rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
        q = cq @ W[p + "uq"].T
    else:
        q = h @ W[p + "q"].T
    q = q.view(T, H, d + r)
    kv = h @ W[p + "dkv"].T
    c = rms(kv[:, :rank], eps) * W[p + "dkv.norm"]
    k_rot = rotate_pairs(kv[:, rank:], pos, mix["rot"]["base"])
    q_rot = rotate_pairs(q[..., d:], pos, mix["rot"]["base"])
    k = (c @ W[p + "uk"].T).view(T, H, d)
    v = (c @ W[p + "uv"].T).view(T, H, dv)
    ok = visible(T, mix["mask"]["size"] if mix.get("mask") else None)
    heads = []
    for n in range(H):
        s = (q[:, n, :d] @ k[:, n].T + q_rot[:, n] @ k_rot.T) * mix["scale"]
        s = s.masked_fill(~ok, -math.inf)
        heads.append(torch.softmax(s, -1) @ v[:, n])
    o = torch.stack(heads, 1)
    o = o * torch.sigmoid(h @ W[p + "g"].T).unsqueeze(-1)
    return o.reshape(T, H * dv) @ W[p + "o"].T


def clamped_glu(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ W[p + "down"].T


def token_side(x, tokens, W, i, dim, eps):
    """x plus layer i's normed per-token input."""
    p = f"l{i}.side."
    e = W["side.embed"][tokens][:, i * dim:(i + 1) * dim]
    y = (gelu_tanh(x @ W[p + "gate"].T) * e) @ W[p + "proj"].T
    return x + rms(y, eps) * W[p + "norm"]


def layer_order(cfg):
    """[(layer index, first of a loop pass?)] in the order they run."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        order += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab]; appends the residual after every layer run to trace."""
    tokens = torch.as_tensor(tokens)
    eps = cfg["norm"]["eps"]
    x = x0 = W["embed"][tokens]
    for i, enters in layer_order(cfg):
        if enters:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T
        spec = cfg["layers"][i]
        h = layer_norm(x, W[f"l{i}.norm1"], eps)
        y = latent_attention(h, W, f"l{i}.mix.", spec["mixer"], eps)
        if spec.get("mlp"):
            y = y + clamped_glu(h, W, f"l{i}.mlp.", spec["mlp"]["limit"])
        x = x + y
        x = token_side(x, tokens, W, i, cfg["token_side"]["dim"], eps)
        if trace is not None:
            trace.append(x)
    return layer_norm(x, W["final.norm"], eps) @ W["embed"].T
