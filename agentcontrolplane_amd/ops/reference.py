"""Plain-PyTorch fp32 reference implementations.

These are the numerics oracles the HIP kernels are tested against
(tests/test_ops_gpu.py compares each kernel to its reference at fp32), and
the compute path for CPU-only engine tests.  Written for clarity, not speed.
"""
from __future__ import annotations

import torch


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5) -> torch.Tensor:
    xf = x.float()
    var = xf.pow(2).mean(-1, keepdim=True)
    out = xf * torch.rsqrt(var + eps) * weight.float()
    return out.to(x.dtype)


def fused_add_rmsnorm(x, residual, weight, eps: float = 1e-5):
    new_residual = (x.float() + residual.float()).to(x.dtype)
    return rmsnorm(new_residual, weight, eps), new_residual


def build_cos_sin(max_position: int, head_dim: int, theta: float, device, dtype=torch.float32,
                  exact: bool = False):
    """[2, max_position, head_dim/2] cos and sin tables of position times
    theta^(-2i/head_dim).  ``exact`` takes the angles in double precision."""
    at = torch.float64 if exact else torch.float32
    inv_freq = 1.0 / (
        theta ** (torch.arange(0, head_dim, 2, device=device, dtype=at) / head_dim)
    )
    t = torch.arange(max_position, device=device, dtype=at)
    freqs = torch.outer(t, inv_freq)
    return torch.stack([freqs.cos(), freqs.sin()], dim=0).to(dtype)  # [2, P, D/2]


def _rope_rotate_half(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor) -> torch.Tensor:
    # x: [N, H, D]; cos/sin: [N, D/2]
    d2 = x.shape[-1] // 2
    x1, x2 = x[..., :d2].float(), x[..., d2:].float()
    c = cos.unsqueeze(1)
    s = sin.unsqueeze(1)
    out = torch.cat([x1 * c - x2 * s, x2 * c + x1 * s], dim=-1)
    return out.to(x.dtype)


def rope_and_cache(q, k, v, positions, slot_mapping, k_cache, v_cache, cos_sin):
    """q:[N,Hq,D] k,v:[N,Hkv,D]; cos_sin:[2,P,D/2];
    k_cache/v_cache: [num_blocks*block_size, Hkv, D] flat-slot view."""
    cos = cos_sin[0][positions]
    sin = cos_sin[1][positions]
    q.copy_(_rope_rotate_half(q, cos, sin))
    k.copy_(_rope_rotate_half(k, cos, sin))
    _flat(k_cache)[slot_mapping] = k.to(k_cache.dtype)
    _flat(v_cache)[slot_mapping] = v.to(v_cache.dtype)
    return q, k


def _gather_kv(k_cache, v_cache, block_table, seq_len, block_size):
    """Contiguous [S, Hkv, D] K and V for one sequence."""
    slots = []
    for pos in range(seq_len):
        b = block_table[pos // block_size]
        slots.append(int(b) * block_size + pos % block_size)
    idx = torch.tensor(slots, device=k_cache.device, dtype=torch.long)
    return k_cache[idx], v_cache[idx]


def attention_prefill(q, k_cache, v_cache, block_table, seq_len, ctx_len, scale):
    """q: [Lq, Hq, D]; returns [Lq, Hq, D].  Causal: query i (global position
    ctx_len+i) attends to kv positions 0..ctx_len+i."""
    Lq, Hq, D = q.shape
    block_size = _block_size_of(k_cache)
    k, v = _gather_kv(_flat(k_cache), _flat(v_cache), block_table, seq_len, block_size)
    Hkv = k.shape[1]
    rep = Hq // Hkv
    kf = k.float().repeat_interleave(rep, dim=1)   # [S, Hq, D]
    vf = v.float().repeat_interleave(rep, dim=1)
    qf = q.float()
    # scores [Hq, Lq, S]
    scores = torch.einsum("lhd,shd->hls", qf, kf) * scale
    pos_q = torch.arange(ctx_len, ctx_len + Lq, device=q.device).view(1, Lq, 1)
    pos_k = torch.arange(seq_len, device=q.device).view(1, 1, seq_len)
    scores = scores.masked_fill(pos_k > pos_q, float("-inf"))
    probs = torch.softmax(scores, dim=-1)
    out = torch.einsum("hls,shd->lhd", probs, vf)
    return out.to(q.dtype)


def attention_prefill_batch(q, k_cache, v_cache, batch, scale, out=None):
    """Loop the per-sequence oracle over a FlatBatch's prefill chunks."""
    outs = []
    row = 0
    for m in batch.prefills:
        outs.append(
            attention_prefill(
                q[row : row + m.query_len], k_cache, v_cache, m.block_table,
                m.seq_len, m.ctx_len, scale,
            )
        )
        row += m.query_len
    res = torch.cat(outs, dim=0) if len(outs) > 1 else outs[0]
    if out is not None:
        out.copy_(res)
        return out
    return res


def attention_decode_batch(q, k_cache, v_cache, batch, scale, out=None):
    """q: [B, Hq, D]; decode tables/lens come from the FlatBatch."""
    res = attention_decode_raw(
        q, k_cache, v_cache, batch.decode_block_tables, batch.decode_seq_lens, scale
    )
    if out is not None:
        out.copy_(res)
        return out
    return res


def attention_decode_raw(q, k_cache, v_cache, block_tables, seq_lens, scale):
    B, Hq, D = q.shape
    outs = []
    for i in range(B):
        out = attention_prefill(
            q[i : i + 1],
            k_cache,
            v_cache,
            block_tables[i].tolist(),
            int(seq_lens[i]),
            int(seq_lens[i]) - 1,
            scale,
        )
        outs.append(out)
    return torch.cat(outs, dim=0)


def _flat(cache):
    """Cache stored [num_blocks, block_size, Hkv, D] → flat [slots, Hkv, D]."""
    if cache.dim() == 4:
        nb, bs, h, d = cache.shape
        return cache.view(nb * bs, h, d)
    return cache


def _block_size_of(cache):
    if cache.dim() == 4:
        return cache.shape[1]
    raise ValueError("pass the 4-D [num_blocks, block_size, H, D] cache")


def swiglu(gate_up: torch.Tensor) -> torch.Tensor:
    gate, up = gate_up.float().chunk(2, dim=-1)
    return (torch.nn.functional.silu(gate) * up).to(gate_up.dtype)


# ------------------------------------------------ fp32-residual norms, GLU, gates


def rmsnorm_rows(x, weight, eps: float, n: int):
    xf = x.float()
    inv = torch.rsqrt(xf[:, :n].pow(2).mean(-1, keepdim=True) + eps)
    return (xf * inv * weight.float()).to(x.dtype)


def layernorm(x, weight, eps: float, dtype):
    xc = x - x.mean(-1, keepdim=True)
    var = xc.pow(2).mean(-1, keepdim=True)
    return (xc * torch.rsqrt(var + eps) * weight.float()).to(dtype)


def residual_norm(x, y, eps: float, y_norm=None, x_norm=None, out=None, center=True,
                  offset=0.0, mult=1.0, depth=None, layer=0, x_norm2=None, out2=None,
                  experts=None, gate=None):
    if y is not None:
        yf = y.float()
        if experts is not None:
            rows, weights = experts
            yf = yf + (rows.float() * weights.unsqueeze(-1)).sum(1)
        if gate is not None:
            yf = yf * torch.sigmoid(gate.float())
        if y_norm is not None:
            yf = yf * torch.rsqrt(yf.pow(2).mean(-1, keepdim=True) + eps)
            yf = yf * (offset + y_norm.float())
        x += mult * yf
    if depth is not None:
        n = layer + 2
        depth.states[n - 1] = x
        x.copy_(torch.einsum("j,jnk->nk", depth.coef[layer, :n], depth.states[:n]))
    if out is None:
        return
    if x_norm is None:
        out.copy_(x)
        return
    xc = x - x.mean(-1, keepdim=True) if center else x
    xc = xc * torch.rsqrt(xc.pow(2).mean(-1, keepdim=True) + eps)
    out.copy_(xc * (offset + x_norm.float()))
    if out2 is not None:
        out2.copy_(xc * (offset + x_norm2.float()))


def embed_positions(token_ids, positions, table, cos_sin, x, copy=None, scale=1.0):
    x.copy_(table[token_ids].float() * scale)
    if cos_sin is not None:
        w = x.shape[1]
        x[:, 0::2] += cos_sin[1][positions]
        x[:, 1::2] += cos_sin[0][positions][:, : w // 2]
    if copy is not None:
        copy.copy_(x)


def softcap(logits, cap):
    return cap * torch.tanh(logits.float() / cap)


def clamped_glu(gate_up, limit: float, alpha: float, offset: float, out, cubic=0.0):
    g, u = gate_up.float().chunk(2, dim=-1)
    g = g.clamp(max=limit)
    z = alpha * (g + cubic * g ** 3) if cubic else alpha * g
    out.copy_(g * torch.sigmoid(z) * (u.clamp(-limit, limit) + offset))


def side_gate(x, y, gate, token_ids, table, offset: int):
    x = x + y.float()
    s = torch.nn.functional.linear(x.to(gate.dtype), gate).float()
    e = table[token_ids, offset : offset + gate.shape[0]].float()
    return x, (torch.nn.functional.gelu(s, approximate="tanh") * e).to(gate.dtype)


# ------------------------------------------------------------ latent attention


def _rotate_interleaved(x, cos, sin):
    """Rotate the pairs (x[..., 2i], x[..., 2i+1]); cos/sin broadcast over
    x's pairs."""
    u, v = x[..., 0::2].float(), x[..., 1::2].float()
    return torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1).flatten(-2)


def latent_inputs(kv, norm_w, eps: float, kv_rank: int, rot_dim: int, rank: int,
                  positions, slot_mapping, cos_sin, cache, q=None, q_norm=None, q_rank=0):
    c = rmsnorm_rows(kv[:, :kv_rank], norm_w, eps, kv_rank)
    k_rot = _rotate_interleaved(
        kv[:, kv_rank : kv_rank + rot_dim], cos_sin[0][positions], cos_sin[1][positions]
    )
    row = torch.zeros(kv.shape[0], cache.shape[-1], dtype=cache.dtype, device=cache.device)
    row[:, :kv_rank] = c.to(cache.dtype)
    row[:, rank : rank + rot_dim] = k_rot.to(cache.dtype)
    cache.view(-1, cache.shape[-1])[slot_mapping] = row
    return None if q is None else rmsnorm_rows(q, q_norm, eps, q_rank)


def head_linear(x, w, out, gate=None):
    y = torch.matmul(x.float().transpose(0, 1), w.float().transpose(1, 2)).transpose(0, 1)
    if gate is not None:
        y = y * torch.sigmoid(gate.float()).unsqueeze(-1)
    out.copy_(y)
    return out


def _sink_softmax(scores, sink):
    """Weights of scores [.., keys]; sink, broadcast over the keys, joins the denominator."""
    if sink is None:
        return torch.softmax(scores, -1)
    scores = torch.cat([scores, sink.expand(*scores.shape[:-1], 1)], -1)
    return torch.softmax(scores, -1)[..., :-1]


def _latent_attention_seq(q, cache, block_table, ctx_len: int, rank: int, scale: float, window,
                          sink):
    """One sequence's rows at positions ctx_len..; q [L, H, row] -> [L, H, rank]."""
    L, bs = q.shape[0], cache.shape[1]
    j = torch.arange(ctx_len + L, device=q.device)
    table = torch.as_tensor(block_table, device=q.device)
    rows = cache.view(-1, cache.shape[-1])[table[j // bs] * bs + j % bs].float()
    i = torch.arange(ctx_len, ctx_len + L, device=q.device).view(-1, 1)
    hidden = j > i
    if window is not None:
        hidden |= (i - j) >= window
    scores = torch.matmul(q.float(), rows.t()) * scale        # [L, H, S]
    scores = scores.masked_fill(hidden.unsqueeze(1), float("-inf"))
    probs = _sink_softmax(scores, None if sink is None else sink.view(1, -1, 1))
    return torch.matmul(probs, rows[:, :rank]).to(q.dtype)


def latent_attention(q, q_rot, cos_sin, rot_dim: int, cache, batch, scale: float, window,
                     row0: int = 0, skip=(), sink=None):
    N, H, rank = q.shape
    pos = batch.positions[row0:]
    rot = torch.zeros(N, H, cache.shape[-1] - rank, dtype=q.dtype, device=q.device)
    rot[:, :, :rot_dim] = _rotate_interleaved(
        q_rot[:, :, :rot_dim], cos_sin[0][pos].unsqueeze(1), cos_sin[1][pos].unsqueeze(1)
    ).to(q.dtype)
    q = torch.cat([q, rot], -1)
    out = torch.empty(N, H, rank, dtype=q.dtype, device=q.device)
    row = -row0
    for n, m in enumerate(batch.prefills):
        if row >= 0 and n not in skip:
            out[row : row + m.query_len] = _latent_attention_seq(
                q[row : row + m.query_len], cache, m.block_table, m.ctx_len, rank, scale, window,
                sink,
            )
        row += m.query_len
    for b in range(batch.num_decode):
        out[row : row + 1] = _latent_attention_seq(
            q[row : row + 1], cache, batch.decode_block_tables[b],
            int(batch.decode_seq_lens[b]) - 1, rank, scale, window, sink,
        )
        row += 1
    return out


# ---------------------------------------- grouped attention: caps, windows, sinks


def cache_keys_values(k, v, slot_mapping, k_cache, v_cache):
    _flat(k_cache)[slot_mapping] = k
    _flat(v_cache)[slot_mapping] = v


def _portions(batch):
    """(first row, rows, cached tokens before them, state slot, pages) per sequence."""
    row = 0
    for m in batch.prefills:
        yield row, m.query_len, m.ctx_len, m.state_slot, m.block_table
        row += m.query_len
    slots = batch.decode_state_slots
    for n in range(batch.num_decode):
        yield (row + n, 1, int(batch.decode_seq_lens[n]) - 1,
               0 if slots is None else int(slots[n]), batch.decode_block_tables[n])


def _short_conv(proj, conv, ring, batch):
    """Causal convolution of every sequence's rows, its ring advanced; fp32."""
    taps, out = conv.shape[0], torch.empty(proj.shape, device=proj.device)
    for row, n, ctx, slot, _ in _portions(batch):
        u = proj[row : row + n]
        past = [ring[slot, p % taps] if p >= 0 else torch.zeros_like(u[0])
                for p in range(ctx - taps + 1, ctx)]
        x = torch.cat([torch.stack(past), u]) if past else u
        out[row : row + n] = sum(x[j : j + n].float() * conv[j].float() for j in range(taps))
        for i in range(max(0, n - taps), n):
            ring[slot, (ctx + i) % taps] = u[i]
    return out


def attention_inputs(proj, heads, dim, vdim, k_cache, v_cache, batch, eps, conv, ring, q_norm,
                     k_norm, v_norm, cos_sin, head_mult, q_temp):
    N, d, e, G = proj.shape[0], k_cache.shape[-1], v_cache.shape[-1], k_cache.shape[2]
    x = proj.float() if conv is None else _short_conv(proj, conv, ring, batch)
    q, k, v = x.split([heads * d, G * d, G * e], 1)
    if q_norm is not None and q_norm.numel() > d:  # over all heads; the padding is zero
        q, k = (
            t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) / (n * dim) + eps) * w.float()
            for t, n, w in ((q, heads, q_norm), (k, G, k_norm))
        )
        q_norm = None
    q, k, v = q.reshape(N, heads, d), k.reshape(N, G, d), v.reshape(N, G, e)

    def rms(t, size):  # the padding is zero
        return t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) / size + eps)

    if q_norm is not None:
        q, k = rms(q, dim) * q_norm.float(), rms(k, dim) * k_norm.float()
    if v_norm:
        v = rms(v, vdim)
    p = batch.positions
    if cos_sin is not None:
        n = 2 * cos_sin.shape[2]
        c, s = (t[p].unsqueeze(1) for t in cos_sin)
        q, k = (torch.cat([_rotate_interleaved(t[..., :n], c, s), t[..., n:]], -1)
                for t in (q, k))
    if head_mult is not None:
        q = q * head_mult.view(1, -1, 1)
    if q_temp is not None:
        coef, every = q_temp
        t = 1 + coef * torch.log(torch.floor((p + 1) / every) + 1)
        q = q * t.view(-1, 1, 1)
    cache_keys_values(k.to(proj.dtype), v.to(proj.dtype), batch.slot_mapping, k_cache, v_cache)
    return q.to(proj.dtype)


def _grouped_attention_seq(q, k_cache, v_cache, block_table, ctx_len: int, scale, cap, window,
                           keep_first, sink, bias, sigmoid, chunk, talk):
    """One sequence's rows at positions ctx_len..; q [L, H, d] -> fp32 [L, H, e]."""
    L, H, bs = q.shape[0], q.shape[1], k_cache.shape[1]
    j = torch.arange(ctx_len + L, device=q.device)
    rows = torch.as_tensor(block_table, device=q.device)[j // bs] * bs + j % bs
    group = H // k_cache.shape[2]
    k = _flat(k_cache)[rows].float().repeat_interleave(group, 1).transpose(0, 1)
    v = _flat(v_cache)[rows].float().repeat_interleave(group, 1).transpose(0, 1)
    scores = torch.matmul(q.float().transpose(0, 1), k.transpose(1, 2)) * scale  # [H, L, S]
    if talk is not None:
        scores = torch.matmul(talk, scores.flatten(1)).view_as(scores)
    if cap is not None:
        scores = cap * torch.tanh(scores / cap)
    i = torch.arange(ctx_len, ctx_len + L, device=q.device).view(-1, 1)
    if bias is not None:
        scores = scores + bias[:, (i - j).clamp(0, bias.shape[1] - 1)]
    hidden = j > i
    if window is not None:
        hidden |= ((i - j) >= window) & (j >= keep_first)
    if chunk is not None:
        hidden |= (i // chunk) != (j // chunk)
    scores = scores.masked_fill(hidden, float("-inf"))
    if sigmoid:
        probs = torch.sigmoid(scores)
    else:
        probs = _sink_softmax(scores, None if sink is None else sink.view(H, 1, 1))
    return torch.matmul(probs, v).transpose(0, 1)


def grouped_attention(q, k_cache, v_cache, batch, scale: float, cap, window, keep_first: int,
                      sink, out, bias=None, sigmoid=False, gate=None, chunk=None, talk=None):
    for row, n, ctx, _, pages in _portions(batch):
        y = _grouped_attention_seq(
            q[row : row + n], k_cache, v_cache, pages, ctx, scale, cap, window, keep_first, sink,
            bias, sigmoid, chunk, talk,
        )
        if gate is not None:
            y = y * torch.sigmoid(gate[row : row + n].float()).unsqueeze(-1)
        out[row : row + n] = y


# -------------------------------------------------------------------- experts


def moe_route(h, router, bias, top: int, sigmoid=False, scale=1.0):
    z = torch.matmul(h.float(), router.float().t())
    s = torch.sigmoid(z) if sigmoid else z
    best = torch.topk(s if bias is None else s + bias, top, -1)
    if not sigmoid:
        return best.indices.int(), scale * torch.softmax(best.values, -1)
    w = s.gather(-1, best.indices)
    return best.indices.int(), scale * w / (w.sum(-1, keepdim=True) + 1e-20)


def moe_experts(h, gate_up, down, ids, glu):
    N, k = ids.shape
    rows = torch.empty(N, k, down.shape[1], dtype=h.dtype, device=h.device)
    for e in range(gate_up.shape[0]):
        token, choice = (ids == e).nonzero(as_tuple=True)
        if len(token):
            x = torch.nn.functional.linear(h[token], gate_up[e])
            act = x.new_empty(len(token), down.shape[2])
            clamped_glu(x, glu.limit, glu.alpha, glu.offset, act, glu.cubic)
            rows[token, choice] = torch.nn.functional.linear(act, down[e])
    return rows


# ----------------------------------------------------------------- delta rule


def _gated_delta_seq(qkv, conv, b, z, A_log, dt_bias, gate, norm, eps, unit_eps, G, S, tail,
                     gate_silu):
    """One sequence's rows from state S [H, D, V] and convolution inputs tail
    [taps - 1, C]; returns the rows and S after them."""
    T, (H, D, V), taps = qkv.shape[0], S.shape, conv.shape[1]
    x = torch.cat([tail, qkv])
    y = sum(x[n : n + T].float() * conv[:, n].float() for n in range(taps))
    y = torch.nn.functional.silu(y).to(qkv.dtype).float()
    q, k, v = y.split([G * D, G * D, H * V], 1)

    def unit(t):
        t = t.reshape(T, G, D)
        t = t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) + unit_eps)
        return t.repeat_interleave(H // G, 1)

    q, k, v = unit(q) * D ** -0.5, unit(k), v.reshape(T, H, V)
    beta = torch.sigmoid(b.float())
    # one decay per head and channel, or one per head
    step = torch.nn.functional.softplus((z.float() + dt_bias).view(T, H, -1), threshold=40.0)
    g = torch.exp(-torch.exp(A_log).view(H, 1) * step)
    out = torch.empty(T, H, V, device=S.device)
    for t in range(T):
        S = g[t].unsqueeze(-1) * S
        u = beta[t].unsqueeze(-1) * (v[t] - torch.matmul(k[t].unsqueeze(1), S).squeeze(1))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out[t] = torch.matmul(q[t].unsqueeze(1), S).squeeze(1)
    out = out * torch.rsqrt(out.pow(2).mean(-1, keepdim=True) + eps) * norm
    gate = gate.float()
    gate = torch.nn.functional.silu(gate) if gate_silu else torch.sigmoid(gate)
    out = out.reshape(T, H * V) * gate
    return out.to(qkv.dtype), S


def gated_delta(qkv, conv, b, z, A_log, dt_bias, gate, norm, eps, unit_eps, kv_heads,
                state, conv_state, batch, gate_silu=False):
    out = torch.empty(gate.shape, dtype=qkv.dtype, device=qkv.device)
    runs, row, taps = [], 0, conv.shape[1]
    for m in batch.prefills:
        runs.append((row, m.query_len, m.state_slot, m.ctx_len))
        row += m.query_len
    for n in range(batch.num_decode):
        runs.append((row + n, 1, int(batch.decode_state_slots[n]),
                     int(batch.decode_seq_lens[n]) - 1))
    for row, n, slot, ctx in runs:
        r, ring = slice(row, row + n), conv_state[slot]
        S = state[slot] if ctx else torch.zeros_like(state[slot])
        tail = torch.zeros(taps - 1, qkv.shape[1], dtype=qkv.dtype, device=qkv.device)
        for i in range(1, min(taps - 1, ctx) + 1):  # the ring's entry of position p is p % taps
            tail[-i] = ring[(ctx - i) % taps]
        out[r], state[slot] = _gated_delta_seq(
            qkv[r], conv, b[r], z[r], A_log, dt_bias, gate[r], norm, eps, unit_eps, kv_heads,
            S, tail, gate_silu,
        )
        for i in range(max(0, n - taps), n):
            ring[(ctx + i) % taps] = qkv[row + i]
    return out


def softmax_sample(logits, temperatures, top_ks, top_ps, gen, mask=None,
                   uniforms=None, mask_map=None):
    """logits: [B, V] float; temperatures/top_ps: [B] float; top_ks: [B] long
    (0 = off); mask: [B, V] bool (True = allowed) or None; uniforms: [B]
    precomputed draws (per-request seeds) — inverse-CDF like the HIP kernel.
    Greedy when temperature == 0."""
    logits = logits.float().clone()
    B, V = logits.shape
    if mask is not None and mask_map is not None:
        # expand the compact [M, V] mask rows (hip kernel indirection)
        for i in range(B):
            mi = int(mask_map[i])
            if mi >= 0:
                logits[i].masked_fill_(~mask[mi], float("-inf"))
    elif mask is not None:
        logits.masked_fill_(~mask, float("-inf"))
    out = torch.empty(B, dtype=torch.long, device=logits.device)
    greedy = temperatures <= 0
    if greedy.any():
        out[greedy] = logits[greedy].argmax(-1)
    rows = (~greedy).nonzero(as_tuple=True)[0]
    for i in rows.tolist():
        row = logits[i] / temperatures[i]
        k = int(top_ks[i])
        if k > 0 and k < V:
            kth = torch.topk(row, k).values[-1]
            row[row < kth] = float("-inf")
        p = float(top_ps[i])
        if p < 1.0:
            sorted_logits, sorted_idx = torch.sort(row, descending=True)
            probs = torch.softmax(sorted_logits, dim=-1)
            cum = torch.cumsum(probs, dim=-1)
            cut = cum - probs > p  # keep tokens until cumulative prob exceeds p
            sorted_logits[cut] = float("-inf")
            row = torch.full_like(row, float("-inf"))
            row[sorted_idx] = sorted_logits
        probs = torch.softmax(row, dim=-1)
        if uniforms is not None:
            cdf = torch.cumsum(probs, dim=-1)
            out[i] = int(torch.searchsorted(cdf, uniforms[i].to(cdf) * cdf[-1]).clamp(max=probs.numel() - 1))
        else:
            out[i] = torch.multinomial(probs, 1, generator=gen).squeeze(-1)
    return out
