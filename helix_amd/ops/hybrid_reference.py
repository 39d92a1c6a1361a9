"""Pure-torch versions of the ops in helix_amd.ops.hybrid, for CPU tensors:
one row or token at a time, 32-bit inside."""
from __future__ import annotations

import torch

from helix_amd.ops.reference import _rms_inv


def residual_norm(x, y, ls, mult, ids, embed, step, w, eps, x_out, tap,
                  dtype):
    v = x + mult * (ls * y.float()) if x is not None else None
    if tap is not None:
        tap.copy_(v)
    if ids is not None:
        e = embed[ids].float()
        v = e if v is None else v + e
    if step is not None:
        v = v + step
    if x_out is not None:
        x_out.copy_(v)
    return (v * _rms_inv(v, eps) * w).to(dtype)


def silu_mul(z, up_at, F):
    g = z[:, :F].float()
    return (torch.nn.functional.silu(g)
            * z[:, up_at:up_at + F].float()).to(z.dtype)


def group_rms_norm(y, groups, w, eps):
    v = y.float().view(y.shape[0], groups, -1)
    return ((v * _rms_inv(v, eps)).flatten(1) * w).to(y.dtype)


# ------------------------------------------------------------ latent attention

def _rotate(v, positions, p):
    """v [..., T, n] float: pairs (2i, 2i+1) of the first 2 * len(freqs)."""
    n = 2 * p.freqs.numel()
    a = positions.double()[:, None] * p.freqs
    c, s = (p.amp * f(a).float() for f in (torch.cos, torch.sin))
    u, w = v[..., 0:n:2], v[..., 1:n:2]
    out = v.clone()
    out[..., 0:n:2] = u * c - w * s
    out[..., 1:n:2] = w * c + u * s
    return out


def latent_epilogue(z, p, positions, norm_w, eps, cache, slots):
    T = z.shape[0]
    q = p.q_view(z)                                       # [T, H, Dq + Rp]
    if p.freqs is not None and p.rot_dim:
        rot = q[..., p.dim_pad:p.dim_pad + p.rot_dim].float().transpose(0, 1)
        q[..., p.dim_pad:p.dim_pad + p.rot_dim] = _rotate(
            rot, positions, p).transpose(0, 1).to(z.dtype)
    kv = z[:, p.kv_at:p.kv_at + p.rank_pad + p.rot_pad]
    row = torch.zeros(T, p.row, dtype=torch.float32)
    c = kv[:, :p.rank].float()
    row[:, :p.rank] = c * _rms_inv(c, eps) * norm_w
    kr = kv[:, p.rank_pad:p.rank_pad + p.rot_dim].float()
    if p.freqs is not None and p.rot_dim:
        kr = _rotate(kr, positions, p)
    row[:, p.rank_pad:p.rank_pad + p.rot_dim] = kr
    bs = cache.shape[2]
    live = slots >= 0
    s = slots[live]
    cache[s // bs, 0, s % bs] = row[live].to(cache.dtype)


def latent_attn_rows(out, z, p, cache, block_tables, row_len, uk, uv, gate,
                     row_seq=None):
    bs = cache.shape[2]
    q = p.q_view(z)
    H, E = p.heads, p.vdim
    ukh = uk.float().view(H, p.dim_pad, p.rank_pad)
    uvh = uv.float().view(H, E, p.rank_pad)
    for r in range(q.shape[0]):
        n = int(row_len[r])
        lo = max(0, n - p.window) if p.window else 0
        b0, b1 = lo // bs, (n + bs - 1) // bs
        seq = r if row_seq is None else int(row_seq[r])
        rows = cache[block_tables[seq, b0:b1].long(), 0].flatten(0, 1)
        rows = rows[lo - b0 * bs:n - b0 * bs].float()
        qr = q[r].float()
        ql = torch.einsum("hd,hdk->hk", qr[:, :p.dim_pad], ukh)
        s = ql @ rows[:, :p.rank_pad].T
        s = s + qr[:, p.dim_pad:] @ rows[:, p.rank_pad:].T
        w = torch.softmax(s * p.scale, -1)
        o = torch.einsum("hk,hek->he", w @ rows[:, :p.rank_pad], uvh)
        if gate is not None:
            o = o * torch.sigmoid(gate[r].float())[:, None]
        out[r] = o.reshape(-1).to(out.dtype)


# ----------------------------------------------------------- state-space mixer

def ssm_span(y, z, p, conv_state, state, slot, start, w):
    """Tokens of one sequence: z rows and y rows, first one at position
    `start`; slot < 0 leaves the state alone."""
    H, P, N, G = p.heads, p.vdim, p.state, p.groups
    taps = p.conv
    live = slot >= 0
    keep = state[slot].clone() if live and start > 0 else \
        torch.zeros(H, N, P, dtype=torch.float32)
    ring = conv_state[slot] if live else torch.zeros_like(conv_state[0])
    decay = -torch.exp(w.A_log)
    for t in range(z.shape[0]):
        pos = start + t
        row = z[t].float()
        ring[pos % taps] = z[t, p.xbc_at:p.xbc_at + p.channels]
        acc = w.conv_b.clone()
        for k in range(taps):
            if pos - k >= 0:
                acc += w.conv[:, taps - 1 - k] * ring[(pos - k) % taps]
        xbc = torch.nn.functional.silu(acc).to(z.dtype).float()
        x, B, C = xbc.split([H * P, G * N, G * N])
        x = x.view(H, P)
        B, C = (v.view(G, N).repeat_interleave(H // G, 0) for v in (B, C))
        dt = torch.nn.functional.softplus(
            row[p.dt_at:p.dt_at + H] + w.dt_bias, threshold=1e9)
        keep = torch.exp(decay * dt)[:, None, None] * keep + \
            dt[:, None, None] * B[:, :, None] * x[:, None, :]
        o = torch.einsum("hnp,hn->hp", keep, C) + w.D[:, None] * x
        gate = row[p.z_at:p.z_at + H * P].view(H, P)
        y[t] = (o * torch.nn.functional.silu(gate)).reshape(-1).to(y.dtype)
    if live:
        state[slot] = keep
