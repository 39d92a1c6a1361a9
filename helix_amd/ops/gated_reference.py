"""Pure-torch versions of the ops in helix_amd.ops.gated, for CPU tensors:
one row or token at a time, 32-bit inside."""
from __future__ import annotations

import torch
import torch.nn.functional as F


def _norm(v, norm, eps):
    return F.layer_norm(v, v.shape[-1:], norm.w, norm.b, eps)


def _split(v, terms):
    if terms is not None:
        terms[0] = v
        terms[1] = v - terms[0].float()


def stream_add(x, y, post, norm, eps, terms, tap):
    x += _norm(y.float(), post, eps)
    if tap is not None:
        tap.copy_(x)
    _split(x, terms)
    return None if norm is None else _norm(x, norm, eps).to(y.dtype)


def stream_embed(x, ids, embed, scale, norm, eps, terms):
    x.copy_(embed[ids].float() * scale)
    _split(x, terms)
    return None if norm is None else _norm(x, norm, eps).to(embed.dtype)


def stream_enter(x, a, a2, e, e_scale, step, norm, eps, dtype):
    v = a if a2 is None else a + a2
    v = v + e_scale * e
    x.copy_(v if step is None else v + step)
    return _norm(x, norm, eps).to(dtype)


def gated_mul(z, up_at, size, act):
    g = z[:, :size].float()
    g = F.silu(g) if act == "silu" else F.gelu(g, approximate="tanh")
    return (g * z[:, up_at:up_at + size].float()).to(z.dtype)


# ------------------------------------------------------------------ attention

def rotary_table(positions, freqs):
    a = positions.double()[:, None] * freqs
    return torch.stack([torch.cos(a), torch.sin(a)], -1).float()


def query_temperature(positions, coef, every):
    n = torch.floor((positions + 1).double() / every) + 1
    return (1 + coef * torch.log(n)).float()


def _turn(v, cs):
    """v [T, heads, D]: pairs (i, i + n) by table cs [T, n, 2]."""
    if cs is None:
        return v
    n = cs.shape[1]
    c, s = cs[:, None, :, 0], cs[:, None, :, 1]
    a, b = v[..., :n], v[..., n:2 * n]
    return torch.cat([a * c - b * s, b * c + a * s, v[..., 2 * n:]], -1)


def attn_epilogue(q, kc, vc, z, p, slots, cs, vcs, q_norm, k_norm, eps):
    def part(at, heads, size, w=None):
        v = z[:, at:at + heads * size].float()
        if w is not None:
            v = F.rms_norm(v, v.shape[-1:], w, eps)
        return v.unflatten(1, (heads, size))

    q.zero_()
    q[..., :p.dim] = _turn(part(p.q_at, p.heads, p.dim, q_norm), cs)
    if p.k_at < 0:
        return
    k = F.pad(_turn(part(p.k_at, p.kv_heads, p.dim, k_norm), cs),
              (0, p.dim_pad - p.dim))
    v = _turn(part(p.v_at, p.kv_heads, p.vdim), vcs)
    bs = kc.shape[2]
    live = slots >= 0
    s = slots[live]
    kc[s // bs, :, s % bs] = k[live].to(kc.dtype)
    vc[s // bs, :, :, s % bs] = v[live].to(vc.dtype)


def attn_rows(out, q, p, kc, vc, block_tables, row_len, vcs, row_seq,
              row_scale, gate):
    bs, per = kc.shape[2], p.heads // p.kv_heads
    for r in range(q.shape[0]):
        n = int(row_len[r])
        seq = r if row_seq is None else int(row_seq[r])
        pages = block_tables[seq, :(n + bs - 1) // bs].long()
        k = kc[pages].transpose(0, 1).flatten(1, 2)[:, :n].float()
        v = vc[pages].permute(1, 2, 0, 3).flatten(2)[..., :n].float()
        s = torch.matmul(k.repeat_interleave(per, 0),
                         q[r].float()[:, :, None])[..., 0] * p.scale
        if row_scale is not None:
            s = s * row_scale[r]
        if p.temp is not None:
            s = s * p.temp[:, None]
        if p.bias is not None:
            s = s + p.bias[:, None]
        w = torch.sigmoid(s) if p.sigmoid else torch.softmax(s, -1)
        o = torch.matmul(v.repeat_interleave(per, 0), w[:, :, None])[..., 0]
        if vcs is not None:
            back = vcs[r:r + 1] * torch.tensor([1.0, -1.0])
            o = _turn(o[None], back)[0]
        o = (p.out_scale * o).reshape(-1)
        if gate is not None:
            o = o * torch.sigmoid(gate[r].float())
        out[r] = o.to(out.dtype)


# ------------------------------------------------------ gated linear attention

def gla_span(y, z, p, w, state, slot, start):
    """Tokens of one sequence: z rows and y rows, first one at position
    `start`; slot < 0 leaves the state alone."""
    H, D, E = p.heads, p.dim, p.vdim
    live = slot >= 0
    keep = state[slot, ..., :E].clone() if live and start > 0 else \
        torch.zeros(H, D, E)
    for t in range(z.shape[0]):
        row = z[t].float()
        q, k = (row[at:at + H * D].view(H, D) for at in (p.q_at, p.k_at))
        v, g = (row[at:at + H * E].view(H, E) for at in (p.v_at, p.g_at))
        a = w.a2[:, :p.rank].float() @ row[p.a_at:p.a_at + p.rank] + w.a2_b
        a = torch.exp(F.logsigmoid(a) / p.tau).view(H, D)
        keep = a[:, :, None] * keep + k[:, :, None] * v[:, None, :]
        o = (keep * (q * p.q_scale)[:, :, None]).sum(1)
        o = F.rms_norm(o, (E,), w.norm, p.eps) * F.silu(g)
        y[t] = (p.out_scale * o).reshape(-1).to(y.dtype)
    if live:
        state[slot, ..., :E] = keep


# --------------------------------------- linear attention, a decay per head

def decay_span(y, z, p, w, state, slot, start):
    """Tokens of one sequence, as gla_span."""
    H, D, E = p.heads, p.dim, p.vdim
    live = slot >= 0
    keep = state[slot, ..., :E].clone() if live and start > 0 else \
        torch.zeros(H, D, E)

    def part(at, size):
        v = F.silu(z[:, at:at + H * size].float()).to(z.dtype)
        return v.float().unflatten(1, (H, size))

    q, k, v = part(p.q_at, D), part(p.k_at, D), part(p.v_at, E)
    a = w.decay[:, None, None]
    o = torch.empty(z.shape[0], H * E)
    for t in range(z.shape[0]):
        keep = a * keep + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (keep * q[t][:, :, None]).sum(1).reshape(-1)
    g = z[:, p.g_at:p.g_at + H * E].float()
    o = F.rms_norm(o.to(z.dtype).float(), (H * E,), w.norm, p.eps)
    y.copy_((o * torch.sigmoid(g)).to(y.dtype))
    if live:
        state[slot, ..., :E] = keep
