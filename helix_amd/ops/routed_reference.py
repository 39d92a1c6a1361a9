"""Pure-torch versions of the ops in helix_amd.ops.routed, for CPU tensors:
32-bit inside, the scan one token at a time."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from .gated import project32

LN2 = 0.6931471805599453


def _norm(u, norm, dtype):
    return (torch.tanh(norm.alpha * u) * norm.w + norm.b).to(dtype)


def _read(x, into):
    return torch.einsum("tsw,s->tw", x, into)


def hyper_embed(x, ids, positions, embed, places, into, norm):
    p = positions.clamp(0, places.shape[0] - 1)
    x.copy_((embed[ids].float() + places[p].float())[:, None, :])
    return _norm(_read(x, into), norm, embed.dtype)


def hyper_step(x, y, back, into, norm, tap):
    if isinstance(y, torch.Tensor):
        dtype, v = y.dtype, y.float()
    else:
        dtype, v = y.rows.dtype, gather_rows(y)
    x.copy_(torch.einsum("tsw,sq->tqw", x, back.mix)
            + back.out[:, None] * v[:, None, :])
    if tap is not None:
        tap.copy_(x.sum(1))
    return _norm(_read(x, into), norm, dtype)


def gather_rows(r):
    rows = r.rows.float()[r.slot.clamp(min=0).long()]
    rows = torch.where((r.slot < 0)[..., None], r.self.float()[:, None, :],
                       rows)
    return (rows * r.weight[..., None]).sum(1)


def softcap(x, cap):
    return x.div_(cap).tanh_().mul_(cap)


# ----------------------------------------------------------- mixture of experts

def choose_experts(z, correction, p):
    s = torch.softmax(z, -1)
    choice = s + correction
    if p.keep < p.groups:
        grouped = choice.unflatten(1, (p.groups, -1))
        best = grouped.amax(-1).topk(p.keep, dim=1).indices
        shut = torch.ones(z.shape[0], p.groups, dtype=torch.bool)
        shut.scatter_(1, best, False)
        choice = grouped.masked_fill(shut[..., None],
                                     float("-inf")).flatten(1)
    ids = choice.topk(p.top, dim=1).indices
    w = s.gather(1, ids)
    return ids.int(), w / (w.sum(1, keepdim=True) + 1e-20)


def expert_mixture(h, z, correction, ups, downs, p):
    from .routed import RoutedRows
    ids, weights = choose_experts(z, correction, p)
    T, K = ids.shape
    rows = torch.zeros(T * K, h.shape[1], dtype=h.dtype)
    slot = torch.arange(T * K, dtype=torch.int32).view(T, K)
    slot = torch.where(ids < p.experts, slot, -1)
    for e in ids.unique().tolist():
        if e < p.experts:
            t, k = torch.nonzero(ids == e, as_tuple=True)
            u = F.relu(F.linear(h[t].float(), ups[e].float())).square()
            u = u.to(h.dtype).float()
            rows[t * K + k] = F.linear(u, downs[e].float()).to(h.dtype)
    return RoutedRows(rows, slot, weights, h)


# --------------------------------------------------------------- selective scan

def selective_span(y, z, p, w, ring, state, slot, start):
    """Tokens of one sequence: z rows and y rows, first one at position
    `start`; slot < 0 leaves ring and state alone."""
    I, K, R, N = p.inner, p.taps, p.dt_rank, p.state
    T, live = z.shape[0], slot >= 0
    raw = z[:, p.x_at:p.x_at + I]
    before = torch.zeros(K - 1, I, dtype=z.dtype)
    if live:
        for k in range(K - 1):
            at = start - (K - 1) + k
            if at >= 0:
                before[k] = ring[slot, at % K]
    seen = torch.cat([before, raw]).float()
    x = w.conv_b + sum(w.conv[k] * seen[k:k + T] for k in range(K))
    x = F.silu(x).to(z.dtype)
    bc = project32(x, w.x)
    dt = project32(bc[:, :R].to(z.dtype), w.dt)
    dt = F.softplus(dt + w.dt_b, threshold=1e9)
    a = torch.exp(w.A[None] * LN2 * dt[:, None, :])         # [T, N, I]
    u = bc[:, p.b_at:p.b_at + N, None] * (dt * x.float())[:, None, :]
    c = bc[:, p.c_at:p.c_at + N, None]
    s = state[slot].clone() if live and start > 0 else torch.zeros(N, I)
    out = torch.empty(T, I)
    for t in range(T):
        s = a[t] * s + u[t]
        out[t] = (s * c[t]).sum(0)
    g = F.silu(z[:, p.z_at:p.z_at + I].float())
    y.copy_(((out + w.D * x.float()) * g).to(y.dtype))
    if live:
        state[slot] = s
        for t in range(max(0, T - K), T):
            ring[slot, (start + t) % K] = raw[t]
