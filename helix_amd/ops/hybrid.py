"""Ops of hybrid models: latent attention over a paged latent cache,
state-space (Mamba-2) mixers over per-sequence state, and the fp32 residual
stream of looped layers. HIP kernels in helix_amd._C_hybrid; CPU tensors run
hybrid_reference."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from . import build
from . import hybrid_reference as ref


def _native():
    return build.load("_C_hybrid")


# ----------------------------------------------------------- residual stream

def residual_norm(x: Optional[torch.Tensor], y: Optional[torch.Tensor],
                  ls: Optional[torch.Tensor], mult: float, w: torch.Tensor,
                  eps: float, dtype: torch.dtype,
                  ids: Optional[torch.Tensor] = None,
                  embed: Optional[torch.Tensor] = None,
                  step: Optional[torch.Tensor] = None,
                  x_out: Optional[torch.Tensor] = None,
                  tap: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One pass over the fp32 stream x [T, W]:

        v = x + mult * (ls * y)      (v = 0 without x)
        tap <- v
        v += embed[ids], v += step   (each if given)
        x_out <- v                   (may be x)

    Returns v's RMS norm times w in `dtype`."""
    if w.is_cuda:
        T = ids.shape[0] if x is None else x.shape[0]
        h = torch.empty(T, w.shape[0], dtype=dtype, device=w.device)
        _native().residual_norm(h, x, y, ls, mult, ids, embed, step, w, eps,
                                x_out, tap)
        return h
    return ref.residual_norm(x, y, ls, mult, ids, embed, step, w, eps, x_out,
                             tap, dtype)


def silu_mul(z: torch.Tensor, up_at: int, size: int) -> torch.Tensor:
    """silu(z[:, :size]) * z[:, up_at:up_at + size]."""
    if z.is_cuda:
        out = torch.empty(z.shape[0], size, dtype=z.dtype, device=z.device)
        _native().silu_mul(out, z, up_at)
        return out
    return ref.silu_mul(z, up_at, size)


def group_rms_norm(y: torch.Tensor, groups: int, w: torch.Tensor,
                   eps: float) -> torch.Tensor:
    """RMS norm of every one of `groups` equal parts of the rows, times w."""
    if y.is_cuda:
        out = torch.empty_like(y)
        _native().group_rms_norm(out, y, groups, w, eps)
        return out
    return ref.group_rms_norm(y, groups, w, eps)


# ---------------------------------------------------------- latent attention

@dataclass
class LatentParams:
    """One latent-attention layer and its columns in the fused projection z.

    q_at: heads of [dim | rot_dim], padded to dim_pad and rot_pad columns;
    kv_at: [latent | shared key part], padded to rank_pad and rot_pad. The
    cache row has the kv layout. freqs: float64 [pairs], None = no rotation.
    """
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    rank: int
    dim_pad: int
    rot_pad: int
    rank_pad: int
    q_at: int
    kv_at: int
    scale: float
    window: int = 0                       # visible tokens (0 = all)
    freqs: Optional[torch.Tensor] = None
    amp: float = 1.0

    @property
    def row(self) -> int:
        return self.rank_pad + self.rot_pad

    @property
    def head_cols(self) -> int:
        return self.dim_pad + self.rot_pad

    def q_view(self, z: torch.Tensor) -> torch.Tensor:
        n = self.heads * self.head_cols
        return z[:, self.q_at:self.q_at + n].unflatten(
            1, (self.heads, self.head_cols))

    def max_keys(self, max_len: int) -> int:
        return min(max_len, self.window) if self.window else max_len


def latent_epilogue(z: torch.Tensor, p: LatentParams,
                    positions: torch.Tensor, norm_w: torch.Tensor,
                    eps: float, cache: torch.Tensor,
                    slots: torch.Tensor) -> None:
    """Rotates the queries in place in z, norms the latent, rotates the
    shared key part and writes both to the cache row of slots[t] (nothing
    where it is negative)."""
    if z.is_cuda:
        _native().latent_epilogue(
            z, p.q_at, p.heads, p.dim_pad, p.head_cols, p.kv_at, p.rank,
            p.rank_pad, p.rot_dim, p.freqs, p.amp, positions, norm_w, eps,
            cache, slots)
        return
    ref.latent_epilogue(z, p, positions, norm_w, eps, cache, slots)


# Cached rows of a partition at least; enough workgroups to fill the chip.
LATENT_PART = 64
LATENT_TARGET_WGS = 512


def latent_parts(rows: int, heads: int, keys: int) -> int:
    """Key partitions per row of the MFMA row kernel."""
    groups = -(-heads // 32)
    return max(1, min(-(-keys // LATENT_PART),
                      LATENT_TARGET_WGS // max(1, rows * groups)))


def latent_scratch_floats(rows: int, p: LatentParams, max_len: int) -> int:
    parts = latent_parts(rows, p.heads, p.max_keys(max_len))
    if parts == 1:
        return 0
    return rows * parts * p.heads * (p.rank_pad + 2)


def latent_attn_rows(out: torch.Tensor, z: torch.Tensor, p: LatentParams,
                     cache: torch.Tensor, block_tables: torch.Tensor,
                     row_len: torch.Tensor, max_len: int, uk: torch.Tensor,
                     ukt: torch.Tensor, uv: torch.Tensor,
                     gate: Optional[torch.Tensor] = None,
                     row_seq: Optional[torch.Tensor] = None,
                     workspace: Optional[torch.Tensor] = None) -> None:
    """out [R, H*E] <- attention of single query rows in latent space: row r
    reads the newest row_len[r] cached rows (its window of them) of table row
    row_seq[r] (r if None). uk [H*dim_pad, rank_pad], ukt its per-head
    transpose, uv [H*E, rank_pad]; gate: [R, H] logits."""
    if not z.is_cuda:
        ref.latent_attn_rows(out, z, p, cache, block_tables, row_len, uk, uv,
                             gate, row_seq)
        return
    R, H, dev = z.shape[0], p.heads, z.device
    C = _native()
    q = torch.empty(R, H, p.row, dtype=z.dtype, device=dev)
    C.latent_absorb(q, z, p.q_at, p.head_cols, p.dim_pad, uk, ukt,
                    p.rank_pad)
    o = torch.empty(R, H, p.rank_pad, dtype=z.dtype, device=dev)
    parts = latent_parts(R, H, p.max_keys(max_len))
    if not C.latent_rows_fits(q, p.rank_pad):
        C.latent_rows_plain(o, q, cache, block_tables, row_seq, row_len,
                            p.scale, p.window)
    elif parts == 1:
        C.latent_rows(o, None, None, q, cache, block_tables, row_seq,
                      row_len, p.rank_pad, p.scale, p.window)
    else:
        need = latent_scratch_floats(R, p, max_len)
        if workspace is None or workspace.numel() < need:
            workspace = torch.empty(need, dtype=torch.float32, device=dev)
        n = R * parts * H
        part = workspace[:n * p.rank_pad].view(R, parts, H, p.rank_pad)
        ml = workspace[n * p.rank_pad:need].view(R, parts, H, 2)
        C.latent_rows(None, part, ml, q, cache, block_tables, row_seq,
                      row_len, p.rank_pad, p.scale, p.window)
        C.latent_merge(o, part, ml)
    C.latent_out(out, o, uv, gate)


# Prompt portions up to this many rows per sequence run as single rows: they
# read the latents once, where spelling out keys and values of their whole
# context would cost more.
LATENT_ROWS_PER_SEQ = 16


def latent_attn_prompt(out: torch.Tensor, z: torch.Tensor, p: LatentParams,
                       cache: torch.Tensor, meta, uk: torch.Tensor,
                       ukt: torch.Tensor, uv: torch.Tensor,
                       gate: Optional[torch.Tensor] = None) -> None:
    """Prompt portions (meta: PrefillMeta). bf16 spells out keys and values
    of the visible context (two GEMMs, values transposed) for the MFMA
    kernel; short portions, fp32 and oversized heads run as rows."""
    T, B = z.shape[0], meta.cu_seqlens.shape[0] - 1
    if not z.is_cuda or T <= LATENT_ROWS_PER_SEQ * B or \
            not _native().latent_prompt_fits(z, p.dim_pad, p.rot_pad, p.vdim):
        latent_attn_rows(out, z, p, cache, meta.block_tables, meta.row_len,
                         meta.max_len, uk, ukt, uv, gate, meta.row_seq)
        return
    rows = cache.view(-1, p.row)
    for c in meta.context(p.window):
        lat = rows.index_select(0, c.slots)
        k = torch.nn.functional.linear(lat[:, :p.rank_pad], uk)
        v = torch.mm(uv, lat[:, :p.rank_pad].t())
        _native().latent_prompt(
            out, z, p.q_at, p.head_cols, p.heads, k, lat[:, p.rank_pad:], v,
            meta.cu_seqlens[c.first:c.last + 1], c.start, c.length,
            meta.max_seqlen, p.scale, p.window, gate)


# --------------------------------------------------------- state-space mixer

@dataclass
class SSMParams:
    """One Mamba-2 mixer and its columns in the fused projection z: gate
    (heads * vdim), [x | B | C] (channels), step sizes (heads)."""
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int                             # taps
    z_at: int
    xbc_at: int
    dt_at: int

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state


@dataclass
class SSMWeights:
    """fp32: conv [channels, taps] (last column = current token), conv_b,
    dt_bias, A_log and D per head."""
    conv: torch.Tensor
    conv_b: torch.Tensor
    dt_bias: torch.Tensor
    A_log: torch.Tensor
    D: torch.Tensor


# Tokens of a chunk of the MFMA prompt kernel.
SSM_CHUNK = 64


def ssm_step(y: torch.Tensor, z: torch.Tensor, p: SSMParams, w: SSMWeights,
             cache, state_slots: torch.Tensor,
             positions: torch.Tensor) -> None:
    """y [R, inner] <- gated output of single tokens, each of its own
    sequence, before the norm. cache = (conv ring [slots, taps, channels],
    state [slots, H, N, P] fp32), both updated in place; ring entry pos %
    taps holds the inputs of position pos. Position 0 starts from zeros,
    whatever the slot holds; a negative slot reads and writes no state."""
    ring, state = cache
    if z.is_cuda:
        _native().ssm_step(y, z, None, p.z_at, p.xbc_at, p.dt_at, w.conv,
                           w.conv_b, w.dt_bias, w.A_log, w.D, ring, state,
                           state_slots, positions, None)
        return
    for r in range(z.shape[0]):
        ref.ssm_span(y[r:r + 1], z[r:r + 1], p, ring, state,
                     int(state_slots[r]), int(positions[r]), w)


def ssm_prompt(y: torch.Tensor, z: torch.Tensor, p: SSMParams, w: SSMWeights,
               cache, meta) -> None:
    """The same for prompt portions (meta: PrefillMeta). bf16 runs chunks of
    the dual (attention-like) form on MFMA; fp32 and oversized states the
    recurrence itself."""
    ring, state = cache
    if not z.is_cuda:
        cu = meta.cu_seqlens.tolist()
        for b in range(len(cu) - 1):
            s = slice(cu[b], cu[b + 1])
            ref.ssm_span(y[s], z[s], p, ring, state,
                         int(meta.state_slots[b]),
                         int(meta.positions[cu[b]]), w)
        return
    C = _native()
    if not C.ssm_chunks_fit(z, p.vdim, p.state, p.conv):
        xbc = torch.empty(z.shape[0], p.channels, dtype=z.dtype,
                          device=z.device)
        C.conv_span(xbc, z, p.xbc_at, w.conv, w.conv_b, ring,
                    meta.state_slots, meta.positions, meta.cu_seqlens,
                    meta.max_seqlen)
        C.ssm_step(y, z, xbc, p.z_at, p.xbc_at, p.dt_at, w.conv, w.conv_b,
                   w.dt_bias, w.A_log, w.D, ring, state, meta.state_slots,
                   meta.positions, meta.cu_seqlens)
        return
    for step in ssm_chunk_steps(y, z, p, w, cache, meta):
        step()


def ssm_chunk_steps(y: torch.Tensor, z: torch.Tensor, p: SSMParams,
                    w: SSMWeights, cache, meta):
    """The two launches of a prompt in chunks: operands, then recurrence."""
    ring, state = cache
    ch, C = meta.chunks(SSM_CHUNK), _native()
    n, dev = ch.seq.shape[0], z.device
    Pp, Np = -(-p.vdim // 16) * 16, -(-p.state // 32) * 32
    xt = torch.empty(n, p.heads, Pp, SSM_CHUNK, dtype=z.dtype, device=dev)
    b = torch.empty(n, SSM_CHUNK, p.groups, Np, dtype=z.dtype, device=dev)
    c = torch.empty_like(b)
    bt = torch.empty(n, p.groups, Np, SSM_CHUNK, dtype=z.dtype, device=dev)
    da = torch.empty(n, p.heads, 3, SSM_CHUNK, dtype=torch.float32,
                     device=dev)

    def operands():
        C.conv_chunks(xt, b, bt, c, da, z, p.xbc_at, p.dt_at, p.vdim,
                      p.state, w.conv, w.conv_b, w.dt_bias, w.A_log, ring,
                      meta.state_slots, meta.positions, meta.cu_seqlens,
                      ch.seq, ch.row, ch.count)

    def recurrence():
        C.ssm_chunks(y, z, p.z_at, p.vdim, p.state, xt, b, bt, c, da, w.D,
                     state, meta.state_slots, meta.positions,
                     meta.cu_seqlens, ch.first)

    return operands, recurrence
