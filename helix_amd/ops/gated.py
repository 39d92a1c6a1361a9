"""Ops of models with rotated paged attention (softmax or sigmoid weights),
linear attention (gated, or with a constant decay) and layer norms on both
sides of a sublayer. HIP
kernels in helix_amd._C_gated; CPU tensors run gated_reference."""
from __future__ import annotations

from dataclasses import dataclass
from typing import NamedTuple, Optional, Tuple

import torch

from . import build
from . import gated_reference as ref


def _native():
    return build.load("_C_gated")


# ----------------------------------------------------------- residual stream

class Norm(NamedTuple):
    """Weight and bias of a layer norm, fp32."""
    w: torch.Tensor
    b: torch.Tensor


def split_terms(x_like: torch.Tensor, dtype: torch.dtype):
    """Room for two bf16 terms of an fp32 [T, W] (the operand of project32),
    or None where fp32 itself is the operand."""
    if dtype == torch.float32:
        return None
    return torch.empty(2, *x_like.shape, dtype=dtype, device=x_like.device)


def _normed(x: torch.Tensor, norm: Optional[Norm], dtype):
    if norm is None:
        return None, None, None
    return (torch.empty(x.shape, dtype=dtype, device=x.device), norm.w,
            norm.b)


def stream_add(x: torch.Tensor, y: torch.Tensor, post: Norm,
               norm: Optional[Norm], eps: float, terms=None,
               tap: Optional[torch.Tensor] = None):
    """x (fp32, in place) <- x + post(y), also to tap and (two terms of it)
    to terms. Returns norm(x) in y's dtype."""
    if not x.is_cuda:
        return ref.stream_add(x, y, post, norm, eps, terms, tap)
    h, w, b = _normed(x, norm, y.dtype)
    _native().stream_add(h, x, y, post.w, post.b, w, b, eps, x, tap, terms)
    return h


def stream_embed(x: torch.Tensor, ids: torch.Tensor, embed: torch.Tensor,
                 scale: float, norm: Optional[Norm], eps: float, terms=None):
    """x (fp32, written) <- scale * embed[ids], two terms of it to terms.
    Returns norm(x) in embed's dtype."""
    if not x.is_cuda:
        return ref.stream_embed(x, ids, embed, scale, norm, eps, terms)
    h, w, b = _normed(x, norm, embed.dtype)
    _native().stream_embed(h, ids, embed, scale, w, b, eps, x, terms)
    return h


def project32(a: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """a [n, K] times w [N, K] transposed, accumulated and left in fp32."""
    if not a.is_cuda or a.dtype == torch.float32:
        return a.float() @ w.float().t()
    return torch.mm(a, w.t(), out_dtype=torch.float32)


def stream_enter(x: torch.Tensor, terms, w_x: torch.Tensor, e: torch.Tensor,
                 e_scale: float, step: Optional[torch.Tensor], norm: Norm,
                 eps: float, dtype: torch.dtype):
    """x (fp32, in place) <- x w_x^T + e_scale * e + step; x itself enters
    the product as its two terms, if given. Returns norm(x) in dtype."""
    if terms is None:
        a, a2 = project32(x, w_x), None
    else:
        a, a2 = project32(terms.flatten(0, 1), w_x).view(
            2, *x.shape).unbind(0)
    if not x.is_cuda:
        return ref.stream_enter(x, a, a2, e, e_scale, step, norm, eps, dtype)
    h = torch.empty(x.shape, dtype=dtype, device=x.device)
    _native().stream_enter(h, a, a2, e, e_scale, step, norm.w, norm.b, eps, x)
    return h


def gated_mul(z: torch.Tensor, up_at: int, size: int,
              act: str = "gelu_tanh") -> torch.Tensor:
    """act(z[:, :size]) * z[:, up_at:up_at + size]."""
    if act not in ("gelu_tanh", "silu"):
        raise ValueError(f"activation {act!r}")
    if not z.is_cuda:
        return ref.gated_mul(z, up_at, size, act)
    out = torch.empty(z.shape[0], size, dtype=z.dtype, device=z.device)
    _native().gated_mul(out, z, up_at, act == "gelu_tanh")
    return out


# ------------------------------------------------------------------ attention

def rotary_table(positions: torch.Tensor,
                 freqs: torch.Tensor) -> torch.Tensor:
    """[T, n, 2] fp32: cosine and sine of every position times each of the n
    (float64) frequencies."""
    if not positions.is_cuda:
        return ref.rotary_table(positions, freqs)
    cs = torch.empty(positions.shape[0], freqs.shape[0], 2,
                     dtype=torch.float32, device=positions.device)
    _native().rotary_table(cs, positions, freqs)
    return cs


def query_temperature(positions: torch.Tensor, coef: float,
                      every: float) -> torch.Tensor:
    """[T] fp32, a query's factor at position p:
    1 + coef * ln(floor((p + 1) / every) + 1)."""
    if not positions.is_cuda:
        return ref.query_temperature(positions, coef, every)
    out = torch.empty(positions.shape[0], dtype=torch.float32,
                      device=positions.device)
    _native().query_temperature(out, positions, coef, every)
    return out


@dataclass
class AttnParams:
    """One attention layer and its columns in the fused projection z. Keys
    are cached in dim_pad columns. v_at == k_at: values are the unrotated
    keys; both negative: the layer has none and reads another's. sigmoid: weights are sigmoids of the scores (temp and bias per
    head) instead of a softmax."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    dim_pad: int
    q_at: int
    k_at: int
    v_at: int
    scale: float
    out_scale: float = 1.0
    sigmoid: bool = False
    temp: Optional[torch.Tensor] = None       # [H] fp32
    bias: Optional[torch.Tensor] = None       # [H] fp32


def attn_epilogue(z: torch.Tensor, p: AttnParams, kv_cache,
                  slots: torch.Tensor, cs: Optional[torch.Tensor] = None,
                  vcs: Optional[torch.Tensor] = None,
                  q_norm: Optional[torch.Tensor] = None,
                  k_norm: Optional[torch.Tensor] = None,
                  eps: float = 0.0) -> torch.Tensor:
    """Norms (over all of q, all of k) and rotation; keys and values, if the
    layer has any, go to the cache slots (nothing where negative). cs, vcs:
    rotary_table of the keys' rotation and of the values'. Returns q [T, H,
    dim_pad]: columns of z where nothing happens to them."""
    if z.is_cuda and cs is None and q_norm is None and \
            p.dim == p.dim_pad and p.q_at % 8 == 0 and z.stride(0) % 8 == 0 \
            and z.data_ptr() % 16 == 0:
        q = z[:, p.q_at:p.q_at + p.heads * p.dim].unflatten(1, (p.heads,
                                                                p.dim))
        made = None
    else:
        q = made = torch.empty(z.shape[0], p.heads, p.dim_pad, dtype=z.dtype,
                               device=z.device)
    if z.is_cuda:
        if made is not None or p.k_at >= 0:
            _native().attn_epilogue(made, *kv_cache, z, p.q_at, p.k_at,
                                    p.v_at, p.heads, p.dim, slots, cs, vcs,
                                    q_norm, k_norm, eps, p.k_at >= 0)
    else:
        ref.attn_epilogue(q, *kv_cache, z, p, slots, cs, vcs, q_norm, k_norm,
                          eps)
    return q


# Keys of a partition at least (every wave has a tile); workgroups that fill
# the chip.
ATTN_PART = 128
ATTN_TARGET_WGS = 512


def attn_parts(rows: int, p: AttnParams, keys: int) -> int:
    """Key partitions per row of the MFMA row kernel."""
    groups = p.kv_heads * -(-(p.heads // p.kv_heads) // 16)
    return max(1, min(-(-keys // ATTN_PART),
                      ATTN_TARGET_WGS // max(1, rows * groups)))


def attn_scratch_floats(rows: int, p: AttnParams, keys: int) -> int:
    parts = attn_parts(rows, p, keys)
    return 0 if parts == 1 else rows * parts * p.heads * (p.vdim + 2)


def attn_rows(out: torch.Tensor, q: torch.Tensor, p: AttnParams, kv_cache,
              block_tables: torch.Tensor, row_len: torch.Tensor,
              max_len: int, vcs: Optional[torch.Tensor] = None,
              row_seq: Optional[torch.Tensor] = None,
              workspace: Optional[torch.Tensor] = None,
              row_scale: Optional[torch.Tensor] = None,
              gate: Optional[torch.Tensor] = None) -> None:
    """out [R, H*E] <- attention of single query rows: row r sees the first
    row_len[r] cached tokens of table row row_seq[r] (r if None). vcs: where
    values were cached turned, the rows' own table to turn results back.
    row_scale [R] fp32: a factor on all scores of a row. gate [R, H*E]: the
    result is multiplied by its sigmoid."""
    if not q.is_cuda:
        ref.attn_rows(out, q, p, *kv_cache, block_tables, row_len, vcs,
                      row_seq, row_scale, gate)
        return
    C, R = _native(), q.shape[0]
    k, v = kv_cache
    if not C.attn_fits(q, p.vdim):
        C.attn_plain(out, q, k, v, block_tables, row_seq, row_len, p.scale,
                     p.out_scale, p.sigmoid, p.temp, p.bias, vcs, row_scale,
                     gate)
        return
    parts = attn_parts(R, p, max_len)
    if parts == 1:
        C.attn_rows(out, None, None, q, k, v, block_tables, row_seq, row_len,
                    p.scale, p.out_scale, p.sigmoid, p.temp, p.bias, vcs,
                    row_scale, gate)
        return
    need = attn_scratch_floats(R, p, max_len)
    if workspace is None or workspace.numel() < need:
        workspace = torch.empty(need, dtype=torch.float32, device=q.device)
    n = R * parts * p.heads
    ml = workspace[:2 * n]
    part = workspace[2 * n:need].view(R, parts, p.heads, p.vdim)
    C.attn_rows(None, part, ml, q, k, v, block_tables, row_seq, row_len,
                p.scale, p.out_scale, p.sigmoid, p.temp, p.bias, None,
                row_scale, None)
    C.attn_merge(out, part, ml, p.out_scale, p.sigmoid, vcs, gate)


# Prompt portions up to this many rows per sequence run as single rows.
ATTN_ROWS_PER_SEQ = 16


def attn_prompt(out: torch.Tensor, q: torch.Tensor, p: AttnParams, kv_cache,
                meta, vcs: Optional[torch.Tensor] = None,
                row_scale: Optional[torch.Tensor] = None,
                gate: Optional[torch.Tensor] = None) -> None:
    """The same for prompt portions (meta: PrefillMeta): 128 queries of a
    head at a time on MFMA; short portions, fp32 and oversized heads run as
    rows."""
    T, B = q.shape[0], meta.cu_seqlens.shape[0] - 1
    if not q.is_cuda or T <= ATTN_ROWS_PER_SEQ * B or \
            not _native().attn_fits(q, p.vdim):
        attn_rows(out, q, p, kv_cache, meta.block_tables, meta.row_len,
                  meta.max_len, vcs, meta.row_seq, row_scale=row_scale,
                  gate=gate)
        return
    _native().attn_prompt(out, q, *kv_cache, meta.block_tables,
                          meta.cu_seqlens, meta.seq_lens, meta.max_seqlen,
                          p.scale, p.out_scale, p.sigmoid, p.temp, p.bias,
                          vcs, row_scale, gate)


# ------------------------------------------------------ gated linear attention

@dataclass
class GLAParams:
    """One gated linear attention layer and its columns in the fused
    projection z: q and k (heads * dim), v and g (heads * vdim), a1 (rank)."""
    heads: int
    dim: int
    vdim: int
    rank: int
    q_at: int
    k_at: int
    v_at: int
    g_at: int
    a_at: int
    tau: float
    eps: float
    out_scale: float = 1.0

    @property
    def q_scale(self) -> float:
        return self.dim ** -0.5

    @property
    def columns(self) -> Tuple[int, ...]:
        return self.q_at, self.k_at, self.v_at, self.g_at, self.a_at


@dataclass
class GLAWeights:
    """a2 [heads * dim, rank padded to 32] in the storage type; fp32: a2_b,
    norm [vdim]."""
    a2: torch.Tensor
    a2_b: torch.Tensor
    norm: torch.Tensor


# Tokens of a chunk of the MFMA prompt kernels.
GLA_CHUNK = 64


def _gla_step(y, z, p: GLAParams, w: GLAWeights, state, slots, positions,
              cu=None):
    _native().gla_step(y, z, *p.columns, p.vdim, p.rank, w.a2, w.a2_b, w.norm,
                       p.tau,
                       p.q_scale, p.out_scale, p.eps, state, slots,
                       positions, cu)


def gla_step(y: torch.Tensor, z: torch.Tensor, p: GLAParams, w: GLAWeights,
             state: torch.Tensor, state_slots: torch.Tensor,
             positions: torch.Tensor) -> None:
    """y [R, heads*vdim] <- normed and gated output of single tokens, each of
    its own sequence. state [slots, heads, dim, vdim padded to 4] fp32 is
    updated in place; position 0 starts from zeros whatever the slot holds,
    a negative slot reads and writes no state."""
    if z.is_cuda:
        _gla_step(y, z, p, w, state, state_slots, positions)
        return
    for r in range(z.shape[0]):
        ref.gla_span(y[r:r + 1], z[r:r + 1], p, w, state,
                     int(state_slots[r]), int(positions[r]))


def gla_prompt(y: torch.Tensor, z: torch.Tensor, p: GLAParams, w: GLAWeights,
               state: torch.Tensor, meta) -> None:
    """The same for prompt portions (meta: PrefillMeta). bf16 runs chunks of
    the dual (attention-like) form on MFMA, fp32 the recurrence itself."""
    if not z.is_cuda:
        cu = meta.cu_seqlens.tolist()
        for b in range(len(cu) - 1):
            s = slice(cu[b], cu[b + 1])
            ref.gla_span(y[s], z[s], p, w, state, int(meta.state_slots[b]),
                         int(meta.positions[cu[b]]))
        return
    if not _native().gla_chunks_fit(z, p.dim):
        _gla_step(y, z, p, w, state, meta.state_slots, meta.positions,
                  meta.cu_seqlens)
        return
    for step in gla_chunk_steps(y, z, p, w, state, meta):
        step()


def _chunk_operands(n: int, p, z: torch.Tensor):
    """Room for the operands of n chunks of p.heads heads."""
    H, L, dev = p.heads, GLA_CHUNK, z.device
    Dp, Pp = -(-p.dim // 32) * 32, -(-p.vdim // 16) * 16
    return (torch.empty(n, H, 2, L, Dp, dtype=z.dtype, device=dev),
            torch.empty(n, H, 2, Dp, L, dtype=z.dtype, device=dev),
            torch.empty(n, H, 2, L, L, dtype=z.dtype, device=dev),
            torch.empty(n, H, Pp, L, dtype=z.dtype, device=dev),
            torch.empty(n, H, Dp, dtype=torch.float32, device=dev))


def gla_chunk_steps(y, z, p: GLAParams, w: GLAWeights, state, meta):
    """The three launches of a prompt in chunks: operands, recurrence, norm
    and gate."""
    ch, C, H = meta.chunks(GLA_CHUNK), _native(), p.heads
    qe, ke, am, vt, ec = _chunk_operands(ch.seq.shape[0], p, z)
    o = torch.empty(z.shape[0], H * p.vdim, dtype=z.dtype, device=z.device)

    def operands():
        C.gla_operands(qe, ke, am, vt, ec, z, p.q_at, p.k_at, p.v_at, p.a_at,
                       p.dim, p.vdim, p.rank, w.a2, w.a2_b, p.tau, p.q_scale,
                       ch.row, ch.count)

    def recurrence():
        C.gla_chunks(o, qe, ke, am, vt, ec, p.vdim, state, meta.state_slots,
                     meta.positions, meta.cu_seqlens, ch.first)

    def norm_gate():
        C.head_norm_gate(y, o, z[:, p.g_at:p.g_at + H * p.vdim], w.norm,
                         p.out_scale, p.eps)

    return operands, recurrence, norm_gate


# --------------------------------------- linear attention, a decay per head

@dataclass
class DecayParams:
    """One linear attention layer with constant decays and its columns in the
    fused projection z: q and k (heads * dim), v and g (heads * vdim)."""
    heads: int
    dim: int
    vdim: int
    q_at: int
    k_at: int
    v_at: int
    g_at: int
    eps: float


class DecayWeights(NamedTuple):
    """fp32: decay and its base-2 logarithm [heads], norm [heads * vdim]."""
    decay: torch.Tensor
    log_decay: torch.Tensor
    norm: torch.Tensor


def _decay_step(y, z, p: DecayParams, w: DecayWeights, state, slots,
                positions, cu=None):
    """Token by token; y <- normed and gated outputs."""
    C = _native()
    o = torch.empty(z.shape[0], p.heads * p.vdim, dtype=z.dtype,
                    device=z.device)
    C.decay_step(o, z, p.q_at, p.k_at, p.v_at, p.vdim, w.decay, state, slots,
                 positions, cu)
    C.row_norm_gate(y, o, _decay_gate(z, p), w.norm, p.eps)


def _decay_gate(z, p: DecayParams):
    return z[:, p.g_at:p.g_at + p.heads * p.vdim]


def decay_step(y: torch.Tensor, z: torch.Tensor, p: DecayParams,
               w: DecayWeights, state: torch.Tensor,
               state_slots: torch.Tensor, positions: torch.Tensor) -> None:
    """S <- decay S + silu(k) silu(v)^T, o = S^T silu(q) per head for single
    tokens, each of its own sequence; y [R, heads*vdim] <- all heads' o
    RMS-normed together, times sigmoid(g). The state is gla_step's."""
    if z.is_cuda:
        _decay_step(y, z, p, w, state, state_slots, positions)
        return
    for r in range(z.shape[0]):
        ref.decay_span(y[r:r + 1], z[r:r + 1], p, w, state,
                       int(state_slots[r]), int(positions[r]))


def decay_prompt(y: torch.Tensor, z: torch.Tensor, p: DecayParams,
                 w: DecayWeights, state: torch.Tensor, meta) -> None:
    """The same for prompt portions (meta: PrefillMeta). bf16 runs chunks of
    the dual form on MFMA, fp32 the recurrence itself."""
    if not z.is_cuda:
        cu = meta.cu_seqlens.tolist()
        for b in range(len(cu) - 1):
            s = slice(cu[b], cu[b + 1])
            ref.decay_span(y[s], z[s], p, w, state, int(meta.state_slots[b]),
                           int(meta.positions[cu[b]]))
        return
    if not _native().gla_chunks_fit(z, p.dim):
        _decay_step(y, z, p, w, state, meta.state_slots, meta.positions,
                    meta.cu_seqlens)
        return
    for step in decay_chunk_steps(y, z, p, w, state, meta):
        step()


def decay_chunk_steps(y, z, p: DecayParams, w: DecayWeights, state, meta):
    """The three launches of a prompt in chunks: operands, recurrence, norm
    and gate."""
    ch, C = meta.chunks(GLA_CHUNK), _native()
    ops = _chunk_operands(ch.seq.shape[0], p, z)
    o = torch.empty(z.shape[0], p.heads * p.vdim, dtype=z.dtype,
                    device=z.device)

    def operands():
        C.decay_operands(*ops, z, p.q_at, p.k_at, p.v_at, p.dim, p.vdim,
                         w.log_decay, ch.row, ch.count)

    def recurrence():
        C.gla_chunks(o, *ops, p.vdim, state, meta.state_slots,
                     meta.positions, meta.cu_seqlens, ch.first)

    def norm_gate():
        C.row_norm_gate(y, o, _decay_gate(z, p), w.norm, p.eps)

    return operands, recurrence, norm_gate
