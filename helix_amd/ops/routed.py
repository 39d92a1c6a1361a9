"""Ops of models with several residual streams (hyper-connections), mixtures
of experts and selective scans. HIP kernels in helix_amd._C_routed; CPU
tensors run routed_reference."""
from __future__ import annotations

from dataclasses import dataclass
from typing import NamedTuple, Optional, Union

import torch

from . import build
from . import routed_reference as ref
from .gated import project32


def _native():
    return build.load("_C_routed")


# ------------------------------------------------------------ residual streams

class TanhNorm(NamedTuple):
    """tanh(alpha * x) * w + b, fp32; alpha has one element."""
    alpha: torch.Tensor
    w: torch.Tensor
    b: torch.Tensor


class Return(NamedTuple):
    """How a sublayer's result y goes back into S streams, fp32:
    x_t <- sum_s mix[s, t] x_s + out[t] y."""
    mix: torch.Tensor            # [S, S]
    out: torch.Tensor            # [S]


class RoutedRows(NamedTuple):
    """A mixture's result before its weighted sum: token t's is the sum of
    weight[t, k] times row slot[t, k] of rows, or times self[t] where that
    is negative."""
    rows: torch.Tensor           # [T * K, W]
    slot: torch.Tensor           # [T, K] int32
    weight: torch.Tensor         # [T, K] fp32
    self: torch.Tensor           # [T, W]


def hyper_embed(x: torch.Tensor, ids: torch.Tensor, positions: torch.Tensor,
                embed: torch.Tensor, places: torch.Tensor,
                into: torch.Tensor, norm: TanhNorm) -> torch.Tensor:
    """Every stream of x (fp32 [T, S, W], written) <- embed[ids] +
    places[positions]. Returns norm(sum_s into[s] x_s) in embed's dtype."""
    if not x.is_cuda:
        return ref.hyper_embed(x, ids, positions, embed, places, into, norm)
    h = torch.empty(x.shape[0], x.shape[2], dtype=embed.dtype,
                    device=x.device)
    _native().hyper_embed(h, x, ids, positions, embed, places, into, *norm)
    return h


def hyper_step(x: torch.Tensor, y: Union[torch.Tensor, RoutedRows],
               back: Return, into: torch.Tensor, norm: TanhNorm,
               tap: Optional[torch.Tensor] = None) -> torch.Tensor:
    """y into the streams x (fp32 [T, S, W], in place); their sum also to
    tap. Returns norm(sum_s into[s] x_s) of the new ones in y's dtype."""
    routed = isinstance(y, RoutedRows)
    if not x.is_cuda:
        return ref.hyper_step(x, y, back, into, norm, tap)
    h = torch.empty(x.shape[0], x.shape[2],
                    dtype=(y.rows if routed else y).dtype, device=x.device)
    if routed:
        _native().hyper_step_routed(h, x, *y, *back, into, *norm, tap)
    else:
        _native().hyper_step(h, x, y, *back, into, *norm, tap)
    return h


def softcap(x: torch.Tensor, cap: float) -> torch.Tensor:
    """x (fp32, in place) <- cap * tanh(x / cap)."""
    if not x.is_cuda:
        return ref.softcap(x, cap)
    _native().softcap(x, cap)
    return x


# ----------------------------------------------------------- mixture of experts

@dataclass(frozen=True)
class RouterParams:
    """`experts` with weights, then `identity` ones that return their input;
    of `groups` equal groups of neighbours the best `keep` stay open, `top`
    experts are chosen per token."""
    experts: int
    top: int
    identity: int = 0
    groups: int = 1
    keep: int = 1

    def __post_init__(self):
        n = self.experts + self.identity
        if self.groups < 1 or n % self.groups or \
                not 1 <= self.keep <= self.groups:
            raise ValueError(f"{n} experts in {self.groups} groups, "
                             f"{self.keep} kept")
        if not 1 <= self.top <= min(64, n // self.groups * self.keep):
            raise ValueError(f"{self.top} of {n // self.groups * self.keep} "
                             "experts chosen")
        if self.experts < 1 or n > 1024:
            raise ValueError(f"{self.experts} + {self.identity} experts")

    @property
    def outputs(self) -> int:
        return self.experts + self.identity


def choose_experts(z: torch.Tensor, correction: torch.Tensor,
                   p: RouterParams):
    """Router outputs z (fp32 [T, outputs]) -> ids [T, top] int32 and weights
    [T, top] fp32: the top of softmax(z) + correction, weighted by softmax(z)
    normalised over the chosen."""
    if not z.is_cuda:
        return ref.choose_experts(z, correction, p)
    return _route(z, correction, p)[:2]


def _tokens_per_group(T: int) -> int:
    """Tokens a routing workgroup counts: at most 256 workgroups."""
    return max(4, -(-T // 1024) * 4)


def _route(z, correction, p: RouterParams):
    T, dev = z.shape[0], z.device
    per = _tokens_per_group(T)
    ids = torch.empty(T, p.top, dtype=torch.int32, device=dev)
    weights = torch.empty(T, p.top, dtype=torch.float32, device=dev)
    rank = torch.empty_like(ids)
    hist = torch.empty(-(-T // per), p.experts, dtype=torch.int32, device=dev)
    _native().route(ids, weights, rank, hist, z, correction, p.experts,
                    p.groups, p.keep, per)
    return ids, weights, rank, hist


class ExpertLists(NamedTuple):
    """Rows of all experts in one list, cut into tiles of one expert each."""
    order: torch.Tensor          # [T * top] int32 (token, choice) of a row
    slot: torch.Tensor           # [T, top] int32 row, -1: identity
    tiles: torch.Tensor          # [n, 4] int32 expert, first row, rows
    height: int                  # rows of a tile at most
    kind: str                    # kernel family: stream, tile or plain


# Height of a tile by the rows an expert has on average (the weights are the
# traffic until there are hundreds).
TILE_HEIGHTS = ((4, 32), (12, 128), (384, 256))


def tile_height(rows: int, p: RouterParams, a: torch.Tensor,
                ups: torch.Tensor, downs: torch.Tensor):
    """(rows of a tile, kernel family) for `rows` (token, choice) pairs."""
    C = _native()
    if not (C.experts_fit(a, ups) and downs.shape[2] % 8 == 0):
        return 32, "plain"
    each = rows / p.outputs
    if each < TILE_HEIGHTS[0][0] or ups.shape[2] % 64 or \
            downs.shape[2] % 64:
        return 32 if each < 16 else 64, "stream"
    return [h for n, h in TILE_HEIGHTS if each >= n][-1], "tile"


def expert_lists(ids, rank, hist, p: RouterParams, height: int,
                 kind: str) -> ExpertLists:
    T, dev = ids.shape[0], ids.device
    P = T * p.top
    order = torch.empty(P, dtype=torch.int32, device=dev)
    slot = torch.empty_like(ids)
    tiles = torch.empty(min(P, P // height + p.experts), 4,
                        dtype=torch.int32, device=dev)
    _native().place(order, slot, tiles, ids, rank, hist,
                    _tokens_per_group(T), height)
    return ExpertLists(order, slot, tiles, height, kind)


def expert_products(h: torch.Tensor, ups: torch.Tensor, downs: torch.Tensor,
                    lists: ExpertLists, top: int):
    """The two launches of the experts' feed-forward: up with the square of
    relu, and down. Returns (their functions, the result rows)."""
    P, C = lists.order.shape[0], _native()
    act = torch.empty(P, ups.shape[1], dtype=h.dtype, device=h.device)
    rows = torch.empty(P, downs.shape[1], dtype=h.dtype, device=h.device)

    def up():
        C.expert_product(act, h, ups, lists.tiles, lists.order, top,
                         lists.height, lists.kind, True)

    def down():
        C.expert_product(rows, act, downs, lists.tiles, None, 1,
                         lists.height, lists.kind, False)

    return (up, down), rows


def expert_mixture(h: torch.Tensor, z: torch.Tensor,
                   correction: torch.Tensor, ups: torch.Tensor,
                   downs: torch.Tensor, p: RouterParams) -> RoutedRows:
    """Feed-forward down_e(relu(up_e h)^2) of every token's chosen experts.
    ups [experts, F, W], downs [experts, W, F]; z: router outputs, fp32."""
    if not h.is_cuda:
        return ref.expert_mixture(h, z, correction, ups, downs, p)
    ids, weights, rank, hist = _route(z, correction, p)
    lists = expert_lists(ids, rank, hist, p,
                         *tile_height(ids.numel(), p, h, ups, downs))
    steps, rows = expert_products(h, ups, downs, lists, p.top)
    for step in steps:
        step()
    return RoutedRows(rows, lists.slot, weights, h)


# --------------------------------------------------------------- selective scan

@dataclass
class ScanParams:
    """One selective scan: its columns x_at and z_at (inner each) in the
    input projection, and b_at, c_at (state each) in the projection of the
    convolved x, whose first dt_rank columns give the step sizes."""
    inner: int
    state: int
    taps: int
    dt_rank: int
    x_at: int
    z_at: int
    b_at: int
    c_at: int

    @property
    def columns(self) -> int:
        return self.c_at + state_columns(self.state)


def state_columns(state: int) -> int:
    """Columns that B and C take each: the registers of a scan (zero past
    the state size)."""
    return max(8, 1 << (state - 1).bit_length())


class ScanWeights(NamedTuple):
    """conv [taps, inner], conv_b and D [inner], A [state, inner] (times
    log2(e)), dt_b [inner]: fp32. x [columns, inner], dt [inner, dt_rank]:
    storage type."""
    conv: torch.Tensor
    conv_b: torch.Tensor
    x: torch.Tensor
    dt: torch.Tensor
    dt_b: torch.Tensor
    A: torch.Tensor
    D: torch.Tensor


# Waves from which whole sequences keep the chip busy; below, chunks of at
# most SCAN_CHUNK tokens, for SCAN_WAVES waves.
SCAN_WHOLE, SCAN_WAVES, SCAN_CHUNK = 2048, 4096, 256


def scan_chunk(inner: int, rows: int, seqs: int) -> int:
    """Tokens of a chunk, 0: sequences as a whole fill the chip."""
    waves = -(-inner // 64)
    if waves * seqs >= SCAN_WHOLE or rows < 128 * seqs:
        return 0
    return min(SCAN_CHUNK,
               max(64, -(-rows * waves // SCAN_WAVES // 32) * 32))


def conv_silu(z: torch.Tensor, p: ScanParams, w: ScanWeights, ring, slots,
              positions, cu=None, max_len: int = 1) -> torch.Tensor:
    """[T, inner] <- silu(causal convolution of z's x); ring [slots, taps,
    inner] holds the last inputs (entry position % taps)."""
    out = torch.empty(z.shape[0], p.inner, dtype=z.dtype, device=z.device)
    _native().conv_silu(out, z, p.x_at, w.conv, w.conv_b, ring, slots,
                        positions, cu, max_len)
    return out


def scan_inputs(x: torch.Tensor, p: ScanParams, w: ScanWeights):
    """Step sizes before their bias [T, inner] and the rows with B and C,
    both fp32, from the convolved x."""
    bc = project32(x, w.x)
    return project32(bc[:, :p.dt_rank].to(x.dtype), w.dt), bc


def selective_step(y: torch.Tensor, z: torch.Tensor, p: ScanParams,
                   w: ScanWeights, cache, state_slots: torch.Tensor,
                   positions: torch.Tensor) -> None:
    """y [R, inner] <- gated output of single tokens, each of its own
    sequence. cache: (ring, state [slots, state, inner] fp32), updated in
    place; position 0 starts from zeros whatever the slot holds, a negative
    slot reads and writes nothing."""
    ring, state = cache
    if not z.is_cuda:
        for r in range(z.shape[0]):
            ref.selective_span(y[r:r + 1], z[r:r + 1], p, w, ring, state,
                               int(state_slots[r]), int(positions[r]))
        return
    x = conv_silu(z, p, w, ring, state_slots, positions)
    dt, bc = scan_inputs(x, p, w)
    _native().scan_step(y, x, z, p.z_at, dt, w.dt_b, bc, p.b_at, p.c_at, w.A,
                        w.D, state, state_slots, positions)


def selective_prompt(y: torch.Tensor, z: torch.Tensor, p: ScanParams,
                     w: ScanWeights, cache, meta) -> None:
    """The same for prompt portions (meta: PrefillMeta)."""
    ring, state = cache
    if not z.is_cuda:
        cu = meta.cu_seqlens.tolist()
        for b in range(len(cu) - 1):
            s = slice(cu[b], cu[b + 1])
            ref.selective_span(y[s], z[s], p, w, ring, state,
                               int(meta.state_slots[b]),
                               int(meta.positions[cu[b]]))
        return
    x = conv_silu(z, p, w, ring, meta.state_slots, meta.positions,
                  meta.cu_seqlens, meta.max_seqlen)
    scan_prompt(y, x, z, p, w, state, *scan_inputs(x, p, w), meta)


def scan_prompt(y, x, z, p: ScanParams, w: ScanWeights, state, dt, bc,
                meta) -> None:
    B = meta.cu_seqlens.shape[0] - 1
    size, parts = scan_chunk(p.inner, x.shape[0], B), (None,) * 5
    if size:
        ch = meta.chunks(size)
        n, dev = ch.seq.shape[0], z.device
        parts = (ch.row, ch.count, ch.first,
                 torch.empty(n, p.state, p.inner, device=dev),
                 torch.empty(n, p.inner, device=dev))
    _native().scan_prompt(y, x, z, p.z_at, dt, w.dt_b, bc, p.b_at, p.c_at,
                          w.A, w.D, state, meta.state_slots, meta.positions,
                          meta.cu_seqlens, *parts)
