"""Plain, slow Nibezen: one function per mechanism, full sequences only.

Every function works on one whole sequence with no cache, no batch and no
chunking, in whatever dtype it is handed (tests use float64). It shares no
code with helix_amd; the framework is compared against it.

Notation: T tokens, W width, H heads, D unrotated and R rotated query/key
size, E value size, K latent size, N state size, G state groups.
"""
import math

import torch


def unit_rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def silu(x):
    return x / (1 + torch.exp(-x))


# ------------------------------------------------------------ latent attention

def rotation_frequencies(dims, base, scaling):
    """(frequency of every pair, factor on cos and sin); scaling stretches
    the slow pairs, ramping between two pair numbers."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0

    def pair_with(turns):
        """Fractional pair number that turns so often over the original
        context."""
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(pair_with(scaling["fast"])), 0)
    hi = min(math.ceil(pair_with(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate(x, rot):
    """x [T, heads, R]: neighbours (2i, 2i+1) turn by position * f_i."""
    if not rot:
        return x
    f, amp = rotation_frequencies(rot["dims"], rot["base"],
                                  rot.get("scaling"))
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=x.dtype)[:, None]
    for i, fi in enumerate(f):
        c, s = amp * torch.cos(pos * fi), amp * torch.sin(pos * fi)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def visible(T, window):
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    ok = dist >= 0
    return ok & (dist < window) if window else ok


def latents(h, w_dkv, norm_w, K, eps):
    """(normed latent [T, K], raw shared key part [T, R])."""
    z = h @ w_dkv.T
    return rms_norm(z[:, :K], norm_w, eps), z[:, K:]


def attend(qn, qr, c, kr, w_uk, w_uv, scale, window):
    """qn [T, H, D], qr [T, H, R] and kr [T, R] (rotated), c [T, K]; keys and
    values are spelled out per head. -> [T, H, E]."""
    T, H, D = qn.shape
    k = (c @ w_uk.T).view(T, H, D)
    v = (c @ w_uv.T).view(T, H, -1)
    out = []
    for h in range(H):
        s = (qn[:, h] @ k[:, h].T + qr[:, h] @ kr.T) * scale
        s = s.masked_fill(~visible(T, window), -math.inf)
        out.append(torch.softmax(s, -1) @ v[:, h])
    return torch.stack(out, 1)


def output_gate(o, logits):
    return o / (1 + torch.exp(-logits))[..., None]


def latent_attention(w, m, h, eps):
    T, H, D, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"]
    q = (h @ w["q"].T).view(T, H, D + R)
    c, kr = latents(h, w["dkv"], w["dkv.norm"], m["kv_rank"], eps)
    rot = m.get("rot")
    o = attend(q[..., :D], rotate(q[..., D:], rot), c,
               rotate(kr[:, None], rot)[:, 0], w["uk"], w["uv"], m["scale"],
               (m.get("mask") or {}).get("size"))
    return output_gate(o, h @ w["g"].T).reshape(T, -1) @ w["o"].T


# ------------------------------------------------------------ state space mixer

def causal_conv(x, taps, bias):
    """x [T, C], taps [C, n], last column on the current token."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x])
    return sum(padded[k:k + T] * taps[:, k] for k in range(n)) + bias


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def state_space(x, B, C, dt, A_log, D):
    """x [T, H, P], B and C [T, G, N], dt [T, H] (positive). One token at a
    time: the head's state decays, takes in B x^T and is read with C."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    state = torch.zeros(H, N, P, dtype=x.dtype)
    y = torch.empty_like(x)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            keep = torch.exp(-torch.exp(A_log[h]) * dt[t, h])
            state[h] = keep * state[h] + \
                dt[t, h] * B[t, g][:, None] * x[t, h][None, :]
            y[t, h] = state[h].T @ C[t, g] + D[h] * x[t, h]
    return y


def group_norm(y, groups, w, eps):
    T = y.shape[0]
    return unit_rms(y.view(T, groups, -1), eps).reshape(T, -1) * w


def mamba2(w, m, h, eps):
    T, H, P, N, G = (h.shape[0], m["heads"], m["vdim"], m["state"],
                     m["groups"])
    inner = H * P
    z, xbc, dt = (h @ w["in"].T).split([inner, inner + 2 * G * N, H], -1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = xbc.split([inner, G * N, G * N], -1)
    y = state_space(x.reshape(T, H, P), B.reshape(T, G, N),
                    C.reshape(T, G, N), softplus(dt + w["dt_bias"]),
                    w["A_log"], w["D"])
    y = group_norm(y.reshape(T, inner) * silu(z), m["norm_groups"],
                   w["norm"], eps)
    return y @ w["o"].T


MIXERS = {"latent_attention": latent_attention, "mamba2": mamba2}


# ------------------------------------------------------------------ the model

def feed_forward(w, h):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def layer_order(cfg):
    """(layer, pass of the loop or -1, first layer of its pass) in order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, -1, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, -1, False) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t, i == a) for i in range(a, b)]
    return out + [(i, -1, False) for i in range(b, n)]


def forward(cfg, weights, ids, layers_out=None, dtype=torch.float64):
    """Logits [T, vocab]; layers_out receives the stream after every layer
    that ran."""
    P = {n: t.to(dtype) for n, t in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]

    def under(prefix):
        return {n[len(prefix):]: t for n, t in P.items()
                if n.startswith(prefix)}

    emb = P["embed"][torch.tensor(ids)]
    x = emb
    for i, t, begins in layer_order(cfg):
        if begins:
            if t > 0:
                x = x + emb
            x = x + P["loop.step"][t]
        spec, p = cfg["layers"][i], f"l{i}."
        y = MIXERS[spec["type"]](under(p + "mix."), spec["mixer"],
                                 rms_norm(x, P[p + "norm1"], eps), eps)
        x = x + m * (y * P[p + "ls1"])
        if spec.get("mlp"):
            y = feed_forward(under(p + "mlp."),
                             rms_norm(x, P[p + "norm2"], eps))
            x = x + m * (y * P[p + "ls2"])
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, P["final.norm"], eps) @ P["head"].T
