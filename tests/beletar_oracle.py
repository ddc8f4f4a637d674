"""Plain, slow implementation of the Beletar design, one function per mechanism, written from the design's equations.  It
shares no code with the product path (no symmetry_amd import): whole-sequence recompute in float64, token by token, no
cache, no paging, no batching.  The tests compare the engine against it.

Notation: ``W`` maps checkpoint tensor names to tensors; matrices are stored [out, in] and applied as ``x @ M.T``; ``cfg``
is the checkpoint's config.json as a dict; positions count from 0.

    e = E[token] * embedding.scale;  x = e
    per layer run:  x += mixer(n1(x));  x += ff(n2(x)),     n(v) = (v - mean) / sqrt(var + eps) * w + b
    layers loop.start .. loop.stop - 1 run loop.times times in a row, x += e in front of every run of them but the first
    logits = E n_f(x)
"""
from __future__ import annotations

import math

import torch


def layer_norm(x, w, b, eps):
    mean = x.mean(-1, keepdim=True)
    var = ((x - mean) ** 2).mean(-1, keepdim=True)
    return (x - mean) / torch.sqrt(var + eps) * w + b


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def short_conv(z, w):
    """z [T, C], w [C, taps]: y_t = sum_j w[:, j] z_(t - taps + 1 + j), zeros before the start."""
    T, taps = z.shape[0], w.shape[1]
    y = torch.zeros_like(z)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * z[s]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_inputs(W, pre, m, h):
    """Queries and keys [T, G, N] (unit vectors, queries times N^(-1/2)) and values [T, H, P] behind their convolutions."""
    H, G, N, P = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]

    def branch(nm):
        return silu(short_conv(h @ W[pre + nm].T, W[pre + nm + ".conv"]))

    q = unit(branch("q").view(T, G, N)) * N ** -0.5
    return q, unit(branch("k").view(T, G, N)), branch("v").view(T, H, P)


def delta_rule(q, k, v, log_g, beta, S=None):
    """q, k [T, G, N], v [T, H, P], log_g [T, H, N] (logarithm of the decay of every key channel), beta [T, H]:
    S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.  -> o [T, H, P], S [H, N, P]."""
    T, G, N = q.shape
    H, P = v.shape[1:]
    S = torch.zeros(H, N, P, dtype=v.dtype) if S is None else S.clone()
    out = torch.zeros(T, H, P, dtype=v.dtype)
    for t in range(T):
        for hd in range(H):
            g = hd // (H // G)
            Sh = torch.exp(log_g[t, hd])[:, None] * S[hd]
            u = beta[t, hd] * (v[t, hd] - Sh.T @ k[t, g])
            Sh = Sh + k[t, g][:, None] * u[None, :]
            S[hd] = Sh
            out[t, hd] = Sh.T @ q[t, g]
    return out, S


def head_decay(W, pre, m, h):
    """log g [T, H, N]: one decay per head."""
    lg = -torch.exp(W[pre + "A_log"]) * softplus(h @ W[pre + "a"].T + W[pre + "dt_bias"])
    return lg[:, :, None].expand(-1, -1, m["dim"])


def channel_decay(W, pre, m, h):
    """log g [T, H, N]: one decay per head and key channel, through a low-rank projection."""
    z = (h @ W[pre + "a1"].T) @ W[pre + "a2"].T + W[pre + "dt_bias"]
    return -torch.exp(W[pre + "A_log"])[None, :, None] * softplus(z).view(h.shape[0], m["heads"], m["dim"])


def delta(W, pre, m, h, eps):
    T = h.shape[0]
    q, k, v = delta_inputs(W, pre, m, h)
    o, _ = delta_rule(q, k, v, head_decay(W, pre, m, h), torch.sigmoid(h @ W[pre + "b"].T))
    o = rms_norm(o, W[pre + "norm"], eps).reshape(T, -1) * silu(h @ W[pre + "g"].T)
    return o @ W[pre + "o"].T


def channel_delta(W, pre, m, h, eps):
    T = h.shape[0]
    q, k, v = delta_inputs(W, pre, m, h)
    o, _ = delta_rule(q, k, v, channel_decay(W, pre, m, h), torch.sigmoid(h @ W[pre + "b"].T))
    o = rms_norm(o, W[pre + "norm"], eps).reshape(T, -1) * torch.sigmoid((h @ W[pre + "g1"].T) @ W[pre + "g2"].T)
    return o @ W[pre + "o"].T


def rotation_angles(positions, rot):
    """(angles [T, dims / 2], magnitude): frequencies base^(-2 i / dims), with ``scaling`` blended towards f / factor."""
    dims, base = rot["dims"], rot["base"]
    mag, freqs = 1.0, []
    sc = rot.get("scaling")
    if sc:
        def dim_at(turns):
            return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

        lo, hi = max(math.floor(dim_at(sc["fast"])), 0), min(math.ceil(dim_at(sc["slow"])), dims - 1)
        mag = 0.1 * math.log(sc["factor"]) + 1.0
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / sc["factor"] * ramp + f * (1.0 - ramp)
        freqs.append(f)
    return positions.double()[:, None] * torch.tensor(freqs, dtype=torch.float64)[None, :], mag


def rotate_pairs(x, positions, rot):
    """Entries 2 i and 2 i + 1 of the last axis turn together by angle i; entries past rot.dims pass.  x [T, ..., D]."""
    a, mag = rotation_angles(positions, rot)
    half = a.shape[1]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [half]
    c, s = (torch.cos(a) * mag).view(shape), (torch.sin(a) * mag).view(shape)
    out = x.clone()
    u, v = x[..., 0:2 * half:2], x[..., 1:2 * half:2]
    out[..., 0:2 * half:2] = u * c - v * s
    out[..., 1:2 * half:2] = v * c + u * s
    return out


def sink_softmax(s, sink):
    """s [H, T, S] (masked entries -inf), sink [H]: weights whose denominator also holds exp(sink_h)."""
    full = torch.cat([s, sink[:, None, None].expand(-1, s.shape[1], 1)], -1)
    return torch.softmax(full, -1)[..., :-1]


def latent_attention(W, pre, m, h, positions, eps):
    H, dn, rot, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).view(T, H, dn + rot)
    z = h @ W[pre + "dkv"].T
    c = rms_norm(z[:, :r], W[pre + "dkv.norm"], eps)
    kr = rotate_pairs(z[:, r:], positions, m["rot"])
    qr = rotate_pairs(q[..., dn:], positions, m["rot"])
    kn, v = (c @ W[pre + "uk"].T).view(T, H, dn), (c @ W[pre + "uv"].T).view(T, H, dv)
    s = (torch.einsum("thd,shd->hts", q[..., :dn], kn) + torch.einsum("thd,sd->hts", qr, kr)) * m["scale"]
    i = torch.arange(T)
    s = s.masked_fill(i[:, None] < i[None, :], float("-inf"))
    o = torch.einsum("hts,shd->thd", sink_softmax(s, W[pre + "sink"]), v)
    o = o * torch.sigmoid(h @ W[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ W[pre + "o"].T


def glu_ff(W, pre, h):
    return (silu(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) @ W[pre + "down"].T


def layer_runs(cfg):
    """The order in which layers run: (layer, True where the embedding output is added in front of it)."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    runs = [(i, False) for i in range(a)]
    for t in range(lp["times"]):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(cfg: dict, W: dict, tokens, trace=None):
    """tokens (list of ids) -> logits [T, vocab] in float64.  ``trace``: a list that receives the stream after every
    layer run."""
    W = {k: (v.double() if v.is_floating_point() else v) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(len(ids))
    e = W["embed"][ids] * cfg["embedding"]["scale"]
    x = e.clone()

    def norm(nm, v):
        return layer_norm(v, W[nm], W[nm + ".b"], eps)

    for i, again in layer_runs(cfg):
        if again:
            x = x + e
        layer, pre = cfg["layers"][i], f"l{i}."
        h = norm(pre + "norm1", x)
        if layer["type"] == "delta":
            x = x + delta(W, pre + "mix.", layer["mixer"], h, eps)
        elif layer["type"] == "channel_delta":
            x = x + channel_delta(W, pre + "mix.", layer["mixer"], h, eps)
        elif layer["type"] == "latent_attention":
            x = x + latent_attention(W, pre + "mix.", layer["mixer"], h, positions, eps)
        else:
            raise ValueError(layer["type"])
        if layer.get("mlp") is not None:
            x = x + glu_ff(W, pre + "mlp.", norm(pre + "norm2", x))
        if trace is not None:
            trace.append(x.clone())
    return norm("final.norm", x) @ W["embed"].T
