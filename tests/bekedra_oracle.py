"""Plain, slow implementation of the Bekedra design, one function per mechanism, written from the design's equations.  It
shares no code with the product path (no symmetry_amd import): whole-sequence recompute in float64, no cache, no paging, no
batching.  The tests compare the engine against it.

Notation: ``W`` maps checkpoint tensor names to tensors; matrices are stored [out, in] and applied as ``x @ M.T``; ``cfg``
is the checkpoint's config.json as a dict; positions count from 0.

    x = E[token] * embedding.scale
    per layer run:  h = rms(x, norm1);  x += mixer(h) + ff(h)
    layers loop.start .. loop.stop - 1 run loop.times times in a row, x += loop.step[t] in front of pass t = 0, 1, ...
    logits = E rms(x, final.norm)
"""
from __future__ import annotations

import math

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def query_temperature(positions, coef, every):
    """1 + coef ln(floor((p + 1) / every) + 1)"""
    return 1.0 + coef * torch.log(torch.floor((positions.double() + 1.0) / every) + 1.0)


def frequencies(rot):
    """base^(-2 i / dims), with ``scaling`` by wavelength: short waves keep theirs, long waves are divided by the factor, a
    linear blend of the two between."""
    out, sc = [], rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def rotate_half(x, positions, rot):
    """Entry i of the last axis turns with entry i + dims / 2; entries past dims pass.  x [T, H, D]."""
    n = rot["dims"] // 2
    a = positions.double()[:, None] * frequencies(rot)[None, :]
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


def causal_scores(q, k, scale):
    """q [T, H, D], k [T, G, D] -> [H, T, T]; query head h reads key head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    kk = k.repeat_interleave(H // G, dim=1)
    return torch.einsum("thd,shd->hts", q, kk) * scale


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap)


def causal_softmax(s, sink=None):
    """s [H, T, T] -> weights over the keys j <= i; sink [H]: the denominator also holds exp(sink_h)."""
    T = s.shape[1]
    i = torch.arange(T)
    s = s.masked_fill(i[:, None] < i[None, :], float("-inf"))
    if sink is None:
        return torch.softmax(s, -1)
    full = torch.cat([s, sink[:, None, None].expand(-1, T, 1)], -1)
    return torch.softmax(full, -1)[..., :-1]


def mix_values(p, v, H):
    """p [H, T, T], v [T, G, P] -> [T, H P]"""
    vv = v.repeat_interleave(H // v.shape[1], dim=1)
    return torch.einsum("hts,shd->thd", p, vv).reshape(p.shape[1], -1)


def key_is_value_attention(W, pre, m, h, positions, eps):
    """Mixer "attention": the values are the projected keys before their norm; the norms run over whole projections."""
    H, G, D, T = m["heads"], m["kv_heads"], m["dim"], h.shape[0]
    q = h @ W[pre + "q"].T + W[pre + "q.b"]
    k = h @ W[pre + "k"].T + W[pre + "k.b"]
    v = k.view(T, G, D)
    q = rms_norm(q, W[pre + "q.norm"], eps).view(T, H, D)
    k = rms_norm(k, W[pre + "k.norm"], eps).view(T, G, D)
    q = q * query_temperature(positions, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    p = causal_softmax(causal_scores(q, k, m["scale"]))
    return mix_values(p, v, H) @ W[pre + "o"].T


def rotary_sink_attention(W, pre, m, h, positions, eps):
    """Mixer "attention_2": norms per head, rotary, soft-capped scores, a sink, an element-wise output gate."""
    H, G, D, T = m["heads"], m["kv_heads"], m["dim"], h.shape[0]
    q = rms_norm((h @ W[pre + "q"].T).view(T, H, D), W[pre + "q.norm"], eps)
    k = rms_norm((h @ W[pre + "k"].T).view(T, G, D), W[pre + "k.norm"], eps)
    v = (h @ W[pre + "v"].T).view(T, G, m["vdim"])
    s = causal_scores(rotate_half(q, positions, m["rot"]), rotate_half(k, positions, m["rot"]), m["scale"])
    p = causal_softmax(soft_cap(s, m["softcap"]), W[pre + "sink"])
    return (mix_values(p, v, H) * torch.sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


def route(W, pre, top, h):
    """-> (chosen experts [T, top], their weights): the largest biased logits, softmax over the chosen ones."""
    z = h @ W[pre + "router"].T + W[pre + "router.b"]
    vals, ids = torch.topk(z, top, dim=-1)
    return ids, torch.softmax(vals, -1)


def expert(W, pre, h):
    return torch.clamp(h @ W[pre + "up"].T, min=0.0) ** 2 @ W[pre + "down"].T


def routed_ff(W, pre, m, h, margins=None):
    """``margins``: a list that receives, per token, the gap between the last chosen and the first passed-over logit."""
    ids, w = route(W, pre, m["router"]["top"], h)
    if margins is not None and m["router"]["top"] < m["router"]["experts"]:
        z = (h @ W[pre + "router"].T + W[pre + "router.b"]).sort(-1, descending=True).values
        margins.append(z[:, m["router"]["top"] - 1] - z[:, m["router"]["top"]])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(ids.shape[1]):
            out[t] += w[t, j] * expert(W, f"{pre}e{int(ids[t, j])}.", h[t])
    return out


def layer_runs(cfg):
    """The order in which layers run: (layer, number of the pass that starts with it or None)."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    runs = [(i, None) for i in range(a)]
    for t in range(lp["times"]):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def forward(cfg: dict, W: dict, tokens, trace=None, margins=None):
    """tokens (list of ids) -> logits [T, vocab] in float64.  ``trace``: a list that receives the stream after every
    layer run."""
    W = {k: (v.double() if v.is_floating_point() else v) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(len(ids))
    x = W["embed"][ids] * cfg["embedding"]["scale"]
    for i, start in layer_runs(cfg):
        if start is not None:
            x = x + W["loop.step"][start]
        layer, pre = cfg["layers"][i], f"l{i}."
        h = rms_norm(x, W[pre + "norm1"], eps)
        mixer = {"attention": key_is_value_attention, "attention_2": rotary_sink_attention}[layer["type"]]
        y = mixer(W, pre + "mix.", layer["mixer"], h, positions, eps)
        if layer.get("mlp") is not None:
            y = y + routed_ff(W, pre + "mlp.", layer["mlp"], h, margins)
        x = x + y
        if trace is not None:
            trace.append(x.clone())
    return rms_norm(x, W["final.norm"], eps) @ W["embed"].T
