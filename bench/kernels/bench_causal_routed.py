#!/usr/bin/env python3
"""Times of the causal attention kernels (prompt rows, single rows by key ranges) and of the routed squared-ReLU feed-forward
(router, expert products, stream sum), each alone, weights and caches rotated so that they come from HBM.

    python bench/kernels/bench_causal_routed.py

One line per case: microseconds, TFLOP/s of the products, TB/s of what has to be read (and written) once."""
from __future__ import annotations

import os
import sys

import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__)))))
from symmetry_amd import ops  # noqa: E402

DEV, BF = "cuda", torch.bfloat16
CAUSAL, BS = 1 << 30, 64


def timed(fn, n=60) -> float:
    """Microseconds per call, replayed from one graph of n calls."""
    fn()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for _ in range(n):
            fn()
    g.replay()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    g.replay()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / n * 1e3


def randn(*shape):
    return torch.randn(*shape, device=DEV).to(BF)


def ints(v):
    return torch.as_tensor(v, dtype=torch.int32, device=DEV)


def prompt(S, L, H, G, D, cap, keyv, gated=False):
    mb, T = L // BS, S * L
    k = randn(S * mb + 1, BS, G, D)
    v = k if keyv else randn(S * mb + 1, BS, G, D)
    ks = torch.rand(S * mb + 1, BS, device=DEV) if keyv else None
    q, out, sink = randn(T, H, D), torch.empty(T, H, D, device=DEV, dtype=BF), torch.randn(H, device=DEV) if cap else None
    bt = (torch.arange(S * mb, device=DEV) + 1).view(S, mb).int()
    pos, rs = ints(list(range(L)) * S), torch.arange(S, device=DEV).repeat_interleave(L).int()
    tiles = ints(sorted(((i, r) for i in range(S) for r in range(0, L, 64)), key=lambda t: -t[1]))
    cu = ints([i * L for i in range(S + 1)])

    gate = randn(T, (H + 2 * G) * D + H * D)[:, (H + 2 * G) * D:] if gated else None

    def run():
        return ops.window_attn(q, k, v, bt, rs, pos, CAUSAL, D ** -0.5, gate, out, tiles, cu, sink=sink, softcap=cap, key_scale=ks)

    us = timed(run, 20)
    print(f"prompt attention  {S} x {L}  heads {H}/{G} x {D}  {'keys = values' if keyv else f'cap {cap}'}"
          f"{'  gated' if gated else ''}  impl {run()}: {us:.1f} us  {S * H * L * L / 2 * 4 * D / us * 1e-6:.0f} TFLOP/s", flush=True)


def single(T, ctx, H, G, D, cap, keyv, bucket):
    copies = max(2, int(600e6 / (T * ctx * G * D * 4)))
    copies = min(copies, 12)
    per = ctx // BS + 1
    K = [randn(T * per + 1, BS, G, D) for _ in range(copies)]
    V = K if keyv else [randn(T * per + 1, BS, G, D) for _ in range(copies)]
    ks = torch.rand(T * per + 1, BS, device=DEV) if keyv else None
    mb = bucket // BS
    bt = torch.zeros(T, mb, dtype=torch.int32)
    bt[:, :per] = (torch.randperm(T * per) + 1).view(T, per).int()
    bt, pos, rs = bt.to(DEV), ints([ctx - 1] * T), ints(list(range(T)))
    q, out, sink = randn(T, H, D), torch.empty(T, H, D, device=DEV, dtype=BF), torch.randn(H, device=DEV) if cap else None
    keys, parts = ops.window_attn_split(T, G, bucket)
    ws = (torch.empty(T, H, parts, D, device=DEV), torch.empty(T, H, parts, 2, device=DEV),
          torch.zeros(T * G, dtype=torch.int32, device=DEV), keys)
    for split in (ws, None):
        n = [0]

        def run():
            n[0] += 1
            return ops.window_attn(q, K[n[0] % copies], V[n[0] % copies], bt, rs, pos, CAUSAL, D ** -0.5, None, out, sink=sink,
                                   softcap=cap, key_scale=ks, split=split)

        us = timed(run)
        print(f"single rows  {T} x {ctx} keys  heads {H}/{G} x {D}  {'keys = values' if keyv else f'cap {cap}'}  impl {run()}"
              f"{f' ({keys} keys a range)' if split else ''}: {us:.1f} us  "
              f"{T * ctx * G * D * 2 * (1 if keyv else 2) / us * 1e-6:.2f} TB/s", flush=True)


def routed(T, d, E, k, ff):
    copies = max(1, min(8, int(1.2e9 / (E * ff * d * 4))))
    x, Wr, b = randn(T, d), randn(E, d) * d ** -0.5, 0.1 * torch.randn(E, device=DEV)
    up, down = [randn(E, ff, d) * d ** -0.5 for _ in range(copies)], [randn(E, d, ff) * ff ** -0.5 for _ in range(copies)]
    R = T * k
    ids, dst, src, off = (torch.zeros(n, dtype=torch.int32, device=DEV) for n in (R, R, R, E + 1))
    w, act, y = torch.zeros(R, device=DEV), torch.empty(R, ff, device=DEV, dtype=BF), torch.empty(R, d, device=DEV, dtype=BF)
    xs, h, wn = torch.randn(T, d, device=DEV), torch.empty(T, d, device=DEV, dtype=BF), torch.rand(d, device=DEV)
    reps = 60 if T <= 512 else 20
    t_r = timed(lambda: ops.route_topk(x, Wr, b, k, ids, w, off, dst, src), reps)
    n = [0]

    def f_up():
        n[0] += 1
        ops.expert_linear(x, src, up[n[0] % copies], off, act, relu2=True)

    def f_down():
        n[0] += 1
        ops.expert_linear(act, None, down[n[0] % copies], off, y)

    t_u, t_d = timed(f_up, reps), timed(f_down, reps)
    t_s = timed(lambda: ops.residual_routed_norm(xs, x, y, dst, w, k, None, wn, 1e-5, h), reps)
    fl, wb = 2.0 * R * d * ff, 2.0 * min(E, R) * d * ff
    print(f"routed ff  {T} x {d}  {E} experts x {ff}, {k} chosen: router {t_r:.1f} us, up {t_u:.1f} us ({fl / t_u * 1e-6:.0f} "
          f"TFLOP/s, weights {wb / t_u * 1e-6:.2f} TB/s), down {t_d:.1f} us ({fl / t_d * 1e-6:.0f}, {wb / t_d * 1e-6:.2f}), sum + "
          f"norm {t_s:.1f} us ({T * d * (14 + 2 * k) / t_s * 1e-6:.2f} TB/s)", flush=True)


def main() -> int:
    for a in ((8, 1024, 16, 4, 128, 0.0, True), (8, 1024, 16, 4, 128, 50.0, False), (8, 1024, 16, 4, 128, 50.0, False, True),
              (8, 1024, 32, 8, 128, 50.0, False),
              (2, 4096, 16, 4, 128, 50.0, False), (8, 1024, 16, 4, 64, 50.0, False)):
        prompt(*a)
    for a in ((8, 1060, 16, 4, 128, 0.0, True, 2048), (8, 1060, 16, 4, 128, 50.0, False, 2048),
              (8, 1060, 32, 8, 128, 50.0, False, 2048), (64, 1060, 16, 4, 128, 50.0, False, 2048),
              (64, 1060, 16, 4, 128, 0.0, True, 2048), (8, 7000, 16, 4, 128, 50.0, False, 8192)):
        single(*a)
    for a in ((8, 2048, 16, 4, 2304), (64, 2048, 16, 4, 2304), (8192, 2048, 16, 4, 2304), (8, 4096, 8, 2, 21504),
              (8192, 4096, 8, 2, 21504)):
        routed(*a)
    return 0


if __name__ == "__main__":
    sys.exit(main())
