"""Beletar decoder forward on the symmetry_amd ops: one code path for CPU (torch references) and MI355X (HIP).

The design, in this file's notation (x: the fp32 stream, one row per token; W stored [out, in]; n(v) = (v - mean) /
sqrt(var + eps) * w + b)::

    e = E[token] * embed_scale;   x = e
    per layer run:   x = x + mixer(n1(x));   x = x + ff(n2(x))
    the layers of cfg.loop run several times in a row with the same weights, x = x + e in front of every pass but the first
    logits = E n_f(x)                                        (the embedding table, without its scale)

    mixers "delta" and "channel_delta" (H heads, G query / key heads, head h reads h // (H / G)):
      q, k, v = silu(conv(W h)) (causal per-channel taps, carried from step to step); q and k heads brought to unit length,
      q times N^(-1/2); beta = sigmoid(W_b h);  log g = -exp(A_h) softplus(z + dt_bias), z = W_a h per head, or
      W_a2 W_a1 h per head and key channel
      S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q            (S [N, P] fp32 per head, carried)
      W_o (rms(o) * w * gate), gate = silu(W_g h), or sigmoid(W_g2 W_g1 h)
    mixer "latent_attention" (H heads; per head dn unrotated + rot rotated query / key dims, dv value dims; rank r):
      q = W_q h = [q_n | q_r] per head, q_r rotated (interleaved pairs, blended frequencies and a magnitude)
      [c' | k'] = W_dkv h,  c = rms(c') * g_kv,  k_r = rotary(k')             -- the cache row [c | k_r]
      score_h(t, j) = scale (q_n . W_uk,h c_j + q_r . k_r,j), causal softmax whose denominator also holds exp(sink_h),
      out_h = sigmoid(W_g h)_h W_uv,h sum_j p_j c_j;  W_o
      evaluated with the up-projections folded into the query / output (ops.latent_attn: multi-query attention over the
      paged latent cache; the head gate is a factor of the whole head, so it is applied to the latents' sum)
    ff: W_down (silu(W_gate h) * W_up h)

Caches and states belong to a layer RUN: a looped layer has one plane or one state slot row per pass.  Every projection
that reads a sublayer's input is one row block of one fused weight (a single library GEMM), except the recurrence's step
sizes and decays, whose GEMMs leave their fp32 accumulator unrounded; the kernels take column ranges as views.  Step
launches per layer run: GEMM (the mixer's projections), then
    delta:   GEMM W_b | W_a (fp32; channel decays: W_b, W_a2), conv_silu_qkv (+ conv_state_update in prompt steps; in
             decode steps W_b | W_a ride along in this launch), delta_rule, (GEMM W_g2,) gated_group_norm, GEMM W_o
    latent:  latent_prep, bmm (absorb W_uk), rope_pairs, latent_attn (sink, gate), bmm (W_uv), GEMM W_o
    residual_layer_norm; GEMM gate|up, silu_mul, GEMM down; residual_layer_norm (+ e in front of a loop's next pass)
All intermediates live in the preallocated Workspace, so decode steps are hipGraph-capturable.

fp32 in both serving dtypes: the stream, norm statistics, rotary angles, attention scores / weights / sink, the recurrent
states and everything that enters a recurrence behind the projections and convolutions.  ``dtype=torch.float32`` runs every
product in true 32-bit as well.
"""
from __future__ import annotations

import torch

from .. import ops
from .config import BeletarConfig
from .lemunex import _Fused
from .transformer import MAX_STEP_SEQS, ForwardBatch, Workspace
from .weights import ModelWeights

GATES_ALONG_ROWS = 64  # decode steps up to this many rows compute beta / decay pre-activations beside the convolution
UNIT_EPS = 1e-6       # inside the root of the queries' and keys' length (fixed by the design)


class BeletarCache:
    """What a Beletar model keeps per sequence, by layer run (a layer that runs three times has three entries).

    ``lat``: one plane [NB, BS, r + rot] per latent-attention run (a row = normalised latent | rotated shared key part), on
    the engine's BlockManager numbering (one block table serves all planes).  Per state slot: ``rec`` [slots, H, N, P] fp32
    per delta-rule run, ``conv`` its newest taps - 1 projected q | k | v rows [slots, taps - 1, C].  Slots are handed out
    by the scheduler's StateSlotManager; a slot's old content is never read by a new sequence (its first run starts from
    zero).  Zero-initialised: every byte finite."""

    def __init__(self, cfg: BeletarConfig, num_blocks: int, block_size: int, num_slots: int, device, dtype):
        self.num_layers, self.num_blocks, self.block_size = cfg.num_layers, num_blocks, block_size
        self.lat, self.rec, self.conv = {}, {}, {}
        for n, (i, _) in enumerate(cfg.layer_runs()):
            m = cfg.layers[i].mixer
            if cfg.layers[i].type == "latent_attention":
                self.lat[n] = torch.zeros(num_blocks, block_size, m.kv_rank + m.rot_dim, device=device, dtype=dtype)
            else:
                self.rec[n] = torch.zeros(num_slots, m.heads, m.dim, m.vdim, device=device, dtype=torch.float32)
                self.conv[n] = torch.zeros(num_slots, m.conv - 1, m.conv_channels, device=device, dtype=dtype)

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for d in (self.lat, self.rec, self.conv) for t in d.values())


class BeletarLM:
    has_seq_state = True      # the engine allots a state slot per live sequence and sends prev_row / save_slot / row_seq
    fused = False
    single_copy = False
    moe = None
    tp = None

    def __init__(self, weights: ModelWeights, device, tp_comm=None, ep_comm=None, max_decode_ctx: int | None = None,
                 decode_weights: str = "auto", kv_reserve_bytes: int = 0, dtype=torch.bfloat16):
        if weights.shard.tp_size > 1 or weights.shard.ep_size > 1:
            raise NotImplementedError("Beletar runs on one GPU per replica")
        self.cfg: BeletarConfig = weights.cfg
        self.w = weights
        self.device = torch.device(device)
        self.dtype = dtype
        self.tp_size, self.tp_rank = 1, 0
        self.ws = Workspace()
        self.last_ids = torch.zeros(MAX_STEP_SEQS, dtype=torch.int32, device=self.device)
        self.last_logits = None
        self.layer_outputs: list | None = None   # set to a list: every forward appends the stream after each layer run
        cfg = self.cfg
        max_pos = min(cfg.max_position, max_decode_ctx or cfg.max_position)
        self._rope: dict = {}
        self.L = [self._prepare_layer(i, max_pos) for i in range(cfg.num_layers)]
        self.embed = weights["embed"].to(dtype)
        self.final_norm = (weights["final.norm"].float(), weights["final.norm.b"].float())
        # the sublayers in execution order: (layer run, prepared tensors, which, embedding output added in front)
        self.subs = []
        for n, (i, again) in enumerate(cfg.layer_runs()):
            P = self.L[i]
            self.subs.append((n, P, 1, again))
            if P["mlp"] is not None:
                self.subs.append((n, P, 2, False))
        self.loops = any(s[3] for s in self.subs)

    # ------------------------------------------------------------------------------------------
    def make_cache(self, num_blocks: int, block_size: int, num_slots: int) -> BeletarCache:
        return BeletarCache(self.cfg, num_blocks, block_size, num_slots, self.device, self.dtype)

    def extra_weight_bytes(self) -> int:
        return 0

    def _rope_table(self, m, max_pos: int) -> torch.Tensor:
        """[max_pos, rot_dim / 2, 2] (cos, sin, times the magnitude): the first rot.dims / 2 pairs turn, later ones pass."""
        key = (m.rot_dim, m.rot_dims, m.rot_base, m.rot_scaling, max_pos)
        if key not in self._rope:
            t = torch.zeros(max_pos, m.rot_dim // 2, 2, dtype=torch.float32)
            t[..., 0] = 1.0
            t[:, : m.rot_dims // 2] = ops.rope_scaled_table(max_pos, m.rot_dims, m.rot_base, *(m.rot_scaling or ()))
            self._rope[key] = t.to(self.device)
        return self._rope[key]

    def _prepare_layer(self, i: int, max_pos: int) -> dict:
        """The fused / converted tensors layer i's launches read.  Matrices in the activation dtype; norm weights and
        biases, sinks and the parameters of decays in fp32."""
        w, layer, dt = self.w, self.cfg.layers[i], self.dtype
        p = f"l{i}."

        def t(name):
            return w[p + name].to(dt)

        def f(name):
            return w[p + name].float().contiguous()

        m = layer.mixer
        fz = _Fused()
        P = {"kind": layer.type, "mixer": m, "mlp": layer.mlp, "norm1": (f("norm1"), f("norm1.b")), "o": t("mix.o")}
        if layer.type == "latent_attention":
            if m.kv_rank > 512:
                raise NotImplementedError(f"layer {i}: kv_rank {m.kv_rank} > 512 (latent_attn's accumulator registers)")
            for nm in ("q", "dkv", "g"):
                fz.add(nm, t("mix." + nm))
            P["gkv"], P["sink"] = t("mix.dkv.norm"), f("mix.sink")
            P["uk"] = t("mix.uk").view(m.heads, m.dim, m.kv_rank)                                   # [H, dn, r]
            P["uv"] = t("mix.uv").view(m.heads, m.vdim, m.kv_rank).transpose(1, 2).contiguous()     # [H, r, dv]
            P["rope"] = self._rope_table(m, max_pos)
        else:
            fz.add("qkv", torch.cat([t("mix.q"), t("mix.k"), t("mix.v")], 0))
            P["conv"] = torch.cat([t("mix.q.conv"), t("mix.k.conv"), t("mix.v.conv")], 0).contiguous()
            P["dt_bias"], P["A_log"], P["norm"] = f("mix.dt_bias"), f("mix.A_log"), f("mix.norm")
            if m.channel:
                fz.add("a1", t("mix.a1"))
                fz.add("g1", t("mix.g1"))
                P["gates"], P["a2"], P["g2"] = t("mix.b").contiguous(), t("mix.a2").contiguous(), t("mix.g2").contiguous()
            else:
                fz.add("g", t("mix.g"))
                P["gates"] = torch.cat([t("mix.b"), t("mix.a")], 0).contiguous()
        if layer.mlp is not None:
            P["norm2"] = (f("norm2"), f("norm2.b"))
            P["w_gu"] = torch.cat([t("mlp.gate"), t("mlp.up")], 0).contiguous()
            P["w_down"] = t("mlp.down")
        P["w_h"], P["cols"] = fz.weight(), fz.cols
        return P

    # ------------------------------------------------------------------------------------------
    def _buf(self, name, shape, dtype=None):
        return self.ws.get(name, shape, dtype or self.dtype, self.device)

    def _linear(self, name: str, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        """x [R, K] @ w[N, K]^T -> [R, N] in the activation dtype (library GEMM, fp32 accumulation)."""
        return ops.linear(x, w, out=self._buf(name, (x.shape[0], w.shape[0])))

    def _linear_f32(self, name: str, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        """x [R, K] @ w[N, K]^T -> fp32 [R, N] (the library GEMM's accumulator, unrounded)."""
        return ops.linear_f32(x, w, self._buf(name, (x.shape[0], w.shape[0]), torch.float32))

    @staticmethod
    def _cols(z: torch.Tensor, P: dict, name: str) -> torch.Tensor:
        c0, n = P["cols"][name]
        return z[:, c0:c0 + n]

    def _delta(self, n: int, P: dict, b: ForwardBatch, cache: BeletarCache, h: torch.Tensor, runs: int) -> torch.Tensor:
        m = P["mixer"]
        T, H, G, N, V = h.shape[0], m.heads, m.kv_heads, m.dim, m.vdim
        prefill = b.kind != "decode"
        cu = b.cu_q if prefill else None
        z = self._linear("z", h, P["w_h"])
        # (a decode step's few rows take these few outputs along in the convolution's launch)
        along = None
        if not prefill and T <= GATES_ALONG_ROWS:
            gates = self._buf("del.gates", (T, P["gates"].shape[0]), torch.float32)
            along = (h, P["gates"], gates)
        else:
            gates = self._linear_f32("del.gates", h, P["gates"])
        dz = self._linear_f32("del.dz", self._cols(z, P, "a1"), P["a2"]) if m.channel else gates[:, H:]
        qkv = self._cols(z, P, "qkv")
        f32 = torch.float32
        q, k = self._buf("del.q", (T, G, N), f32), self._buf("del.k", (T, G, N), f32)
        v = self._buf("del.v", (T, H, V))
        ops.conv_silu_qkv(qkv, P["conv"], cache.conv[n], cu, b.row_seq, b.prev_row, runs, G, N, H, V, N ** -0.5, UNIT_EPS,
                          q, k, v, save_slot=None if prefill else b.save_slot, gates=along)
        if prefill and m.conv > 1:
            ops.conv_state_update(qkv, cache.conv[n], cu, b.prev_row, b.save_slot, runs)
        y = self._buf("del.y", (T, H * V), f32)
        tiles = ws = None
        if prefill and self.dtype == torch.bfloat16 and self.device.type != "cpu":   # (the 32-bit model walks token by token)
            tiles, ws = b.tiles, self._buf("del.ws", (T, H, ops.delta_ws_cols(m.channel, N)), f32)
        ops.delta_rule(m.channel, q, k, v, dz, P["dt_bias"], P["A_log"], gates[:, :H], cache.rec[n], cu, b.prev_row,
                       b.save_slot, runs, y, tiles, ws)
        gate = self._linear("del.g", self._cols(z, P, "g1"), P["g2"]) if m.channel else self._cols(z, P, "g")
        gy = self._buf("del.gy", (T, H * V))
        ops.gated_group_norm(y, gate, P["norm"], self.cfg.norm_eps, V, False, gy, sigmoid=m.channel)
        return self._linear("mix.out", gy, P["o"])

    def _latent(self, n: int, P: dict, b: ForwardBatch, cache: BeletarCache, h: torch.Tensor) -> torch.Tensor:
        m = P["mixer"]
        T, H, r, rot, dn = h.shape[0], m.heads, m.kv_rank, m.rot_dim, m.dim
        plane = cache.lat[n]
        z = self._linear("z", h, P["w_h"])
        ops.latent_prep(self._cols(z, P, "dkv"), 0, r, rot, None, P["gkv"], self.cfg.norm_eps, b.positions, b.slot_mapping,
                        P["rope"], None, plane)
        q = self._cols(z, P, "q").unflatten(1, (H, dn + rot))
        qa = self._buf("lat.qa", (T, H, r + rot))
        torch.bmm(q[:, :, :dn].transpose(0, 1), P["uk"], out=qa[:, :, :r].transpose(0, 1))
        ops.rope_pairs(q[:, :, dn:], qa[:, :, r:], b.positions, P["rope"])
        olat = self._buf("lat.o", (T, H, r))
        part_o = part_ml = None
        if b.kind == "decode" and self.device.type != "cpu":
            parts = ops.latent_attn_parts(T, b.block_tables.shape[1] * cache.block_size)
            if parts > 1:
                part_o = self._buf("lat.part_o", (T, H, parts, r), torch.float32)
                part_ml = self._buf("lat.part_ml", (T, H, parts, 2), torch.float32)
        tiled = b.kind != "decode" and self.dtype == torch.bfloat16
        ops.latent_attn(qa, plane, b.block_tables, b.row_seq, b.positions, m.scale, r, olat, part_o, part_ml,
                        b.tiles if tiled else None, b.cu_q if tiled else None, sink=P["sink"], gate=self._cols(z, P, "g"))
        ov = self._buf("lat.ov", (T, H * m.vdim))
        torch.bmm(olat.transpose(0, 1), P["uv"], out=ov.view(T, H, m.vdim).transpose(0, 1))
        return self._linear("mix.out", ov, P["o"])

    def _ff(self, P: dict, h: torch.Tensor) -> torch.Tensor:
        F = P["mlp"].ff
        gu = self._linear("ff.gu", h, P["w_gu"])
        act = self._buf("ff.act", (h.shape[0], F))
        ops.silu_mul(gu[:, :F], gu[:, F:], act)
        return self._linear("ff.down", act, P["w_down"])

    @torch.no_grad()
    def forward(self, b: ForwardBatch, cache: BeletarCache) -> torch.Tensor:
        """Run one step; returns sampled token ids [num_seqs] int32 (device).  ``b.logit_rows`` (prefill-kind steps)
        or ``b.need_logits`` (decode steps: every row) leave fp32 logits in ``self.last_logits``."""
        cfg = self.cfg
        T, d, eps = b.num_tokens, cfg.hidden_size, cfg.norm_eps
        prefill = b.kind != "decode"
        runs = b.num_seqs if prefill else T
        x = self._buf("x", (T, d), torch.float32)
        # the embedding output is kept where a loop adds it again; the stream then starts from it in the first sum
        e = self._buf("e", (T, d), torch.float32) if self.loops else x
        h = self._buf("h", (T, d))
        src = b.src if b.src is not None and not prefill else None
        ops.embed_scale(b.input_ids, self.embed, cfg.embed_scale, e, src, self.last_ids if src is not None else None)
        w, bias = self.subs[0][1]["norm1"]
        ops.residual_layer_norm(e, w=w, bias=bias, eps=eps, out=h)
        base = e if self.loops else None
        for s, (n, P, which, _) in enumerate(self.subs):
            if which == 2:
                y = self._ff(P, h)
            elif P["kind"] == "latent_attention":
                y = self._latent(n, P, b, cache, h)
            else:
                y = self._delta(n, P, b, cache, h, runs)
            nxt = self.subs[s + 1] if s + 1 < len(self.subs) else None
            again = e if nxt is not None and nxt[3] else None
            kw = {}
            if nxt is not None:
                w, bias = nxt[1][f"norm{nxt[2]}"]
                kw = {"w": w, "bias": bias, "eps": eps, "out": h}
            if self.layer_outputs is not None and (nxt is None or nxt[0] != n):
                ops.residual_layer_norm(x, y, base=base)
                self.layer_outputs.append(x.clone())
                if nxt is not None:
                    ops.residual_layer_norm(x, again, **kw)
            else:
                ops.residual_layer_norm(x, y, again, base=base, **kw)
            base = None
        n = b.num_seqs
        ids = self.last_ids[:n]
        self.last_logits = None
        if b.sample or b.need_logits:
            rows = None if not prefill else b.last_idx
            logits = self._logits("logits", x, rows, n)
            if b.need_logits:
                self.last_logits = logits
            if b.sample:
                keys = self._buf("keys", (n,), torch.int64)
                ops.logits_argmax(logits, b.temps, b.seeds, b.step, keys, ids, 0)
                if b.filtered:
                    ops.sample_filtered(logits, b.temps, b.top_k, b.top_p, b.seeds, b.step, ids)
        if b.logit_rows is not None and b.logit_rows.numel():
            self.last_logits = self._logits("want_logits", x, b.logit_rows, int(b.logit_rows.numel()))
        return ids

    def _logits(self, name: str, x: torch.Tensor, rows, n: int) -> torch.Tensor:
        """fp32 logits [n, V] = n_f(x[rows]) . E^T (fp32 output from the library GEMM)."""
        xn = self._buf(name + ".xn", (n, self.cfg.hidden_size))
        w, bias = self.final_norm
        ops.residual_layer_norm(x, w=w, bias=bias, eps=self.cfg.norm_eps, rows=rows, out=xn)
        return self._linear_f32(name, xn, self.embed)
