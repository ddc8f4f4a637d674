"""Bekedra decoder forward on the symmetry_amd ops: one code path for CPU (torch references) and MI355X (HIP).

The design, in this file's notation (x: the fp32 stream, one row per token; W stored [out, in]; n(v, g) =
v / sqrt(mean(v^2) + eps) * g)::

    x = E[token] * embed_scale
    per layer run:   h = n(x, g_i);   x = x + mixer(h) + ff(h)              (one norm feeds both sublayers)
    the layers of cfg.loop run several times in a row with the same weights, x = x + s_t in front of pass t = 0, 1, ...
    logits = E n(x, g_f)                                        (the embedding table, without its scale)

    mixer "attention" (H query heads on G key heads; no rotation; the values are the projected keys):
      q = n(W_q h + b_q, g_q) temp_p,  k' = W_k h + b_k,  k = n(k', g_k)  (norms over whole projections),
      temp_p = 1 + c ln(floor((p + 1) / m) + 1);   score(t, j) = scale q . k_j over j <= t, softmax over the values k'_j, W_o
      evaluated on ONE cached plane of k' plus a number per key: q . k_j = (q * g_k) . k'_j / rms(k'_j)
    mixer "attention_2" (H query heads on G key / value heads):
      q = n_head(W_q h, g_q), k = n_head(W_k h, g_k), turned (entry i with i + dims / 2, frequencies scaled by wavelength)
      score(t, j) = c tanh(scale q . k_j / c) over j <= t, softmax whose denominator also holds exp(sink_h),
      W_o (heads * sigmoid(W_g h))
    ff: z = W_r h + b_r, the ``top`` largest logits, weights = softmax over them; expert = W_down relu(W_up h)^2

Caches belong to a layer RUN: a looped layer has planes per pass.  Nothing else is kept per sequence, so the model needs no
state slots and cached prompt prefixes are adopted as they are.  Every bf16 projection that reads h is one row block of one
fused weight (a single library GEMM); the kernels take column ranges as views.  Step launches per layer run:
    attention:    GEMM q | k, qk_row_norm_cache, window_attn (key scales; decode: key ranges), GEMM W_o
    attention_2:  GEMM q | k | v | gate, qk_norm_cache (rotary), window_attn (soft cap, sink, gate), GEMM W_o
    ff:           route_topk, expert_linear (gathers its rows, squared ReLU), expert_linear
    residual_routed_norm (stream + mixer + weighted expert rows + the next pass's vector, and the next layer's h)
All intermediates live in the preallocated Workspace, so decode steps are hipGraph-capturable.  In decode steps the experts
(bound by their weights' traffic) run on a second stream beside the attention (bound by latency): two branches of the graph,
joined in front of the sum.

fp32 in both serving dtypes: the stream, norm statistics, rotary angles, temperatures, attention scores / weights / sink /
cap, router logits and weights.  ``dtype=torch.float32`` runs every product in true 32-bit as well.
"""
from __future__ import annotations

import torch

from .. import ops
from .config import BekedraConfig
from .lemunex import _Fused
from .transformer import MAX_STEP_SEQS, ForwardBatch, Workspace
from .weights import ModelWeights

CAUSAL = 1 << 30      # a window that never ends: plain causal attention through the windowed kernel


class BekedraCache:
    """What a Bekedra model keeps: paged planes by layer run, on the engine's BlockManager numbering (one block table serves
    all): ``k`` [NB, BS, G, dk] and ``v`` [NB, BS, G, dv]; runs whose values are their keys have the projected keys in ``k``,
    no ``v``, and ``ks`` [NB, BS] fp32, the keys' norm statistics.  Zero-initialised: every byte finite."""

    def __init__(self, cfg: BekedraConfig, num_blocks: int, block_size: int, device, dtype):
        self.num_layers, self.num_blocks, self.block_size = cfg.num_layers, num_blocks, block_size
        self.k, self.v, self.ks = {}, {}, {}
        for n, (i, _) in enumerate(cfg.layer_runs()):
            m = cfg.layers[i].mixer
            self.k[n] = torch.zeros(num_blocks, block_size, m.kv_heads, m.dim, device=device, dtype=dtype)
            if m.key_values:
                self.ks[n] = torch.zeros(num_blocks, block_size, device=device, dtype=torch.float32)
            else:
                self.v[n] = torch.zeros(num_blocks, block_size, m.kv_heads, m.vdim, device=device, dtype=dtype)

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for d in (self.k, self.v, self.ks) for t in d.values())


class BekedraLM:
    has_seq_state = False     # the paged cache is all there is
    row_metadata = True       # the attention kernels read the runner's row -> sequence map
    serves_float32 = True
    fused = False
    single_copy = False
    moe = None
    tp = None

    def __init__(self, weights: ModelWeights, device, tp_comm=None, ep_comm=None, max_decode_ctx: int | None = None,
                 decode_weights: str = "auto", kv_reserve_bytes: int = 0, dtype=torch.bfloat16):
        if weights.shard.tp_size > 1 or weights.shard.ep_size > 1:
            raise NotImplementedError("Bekedra runs on one GPU per replica")
        self.cfg: BekedraConfig = weights.cfg
        self.w = weights
        self.device = torch.device(device)
        self.dtype = dtype
        self.tp_size, self.tp_rank = 1, 0
        self.ws = Workspace()
        self.last_ids = torch.zeros(MAX_STEP_SEQS, dtype=torch.int32, device=self.device)
        self.last_logits = None
        self.layer_outputs: list | None = None   # set to a list: every forward appends the stream after each layer run
        self.side = torch.cuda.Stream(self.device) if self.device.type != "cpu" else None
        cfg = self.cfg
        max_pos = min(cfg.max_position, max_decode_ctx or cfg.max_position)
        self._rope: dict = {}
        self.L = [self._prepare_layer(i, max_pos) for i in range(cfg.num_layers)]
        self.embed = weights["embed"].to(dtype)
        self.final_norm = weights["final.norm"].float()
        # the layer runs in order: (prepared tensors, vector added in front of it or None)
        steps = weights["loop.step"].float() if cfg.loop else None
        self.runs = [(self.L[i], None if t is None else steps[t].contiguous()) for i, t in cfg.layer_runs()]

    # ------------------------------------------------------------------------------------------
    def make_cache(self, num_blocks: int, block_size: int, num_slots: int = 0) -> BekedraCache:
        return BekedraCache(self.cfg, num_blocks, block_size, self.device, self.dtype)

    def extra_weight_bytes(self) -> int:
        return 0

    def _rope_table(self, rot, max_pos: int) -> torch.Tensor:
        """[max_pos, dims / 2, 2] (cos, sin)"""
        key = (rot, max_pos)
        if key not in self._rope:
            scaling = None
            if rot.factor > 0:
                scaling = {"rope_type": "llama3", "factor": rot.factor, "low_freq_factor": rot.low,
                           "high_freq_factor": rot.high, "original_max_position_embeddings": rot.original}
            t = ops.rope_table(max_pos, rot.dims, rot.base, scaling)                   # [max_pos, cos | sin]
            self._rope[key] = t.view(max_pos, 2, rot.dims // 2).transpose(1, 2).contiguous().to(self.device)
        return self._rope[key]

    def _prepare_layer(self, i: int, max_pos: int) -> dict:
        """The fused / converted tensors layer i's launches read.  Matrices in the activation dtype; norm weights, biases
        and sinks in fp32."""
        w, layer, dt = self.w, self.cfg.layers[i], self.dtype
        p = f"l{i}."

        def t(name):
            return w[p + name].to(dt)

        def f(name):
            return w[p + name].float().contiguous()

        m = layer.mixer
        if m.vdim > 512:
            raise NotImplementedError(f"layer {i}: value heads wider than 512")
        fz = _Fused()
        P = {"mixer": m, "mlp": layer.mlp, "norm1": f("norm1"), "gq": f("mix.q.norm"), "gk": f("mix.k.norm"), "o": t("mix.o")}
        fz.add("qkv", torch.cat([t("mix." + nm) for nm in (("q", "k") if m.key_values else ("q", "k", "v"))], 0))
        P["bias"] = torch.cat([f("mix.q.b"), f("mix.k.b")]).contiguous() if m.bias else None
        P["sink"] = f("mix.sink") if m.sink else None
        P["rope"] = self._rope_table(m.rot, max_pos) if m.rot is not None and m.rot.dims else None
        if m.gate:
            fz.add("g", t("mix.g"))
        if layer.mlp is not None:
            E = layer.mlp.experts
            P["router"], P["router.b"] = t("mlp.router").contiguous(), f("mlp.router.b")
            P["up"] = torch.stack([t(f"mlp.e{e}.up") for e in range(E)]).contiguous()
            P["down"] = torch.stack([t(f"mlp.e{e}.down") for e in range(E)]).contiguous()
        P["w_h"], P["cols"] = fz.weight(), fz.cols
        return P

    # ------------------------------------------------------------------------------------------
    def _buf(self, name, shape, dtype=None):
        return self.ws.get(name, shape, dtype or self.dtype, self.device)

    def _linear(self, name: str, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        """x [R, K] @ w[N, K]^T -> [R, N] in the activation dtype (library GEMM, fp32 accumulation)."""
        return ops.linear(x, w, out=self._buf(name, (x.shape[0], w.shape[0])))

    @staticmethod
    def _cols(z: torch.Tensor, P: dict, name: str) -> torch.Tensor:
        c0, n = P["cols"][name]
        return z[:, c0:c0 + n]

    def _attention(self, n: int, P: dict, b: ForwardBatch, cache: BekedraCache, h: torch.Tensor) -> torch.Tensor:
        """Either mixer of layer run n -> [T, d]."""
        m, eps = P["mixer"], self.cfg.norm_eps
        T = h.shape[0]
        prefill = b.kind != "decode"
        z = self._linear("z", h, P["w_h"])
        qkv = self._cols(z, P, "qkv")
        q = self._buf("att.q", (T, m.heads, m.dim))
        if m.key_values:
            ops.qk_row_norm_cache(qkv, P["bias"], m.heads, m.kv_heads, m.dim, P["gq"], P["gk"], eps, m.temp_coef, m.temp_every,
                                  b.positions, b.slot_mapping, q, cache.k[n], cache.ks[n])
        else:
            ops.qk_norm_cache(qkv, m.heads, m.kv_heads, m.dim, m.vdim, P["gq"], P["gk"], None, eps, b.slot_mapping, q,
                              cache.k[n], cache.v[n], rope=P["rope"], positions=b.positions)
        att = self._buf("att.o", (T, m.heads, m.vdim))
        split = None
        if not prefill and self.device.type != "cpu" and self.dtype == torch.bfloat16:
            keys, parts = ops.window_attn_split(T, m.kv_heads, b.block_tables.shape[1] * cache.block_size)
            split = (self._buf("att.part_o", (T, m.heads, parts, m.vdim), torch.float32),
                     self._buf("att.part_ml", (T, m.heads, parts, 2), torch.float32),
                     self.ws.get("att.counters", (T * m.kv_heads,), torch.int32, self.device, zeros=True), keys)
        ops.window_attn(q, cache.k[n], cache.k[n] if m.key_values else cache.v[n], b.block_tables, b.row_seq, b.positions,
                        CAUSAL, m.scale, self._cols(z, P, "g") if m.gate else None, att, b.tiles if prefill else None,
                        b.cu_q if prefill else None, sink=P["sink"], softcap=m.softcap, key_scale=cache.ks.get(n), split=split)
        return self._linear("att.out", att.view(T, m.heads * m.vdim), P["o"])

    def _routed(self, P: dict, h: torch.Tensor):
        """The chosen experts' rows -> (y [T top, d] in expert order, place of every (token, choice), weights).  Segment
        bounds stay on the device (no host sync: graph-capturable)."""
        spec = P["mlp"]
        T, d = h.shape
        R, i32 = T * spec.top, torch.int32
        ids, wts = self._buf("moe.ids", (R,), i32), self._buf("moe.w", (R,), torch.float32)
        offsets = self._buf("moe.offsets", (spec.experts + 1,), i32)
        dst, src = self._buf("moe.dst", (R,), i32), self._buf("moe.src", (R,), i32)
        ops.route_topk(h, P["router"], P["router.b"], spec.top, ids, wts, offsets, dst, src)
        act = self._buf("moe.act", (R, spec.expert_ff))
        ops.expert_linear(h, src, P["up"], offsets, act, relu2=True)
        y = self._buf("moe.y", (R, d))
        ops.expert_linear(act, None, P["down"], offsets, y)
        return y, dst, wts

    @torch.no_grad()
    def forward(self, b: ForwardBatch, cache: BekedraCache) -> torch.Tensor:
        """Run one step; returns sampled token ids [num_seqs] int32 (device).  ``b.logit_rows`` (prefill-kind steps)
        or ``b.need_logits`` (decode steps: every row) leave fp32 logits in ``self.last_logits``."""
        cfg = self.cfg
        T, d, eps = b.num_tokens, cfg.hidden_size, cfg.norm_eps
        prefill = b.kind != "decode"
        x = self._buf("x", (T, d), torch.float32)
        h = self._buf("h", (T, d))
        src = b.src if b.src is not None and not prefill else None
        ops.embed_scale(b.input_ids, self.embed, cfg.embed_scale, x, src, self.last_ids if src is not None else None)
        P0, step = self.runs[0]
        ops.residual_routed_norm(x, None, None, None, None, 0, step, P0["norm1"], eps, h)
        side, main = (None, None) if prefill or self.side is None else (self.side, torch.cuda.current_stream(self.device))
        for n, (P, _) in enumerate(self.runs):
            y = dst = wts = None
            top = 0
            if P["mlp"] is not None:
                top = P["mlp"].top
                if side is None:
                    y, dst, wts = self._routed(P, h)
                else:      # both sublayers read h: two branches of the step's graph
                    side.wait_stream(main)
                    with torch.cuda.stream(side):
                        y, dst, wts = self._routed(P, h)
            att = self._attention(n, P, b, cache, h)
            if top and side is not None:
                main.wait_stream(side)
            nxt, step = self.runs[n + 1] if n + 1 < len(self.runs) else (None, None)
            w, out = (nxt["norm1"], h) if nxt is not None else (None, None)
            if self.layer_outputs is not None:
                ops.residual_routed_norm(x, att, y, dst, wts, top, None)
                self.layer_outputs.append(x.clone())
                if nxt is not None:
                    ops.residual_routed_norm(x, None, None, None, None, 0, step, w, eps, out)
            else:
                ops.residual_routed_norm(x, att, y, dst, wts, top, step, w, eps, out)
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
        """fp32 logits [n, V] = n(x[rows], g_f) . E^T (fp32 output from the library GEMM)."""
        xn = self._buf(name + ".xn", (n, self.cfg.hidden_size))
        ops.rms_norm_rows(x, rows, self.final_norm, self.cfg.norm_eps, 0.0, xn)
        return ops.linear_f32(xn, self.embed, self._buf(name, (n, self.cfg.vocab_size), torch.float32))
