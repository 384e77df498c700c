"""Vivesun decoder on the gfx950 kernel set: pre-norm layers on an fp32 residual stream, a bigram
embedding, delta-rule recurrences (one of them side by side with chunked attention), gelu experts and
a per-layer input from the token itself.

Per layer (``x`` is the fp32 residual stream, activations in the model dtype; norm weights are stored
around zero and applied as ``1 + w``):

    h  = norm1(x)                                    fused into the previous layer's last step
    x += mixer(h); h2 = norm2(x)                     ops.residual_add_rmsnorm_
    x += experts(h2), copy of x for the gate         ops.moe_router, ops.residual_plain_experts_
    g  = gelu_tanh(gate x) * token vector of layer i ops.gelu_gate_rows
    x += rmsnorm(proj g) * w; h = next norm1(x)      ops.rmsnorm_residual_next_

The first rows are ``embed[id] + bigram[(previous id, id) hash]`` (``ops.bigram_embed``); the previous
id of a sequence is part of its state. The logits are the embedding table applied to the final norm.

Mixers:

* ``delta`` - one GEMM gives ``q | k | v | output gate | b | a``; ``ops.short_conv`` runs the causal
  convolution of q, k, v (its last inputs in the state slot), ``ops.gated_delta_scan`` the gated delta rule
  with the fp32 state in the slot, ``ops.group_rmsnorm`` the head norm with the silu gate.
* ``parallel`` - one GEMM gives the projections of both halves. Left: rotary positions and page write
  (``ops.rope_headnorm_cache_``), chunked softmax attention with a valueless sink. Right: ``ops.tanh_rows`` +
  a small GEMM for the decay, ``ops.channel_delta_scan``, head norm with the sigmoid gate. Both halves
  write their columns of one row, already times their scale, so one GEMM applies both output
  projections and adds them.

The serving engine drives this class as it drives the other decoders (``forward`` on a step's token
rows + ``logits``); ``AttnMeta`` carries the per-step row maps (``tok_seq``, ``shift_src``, state slots).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

from .. import ops
from ..parallel.dist import ParallelContext, get_context
from .config import VivesunConfig
from .llama import AttnMeta

DECAY = math.exp(-0.5)    # decay of the channel-wise delta rule: exp(-DECAY * sigmoid(.))


def _ceil8(n: int) -> int:
    return (n + 7) // 8 * 8


class VivesunModel:
    stateful = True                # recurrent layers keep per-sequence state in scheduler slots
    uses_decode_workspace = False
    supports_step_graphs = False   # prefill / mixed steps run eagerly (decode steps are graphs)
    supports_prefix_cache = False  # a cached page carries no recurrent state

    def __init__(self, cfg: VivesunConfig, device="cuda", dtype=torch.bfloat16,
                 pctx: Optional[ParallelContext] = None, seed: int = 0,
                 weights: Optional[Dict[str, torch.Tensor]] = None, fp8: bool = False):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Vivesun runs in bfloat16 or float32")
        if fp8:
            raise NotImplementedError("FP8 projections cover the Llama-layout decoders")
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.p = pctx or get_context()
        if self.p.tp_size > 1 or self.p.pp_size > 1:
            raise NotImplementedError("Vivesun runs on one GPU per replica (no TP / PP split)")
        self.fp8 = False
        self.kv_dtype, self.kv_scales = "auto", (1.0, 1.0)
        self.sequence_parallel, self.sp_min_tokens, self.split_mixed, self.moe_ws = False, 0, False, None
        att = [b.mixer.left for b in cfg.blocks if b.type == "parallel"]
        self.hq, self.hkv, self.D = (att[0].heads, att[0].kv_heads, att[0].dim) if att else (1, 1, 1)
        self.n_experts = cfg.num_experts
        self.vocab_local = cfg.vocab_size
        self.k_cache: List[Optional[torch.Tensor]] = []
        self.v_cache: List[Optional[torch.Tensor]] = []
        self.rec_state: List[torch.Tensor] = []
        self.conv_state: List[Optional[torch.Tensor]] = []
        self.prev_token: Optional[torch.Tensor] = None
        self.skinny = (self.device.type == "cuda" and dtype == torch.bfloat16 and ops.skinny.enabled())
        self.mfma = True   # MFMA attention kernels where they apply (bf16, tile sizes)
        if weights is None:
            weights = random_weights(cfg, seed, dtype)
        self._load(weights)

    # ------------------------------------------------------------------ weights
    def _load(self, w: Dict[str, torch.Tensor]):
        cfg, dev, dt = self.cfg, self.device, self.dtype
        W = cfg.hidden

        def mat(name, shape, dtype=dt):
            t = w[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"{name}: shape {tuple(t.shape)}, config says {tuple(shape)}")
            t = t.to(dev, dtype).contiguous()
            return t.clone() if t.data_ptr() % 16 else t   # (a memory-mapped file need not be aligned)

        def vec(name, n):
            t = w[name].to(dev, torch.float32).reshape(-1).contiguous()
            if t.numel() != n:
                raise ValueError(f"{name}: {t.numel()} elements, config says {n}")
            return t

        def fused(*mats):
            """Row-stacked GEMM weight, padded with zero rows to a multiple of 8 outputs."""
            M = torch.cat(mats)
            pad = _ceil8(M.shape[0]) - M.shape[0]
            if pad:
                M = torch.cat([M, torch.zeros(pad, M.shape[1], dtype=M.dtype, device=M.device)])
            return M.contiguous()

        self.norm_weights: Dict[str, torch.Tensor] = {}     # as stored, around zero

        def norm(name):
            self.norm_weights[name] = vec(name, W)
            return 1.0 + self.norm_weights[name]

        self.embed = mat("embed", (cfg.vocab_size, W))
        self.bigram = mat("bigram", (cfg.bigram.buckets + 1, W)) if cfg.bigram is not None else None
        S = cfg.side_dim
        self.side_embed = mat("side.embed", (cfg.vocab_size, cfg.layers * S)) if S else None
        self.layers: List[dict] = []
        for i, b in enumerate(cfg.blocks):
            p, m = f"l{i}.", b.mixer
            L = {"type": b.type, "spec": m, "mlp": b.mlp, "norm1": norm(p + "norm1")}
            if b.type == "delta":
                nq, nv, Hh = m.kv_heads * m.dim, m.heads * m.vdim, m.heads
                L["w_in"] = fused(mat(p + "mix.q", (nq, W)), mat(p + "mix.k", (nq, W)), mat(p + "mix.v", (nv, W)),
                                  mat(p + "mix.g", (nv, W)), mat(p + "mix.b", (Hh, W)), mat(p + "mix.a", (Hh, W)))
                L["taps"] = torch.cat([mat(p + "mix.q.conv", (nq, m.conv), torch.float32),
                                       mat(p + "mix.k.conv", (nq, m.conv), torch.float32),
                                       mat(p + "mix.v.conv", (nv, m.conv), torch.float32)]).t().contiguous()
                L["a_log"], L["dt_bias"] = vec(p + "mix.A_log", Hh), vec(p + "mix.dt_bias", Hh)
                L["on"] = vec(p + "mix.norm", m.vdim)
                L["wo"] = mat(p + "mix.o", (W, nv))
            elif b.type == "parallel":
                a, r = m.left, m.right
                pl, pr = p + "mix.left.", p + "mix.right."
                nq, nk, nv, nr = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim, r.heads * r.dim
                rank = w[pr + "w1"].shape[0]       # (the low rank of the decay is the tensor's own)
                L["w_in"] = fused(mat(pl + "q", (nq, W)), mat(pl + "k", (nk, W)), mat(pl + "v", (nv, W)),
                                  mat(pr + "r", (nr, W)), mat(pr + "k", (nr, W)), mat(pr + "v", (nr, W)),
                                  mat(pr + "g", (nr, W)), mat(pr + "a", (nr, W)), mat(pr + "w1", (rank, W)))
                L["rank"], L["r_off"] = rank, nq + nk + nv
                L["w2"] = mat(pr + "w2", (nr, rank))
                L["w0"], L["ab"] = vec(pr + "w0", nr), vec(pr + "a.b", nr)
                L["on"] = vec(pr + "norm", nr)
                L["on_scaled"] = L["on"] * m.right_scale
                f, mag = ops.rotary_frequencies(a.rot.dims, a.rot.base, bands=a.rot.bands)
                L["freq"], L["mag"] = f.to(dev), mag
                L["wo"] = torch.cat([mat(pl + "o", (W, a.heads * a.vdim)), mat(pr + "o", (W, nr))], dim=1).contiguous()
            else:
                raise ValueError(f"layer {i}: unknown mixer type {b.type!r}")
            f = b.mlp
            if f is not None:
                L["norm2"] = norm(p + "norm2")
                L["router"] = mat(p + "mlp.router", (f.experts, W), torch.float32)
                L["w1"] = torch.stack([mat(f"{p}mlp.e{e}.up", (f.ff, W)) for e in range(f.experts)]).contiguous()
                L["wd"] = torch.stack([mat(f"{p}mlp.e{e}.down", (W, f.ff)) for e in range(f.experts)]).contiguous()
            if S:
                L["sg"], L["sp"] = mat(p + "side.gate", (S, W)), mat(p + "side.proj", (W, S))
                L["sn"] = vec(p + "side.norm", W)
            self.layers.append(L)
        self.final_norm = norm("final.norm")

    def state_dict(self) -> Dict[str, torch.Tensor]:
        dt, cfg = self.dtype, self.cfg
        out = {"embed": self.embed, **{k: v.to(dt) for k, v in self.norm_weights.items()}}
        if self.bigram is not None:
            out["bigram"] = self.bigram
        if self.side_embed is not None:
            out["side.embed"] = self.side_embed
        for i, L in enumerate(self.layers):
            p, m, f, Wi = f"l{i}.", L["spec"], L["mlp"], L["w_in"]

            def rows(prefix, parts, at=0):
                for name, n in parts:
                    out[prefix + name] = Wi[at:at + n]
                    at += n

            if L["type"] == "delta":
                nq, nv, Hh = m.kv_heads * m.dim, m.heads * m.vdim, m.heads
                rows(p + "mix.", (("q", nq), ("k", nq), ("v", nv), ("g", nv), ("b", Hh), ("a", Hh)))
                t = L["taps"].t().to(dt)
                out.update({p + "mix.q.conv": t[:nq], p + "mix.k.conv": t[nq:2 * nq], p + "mix.v.conv": t[2 * nq:],
                            p + "mix.A_log": L["a_log"].to(dt), p + "mix.dt_bias": L["dt_bias"].to(dt),
                            p + "mix.norm": L["on"].to(dt), p + "mix.o": L["wo"]})
            else:
                a, nr = m.left, m.right.heads * m.right.dim
                rows(p + "mix.left.", (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim)))
                rows(p + "mix.right.", (("r", nr), ("k", nr), ("v", nr), ("g", nr), ("a", nr), ("w1", L["rank"])), L["r_off"])
                na = a.heads * a.vdim
                out.update({p + "mix.left.o": L["wo"][:, :na], p + "mix.right.o": L["wo"][:, na:],
                            p + "mix.right.w2": L["w2"], p + "mix.right.w0": L["w0"].to(dt),
                            p + "mix.right.a.b": L["ab"].to(dt), p + "mix.right.norm": L["on"].to(dt)})
            if f is not None:
                out[p + "mlp.router"] = L["router"].to(dt)
                for e in range(f.experts):
                    out.update({f"{p}mlp.e{e}.up": L["w1"][e], f"{p}mlp.e{e}.down": L["wd"][e]})
            if cfg.side_dim:
                out.update({p + "side.gate": L["sg"], p + "side.proj": L["sp"], p + "side.norm": L["sn"].to(dt)})
        return out

    # ------------------------------------------------------------------ cache and state
    def allocate_kv_cache(self, num_blocks: int, block_size: int = 64, kv_dtype: str = "auto",
                          kv_scales=(1.0, 1.0)):
        """Row-major pages in the model dtype, one K [blocks, kv_heads, 64, dim] and one V [blocks,
        kv_heads, 64, vdim] tensor per ``parallel`` layer, all addressed by the same page numbers;
        ``delta`` layers have none."""
        if block_size != 64:
            raise ValueError("the gfx950 attention kernels use 64-token KV pages")
        if kv_dtype not in ("auto", "bf16"):
            raise ValueError("Vivesun keeps its KV pages in the model dtype")
        self.k_cache, self.v_cache = [], []
        for L in self.layers:
            if L["type"] == "delta":
                self.k_cache.append(None)
                self.v_cache.append(None)
            else:
                a = L["spec"].left
                self.k_cache.append(torch.zeros(num_blocks, a.kv_heads, block_size, a.dim, device=self.device, dtype=self.dtype))
                self.v_cache.append(torch.zeros(num_blocks, a.kv_heads, block_size, a.vdim, device=self.device, dtype=self.dtype))
        return self.k_cache, self.v_cache

    def allocate_state(self, slots: int) -> None:
        """Per-sequence state by slot: the previous token (bigram embedding), per layer the fp32
        matrix memory [slots, heads, dim, vdim] and, for ``delta`` layers, the last inputs of the short
        convolution [slots, taps - 1, channels]. A slot needs no clearing when it is given to a new
        sequence: a segment that starts at position 0 starts from zeros, not from the slot."""
        n = max(1, slots)
        self.prev_token = torch.zeros(n, device=self.device, dtype=torch.int32)
        self.rec_state, self.conv_state = [], []
        for L in self.layers:
            m = L["spec"]
            h, d, dv = (m.heads, m.dim, m.vdim) if L["type"] == "delta" else (m.right.heads, m.right.dim, m.right.dim)
            self.rec_state.append(torch.zeros(n, h, d, dv, device=self.device, dtype=torch.float32))
            self.conv_state.append(torch.zeros(n, m.conv - 1, L["taps"].shape[1], device=self.device, dtype=self.dtype)
                                   if L["type"] == "delta" else None)

    def kv_block_bytes(self, block_size: int = 64, kv_dtype: str = "auto") -> int:
        elem = torch.finfo(self.dtype).bits // 8
        n = sum(b.mixer.left.kv_heads * (b.mixer.left.dim + b.mixer.left.vdim) for b in self.cfg.blocks
                if b.type == "parallel")
        return max(1, n) * block_size * elem

    def copy_kv_blocks(self, src, dst) -> None:
        raise NotImplementedError("beam search forks need a copy of the recurrent state")

    def ipc_collectives_cover(self, rows: int, tokens: int) -> bool:
        return True

    def quantize_fp8(self) -> None:
        raise NotImplementedError("FP8 projections cover the Llama-layout decoders")

    # ------------------------------------------------------------------ forward
    def _lin(self, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        """x @ w^T: decode-shape rows take the skinny MFMA GEMM where the measured table
        (ops.skinny) holds this (N, K) and prefers it over the library GEMM."""
        if self.skinny and x.shape[0] <= 512 and x.stride(1) == 1 and x.stride(0) % 8 == 0:
            pk = ops.skinny.table().pick(w.shape[0], w.shape[1], x.shape[0])
            if pk is not None:
                cfg, split = pk
                if split == 1:
                    return ops.skinny_gemm(x, w, cfg, 1, 0)
                return ops.PartialSum(ops.skinny_gemm(x, w, cfg, split, 1)).materialize()
        return ops.linear(x, w)

    @staticmethod
    def _segments(meta: AttnMeta) -> dict:
        """A step's segments as the scans take them: single rows first, then portions."""
        if meta.kind == "decode":
            return dict(cu=None, slots=meta.state_slots)
        return dict(cu=meta.cu_q, slots=meta.state_slots, max_q=meta.max_q_len,
                    n_single=meta.n_decode if meta.kind == "mixed" else 0)

    def _attend(self, q, kc, vc, pos, meta: AttnMeta, a, out, **kw):
        """Softmax attention of a step's rows: prompt portions on the MFMA tile kernel and
        single-token rows on the page-parallel kernel where they apply (bf16, tile-sized heads),
        everything else on the row kernel."""
        H, G, dk, dv = a.heads, a.kv_heads, a.dim, a.vdim
        if self.mfma and ops.softmax_attention_mfma_ok(q, dk, dv, H // G, 1):
            nd = meta.n_decode if meta.kind == "mixed" else (q.shape[0] if meta.kind == "decode" else 0)
            if nd:
                ops.softmax_attention_rows(q[:nd], kc, vc, meta.block_tables, meta.tok_seq[:nd], pos[:nd], H, G, dk, dv,
                                           max_ctx=meta.max_ctx, out=out[:nd], **kw)
            if nd < q.shape[0]:
                ops.softmax_attention_prefill(q[nd:], kc, vc, meta.block_tables[nd:],
                                              meta.cu_q_prefill if nd else meta.cu_q, meta.ctx_lens[nd:],
                                              meta.max_q_len, H, G, dk, dv, out=out[nd:], **kw)
            return
        ops.softmax_attention(q, kc, vc, meta.block_tables, meta.tok_seq, pos, H, G, dk, dv, out=out, **kw)

    def _mix_delta(self, li: int, L: dict, h, pos, meta: AttnMeta):
        m = L["spec"]
        proj = self._lin(h, L["w_in"])
        C, nv = L["taps"].shape[1], m.heads * m.vdim
        seg = self._segments(meta)
        x = ops.short_conv(proj[:, :C], L["taps"], self.conv_state[li], seg["cu"], seg["slots"], meta.tok_seq, pos)
        o = ops.gated_delta_scan(x, proj[:, C + nv:], L["a_log"], L["dt_bias"], self.rec_state[li], m.heads, m.kv_heads,
                                 m.dim, m.vdim, pos=pos, **seg)
        return self._lin(ops.group_rmsnorm(o, L["on"], m.heads, self.cfg.eps, self.dtype, gate=proj[:, C:C + nv],
                                           gate_act="silu"), L["wo"])

    def _mix_parallel(self, li: int, L: dict, h, pos, meta: AttnMeta):
        m = L["spec"]
        a, r = m.left, m.right
        proj = self._lin(h, L["w_in"])
        nl, nr = a.heads * a.vdim, r.heads * r.dim
        y = torch.empty(h.shape[0], _ceil8(nl + nr), dtype=self.dtype, device=h.device)[:, :nl + nr]
        # left: rotated rows into the pages, chunked attention times its scale
        kc, vc = self.k_cache[li], self.v_cache[li]
        ops.rope_headnorm_cache_(proj, pos, meta.slots, kc, vc, a.heads, a.kv_heads, a.dim, a.vdim, L["freq"], L["mag"],
                                 a.rot.dims, self.cfg.eps, v_off=(a.heads + a.kv_heads) * a.dim)
        self._attend(proj[:, :a.heads * a.dim], kc, vc, pos, meta, a, y[:, :nl], scale=a.scale, chunk=a.chunk, sink=0.0,
                     factor=m.left_scale)
        # right: r | k | v | gate | removal rate | low-rank decay columns
        c = [L["r_off"] + j * nr for j in range(6)]
        w = self._lin(ops.tanh_rows(proj[:, c[5]:c[5] + L["rank"]]), L["w2"])
        o = ops.channel_delta_scan(proj[:, c[0]:c[1]], proj[:, c[1]:c[2]], proj[:, c[2]:c[3]], proj[:, c[4]:c[5]], w,
                                   L["ab"], L["w0"], self.rec_state[li], r.heads, r.dim, r.dim, DECAY, pos=pos,
                                   **self._segments(meta))
        ops.group_rmsnorm(o, L["on_scaled"], r.heads, self.cfg.eps, self.dtype, gate=proj[:, c[3]:c[4]], out=y[:, nl:])
        return self._lin(y, L["wo"])

    def _embed(self, ids, meta: AttnMeta):
        g = self.cfg.bigram
        if g is None:
            return ops.embed_rows(ids, self.embed, 1.0)
        if meta.kind == "decode":   # one token per sequence: the same launch leaves the id in the slot
            return ops.bigram_embed(ids, self.embed, self.bigram, meta.shift_src, self.prev_token, g.mul_prev, g.mul_cur,
                                    save_slots=meta.state_slots)
        x = ops.bigram_embed(ids, self.embed, self.bigram, meta.shift_src, self.prev_token, g.mul_prev, g.mul_cur)
        ops.token_save_(self.prev_token, ids, meta.state_rows, meta.state_slots)
        return x

    def forward(self, ids: torch.Tensor, pos: torch.Tensor, meta: AttnMeta,
                sample_idx: Optional[torch.Tensor] = None, embed_override=None,
                layer_tap: Optional[list] = None) -> torch.Tensor:
        """Final-normed rows selected by ``sample_idx`` (all rows if None) of a step's token rows.
        ``layer_tap``: a list that receives a copy of the residual stream after every layer."""
        if embed_override is not None:
            raise NotImplementedError("Vivesun takes token ids only")
        if meta.tok_seq is None or meta.shift_src is None or meta.state_slots is None:
            raise ValueError("Vivesun steps need the engine's row maps (tok_seq, shift_src, state slots)")
        eps, dt, S = self.cfg.eps, self.dtype, self.cfg.side_dim
        x = self._embed(ids, meta)
        h = ops.rmsnorm_f32(x, self.layers[0]["norm1"], eps, dtype=dt) if self.layers else None
        for li, L in enumerate(self.layers):
            y = (self._mix_delta if L["type"] == "delta" else self._mix_parallel)(li, L, h, pos, meta)
            nxt = self.layers[li + 1]["norm1"] if li + 1 < len(self.layers) else None
            f = L["mlp"]
            if f is not None:
                h2 = ops.residual_add_rmsnorm_(x, y, L["norm2"], eps, dt)
                eid, ew = ops.moe_router(h2, L["router"], f.top, f.scale, ws=self.moe_ws)
                h = ops.residual_plain_experts_(x, h2, eid, ew, L["w1"], L["wd"], nxt, eps, dt, copy=S > 0, ws=self.moe_ws)
            elif S:
                h = ops.residual_add_cast_(x, y, dt)
            else:
                h = ops.residual_add_rmsnorm_(x, y, nxt, eps, dt)
            if S:      # h is a copy of the stream
                y = self._lin(ops.gelu_gate_rows(self._lin(h, L["sg"]), ids, self.side_embed, li * S), L["sp"])
                if nxt is not None:
                    h = ops.rmsnorm_residual_next_(x, y, L["sn"], eps, nxt, dt)
                else:
                    ops.rmsnorm_residual_(x, y, L["sn"], eps)
            if layer_tap is not None:
                layer_tap.append(x.clone())
        return ops.rmsnorm_f32(x, self.final_norm, eps, rows=sample_idx, dtype=dt)

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        return ops.linear(h, self.embed).float()


def random_weights(cfg: VivesunConfig, seed: int = 0, dtype=torch.bfloat16) -> Dict[str, torch.Tensor]:
    """Random weights under the checkpoint's tensor names (benchmarks, tests, smoke runs)."""
    g = torch.Generator().manual_seed(seed)
    W, S = cfg.hidden, cfg.side_dim

    def rnd(*shape, std):
        return (torch.randn(*shape, generator=g) * std).to(dtype)

    def around1(n):
        return (1.0 + 0.1 * torch.randn(n, generator=g)).to(dtype)

    sd = W ** -0.5
    w = {"embed": rnd(cfg.vocab_size, W, std=1.0), "final.norm": rnd(W, std=0.1)}
    if cfg.bigram is not None:
        w["bigram"] = rnd(cfg.bigram.buckets + 1, W, std=0.7)
    if S:
        w["side.embed"] = rnd(cfg.vocab_size, cfg.layers * S, std=1.0)
    for i, b in enumerate(cfg.blocks):
        p, m = f"l{i}.", b.mixer
        w[p + "norm1"] = rnd(W, std=0.1)
        if b.type == "delta":
            nq, nv, Hh = m.kv_heads * m.dim, m.heads * m.vdim, m.heads
            w.update({p + "mix.q": rnd(nq, W, std=sd), p + "mix.k": rnd(nq, W, std=sd), p + "mix.v": rnd(nv, W, std=sd),
                      p + "mix.g": rnd(nv, W, std=sd), p + "mix.b": rnd(Hh, W, std=sd), p + "mix.a": rnd(Hh, W, std=sd),
                      p + "mix.q.conv": rnd(nq, m.conv, std=0.6), p + "mix.k.conv": rnd(nq, m.conv, std=0.6),
                      p + "mix.v.conv": rnd(nv, m.conv, std=0.6),
                      p + "mix.A_log": (-1.0 + torch.randn(Hh, generator=g)).to(dtype),
                      p + "mix.dt_bias": (-2.0 + torch.randn(Hh, generator=g)).to(dtype),
                      p + "mix.norm": around1(m.vdim), p + "mix.o": rnd(W, nv, std=nv ** -0.5)})
        else:
            a, nr = m.left, m.right.heads * m.right.dim
            rank = m.right.decay_rank or max(1, min(64, W // 4))
            pl, pr = p + "mix.left.", p + "mix.right."
            w.update({pl + "q": rnd(a.heads * a.dim, W, std=sd), pl + "k": rnd(a.kv_heads * a.dim, W, std=sd),
                      pl + "v": rnd(a.kv_heads * a.vdim, W, std=sd),
                      pl + "o": rnd(W, a.heads * a.vdim, std=(a.heads * a.vdim) ** -0.5)})
            w.update({pr + n: rnd(nr, W, std=sd) for n in ("r", "k", "v", "g", "a")})
            w.update({pr + "a.b": rnd(nr, std=0.5), pr + "w1": rnd(rank, W, std=sd), pr + "w2": rnd(nr, rank, std=rank ** -0.5),
                      pr + "w0": (-3.0 + torch.randn(nr, generator=g)).to(dtype), pr + "norm": around1(nr),
                      pr + "o": rnd(W, nr, std=nr ** -0.5)})
        f = b.mlp
        if f is not None:
            w.update({p + "norm2": rnd(W, std=0.1), p + "mlp.router": rnd(f.experts, W, std=sd)})
            for e in range(f.experts):
                w.update({f"{p}mlp.e{e}.up": rnd(f.ff, W, std=sd), f"{p}mlp.e{e}.down": rnd(W, f.ff, std=f.ff ** -0.5)})
        if S:
            w.update({p + "side.gate": rnd(S, W, std=sd), p + "side.proj": rnd(W, S, std=S ** -0.5), p + "side.norm": around1(W)})
    return w
