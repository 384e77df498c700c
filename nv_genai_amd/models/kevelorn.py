"""Kevelorn decoder on the gfx950 kernel set: pre-norm layers with scaled sub-layer outputs on an
fp32 residual stream, linear recurrences with a diagonal decay (one of them side by side with
windowed attention), dense or routed feed-forwards, and a span of layers that runs several times.

Per layer run (``x`` is the fp32 residual stream, activations in the model dtype; norm weights of the
model width are stored around zero and applied as ``1 + w``; m = ``residual_mult``):

    h  = norm1(x)                                   fused into the previous run's last step
    x += m mixer(h); h2 = norm2(x)                  ops.residual_step_
    x += m ff(h2) [+ x0] [+ step_t]; h = next norm  ops.residual_step_ / ops.residual_glu_experts_

The bracketed additions (x0 = the embedding rows) are those in front of a pass of the repeated span; they
ride on the step in front of it. Every layer *run* has pages / a state slot tensor of its own, so the
passes of the span do not share a cache.

Mixers:

* ``lightning`` - one GEMM gives ``q | k | v | output gate``; ``ops.linear_scan`` carries the fp32 state of
  every sequence in a state slot handed out by the scheduler (silu on q, k, v, one decay per head);
  ``ops.group_rmsnorm`` norms all heads together and applies the weight and the sigmoid gate.
* ``gla`` - the same with a decay per key channel and token: ``a1`` columns of the same GEMM, a small GEMM
  for ``a2``, sigmoid^(1 / tau) inside the scan; a norm per head, a silu gate.
* ``parallel`` - one GEMM gives the projections of both halves. Left: rotary positions, unit RMS of the heads
  and page write (``ops.rope_headnorm_cache_``), windowed softmax attention with a gate per element. Right: a
  ``lightning`` recurrence. Both outputs are normed over the width and summed in the residual step.

The serving engine drives this class as it drives the other decoders (``forward`` on a step's token
rows + ``logits``); ``AttnMeta`` carries the per-step row maps (``tok_seq``, state slots).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

from .. import ops
from ..parallel.dist import ParallelContext, get_context
from .config import KevelornConfig, SharedMoeSpec
from .llama import AttnMeta

MAX_KEY = 256       # widest key of a recurrent head the scan kernels take
MIN_LOG = -1.0e4    # log of a decay of zero (its first power is already zero in fp32)


def _ceil8(n: int) -> int:
    return (n + 7) // 8 * 8


class KevelornModel:
    stateful = True                # recurrent layers keep per-sequence state in scheduler slots
    uses_decode_workspace = False
    supports_step_graphs = False   # prefill / mixed steps run eagerly (decode steps are graphs)
    supports_prefix_cache = False  # a cached page carries no recurrent state

    def __init__(self, cfg: KevelornConfig, device="cuda", dtype=torch.bfloat16,
                 pctx: Optional[ParallelContext] = None, seed: int = 0,
                 weights: Optional[Dict[str, torch.Tensor]] = None, fp8: bool = False):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Kevelorn runs in bfloat16 or float32")
        if fp8:
            raise NotImplementedError("FP8 projections cover the Llama-layout decoders")
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.p = pctx or get_context()
        if self.p.tp_size > 1 or self.p.pp_size > 1:
            raise NotImplementedError("Kevelorn runs on one GPU per replica (no TP / PP split)")
        for b in cfg.blocks:
            if (b.mixer.right if b.type == "parallel" else b.mixer).dim > MAX_KEY:
                raise ValueError(f"recurrent heads of more than {MAX_KEY} key channels")
        self.fp8 = False
        self.kv_dtype, self.kv_scales = "auto", (1.0, 1.0)
        self.sequence_parallel, self.sp_min_tokens, self.split_mixed, self.moe_ws = False, 0, False, None
        att = [b.mixer.left for b in cfg.blocks if b.type == "parallel"]
        self.hq, self.hkv, self.D = (att[0].heads, att[0].kv_heads, att[0].dim) if att else (1, 1, 1)
        self.n_experts = cfg.num_experts
        self.vocab_local = cfg.vocab_size
        self.runs = cfg.runs               # (layer, number of the pass that begins here or None) in running order
        self.k_cache: List[Optional[torch.Tensor]] = []   # per run
        self.v_cache: List[Optional[torch.Tensor]] = []
        self.rec_state: List[torch.Tensor] = []
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

        def pad8(M):
            """Zero rows up to a multiple of 8 outputs."""
            pad = _ceil8(M.shape[0]) - M.shape[0]
            return torch.cat([M, torch.zeros(pad, M.shape[1], dtype=M.dtype, device=M.device)]) if pad else M

        self.norm_weights: Dict[str, torch.Tensor] = {}     # as stored, around zero

        def norm(name):
            self.norm_weights[name] = vec(name, W)
            return 1.0 + self.norm_weights[name]

        def lightning(p, m):
            """(q | k | v | g matrices, the rest of a lightning recurrence's parameters)."""
            nq, nv = m.heads * m.dim, m.heads * m.vdim
            log = [max(MIN_LOG, math.log(v)) if v > 0 else MIN_LOG for v in m.decay]
            return ([mat(p + "q", (nq, W)), mat(p + "k", (nq, W)), mat(p + "v", (nv, W)), mat(p + "g", (nv, W))],
                    {"on": vec(p + "norm", nv), "log_decay": torch.tensor(log, dtype=torch.float32, device=dev)})

        self.embed = mat("embed", (cfg.vocab_size, W))
        self.loop_step = mat("loop.step", (cfg.loop.times, W), torch.float32) if cfg.loop is not None else None
        self.layers: List[dict] = []
        for i, b in enumerate(cfg.blocks):
            p, m = f"l{i}.", b.mixer
            L = {"type": b.type, "spec": m, "mlp": b.mlp, "norm1": norm(p + "norm1")}
            if b.type == "lightning":
                mats, rest = lightning(p + "mix.", m)
                L.update(rest)
                L["w_in"], L["off"] = pad8(torch.cat(mats)).contiguous(), 0
                L["wo"] = mat(p + "mix.o", (W, m.heads * m.vdim))
            elif b.type == "gla":
                nq, nv = m.heads * m.dim, m.heads * m.vdim
                rank = w[p + "mix.a1"].shape[0]        # (the low rank of the decay is the tensor's own)
                a1 = pad8(mat(p + "mix.a1", (rank, W)))
                L["w_in"] = pad8(torch.cat([a1, mat(p + "mix.q", (nq, W)), mat(p + "mix.k", (nq, W)),
                                            mat(p + "mix.v", (nv, W)), mat(p + "mix.g", (nv, W))])).contiguous()
                L["rank"], L["off"] = rank, a1.shape[0]
                L["wa"], L["ab"] = mat(p + "mix.a2", (nq, rank)), vec(p + "mix.a2.b", nq)
                L["on"] = vec(p + "mix.norm", m.vdim)
                L["wo"] = mat(p + "mix.o", (W, nv))
            elif b.type == "parallel":
                a, r = m.left, m.right
                pl, pr = p + "mix.left.", p + "mix.right."
                nq, nk, nv, ng = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim, a.heads * a.vdim
                mats, rest = lightning(pr, r)
                L.update(rest)
                L["w_in"] = pad8(torch.cat([mat(pl + "q", (nq, W)), mat(pl + "k", (nk, W)), mat(pl + "v", (nv, W)),
                                            mat(pl + "g", (ng, W)), *mats])).contiguous()
                L["off"] = nq + nk + nv + ng
                L["freq"] = ops.rotary_frequencies(a.rot.dims, a.rot.base, linear=a.rot.linear)[0].to(dev)
                L["wo_left"], L["wo"] = mat(pl + "o", (W, ng)), mat(pr + "o", (W, r.heads * r.vdim))
                L["pair"] = (vec(pl + "out", W), vec(pr + "out", W))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {b.type!r}")
            f = b.mlp
            if f is not None:
                L["norm2"] = norm(p + "norm2")
            if isinstance(f, SharedMoeSpec):
                L["router"] = mat(p + "mlp.router", (f.experts, W), torch.float32)
                L["w13"] = torch.stack([torch.cat([mat(f"{p}mlp.e{e}.gate", (f.ff, W)), mat(f"{p}mlp.e{e}.up", (f.ff, W))])
                                        for e in range(f.experts)]).contiguous()
                L["w2"] = torch.stack([mat(f"{p}mlp.e{e}.down", (W, f.ff)) for e in range(f.experts)]).contiguous()
                if f.shared:
                    ps = p + "mlp.shared."
                    L["wsgu"] = pad8(torch.cat([mat(ps + "gate", (f.shared, W)), mat(ps + "up", (f.shared, W)),
                                                mat(ps + "sg", (1, W))])).contiguous()
                    L["wsd"] = mat(ps + "down", (W, f.shared))
            elif f is not None:
                L["wgu"] = torch.cat([mat(p + "mlp.gate", (f.ff, W)), mat(p + "mlp.up", (f.ff, W))]).contiguous()
                L["wd"] = mat(p + "mlp.down", (W, f.ff))
            self.layers.append(L)
        self.final_norm = norm("final.norm")
        self.lm_head = mat("head", (cfg.vocab_size, W))

    def state_dict(self) -> Dict[str, torch.Tensor]:
        dt = self.dtype
        out = {"embed": self.embed, "head": self.lm_head, **{k: v.to(dt) for k, v in self.norm_weights.items()}}
        if self.loop_step is not None:
            out["loop.step"] = self.loop_step.to(dt)
        for i, L in enumerate(self.layers):
            p, m, f, Wi = f"l{i}.", L["spec"], L["mlp"], L["w_in"]

            def rows(prefix, at, *parts):
                for name, n in parts:
                    out[prefix + name] = Wi[at:at + n]
                    at += n

            pm, r = p + "mix.", m
            if L["type"] == "parallel":
                a, r = m.left, m.right
                rows(pm + "left.", 0, ("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim),
                     ("g", a.heads * a.vdim))
                out.update({pm + "left.o": L["wo_left"], pm + "left.out": L["pair"][0].to(dt),
                            pm + "right.out": L["pair"][1].to(dt)})
                pm += "right."
            elif L["type"] == "gla":
                out.update({pm + "a1": Wi[:L["rank"]], pm + "a2": L["wa"], pm + "a2.b": L["ab"].to(dt)})
            nq, nv = r.heads * r.dim, r.heads * r.vdim
            rows(pm, L["off"], ("q", nq), ("k", nq), ("v", nv), ("g", nv))
            out.update({pm + "norm": L["on"].to(dt), pm + "o": L["wo"]})
            if isinstance(f, SharedMoeSpec):
                out[p + "mlp.router"] = L["router"].to(dt)
                for e in range(f.experts):
                    out.update({f"{p}mlp.e{e}.gate": L["w13"][e, :f.ff], f"{p}mlp.e{e}.up": L["w13"][e, f.ff:],
                                f"{p}mlp.e{e}.down": L["w2"][e]})
                if f.shared:
                    s = f.shared
                    out.update({p + "mlp.shared.gate": L["wsgu"][:s], p + "mlp.shared.up": L["wsgu"][s:2 * s],
                                p + "mlp.shared.sg": L["wsgu"][2 * s:2 * s + 1], p + "mlp.shared.down": L["wsd"]})
            elif f is not None:
                out.update({p + "mlp.gate": L["wgu"][:f.ff], p + "mlp.up": L["wgu"][f.ff:], p + "mlp.down": L["wd"]})
        return out

    # ------------------------------------------------------------------ cache and state
    def allocate_kv_cache(self, num_blocks: int, block_size: int = 64, kv_dtype: str = "auto",
                          kv_scales=(1.0, 1.0)):
        """Row-major pages in the model dtype, one K [blocks, kv_heads, 64, dim] and one V [blocks,
        kv_heads, 64, vdim] tensor per *run* of a ``parallel`` layer (a layer of the repeated span has
        one pair per pass), all addressed by the same page numbers; the other runs have none."""
        if block_size != 64:
            raise ValueError("the gfx950 attention kernels use 64-token KV pages")
        if kv_dtype not in ("auto", "bf16"):
            raise ValueError("Kevelorn keeps its KV pages in the model dtype")
        self.k_cache, self.v_cache = [], []
        for li, _ in self.runs:
            L = self.layers[li]
            if L["type"] == "parallel":
                a = L["spec"].left
                self.k_cache.append(torch.zeros(num_blocks, a.kv_heads, block_size, a.dim, device=self.device, dtype=self.dtype))
                self.v_cache.append(torch.zeros(num_blocks, a.kv_heads, block_size, a.vdim, device=self.device, dtype=self.dtype))
            else:
                self.k_cache.append(None)
                self.v_cache.append(None)
        return self.k_cache, self.v_cache

    def allocate_state(self, slots: int) -> None:
        """Recurrent state: per run the fp32 matrix memory [slots, heads, dim, vdim]. A slot needs no
        clearing when it is given to a new sequence: a segment that starts at position 0 starts from
        zeros, not from the slot."""
        self.rec_state = []
        for li, _ in self.runs:
            m = self.layers[li]["spec"]
            m = m.right if self.layers[li]["type"] == "parallel" else m
            self.rec_state.append(torch.zeros(max(1, slots), m.heads, m.dim, m.vdim, device=self.device, dtype=torch.float32))

    def kv_block_bytes(self, block_size: int = 64, kv_dtype: str = "auto") -> int:
        elem = torch.finfo(self.dtype).bits // 8
        n = 0
        for li, _ in self.runs:
            b = self.cfg.blocks[li]
            if b.type == "parallel":
                n += b.mixer.left.kv_heads * (b.mixer.left.dim + b.mixer.left.vdim)
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

    def _attend(self, q, gate, kc, vc, pos, meta: AttnMeta, a, **kw):
        """Softmax attention of a step's rows: prompt portions on the MFMA tile kernel and
        single-token rows on the page-parallel kernel where they apply (bf16, tile-sized
        heads), everything else on the row kernel."""
        H, G, dk, dv = a.heads, a.kv_heads, a.dim, a.vdim
        if self.mfma and ops.softmax_attention_mfma_ok(q, dk, dv, H // G, 1):
            nd = meta.n_decode if meta.kind == "mixed" else (q.shape[0] if meta.kind == "decode" else 0)
            out = torch.empty(q.shape[0], H * dv, dtype=q.dtype, device=q.device)
            if nd:
                ops.softmax_attention_rows(q[:nd], kc, vc, meta.block_tables, meta.tok_seq[:nd], pos[:nd], H, G, dk,
                                           dv, max_ctx=meta.max_ctx, gate=gate[:nd], out=out[:nd], **kw)
            if nd < q.shape[0]:
                ops.softmax_attention_prefill(q[nd:], kc, vc, meta.block_tables[nd:],
                                              meta.cu_q_prefill if nd else meta.cu_q, meta.ctx_lens[nd:],
                                              meta.max_q_len, H, G, dk, dv, gate=gate[nd:], out=out[nd:], **kw)
            return out
        return ops.softmax_attention(q, kc, vc, meta.block_tables, meta.tok_seq, pos, H, G, dk, dv, gate=gate, **kw)

    def _recurrence(self, ri: int, L: dict, m, proj, pos, meta: AttnMeta, **decay):
        """Rows of the recurrence whose ``q | k | v | gate`` columns start at ``L["off"]``, normed and gated."""
        nq, nv, c = m.heads * m.dim, m.heads * m.vdim, L["off"]
        light = L["type"] != "gla"
        o = ops.linear_scan(proj[:, c:c + nq], proj[:, c + nq:c + 2 * nq], proj[:, c + 2 * nq:c + 2 * nq + nv],
                            self.rec_state[ri], m.heads, m.dim, m.vdim, pos=pos, silu=light,
                            q_scale=1.0 if light else m.dim ** -0.5, **decay, **self._segments(meta))
        return ops.group_rmsnorm(o, L["on"], 1 if light else m.heads, self.cfg.eps, self.dtype,
                                 gate=proj[:, c + 2 * nq + nv:c + 2 * nq + 2 * nv], gate_act="sigmoid" if light else "silu")

    def _mix(self, ri: int, L: dict, h, pos, meta: AttnMeta) -> dict:
        """The mixer's output(s) as :func:`ops.residual_step_` takes them."""
        m = L["spec"]
        proj = self._lin(h, L["w_in"])
        if L["type"] == "lightning":
            return dict(y=self._lin(self._recurrence(ri, L, m, proj, pos, meta, log_decay=L["log_decay"]), L["wo"]))
        if L["type"] == "gla":
            z = self._lin(proj[:, :L["rank"]], L["wa"])
            return dict(y=self._lin(self._recurrence(ri, L, m, proj, pos, meta, z=z, z_bias=L["ab"], tau=m.tau), L["wo"]))
        a = m.left
        nq = a.heads * a.dim
        g0 = (a.heads + a.kv_heads) * a.dim + a.kv_heads * a.vdim
        kc, vc = self.k_cache[ri], self.v_cache[ri]
        ops.rope_headnorm_cache_(proj, pos, meta.slots, kc, vc, a.heads, a.kv_heads, a.dim, a.vdim, L["freq"], 1.0,
                                 a.rot.dims, self.cfg.eps, v_off=(a.heads + a.kv_heads) * a.dim,
                                 interleaved=a.rot.interleaved, unit=True)
        left = self._attend(proj[:, :nq], proj[:, g0:g0 + a.heads * a.vdim], kc, vc, pos, meta, a, scale=a.scale,
                            window=a.window)
        right = self._recurrence(ri, L, m.right, proj, pos, meta, log_decay=L["log_decay"])
        return dict(y=self._lin(left, L["wo_left"]), y2=self._lin(right, L["wo"]), pair=L["pair"],
                    mult=0.5 * self.cfg.residual_mult)

    def forward(self, ids: torch.Tensor, pos: torch.Tensor, meta: AttnMeta,
                sample_idx: Optional[torch.Tensor] = None, embed_override=None,
                layer_tap: Optional[list] = None) -> torch.Tensor:
        """Final-normed rows selected by ``sample_idx`` (all rows if None) of a step's token rows.
        ``layer_tap``: a list that receives a copy of the residual stream after every layer run."""
        if embed_override is not None:
            raise NotImplementedError("Kevelorn takes token ids only")
        if meta.tok_seq is None or meta.state_slots is None:
            raise ValueError("Kevelorn steps need the engine's row maps (tok_seq, state slots)")
        eps, dt, mult = self.cfg.eps, self.dtype, self.cfg.residual_mult
        x0 = ops.embed_rows(ids, self.embed, 1.0)
        x = x0.clone() if self.loop_step is not None else x0

        def ahead(ri):
            """(additions in front of run ri, weight of its first norm)."""
            if ri == len(self.runs):
                return {}, None
            li, t = self.runs[ri]
            add = {} if t is None else dict(row=self.loop_step[t], x0=x0 if t else None)
            return add, self.layers[li]["norm1"]

        def first(ri):
            add, w = ahead(ri)
            return ops.residual_step_(x, None, w, eps, dt, **add) if add else None if w is None else ops.rmsnorm_f32(x, w, eps, dtype=dt)

        h = first(0)
        for ri, (li, _) in enumerate(self.runs):
            L = self.layers[li]
            # (a tapped stream is the one ahead of the next pass's additions: they take a step of their own then)
            add, nxt = ahead(ri + 1) if layer_tap is None else ({}, None)
            y = {"mult": mult, **self._mix(ri, L, h, pos, meta)}
            f = L["mlp"]
            if f is None:
                h = ops.residual_step_(x, norm_w=nxt, eps=eps, dtype=dt, **y, **add)
            else:
                h2 = ops.residual_step_(x, norm_w=L["norm2"], eps=eps, dtype=dt, **y)
                if isinstance(f, SharedMoeSpec):
                    eid, ew = ops.moe_router(h2, L["router"], f.top, ws=self.moe_ws)
                    shared = None
                    if f.shared:
                        shared = self._lin(ops.clamped_glu(self._lin(h2, L["wsgu"]), f.shared, math.inf, 1.0, 2 * f.shared,
                                                           shift=0.0), L["wsd"])
                    h = ops.residual_glu_experts_(x, h2, eid, ew, L["w13"], L["w2"], nxt, eps, dt, mult, shared,
                                                  ws=self.moe_ws, **add)
                else:
                    h = ops.residual_step_(x, self._lin(ops.glu_gelu_tanh(self._lin(h2, L["wgu"])), L["wd"]), nxt, eps, dt,
                                           mult, **add)
            if layer_tap is not None:
                layer_tap.append(x.clone())
                h = first(ri + 1)
        return ops.rmsnorm_f32(x, self.final_norm, eps, rows=sample_idx, dtype=dt)

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        return ops.linear(h, self.lm_head).float()


def random_weights(cfg: KevelornConfig, seed: int = 0, dtype=torch.bfloat16) -> Dict[str, torch.Tensor]:
    """Random weights under the checkpoint's tensor names (benchmarks, tests, smoke runs)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg.hidden

    def rnd(*shape, std):
        return (torch.randn(*shape, generator=g) * std).to(dtype)

    def around1(n):
        return (1.0 + 0.1 * torch.randn(n, generator=g)).to(dtype)

    def recurrence(p, m, norm):
        nq, nv = m.heads * m.dim, m.heads * m.vdim
        return {p + "q": rnd(nq, W, std=sd), p + "k": rnd(nq, W, std=sd), p + "v": rnd(nv, W, std=sd),
                p + "g": rnd(nv, W, std=sd), p + "norm": around1(norm), p + "o": rnd(W, nv, std=nv ** -0.5)}

    def glu(p, ff):
        return {p + "gate": rnd(ff, W, std=sd), p + "up": rnd(ff, W, std=sd), p + "down": rnd(W, ff, std=ff ** -0.5)}

    sd = W ** -0.5
    w = {"embed": rnd(cfg.vocab_size, W, std=1.0), "head": rnd(cfg.vocab_size, W, std=sd), "final.norm": rnd(W, std=0.1)}
    if cfg.loop is not None:
        w["loop.step"] = rnd(cfg.loop.times, W, std=0.5)
    for i, b in enumerate(cfg.blocks):
        p, m = f"l{i}.", b.mixer
        w[p + "norm1"] = rnd(W, std=0.1)
        if b.type == "lightning":
            w.update(recurrence(p + "mix.", m, m.heads * m.vdim))
        elif b.type == "gla":
            nq, rank = m.heads * m.dim, m.rank or max(1, min(64, W // 16))
            w.update(recurrence(p + "mix.", m, m.vdim))
            w.update({p + "mix.a1": rnd(rank, W, std=sd), p + "mix.a2": rnd(nq, rank, std=rank ** -0.5),
                      p + "mix.a2.b": rnd(nq, std=1.0)})
        else:
            a, pl = m.left, p + "mix.left."
            na = a.heads * a.vdim
            w.update({pl + "q": rnd(a.heads * a.dim, W, std=sd), pl + "k": rnd(a.kv_heads * a.dim, W, std=sd),
                      pl + "v": rnd(a.kv_heads * a.vdim, W, std=sd), pl + "g": rnd(na, W, std=sd),
                      pl + "o": rnd(W, na, std=na ** -0.5), pl + "out": around1(W), p + "mix.right.out": around1(W)})
            w.update(recurrence(p + "mix.right.", m.right, m.right.heads * m.right.vdim))
        f = b.mlp
        if f is not None:
            w[p + "norm2"] = rnd(W, std=0.1)
        if isinstance(f, SharedMoeSpec):
            w[p + "mlp.router"] = rnd(f.experts, W, std=sd)
            for e in range(f.experts):
                w.update(glu(f"{p}mlp.e{e}.", f.ff))
            if f.shared:
                w.update(glu(p + "mlp.shared.", f.shared))
                w[p + "mlp.shared.sg"] = rnd(1, W, std=sd)
        elif f is not None:
            w.update(glu(p + "mlp.", f.ff))
    return w
