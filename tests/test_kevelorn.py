"""Kevelorn on the serving engine against the plain oracle (tests/kevelorn_oracle.py).

Every case runs on the CPU (the engine on the fp32 reference ops: scheduling, pages, state slots,
row maps) and, marked ``gpu``, on the HIP kernels in float32 and bfloat16. The models are small
random ones built here; sizes are chosen so that heads, dims, window and page size do not coincide
(``odd``: a rotation on part of the head, a window that is no multiple of the page, layers without
feed-forward or shared expert), or so that the MFMA tile kernels run (``tiles``).
"""
import json
import math

import pytest
import torch

import kevelorn_oracle as O
from nv_genai_amd import ops
from nv_genai_amd.engine.llm_engine import EngineConfig, LLMEngine, SamplingParams
from nv_genai_amd.models.config import KevelornConfig, kevelorn_layers
from nv_genai_amd.models.kevelorn import KevelornModel, random_weights

GPU = pytest.param("cuda", marks=pytest.mark.gpu)
DEVICES = ["cpu", GPU]
DTYPES = [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
          pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)]


def moe(experts=5, top=3, ff=14, shared=10):
    d = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared:
        d["shared"] = {"ff": shared}
    return d


def dense(ff=22):
    return {"kind": "dense", "ff": ff}


def light(heads=3, dim=9, vdim=7, decay=(0.3, 0.93, 0.9975)):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def lightning(mlp=None, **kw):
    return {"type": "lightning", "mixer": light(**kw), "mlp": mlp}


def gla(heads=3, dim=10, vdim=13, tau=7.0, rank=5, mlp=None):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "rank": rank}, "mlp": mlp}


def par(heads=4, kv=2, dim=12, vdim=6, window=27, dims=8, base=50.0, factor=3.0, scale=0.8, right=None, mlp=None):
    rot = {"base": base, "dims": dims}
    if factor:
        rot["scaling"] = {"factor": factor}
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    if window:
        left["mask"] = {"size": window}
    return {"type": "parallel", "mixer": {"left": left, "right": right or light()}, "mlp": mlp}


def cfg_dict(layers, width=40, vocab=97, eps=1e-5, mult=0.6, loop=None):
    d = {"architecture": "Kevelorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
         "layers": layers}
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


def cfg_odd():
    return cfg_dict([lightning(mlp=dense()), par(mlp=moe()), gla(mlp=moe(3, 2, 9, 0)), lightning(heads=2, dim=5, vdim=11, decay=(0.8, 0.99)),
                     par(heads=3, kv=1, dim=6, vdim=10, window=100, dims=6, factor=None, right=light(heads=1, dim=17, vdim=4, decay=(0.97,)),
                         mlp=dense(13))], loop=(1, 4, 2))


def cfg_tiles():
    """Sizes the MFMA kernels take: 128-wide heads with GQA, experts of 128 on a width of 256, a window longer
    than a page and no multiple of it; a span that starts at the first layer and runs three times."""
    return cfg_dict([par(heads=8, kv=2, dim=128, vdim=64, window=80, dims=32, base=1e4, scale=0.2,
                         right=light(heads=4, dim=32, vdim=64, decay=(0.5, 0.9, 0.99, 0.999)), mlp=dense(96)),
                     gla(heads=2, dim=64, vdim=32, tau=16.0, rank=8, mlp=moe(4, 2, 128, 64))], width=256, loop=(0, 2, 3))


CFGS = {"odd": cfg_odd, "tiles": cfg_tiles}


def build(device, dtype="float32", seed=0, pages=24, seqs=4, cd=None, graphs=None, **eng):
    cd = cd or cfg_odd()
    cfg = KevelornConfig.from_dict(cd)
    w = random_weights(cfg, seed, torch.bfloat16)       # bf16 values, as a checkpoint holds them
    for k in w:
        if k.endswith("mlp.router"):
            w[k] = w[k] * 4.0                           # wide logits: few near ties between experts
    tdt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype]
    model = KevelornModel(cfg, device, tdt, weights=w)
    kw = dict(model="kevelorn-test", dtype=dtype, max_num_seqs=seqs, max_batched_tokens=512, max_model_len=512,
              kv_cache_blocks=pages, detokenize=False, use_graphs=(device == "cuda") if graphs is None else graphs,
              graph_batch_sizes=(1, 2, 4), mixed_graphs=False, logits_tap=True, tuned_gemms=False, async_decode=False)
    kw.update(eng)
    e = LLMEngine(EngineConfig(**kw), device=device, model=model)
    return e, cd, w


def tokens(n, vocab=97, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def tol(dtype):
    return 2e-4 if dtype == "float32" else 6e-2


def close(got, want, dtype, what=""):
    got, want = got.double().cpu(), want.double()
    err = (got - want).abs().max().item() / max(1.0, want.abs().max().item())
    assert err < tol(dtype), f"{what}: relative error {err:.3e}"


def close_rows(got, want, dtype, what=""):
    """Model outputs, one row per token. In bfloat16 the router reads rounded activations, so a token
    whose k-th and (k+1)-th choice nearly tie may take another expert than the oracle does: there
    the comparison allows a few rows (two, or 3 %) to differ; every other row, and every row in
    float32, must agree. (The test models' routers are scaled up so that near ties are rare.)"""
    if dtype == "float32":
        return close(got, want, dtype, what)
    got, want = got.double().cpu(), want.double()
    err = (got - want).abs().flatten(1).max(dim=1).values / max(1.0, want.abs().max().item())
    bad = int((err >= tol(dtype)).sum())
    assert bad <= max(2, 0.03 * err.numel()), f"{what}: {bad} of {err.numel()} rows differ (worst {err.max().item():.3e})"


def tdtype(dtype):
    return {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype]


def i32(*v, device="cpu"):
    return torch.tensor(v, dtype=torch.int32, device=device)


def replay_cuts(eng, toks, cuts, rid=1, finish=True):
    """Feed ``toks`` in portions of the given sizes (the rest one token at a time); all logits."""
    out, at, cuts = [], 0, list(cuts)
    while at < len(toks):
        n = min(cuts.pop(0) if cuts else 1, len(toks) - at)
        done = at + n == len(toks)
        out.append(eng.replay_step([(rid, toks[at:at + n], list(range(n)))], [rid] if done and finish else []))
        at += n
    return torch.cat(out)


# ---------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("T,H", [(9, 30), (5, 40), (33, 1024), (40, 5120), (7, 4098)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_residual_step_forms(device, dtype, T, H):
    """Scaled sum, sum of two outputs, pair of norms, additions in front of a pass, expert rows summed straight
    into the stream, with and without the norm behind it."""
    check_residual_step(device, dtype, T, H)


@pytest.mark.gpu
@pytest.mark.parametrize("T,H", [(4100, 256), (4097, 1000), (4100, 3000)])
def test_residual_step_of_many_rows(T, H):
    check_residual_step("cuda", "bfloat16", T, H)


def check_residual_step(device, dtype, T, H):
    tdt, eps, m = tdtype(dtype), 1e-3, 0.37
    g = torch.Generator().manual_seed(37)
    x, x0 = 3.0 * torch.randn(T, H, generator=g), torch.randn(T, H, generator=g)
    y, y2 = (torch.randn(T, H, generator=g).to(tdt) for _ in range(2))
    w, w1, w2, row = (1 + 0.3 * torch.randn(H, generator=g) for _ in range(4))
    xd, yd, y2d = x.double(), y.double(), y2.double()
    pair = O.unit_rms(yd, eps) * w1.double() + O.unit_rms(y2d, eps) * w2.double()
    d = lambda t: t.to(device)   # noqa: E731
    cases = {
        "scaled": (dict(y=d(y)), xd + m * yd),
        "two outputs": (dict(y=d(y), y2=d(y2)), xd + m * (yd + y2d)),
        "pair of norms": (dict(y=d(y), y2=d(y2), pair=(d(w1), d(w2))), xd + m * pair),
        "first pass": (dict(y=d(y), row=d(row)), xd + m * yd + row.double()),
        "later pass": (dict(y=d(y), row=d(row), x0=d(x0)), xd + m * yd + row.double() + x0.double()),
        "pair in front of a pass": (dict(y=d(y), y2=d(y2), pair=(d(w1), d(w2)), row=d(row), x0=d(x0)),
                                    xd + m * pair + row.double() + x0.double()),
        "additions alone": (dict(y=None, row=d(row), x0=d(x0)), xd + row.double() + x0.double())}
    for what, (kw, want) in cases.items():
        s = d(x.clone())
        h = ops.residual_step_(s, norm_w=d(w), eps=eps, dtype=tdt, mult=m, **kw)
        close(s, want, "float32", what + ": stream")
        close(h, O.unit_rms(want, eps) * w.double(), dtype, what + ": norm")
        s = d(x.clone())
        assert ops.residual_step_(s, norm_w=None, eps=eps, dtype=tdt, mult=m, **kw) is None
        close(s, want, "float32", what + ": no norm")


@pytest.mark.parametrize("W,E,k,F", [(40, 5, 3, 14), (37, 1, 1, 9), (256, 4, 2, 128), (256, 6, 6, 96)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_experts_summed_into_the_scaled_stream(device, dtype, W, E, k, F):
    """Router, SwiGLU experts, shared expert times its gate, all into the stream times the multiplier."""
    tdt, m, eps = tdtype(dtype), 0.45, 1e-5
    g = torch.Generator().manual_seed(3)
    for T in (33, 600):
        x, h = torch.randn(T, W, generator=g), torch.randn(T, W, generator=g).to(tdt)
        w = {f"e{e}.{n}": (torch.randn(*s, generator=g) * s[1] ** -0.5).to(tdt) for e in range(E)
             for n, s in (("gate", (F, W)), ("up", (F, W)), ("down", (W, F)))}
        w["router"] = 3.0 * torch.randn(E, W, generator=g) * W ** -0.5
        if E > 2:
            w["router"][2] = w["router"][1]                 # equal logits: the lower index first
        want = x.double() + m * O.moe_ff(h.double(), {"router": {"top": k}}, w, "")
        ids, wts = ops.moe_router(h.to(device), w["router"].to(device), k)
        w13 = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)]).to(device)
        w2 = torch.stack([w[f"e{e}.down"] for e in range(E)]).to(device)
        add = torch.randn(T, W, generator=g).to(tdt)
        nw = 1 + 0.2 * torch.randn(W, generator=g)
        s = x.clone().to(device)
        out = ops.residual_glu_experts_(s, h.to(device), ids, wts, w13, w2, nw.to(device), eps, tdt, m, add.to(device))
        close(s, want + m * add.double(), dtype, f"stream, {T} rows")
        close(out, O.unit_rms(want + m * add.double(), eps) * nw.double(), dtype, "norm")
        s, row, x0 = x.clone().to(device), torch.randn(W, generator=g), torch.randn(T, W, generator=g)
        assert ops.residual_glu_experts_(s, h.to(device), ids, wts, w13, w2, None, eps, tdt, m, x0=x0.to(device),
                                         row=row.to(device)) is None
        close(s, want + x0.double() + row.double(), dtype, "no shared expert, in front of a pass")


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_gated_norms_over_heads_and_over_the_row(device, dtype):
    """One norm per head (one weight per element, silu gate) and one over all columns (a weight per column,
    sigmoid gate), narrow rows and rows of several registers per thread."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(8)
    for T, H, n in ((9, 3, 13), (5, 1, 7), (20, 4, 64), (6, 8, 128), (3, 5, 500), (4, 16, 256), (3, 24, 256)):
        x = torch.randn(T, H * n, generator=g)
        x[0] *= 1e-3                                        # eps matters
        wide = torch.randn(T, H * n + 8, generator=g).to(tdt)
        gate = wide[:, :H * n]
        w, wr = 1 + 0.3 * torch.randn(n, generator=g), 1 + 0.3 * torch.randn(H * n, generator=g)
        gd = wide.to(device)[:, :H * n]
        got = ops.group_rmsnorm(x.to(device), w.to(device), H, 1e-5, tdt, gate=gd, gate_act="silu")
        want = (O.unit_rms(x.double().view(T, H, n), 1e-5) * w.double()).reshape(T, -1) * O.silu(gate.double())
        close(got, want, dtype, f"per head {T, H, n}")
        got = ops.group_rmsnorm(x.to(device), wr.to(device), 1, 1e-5, tdt, gate=gd)
        close(got, O.unit_rms(x.double(), 1e-5) * wr.double() * torch.sigmoid(gate.double()), dtype, f"whole row {T, H, n}")


def test_rotary_scaling_against_the_oracle():
    for dims, base, factor in ((8, 50.0, 3.0), (2, 1e4, 1.0), (64, 5e5, 0.5), (30, 7.0, 12.0)):
        f, mag = ops.rotary_frequencies(dims, base, linear=factor)
        want = O.rotary_frequencies({"dims": dims, "base": base, "scaling": {"factor": factor}})
        assert mag == 1.0 and (f - want).abs().max().item() < 1e-15
    assert torch.equal(O.rotary_frequencies({"dims": 8, "base": 9.0}), ops.rotary_frequencies(8, 9.0)[0])


@pytest.mark.parametrize("sizes", [(6, 2, 12, 8, 6), (4, 2, 64, 32, 64), (3, 1, 128, 128, 32), (9, 3, 32, 16, 24), (2, 2, 48, 48, 48),
                                   (1, 1, 2, 2, 1)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_rotation_then_unit_norm_and_page_write(device, dtype, sizes):
    """Neighbouring elements rotated together on part of the head or all of it, unit RMS of the rotated head
    (short heads: eps matters), positions far out, a row that is not written, the other columns untouched."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(5)
    H, G, dk, dims, dv = sizes
    T, eps = 9, 1e-4
    rot = {"dims": dims, "base": 30.0, "scaling": {"factor": 2.5}}
    freq, _ = ops.rotary_frequencies(dims, 30.0, linear=2.5)
    proj0 = torch.randn(T, (H + G) * dk + G * dv + 8, generator=g)
    proj0[3] *= 0.01
    proj0 = proj0.to(tdt)
    pos = i32(0, 1, 63, 64, 1000, 65535, 99999, 7, 2)
    slots = i32(0, 1, 63, 64, 130, 191, 5, -1, 70)
    kc = torch.zeros(3, G, 64, dk, dtype=tdt, device=device)
    vc = torch.zeros(3, G, 64, dv, dtype=tdt, device=device)
    proj = proj0.clone().to(device)
    ops.rope_headnorm_cache_(proj, pos.to(device), slots.to(device), kc, vc, H, G, dk, dv, freq.to(device), 1.0, dims, eps,
                             v_off=(H + G) * dk, interleaved=True, unit=True)
    pd = proj0.double()
    q, k = pd[:, :H * dk].view(T, H, dk), pd[:, H * dk:(H + G) * dk].view(T, G, dk)
    v = pd[:, (H + G) * dk:(H + G) * dk + G * dv].view(T, G, dv)
    qr, kr = (O.unit_rms(torch.stack([O.rotate(x[t:t + 1], rot, int(pos[t]))[0] for t in range(T)]), eps) for x in (q, k))
    close(proj[:, :H * dk], qr.reshape(T, -1), dtype, "queries")
    close(proj[:, H * dk:(H + G) * dk], kr.reshape(T, -1), dtype, "keys")
    assert torch.equal(proj[:, (H + G) * dk:].cpu(), proj0[:, (H + G) * dk:]), "the other columns stay"
    for t in range(T):
        s = int(slots[t])
        if s >= 0:
            close(kc[s // 64, :, s % 64], kr[t], dtype, f"K page row of token {t}")
            close(vc[s // 64, :, s % 64], v[t], dtype, f"V page row of token {t}")
    # neighbouring pairs without a norm
    proj = proj0.clone().to(device)
    ops.rope_headnorm_cache_(proj, pos.to(device), slots.to(device), kc, vc, H, G, dk, dv, freq.to(device), 1.0, dims, eps,
                             v_off=(H + G) * dk, interleaved=True)
    close(proj[:, :H * dk], torch.stack([O.rotate(q[t:t + 1], rot, int(pos[t]))[0] for t in range(T)]).reshape(T, -1), dtype, "no norm")


def _pages(rows, device, tdt, bt_row, nb):
    """Token rows [n, G, d] laid into pages [nb, G, 64, d] through the block-table row."""
    n, G, d = rows.shape
    page = torch.zeros(nb, G, 64, d, dtype=tdt, device=device)
    j = torch.arange(n)
    page[bt_row[j // 64].long(), :, j % 64] = rows.to(tdt).to(device)
    return page


def o_attention(q, K, V, scale, window, pos, gate):
    """Plain form: query t at position pos[t] sees itself and the window - 1 keys before it; q [T, H, d]."""
    T, H, _ = q.shape
    G = K.shape[1]
    out = torch.zeros(T, H, V.shape[2], dtype=torch.float64)
    for t in range(T):
        lo = max(0, int(pos[t]) - window + 1) if window else 0
        for h in range(H):
            kk, vv = (X[lo:int(pos[t]) + 1, h // (H // G)].double() for X in (K, V))
            out[t, h] = torch.softmax((kk @ q[t, h].double()) * scale, -1) @ vv
    return out.reshape(T, -1) * torch.sigmoid(gate.double())


@pytest.mark.parametrize("window", [0, 1, 50, 64, 128, 200])
@pytest.mark.parametrize("shape", [(6, 2, 10, 6), (4, 2, 64, 64), (8, 1, 128, 128), (9, 3, 96, 64), (2, 2, 32, 128), (5, 1, 48, 3)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_one_key_stands_out_in_windows(device, dtype, shape, window):
    """One key is made to match a scaled query: just inside and just outside the window, on both sides of
    page borders, far back, at the query's own position and one position after it. A key in sight takes
    nearly all the weight, one out of sight none. Through the row kernel, the single-token kernel and the
    prompt kernel, with a gate per output element whose rows lie inside a wider projection."""
    H, G, dk, dv = shape
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(11)
    n = 460
    K = (0.3 * torch.randn(n, G, dk, generator=g)).to(tdt).float()
    V = torch.randn(n, G, dv, generator=g).to(tdt).float()
    bt = torch.randperm(12, generator=g)[:8].to(torch.int32)
    scale = dk ** -0.5
    dev = lambda t: t.to(device)   # noqa: E731
    w = window or 300
    for hot in (3, 63, 64, 128, 191, 200, 255, 256):
        KK = K.clone()
        u = torch.randn(dk, generator=g)
        u = u / u.norm()
        KK[hot, 0] = (6.0 * u).to(tdt).float()
        kc, vc = _pages(KK, device, tdt, bt, 12), _pages(V, device, tdt, bt, 12)
        qpos = sorted({hot - 1, hot, hot + 1, hot + w - 2, hot + w - 1, hot + w, hot + w + 1, 459, 64, 63, 0} & set(range(n)))
        q = 0.3 * torch.randn(len(qpos), H, dk, generator=g)
        q[:, 0] = 20.0 * u / scale / 6.0      # head 0 (kv head 0): score 20 on the hot key
        q = q.to(tdt)
        wide = torch.randn(len(qpos), H * dv + 16, generator=g).to(tdt)
        pos = i32(*qpos)
        want = o_attention(q.float(), KK, V, scale, window, pos, wide[:, 8:8 + H * dv])
        qd, gd = dev(q.reshape(len(qpos), H * dk)), dev(wide)[:, 8:8 + H * dv]
        seq = torch.zeros(len(qpos), dtype=torch.int32, device=device)
        btd = dev(bt.view(1, -1))
        out = ops.softmax_attention(qd, kc, vc, btd, seq, dev(pos), H, G, dk, dv, scale=scale, window=window, gate=gd)
        close(out, want, dtype, f"row form, hot key {hot}")
        out = ops.softmax_attention_rows(qd, kc, vc, btd, seq, dev(pos), H, G, dk, dv, max_ctx=512, scale=scale, window=window, gate=gd)
        close(out, want, dtype, f"single form, hot key {hot}")
        gs = torch.sigmoid(wide[:, 8:8 + dv].double())
        for t, p in enumerate(qpos):
            seen = hot <= p and (not window or p - hot < window)
            hit = (out[t, :dv].double().cpu() - gs[t] * V[hot, 0].double()).abs().max().item() < 0.05
            if p > 0 and window != 1:
                assert hit == seen, f"query at {p}, hot key at {hot}: seen={seen}"
    # a portion that starts in the middle of a window and of a page
    lo, nq = 173, 460 - 173
    q = 0.3 * torch.randn(nq, H, dk, generator=g)
    q[:, H - 1] = 20.0 * u / scale / 6.0
    q = q.to(tdt)
    KK = K.clone()
    KK[250, G - 1] = (6.0 * u).to(tdt).float()
    kc, vc = _pages(KK, device, tdt, bt, 12), _pages(V, device, tdt, bt, 12)
    wide = torch.randn(nq, H * dv + 16, generator=g).to(tdt)
    want = o_attention(q.float(), KK, V, scale, window, torch.arange(lo, 460), wide[:, 8:8 + H * dv])
    out = ops.softmax_attention_prefill(dev(q.reshape(nq, H * dk)), kc, vc, dev(bt.view(1, -1)), i32(0, nq, device=device),
                                        i32(460, device=device), nq, H, G, dk, dv, scale=scale, window=window,
                                        gate=dev(wide)[:, 8:8 + H * dv])
    close(out, want, dtype, "portion")
    for p in {249, 250, 251, 250 + w - 2, 250 + w - 1, 250 + w, 459} & set(range(lo, 460)):
        seen = p >= 250 and (not window or p - 250 < window)
        gs = torch.sigmoid(wide[p - lo, 8 + (H - 1) * dv:8 + H * dv].double())
        hit = (out[p - lo, (H - 1) * dv:].double().cpu() - gs * V[250, G - 1].double()).abs().max().item() < 0.05
        if window != 1:
            assert hit == seen, f"portion: query at {p}"


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_one_gate_per_head_beside_one_per_element(device, dtype):
    """The two forms of the output gate in all three kernels."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(12)
    for (H, G, dk, dv) in ((3, 1, 10, 6), (4, 2, 64, 32), (2, 1, 32, 64)):
        K, V = torch.randn(100, G, dk, generator=g).to(tdt).float(), torch.randn(100, G, dv, generator=g).to(tdt).float()
        q = torch.randn(2, H, dk, generator=g).to(tdt)
        bt = i32(1, 0)
        kc, vc = _pages(K, device, tdt, bt, 2), _pages(V, device, tdt, bt, 2)
        pos = i32(99, 40)
        args = (q.reshape(2, -1).to(device), kc, vc, bt.view(1, -1).to(device))
        rows = (torch.zeros(2, dtype=torch.int32, device=device), pos.to(device), H, G, dk, dv)
        for cols in (H, H * dv):
            gate = (2.0 * torch.randn(2, cols, generator=g)).to(tdt)
            full = gate.double().view(2, H, -1).expand(2, H, dv).reshape(2, -1)
            want = o_attention(q.float(), K, V, 0.4, 0, pos, full)
            gd = gate.to(device)
            close(ops.softmax_attention(*args, *rows, scale=0.4, gate=gd), want, dtype, f"row, {cols} gates")
            close(ops.softmax_attention_rows(*args, *rows, scale=0.4, max_ctx=128, gate=gd), want, dtype, f"single, {cols} gates")
            one = ops.softmax_attention_prefill(args[0][:1], *args[1:], i32(0, 1, device=device), i32(100, device=device), 1,
                                                H, G, dk, dv, scale=0.4, gate=gd[:1])
            close(one, want[:1], dtype, f"portion, {cols} gates")


# ---------------------------------------------------------------------------- linear recurrences
def scan_call(device, q, k, v, state, H, d, dv, **decay):
    """call(segments, slots, single, n_single) on rows of one sequence; rows lie in one wider row."""
    z = decay.pop("z", None)
    row = torch.cat([q, k, v], 1).to(device)
    kw = {n: (t.to(device) if torch.is_tensor(t) else t) for n, t in decay.items()}
    zd = None if z is None else z.to(device)

    def call(segs, slots, single=False, n_single=0):
        rows = torch.cat([torch.arange(a, b) for a, b in segs]).to(device)
        cu = None if single else torch.tensor([0] + [b - a for a, b in segs]).cumsum(0).to(torch.int32).to(device)
        p = row[rows]
        zz = {} if zd is None else {"z": zd[rows]}
        return ops.linear_scan(p[:, :H * d], p[:, H * d:2 * H * d], p[:, 2 * H * d:], state, H, d, dv, cu,
                               i32(*slots, device=device), rows.to(torch.int32), n_single=n_single,
                               max_q=max(b - a for a, b in segs), **zz, **kw)

    return call


def check_scan(call, want, dtype, state, sp):
    """Portions of many sizes, single rows, slots, two segments with single rows in front."""
    T = want.shape[0]
    cuts = [0, 1, 20, 22, 27, 43, 44, 60]
    got = [call([(a, b)], [1]) for a, b in zip(cuts, cuts[1:])] + [call([(t, t + 1)], [1], single=True) for t in range(60, T)]
    close(torch.cat(got), want, dtype, "portions, then single rows")
    assert float((state[0] - sp).abs().max()) == 0.0 and float((state[2] - sp).abs().max()) == 0.0
    close(torch.cat([call([(t, t + 1)], [1], single=True) for t in range(T)]), want, dtype, "single rows from the first")
    keep = state.clone()
    close(call([(0, 30)], [-1]), want[:30], dtype, "no slot")
    assert torch.equal(keep, state)
    call([(0, 40)], [2])
    # two single rows (one that goes on, one fresh into a stale slot), then two portions
    call([(0, 50)], [3])
    out = call([(50, 51), (0, 1), (40, T), (0, 17)], [3, 4, 2, 0], n_single=2)
    close(out[0], want[50], dtype, "single row beside portions")
    close(out[1], want[0], dtype, "first row of a sequence in a stale slot")
    close(out[2:2 + T - 40], want[40:], dtype, "continued segment")
    close(out[2 + T - 40:], want[:17], dtype, "fresh segment into a stale slot")
    close(call([(1, 3), (51, 68)], [4, 3]), torch.cat([want[1:3], want[51:68]]), dtype, "both go on")


def heads(t, H, n):
    return t.double().view(t.shape[0], H, n)


def o_scan(q, k, v, w):
    """q, k, w [T, H, d], v [T, H, dv]."""
    return torch.stack([O.linear_cell(q[:, h], k[:, h], v[:, h], w[:, h]) for h in range(q.shape[1])], 1).reshape(q.shape[0], -1)


SCANS = [(3, 9, 7), (2, 17, 17), (4, 32, 32), (1, 1, 1), (2, 48, 100), (2, 130, 24), (1, 256, 40), (2, 96, 64)]


@pytest.mark.parametrize("shape", SCANS)
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_constant_decay_scan_portions_and_slots(device, dtype, shape):
    """One decay per head (silu on q, k, v) against the whole-sequence cell: heads that forget everything at
    once (a decay of zero), nearly everything, next to nothing, and nothing at all."""
    H, d, dv = shape
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(17)
    T = 83
    q, k, v = (torch.randn(T, n, generator=g).to(tdt) for n in (H * d, H * d, H * dv))
    for decay in ((0.9, 0.0, 0.999, 0.5), (1e-30, 1.0, 0.02, 0.97)):
        decay = decay[:H]
        w = torch.tensor(decay, dtype=torch.float64)[None, :, None].expand(T, H, d)
        want = o_scan(*(O.silu(heads(t, H, n)) for t, n in ((q, d), (k, d), (v, dv))), w)
        log = torch.tensor([max(-1e4, math.log(x)) if x > 0 else -1e4 for x in decay])
        state = torch.full((5, H, d, dv), 7.0, device=device)
        check_scan(scan_call(device, q, k, v, state, H, d, dv, log_decay=log, silu=True), want, dtype, state, 7.0)


@pytest.mark.parametrize("tau", [16.0, 1.0, 0.3])
@pytest.mark.parametrize("shape", SCANS)
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_channel_decay_scan_portions_and_slots(device, dtype, shape, tau):
    """A decay per key channel and row: pre-activations wide enough for channels that keep everything and
    channels that vanish within a block of rows (also both in one block), a scale on q."""
    H, d, dv = shape
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(19)
    T = 83
    q, k, v = (torch.randn(T, n, generator=g).to(tdt) for n in (H * d, H * d, H * dv))
    z, zb = 4.0 * torch.randn(T, H * d, generator=g), torch.randn(H * d, generator=g)
    z[30:34] -= 40.0                                        # rows behind which next to nothing is left
    z[60:70, ::2] = 30.0
    z = z.to(tdt)
    w = O.gla_decay(heads(z.double() + zb.double(), H, d), tau)
    want = o_scan(heads(q, H, d) * 0.3, heads(k, H, d), heads(v, H, dv), w)
    state = torch.full((5, H, d, dv), -3.0, device=device)
    check_scan(scan_call(device, q, k, v, state, H, d, dv, z=z, z_bias=zb, tau=tau, q_scale=0.3), want, dtype, state, -3.0)


@pytest.mark.parametrize("channels", [False, True])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_long_portions_in_parts(device, dtype, channels):
    """Few long segments (walked in parts side by side on the GPU) beside short ones, fresh and going on from
    slots, borders anywhere; a key written early and read back hundreds of rows later."""
    H, d, dv, T = 2, 24, 20, 700
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(29)
    q, k, v = (torch.randn(T, n, generator=g).to(tdt) for n in (H * d, H * d, H * dv))
    k[:, 5] = 0.0
    k[11, 5], q[640, :d] = 30.0, 0.0                        # head 0: only row 11 writes channel 5, row 640 reads it alone
    q[640, 5] = 1.0
    if channels:
        zb = torch.full((H * d,), 6.0)
        z = (2.0 * torch.randn(T, H * d, generator=g)).to(tdt)
        z[:, 5] = 20.0
        w = O.gla_decay(heads(z.double() + zb.double(), H, d), 9.0)
        decay = dict(z=z, z_bias=zb, tau=9.0)
    else:
        w = torch.tensor([0.9995, 0.8], dtype=torch.float64)[None, :, None].expand(T, H, d)
        decay = dict(log_decay=torch.log(torch.tensor([0.9995, 0.8])))
    want = o_scan(heads(q, H, d), heads(k, H, d), heads(v, H, dv), w)
    held = want[640, :dv]
    assert held.abs().max() > 10.0 and torch.nn.functional.cosine_similarity(held, v[11, :dv].double(), dim=0) > 0.99
    state = torch.full((4, H, d, dv), 5.0, device=device)
    call = scan_call(device, q, k, v, state, H, d, dv, **decay)
    close(call([(0, T)], [1]), want, dtype, "one segment")
    close(call([(0, 17)], [2]), want[:17], dtype, "a short one")
    end = state[1].clone()
    got = call([(0, 390), (17, 19), (0, 45)], [3, 2, 0])
    close(got, torch.cat([want[:390], want[17:19], want[:45]]), dtype, "unequal segments")
    got = call([(390, T), (19, 400)], [3, 2])
    close(got, torch.cat([want[390:], want[19:400]]), dtype, "going on")
    close(state[3], end.double().cpu(), "float32", "the same state, however the rows were cut")
    close(call([(400, T)], [2]), want[400:], dtype, "last portion")
    close(state[2], end.double().cpu(), "float32", "and again")


def test_scan_arguments():
    z = torch.zeros(1, 2)
    for kw in ({}, {"z": z}, {"z": z, "z_bias": z[0], "log_decay": z[0]}, {"z": z, "z_bias": z[0], "tau": 0.0}):
        with pytest.raises(ValueError):
            ops.linear_scan(z, z, z, torch.zeros(1, 1, 2, 2), 1, 2, 2, None, i32(0), i32(0), **kw)


# ---------------------------------------------------------------------------- the model on the engine
@pytest.mark.parametrize("shape", sorted(CFGS))
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_whole_prompt_and_layers(device, dtype, shape):
    eng, cd, W = build(device, dtype, cd=CFGS[shape]())
    toks = tokens(200)
    runs = []
    want = O.forward(cd, W, toks, runs)
    tap = []
    got = eng.replay_step([(1, toks, list(range(len(toks))))], [1], layer_tap=tap)
    assert len(tap) == len(runs) == len(KevelornConfig.from_dict(cd).runs)
    for i, (a, b) in enumerate(zip(tap, runs)):
        close_rows(a, b, dtype, f"residual stream after layer run {i}")
    close_rows(got, want, dtype, "logits with a tap")
    close_rows(eng.replay_step([(1, toks, list(range(len(toks))))], [1]), want, dtype, "logits")
    close_rows(got[:3], O.forward(cd, W, toks[:3]), dtype, "first tokens")
    close_rows(eng.replay_step([(2, toks[:1], [0])], [2]), O.forward(cd, W, toks[:1]), dtype, "a prompt of one token")


@pytest.mark.parametrize("shape", sorted(CFGS))
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_prefill_then_decode_and_portions(device, dtype, shape):
    eng, cd, W = build(device, dtype, cd=CFGS[shape]())
    toks = tokens(230, seed=5)
    want = O.forward(cd, W, toks)
    close_rows(replay_cuts(eng, toks, [70]), want, dtype, "prompt then token by token (160 decoded)")
    close_rows(replay_cuts(eng, toks, [1] * 3 + [2, 61, 2, 3, 64, 2, 63, 2, 17]), want, dtype, "portions down to two tokens")
    if shape == "odd":
        close_rows(replay_cuts(eng, toks, []), want, dtype, "token by token from the first")
    assert eng.sched.free_blocks() == eng.num_blocks


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_window_edges_in_the_model(device, dtype):
    """A model that is one attention layer whose scores are sharp: changing one token changes the logits of
    positions up to the window's edge and of none past it, in a prompt and in decoding."""
    cd = cfg_dict([par(heads=2, kv=1, dim=16, vdim=8, window=65, dims=16, scale=6.0, right=light(1, 4, 4, (0.0,)))], mult=1.0)
    eng, _, W = build(device, dtype, cd=cd)
    a = tokens(150, seed=61)
    b = list(a)
    b[40] = (a[40] + 31) % 97
    want = [O.forward(cd, W, t) for t in (a, b)]
    far = (want[0] - want[1]).abs().amax(1)
    assert float(far[105:].max()) < 1e-12 and float(far[40]) > 0.1 and float(far[41:105].max()) > 0.1
    for cuts in ([150], [39, 2, 63, 2, 9], [30]):
        got = [replay_cuts(eng, t, cuts, rid=i + 1) for i, t in enumerate((a, b))]
        for x, y in zip(got, want):
            close_rows(x, y, dtype, f"cuts {cuts}")
        same = (got[0] - got[1]).abs().amax(1).cpu()
        assert float(same[:40].max()) < tol(dtype) and float(same[105:].max()) < tol(dtype), "past the edge nothing is left"


@pytest.mark.parametrize("shape", sorted(CFGS))
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_mixed_batches_and_reuse(device, dtype, shape):
    """Unequal requests interleaved (portions beside single tokens, a request that skips steps),
    in a pool that only holds the live ones: pages and state slots are freed and used again by
    requests that start later. Every request must equal its run alone (the oracle)."""
    eng, cd, W = build(device, dtype, pages=9, seqs=3, cd=CFGS[shape]())
    reqs = {i: tokens(n, seed=10 + i) for i, n in enumerate((150, 65, 1, 200, 129, 64, 3))}
    want = {i: O.forward(cd, W, t) for i, t in reqs.items()}
    got = {i: [] for i in reqs}
    at = {i: 0 for i in reqs}
    waiting, live, step = sorted(reqs), [], 0
    plans = {0: [64, 1, 1, 30], 1: [2, 62], 3: [100, 2], 4: [128], 5: [63]}
    while waiting or live:
        while waiting and len(live) < 3:
            nxt = waiting[0]
            need = sum(-(-len(reqs[i]) // 64) for i in live) + -(-len(reqs[nxt]) // 64)
            if need > 9:
                break
            live.append(waiting.pop(0))
        rows, fin = [], []
        for i in list(live):
            if i == 3 and step % 3 == 1:
                continue                                  # left out of this step, goes on later
            plan = plans.get(i, [])
            n = min(plan.pop(0) if plan else 1, len(reqs[i]) - at[i])
            rows.append((100 + i, reqs[i][at[i]:at[i] + n], list(range(n))))
            at[i] += n
            if at[i] == len(reqs[i]):
                fin.append(100 + i)
                live.remove(i)
        lg = eng.replay_step(rows, fin)
        k = 0
        for rid, t, _ in rows:
            got[rid - 100].append(lg[k:k + len(t)])
            k += len(t)
        step += 1
    for i in reqs:
        close_rows(torch.cat(got[i]), want[i], dtype, f"request {i} in the batch")
    assert eng.sched.free_blocks() == 9 and eng.sched.free_state_slots() == 3


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_sizes_that_coincide_elsewhere(device, dtype):
    """One head, k / v heads as many as heads and one for all, one expert with top 1, all experts chosen, a
    rotation of one pair and of the whole head, vdim = dim, a window of one token and none, tau 1, a low
    rank of one, a multiplier of 1, no scaling, no shared expert, no feed-forward, no repeated span, a span of
    one pass over all layers and of the last layer only, a width that is no multiple of 8. (A head of one
    value column is brought to plus or minus one by its norm, so a rounding can turn its sign: heads of one
    column in float32 only.)"""
    one = 1 if dtype == "float32" else 4
    a = [par(heads=1, kv=1, dim=2, vdim=3, dims=2, window=1, factor=None, scale=1.0, right=light(1, one, one, (1.0,))),
         gla(heads=1, dim=one, vdim=one, tau=1.0, rank=1, mlp=moe(1, 1, 8, 0)),
         lightning(heads=4, dim=6, vdim=6, decay=(0.9,) * 4, mlp=moe(3, 3, 5, 1)),
         par(heads=6, kv=6, dim=4, vdim=4, dims=4, window=0, right=light(2, 4, 4, (0.5, 0.99)), mlp=dense(1))]
    toks = tokens(140, vocab=61, seed=9)
    for layers, mult, loop in ((a, 1.0, None), (a, 0.7, (0, 4, 1)), (a[2:3], 0.3, (0, 1, 4)), (a[1:], 1.0, (2, 3, 2))):
        eng, cd, W = build(device, dtype, cd=cfg_dict(layers, width=36, vocab=61, mult=mult, loop=loop))
        close_rows(replay_cuts(eng, toks, [66, 5]), O.forward(cd, W, toks), dtype, f"loop {loop}, multiplier {mult}")


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_long_decoding(device, dtype):
    """300 tokens decoded one by one after a short prompt: recurrent states carried through hundreds of
    single-row steps, window and page borders crossed by decoded tokens only."""
    eng, cd, W = build(device, dtype, cd=cfg_dict([gla(mlp=moe()), par(window=70), lightning(mlp=dense())], loop=(1, 3, 2)))
    toks = tokens(330, seed=6)
    close_rows(replay_cuts(eng, toks, [30]), O.forward(cd, W, toks), dtype, "long decoding")


@pytest.mark.parametrize("device,dtype", [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu)])
def test_greedy_generation_through_the_scheduler(device, dtype):
    """LLMEngine.generate: the engine's own scheduler chunks the prompts (a small token budget),
    batches the requests and decodes (hipGraph decode steps on the GPU); greedy tokens must
    equal the oracle's."""
    eng, cd, W = build(device, dtype, pages=16, max_batched_tokens=48, token_alignment=1, mixed_prefill_tokens=16)
    prompts = [tokens(90, seed=21), tokens(5, seed=22), tokens(67, seed=23)]
    reqs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    for p, r in zip(prompts, reqs):
        assert r.output_ids == O.greedy(cd, W, p, 12)
    assert eng.stats["prefill_steps"] > 2 and eng.sched.free_blocks() == 16


@pytest.mark.parametrize("device", DEVICES)
def test_pipelined_generation_matches_synchronous(device):
    a, cd, W = build(device, "float32", async_decode=True)
    b, _, _ = build(device, "float32", async_decode=False)
    prompts = [tokens(40, seed=31), tokens(70, seed=32)]
    sp = SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True)
    assert [r.output_ids for r in a.generate(prompts, sp)] == [r.output_ids for r in b.generate(prompts, sp)]


@pytest.mark.parametrize("device", DEVICES)
def test_preemption_recomputes(device):
    """A pool too small for both sequences to grow: the scheduler preempts one (its pages and
    state slot go back), recomputes it later from its first token, and the tokens do not change."""
    small, cd, W = build(device, "float32", pages=5)
    big, _, _ = build(device, "float32", pages=16)
    prompts = [tokens(120, seed=41), tokens(120, seed=42)]
    sp = SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True)
    got = [r.output_ids for r in small.generate(prompts, sp)]
    assert small.sched.preemptions() > 0
    assert got == [r.output_ids for r in big.generate(prompts, sp)]
    assert got[0] == O.greedy(cd, W, prompts[0], 20)
    assert small.sched.free_blocks() == 5


@pytest.mark.gpu
def test_captured_decode_graph_replays():
    """Decode steps from the captured graph, several in a row with eager steps of other sequences in
    between, against eager decoding of the same tokens: the states are written by the replays."""
    a, cd, _ = build("cuda", "float32", graphs=True)
    b, _, _ = build("cuda", "float32", graphs=False)
    t1, t2 = tokens(60, seed=71), tokens(45, seed=72)
    for i in range(0, 40):
        rows = [(1, t1[:20] if i == 0 else t1[19 + i:20 + i], [0])]
        if i % 5 == 0:
            n = i // 5
            rows.append((2, t2[5 * n:5 * n + 5], [4]))
        la, lb = a.replay_step(rows), b.replay_step(rows)
        assert (la - lb).abs().max().item() < 1e-4 * max(1.0, lb.abs().max().item()), f"step {i}"
    assert a.graphs and not b.graphs


@pytest.mark.gpu
def test_mfma_forms_run_and_agree_with_the_plain_kernels():
    """At layer sizes (bf16): windowed attention with a gate per element on the MFMA prompt and single-token
    kernels against the row kernel, and the block form of both scans (one segment in parts, and many) against
    their single-row form."""
    dev = "cuda"
    g = torch.Generator().manual_seed(2)
    H, G, dk, dv, npg, window = 8, 2, 128, 128, 40, 300
    kc = (0.5 * torch.randn(npg, G, 64, dk, generator=g)).bfloat16().to(dev)
    vc = torch.randn(npg, G, 64, dv, generator=g).bfloat16().to(dev)
    bt = torch.randperm(npg, generator=g).to(torch.int32).view(2, 20).to(dev)
    cu, ctx = i32(0, 301, 370, device=dev), i32(1000, 69, device=dev)
    qq = (2.0 * torch.randn(370, H * dk, generator=g)).bfloat16().to(dev)
    gate = torch.randn(370, H * dv, generator=g).bfloat16().to(dev)
    assert ops.softmax_attention_mfma_ok(qq, dk, dv, 4, 1)
    seq, pos = ops._rows_of_portions(cu, ctx, 370, dev)
    kw = dict(scale=dk ** -0.5, window=window, gate=gate)
    want = ops.softmax_attention(qq, kc, vc, bt, seq, pos, H, G, dk, dv, **kw).float()
    free = ops.softmax_attention(qq, kc, vc, bt, seq, pos, H, G, dk, dv, scale=dk ** -0.5, gate=gate).float()
    assert (want - free).abs().max().item() > 0.1, "the window changes the result"
    for got in (ops.softmax_attention_prefill(qq, kc, vc, bt, cu, ctx, 301, H, G, dk, dv, **kw),
                ops.softmax_attention_rows(qq, kc, vc, bt, seq, pos, H, G, dk, dv, max_ctx=1024, **kw)):
        assert (got.float() - want).abs().max().item() < 0.03 * max(1.0, want.abs().max().item())
    H, d, dv = 4, 128, 128
    for T, n in ((300, 1), (272, 1), (130, 40)):
        q, k, v = (torch.randn(n * T, H * m, generator=g).bfloat16().to(dev) for m in (d, d, dv))
        z = torch.randn(n * T, H * d, generator=g).bfloat16().to(dev)
        for kw in (dict(z=z, z_bias=torch.ones(H * d, device=dev), tau=16.0, q_scale=d ** -0.5),
                   dict(log_decay=torch.tensor([-0.5, -0.05, -0.01, -0.001], device=dev), silu=True)):
            s1, s2 = (torch.zeros(n, H, d, dv, device=dev) for _ in range(2))
            slot = torch.arange(n, dtype=torch.int32, device=dev)
            p = torch.arange(T, dtype=torch.int32, device=dev)
            a = ops.linear_scan(q, k, v, s1, H, d, dv, torch.arange(0, n * T + 1, T, dtype=torch.int32, device=dev), slot,
                                p.repeat(n), max_q=T, **kw).view(n, T, -1)
            b = []
            for t in range(T):
                kt = dict(kw, z=z.view(n, T, -1)[:, t]) if "z" in kw else kw
                qt, ktt, vt = (x.view(n, T, -1)[:, t] for x in (q, k, v))
                b.append(ops.linear_scan(qt, ktt, vt, s2, H, d, dv, None, slot, p[t:t + 1].repeat(n), **kt))
            b = torch.stack(b, 1)
            assert (a - b).abs().max().item() < 1e-4 * max(1.0, b.abs().max().item())
            assert (s1 - s2).abs().max().item() < 1e-4 * max(1.0, s2.abs().max().item())


def test_model_folder_roundtrip(tmp_path):
    """config.json + safetensors -> registry -> engine (EngineConfig.model as a folder)."""
    from nv_genai_amd.models.registry import read_config
    from nv_genai_amd.utils.checkpoint import save_weights

    cd = cfg_odd()
    cfg = KevelornConfig.from_dict(cd)
    assert cfg.to_json_dict() == cd
    assert cfg.is_moe and cfg.experts_per_tok == 3 and cfg.num_experts == 5
    assert cfg.runs == ((0, None), (1, 0), (2, None), (3, None), (1, 1), (2, None), (3, None), (4, None))
    w = random_weights(cfg, 3, torch.bfloat16)
    save_weights(w, str(tmp_path))
    for b in cd["layers"]:      # the rank of the decay may also come from the tensors alone
        b["mixer"].pop("rank", None)
    (tmp_path / "config.json").write_text(json.dumps(cd))
    got, cls = read_config(str(tmp_path))
    assert cls is KevelornModel and got == KevelornConfig.from_dict(cd)
    eng = LLMEngine(EngineConfig(model=str(tmp_path), dtype="float32", max_num_seqs=2, max_batched_tokens=128,
                                 max_model_len=128, kv_cache_blocks=4, detokenize=False, use_graphs=False,
                                 mixed_graphs=False, tuned_gemms=False, async_decode=False), device="cpu")
    toks = tokens(50, seed=7)
    close_rows(eng.replay_step([(1, toks, list(range(50)))], [1]), O.forward(cd, w, toks), "float32", "model folder")
    sd = eng.model.state_dict()
    assert set(sd) == set(w)
    for k in w:
        assert torch.equal(sd[k].cpu().reshape(w[k].shape).to(w[k].dtype), w[k]), k


def test_config_errors_and_builder():
    bad = cfg_odd()
    bad["layers"][0]["type"] = "conv"
    with pytest.raises(ValueError):
        KevelornConfig.from_dict(bad)
    for layer in (lightning(mlp=moe(3, 5)), par(dim=4, dims=6), par(heads=5, kv=2), lightning(heads=2), gla(tau=0.0),
                  lightning(mlp={"kind": "sparse", "ff": 4}), lightning(mlp=dense(0)), par(factor=-1.0), gla(dim=0),
                  lightning(decay=(0.5, 1.5, 0.1))):
        with pytest.raises(ValueError):
            KevelornConfig.from_dict(cfg_dict([layer]))
    for loop in ((1, 1, 2), (0, 2, 1), (0, 1, 0)):
        with pytest.raises(ValueError):
            KevelornConfig.from_dict(cfg_dict([lightning()], loop=loop))
    cfg = KevelornConfig.from_dict(cfg_odd())
    w = random_weights(cfg, 0)
    w["l0.mix.norm"] = w["l0.mix.norm"][:-1]
    with pytest.raises(ValueError):
        KevelornModel(cfg, "cpu", torch.float32, weights=w)
    with pytest.raises(ValueError):
        KevelornModel(KevelornConfig.from_dict(cfg_dict([gla(heads=1, dim=300)])), "cpu", torch.float32)
    c = kevelorn_layers(["parallel", "gla", "lightning"], 64, 4, 2, 16, 8, ff=24, window=70, rec_heads=3, rec_dim=8, rec_vdim=16,
                        tau=4.0, rank=6, experts=4, top=2, expert_ff=16, shared_ff=8, rot_dims=8, rot_factor=2.0,
                        residual_mult=0.5, loop=(0, 2, 2))
    assert KevelornConfig.from_dict(c.to_json_dict()) == c
    assert c.blocks[0].mixer.left.window == 70 and c.blocks[0].mlp.kind == "dense" and c.blocks[1].mlp.shared == 8


@pytest.mark.parametrize("device", DEVICES)
def test_trace_runner_replays_a_schedule(device, tmp_path, monkeypatch, capsys):
    """The trace runner on a model folder: steps as JSON lines on standard input (a prompt in two
    portions, a second request beside single tokens of the first, requests ended and their names
    used again), logits files of the wanted places, a ``done`` line per step."""
    import io

    import numpy as np

    from nv_genai_amd.tools import trace_run
    from nv_genai_amd.utils.checkpoint import save_weights

    cd = cfg_dict([gla(mlp=moe()), par(window=33)], loop=(1, 2, 2))
    cfg = KevelornConfig.from_dict(cd)
    w = random_weights(cfg, 8, torch.bfloat16)
    model_dir, out_dir = tmp_path / "model", tmp_path / "out"
    save_weights(w, str(model_dir))
    (model_dir / "config.json").write_text(json.dumps(cd))
    a, b = tokens(80, seed=51), tokens(30, seed=52)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:65], "want": [0, 64]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[65:78], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[:29], "want": [28]}, {"id": "a", "tokens": a[78:79], "want": [0]}],
              "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[79:], "want": [0]}, {"id": "b", "tokens": b[29:], "want": [0]}],
              "end": ["a", "b"]},
             {"step": 4, "entries": [{"id": "a", "tokens": b[:5], "want": [4]}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    rc = trace_run.main(["--model", str(model_dir), "--dtype", "float32", "--out", str(out_dir), "--max-tokens", "192",
                         "--device", device])
    assert rc == 0
    assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    wa, wb = O.forward(cd, w, a), O.forward(cd, w, b)
    V = cd["vocab"]

    def rows(i):
        return torch.from_numpy(np.fromfile(out_dir / f"{i}.f32", dtype="<f4").reshape(-1, V).copy())

    assert not (out_dir / "1.f32").exists()
    close_rows(rows(0), wa[[0, 64]], "float32", "first portion")
    close_rows(rows(2), torch.stack([wb[28], wa[78]]), "float32", "a portion beside a single token")
    close_rows(rows(3), torch.stack([wa[79], wb[29]]), "float32", "last tokens")
    close_rows(rows(4), wb[4:5], "float32", "a name used again")
