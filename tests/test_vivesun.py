"""Vivesun on the serving engine against the plain oracle (tests/vivesun_oracle.py).

Every case runs on the CPU (the engine on the fp32 reference ops: scheduling, pages, state slots,
row maps) and, marked ``gpu``, on the HIP kernels in float32 and bfloat16. The models are small
random ones built here; sizes are chosen so that heads, dims, taps, chunk and page size do not
coincide (``odd``: a rotation on part of the head, a chunk that is no multiple of the page, a layer
without feed-forward), or so that the MFMA tile kernels run (``tiles``).
"""
import json
import math

import pytest
import torch

import vivesun_oracle as O
from nv_genai_amd import ops
from nv_genai_amd.engine.llm_engine import EngineConfig, LLMEngine, SamplingParams
from nv_genai_amd.models.config import VivesunConfig, vivesun_layers
from nv_genai_amd.models.vivesun import VivesunModel, random_weights

GPU = pytest.param("cuda", marks=pytest.mark.gpu)
DEVICES = ["cpu", GPU]
DTYPES = [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
          pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)]
BANDS = {"factor": 8.0, "low": 1.5, "high": 6.0, "original": 48}


def moe(experts=5, top=3, ff=14, scale=1.7):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff}}


def delta(heads=6, kv=2, dim=10, vdim=7, conv=3, mlp=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def par(heads=4, kv=2, dim=12, vdim=6, chunk=27, dims=8, base=50.0, scale=0.3, scaling=BANDS, rheads=3, rdim=9, rank=5,
        left_scale=0.8, right_scale=1.3, mlp=None):
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = dict(scaling)
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    if chunk:
        left["mask"] = {"size": chunk}
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": rheads, "dim": rdim, "decay_rank": rank},
                                          "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def cfg_dict(layers, width=40, vocab=97, eps=1e-5, bigram=(53, 7, 11), side=6):
    d = {"architecture": "Vivesun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if bigram:
        d["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    if side:
        d["token_side"] = {"dim": side}
    return d


def cfg_odd():
    return cfg_dict([delta(mlp=moe()), par(mlp=moe(3, 2, 9, 0.6)), delta(heads=3, kv=3, dim=5, vdim=11, conv=5),
                     par(heads=3, kv=1, dim=6, vdim=10, chunk=100, dims=6, scaling=None, rheads=2, rdim=17, rank=3, mlp=moe(4, 1, 8))])


def cfg_tiles():
    """Sizes the MFMA kernels take: 128-wide heads with GQA, experts of 64 / 192 on a width of 256,
    a chunk longer than a page and no multiple of it."""
    return cfg_dict([delta(heads=4, kv=2, dim=64, vdim=64, conv=4, mlp=moe(4, 2, 64, 2.5)),
                     par(heads=8, kv=2, dim=128, vdim=64, chunk=80, dims=32, base=1e4, scale=0.09, rheads=4, rdim=32, rank=16,
                         scaling={"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}, mlp=moe(6, 3, 192, 1.0))],
                    width=256, side=24)


CFGS = {"odd": cfg_odd, "tiles": cfg_tiles}


def build(device, dtype="float32", seed=0, pages=24, seqs=4, cd=None, graphs=None, **eng):
    cd = cd or cfg_odd()
    cfg = VivesunConfig.from_dict(cd)
    w = random_weights(cfg, seed, torch.bfloat16)       # bf16 values, as a checkpoint holds them
    for k in w:
        if k.endswith("mlp.router"):
            w[k] = w[k] * 4.0                           # wide logits: few near ties between experts
    tdt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype]
    model = VivesunModel(cfg, device, tdt, weights=w)
    kw = dict(model="vivesun-test", dtype=dtype, max_num_seqs=seqs, max_batched_tokens=512, max_model_len=512,
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
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_bigram_embedding(device, dtype):
    """Rows of a step: a first token (the last row of the table), pairs inside the step, a pair whose
    first half lies in a slot; ids and multipliers whose product leaves 32 bits; what the step
    leaves in the slots, by the launch itself for single rows and by token_save_ for portions."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(3)
    V, H, B, a, b = 70000, 19, 1009, 99991, 7919
    E, Tb = torch.randn(V, H, generator=g).to(tdt), torch.randn(B + 1, H, generator=g).to(tdt)
    seq1, seq2 = [69999, 65000, 65000, 3], [0, 69998]
    bg = {"buckets": B, "mul_prev": a, "mul_cur": b}

    def want(toks):
        return E[torch.tensor(toks)].double() + Tb[torch.tensor(O.bigram_rows(toks, bg))].double()

    dv = lambda t: t.to(device)   # noqa: E731
    prev = dv(torch.full((3,), 12345, dtype=torch.int32))
    # portions: two rows of sequence 1 into slot 2, sequence 2 into slot 0
    x = ops.bigram_embed(dv(i32(*seq1[:2], *seq2)), dv(E), dv(Tb), dv(i32(-1, 0, -1, 2)), prev, a, b)
    close(x, torch.cat([want(seq1)[:2], want(seq2)]), "float32", "portions")
    ops.token_save_(prev, dv(i32(*seq1[:2], *seq2)), dv(i32(1, 3, -1)), dv(i32(2, 0, 1)))
    assert prev.tolist() == [69998, 12345, 65000]
    # single rows: sequence 1 goes on from slot 2, a fresh one into the stale slot 1, a padding row
    x = ops.bigram_embed(dv(i32(seq1[2], 5, 0)), dv(E), dv(Tb), dv(i32(-(2 + 2), -1, -1)), prev, a, b, save_slots=dv(i32(2, 1, -1)))
    close(x[:2], torch.stack([want(seq1)[2], want([5])[0]]), "float32", "single rows")
    assert prev.tolist() == [69998, 5, 65000]
    x = ops.bigram_embed(dv(i32(seq1[3])), dv(E), dv(Tb), dv(i32(-(2 + 2))), prev, a, b, save_slots=dv(i32(2)))
    close(x, want(seq1)[3:], "float32", "next single row")


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_stream_and_row_ops(device, dtype):
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(4)
    T, H = 37, 41
    dv = lambda t: t.to(device)   # noqa: E731
    x0, y = 3.0 * torch.randn(T, H, generator=g), torch.randn(T, H, generator=g).to(tdt)
    x = dv(x0.clone())
    c = ops.residual_add_cast_(x, dv(y), tdt)
    xs = x0.double() + y.double()
    close(x, xs, "float32", "the sum stays fp32")
    close(c, xs, dtype, "copy of the sum")
    z = (2.0 * torch.randn(T, 6, generator=g)).to(tdt)
    table, ids = torch.randn(11, 20, generator=g).to(tdt), torch.randint(0, 11, (T,), generator=g).to(torch.int32)
    close(ops.gelu_gate_rows(dv(z), dv(ids), dv(table), 7), O.gelu_tanh(z.double()) * table[ids.long(), 7:13].double(), dtype,
          "gate on the token's vector")
    w = torch.randn(T, 30, generator=g).to(tdt)
    close(ops.tanh_rows(dv(w)[:, 5:16]), torch.tanh(w[:, 5:16].double()), dtype, "tanh of a column slice")
    # head norm: a weight per element of a head, silu gate, columns of a wider row as the output
    for gs in (7, 8):
        o, wn = torch.randn(T, 3 * gs, generator=g), 1 + 0.1 * torch.randn(gs, generator=g)
        gate = (2.0 * torch.randn(T, 3 * gs + 8, generator=g)).to(tdt)
        want = (O.unit_rms(o.double().view(T, 3, gs), 1e-5) * wn.double()).reshape(T, 3 * gs)
        row = torch.zeros(T, 3 * gs + 16, dtype=tdt, device=device)
        ops.group_rmsnorm(dv(o), dv(wn), 3, 1e-5, tdt, gate=dv(gate)[:, 8:], gate_act="silu", out=row[:, 8:8 + 3 * gs])
        close(row[:, 8:8 + 3 * gs], want * O.silu(gate[:, 8:].double()), dtype, "silu gate, output columns")
        assert float(row[:, :8].abs().max()) == 0.0 and float(row[:, 8 + 3 * gs:].abs().max()) == 0.0
        close(ops.group_rmsnorm(dv(o), dv(wn), 3, 1e-5, tdt, gate=dv(gate)[:, 8:]), want * torch.sigmoid(gate[:, 8:].double()),
              dtype, "sigmoid gate")


def test_rotary_bands_against_the_oracle():
    """Frequencies kept, divided and in between (all three occur), and no scaling."""
    for rot in ({"dims": 8, "base": 50.0, "scaling": BANDS}, {"dims": 6, "base": 100.0},
                {"dims": 128, "base": 500000.0, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}):
        sc = rot.get("scaling")
        f, mag = ops.rotary_frequencies(rot["dims"], rot["base"], bands=None if not sc else tuple(sc[k] for k in (
            "factor", "low", "high", "original")))
        assert torch.allclose(f, O.rotary_frequencies(rot), rtol=1e-13, atol=0) and mag == 1.0
    plain = O.rotary_frequencies({"dims": 128, "base": 500000.0})
    kept, cut = (f / plain > 0.999).sum(), ((f / plain - 1 / 8).abs() < 1e-9).sum()
    assert kept > 0 and cut > 0 and kept + cut < 64


@pytest.mark.parametrize("sizes", [(6, 2, 12, 8, 6), (4, 2, 64, 32, 64), (3, 1, 128, 32, 128), (9, 3, 32, 16, 24)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_partial_rotation_and_page_write(device, dtype, sizes):
    """A rotation on part of the head (the rest passes unchanged), no head norm, values with columns
    of their own, positions far out, a row that is not written."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(5)
    H, G, dk, dims, dv = sizes
    T = 9
    rot = {"dims": dims, "base": 30.0, "scaling": BANDS}
    freq, mag = ops.rotary_frequencies(dims, 30.0, bands=tuple(BANDS[k] for k in ("factor", "low", "high", "original")))
    proj0 = torch.randn(T, (H + G) * dk + G * dv + 8, generator=g).to(tdt)
    pos = i32(0, 1, 63, 64, 1000, 65535, 99999, 7, 2)
    slots = i32(0, 1, 63, 64, 130, 191, 5, -1, 70)
    kc = torch.zeros(3, G, 64, dk, dtype=tdt, device=device)
    vc = torch.zeros(3, G, 64, dv, dtype=tdt, device=device)
    proj = proj0.clone().to(device)
    ops.rope_headnorm_cache_(proj, pos.to(device), slots.to(device), kc, vc, H, G, dk, dv, freq.to(device), mag, dims, 1e-5,
                             v_off=(H + G) * dk)
    pd = proj0.double()
    q, k = pd[:, :H * dk].view(T, H, dk), pd[:, H * dk:(H + G) * dk].view(T, G, dk)
    v = pd[:, (H + G) * dk:(H + G) * dk + G * dv].view(T, G, dv)
    qr, kr = (torch.stack([O.rotate(x[t:t + 1], rot, int(pos[t]))[0] for t in range(T)]) for x in (q, k))
    close(proj[:, :H * dk], qr.reshape(T, -1), dtype, "rotated queries")
    close(proj[:, H * dk:(H + G) * dk], kr.reshape(T, -1), dtype, "rotated keys")
    assert torch.equal(proj[:, (H + G) * dk:].cpu(), proj0[:, (H + G) * dk:]), "the other columns stay"
    if dims < dk:
        assert torch.equal(proj[:, :H * dk].cpu().view(T, H, dk)[..., dims:], proj0[:, :H * dk].view(T, H, dk)[..., dims:])
    for t in range(T):
        s = int(slots[t])
        if s >= 0:
            close(kc[s // 64, :, s % 64], kr[t], dtype, f"K page row of token {t}")
            close(vc[s // 64, :, s % 64], v[t], dtype, f"V page row of token {t}")


def _pages(rows, device, tdt, bt_row, nb):
    """Token rows [n, G, d] laid into pages [nb, G, 64, d] through the block-table row."""
    n, G, d = rows.shape
    page = torch.zeros(nb, G, 64, d, dtype=tdt, device=device)
    j = torch.arange(n)
    page[bt_row[j // 64].long(), :, j % 64] = rows.to(tdt).to(device)
    return page


def o_attention(q, K, V, scale, chunk, sink, pos):
    """Plain form: query t at position pos[t] sees keys of its chunk up to itself; q [T, H, d]."""
    T, H, _ = q.shape
    G = K.shape[1]
    out = torch.zeros(T, H, V.shape[2], dtype=torch.float64)
    for t in range(T):
        lo = int(pos[t]) // chunk * chunk if chunk else 0
        for h in range(H):
            kk, vv = (X[lo:int(pos[t]) + 1, h // (H // G)].double() for X in (K, V))
            s = (kk @ q[t, h].double()) * scale
            out[t, h] = (O.sink_weights(s) if sink else torch.softmax(s, -1)) @ vv
    return out.reshape(T, -1)


@pytest.mark.parametrize("chunk", [0, 50, 64, 128, 200])
@pytest.mark.parametrize("shape", [(6, 2, 10, 6), (4, 2, 64, 64), (8, 1, 128, 128), (9, 3, 96, 64), (2, 2, 32, 128)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_one_key_stands_out_in_chunks(device, dtype, shape, chunk):
    """One key is made to match a scaled query: just inside and just outside chunk edges, on both
    sides of page borders, far back, at the query's own position and one position after it. A key in
    sight takes nearly all the weight, one out of sight none. Through the row kernel, the
    single-token kernel and the prompt kernel, the result in columns of a wider row times a factor."""
    H, G, dk, dv = shape
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(11)
    n = 460
    K = (0.3 * torch.randn(n, G, dk, generator=g)).to(tdt).float()
    V = torch.randn(n, G, dv, generator=g).to(tdt).float()
    bt = torch.randperm(12, generator=g)[:8].to(torch.int32)
    qpos = [459, 401, 400, 399, 384, 250, 249, 200, 199, 128, 127, 64, 63, 5, 0]
    scale = dk ** -0.5
    w8 = (H * dv + 7) // 8 * 8 + 16
    dev = lambda t: t.to(device)   # noqa: E731
    pos = i32(*qpos)
    for hot in (3, 63, 64, 128, 199, 200, 249, 250, 383, 384, 399, 400):
        KK = K.clone()
        u = torch.randn(dk, generator=g)
        u = u / u.norm()
        KK[hot, 0] = (6.0 * u).to(tdt).float()
        kc, vc = _pages(KK, device, tdt, bt, 12), _pages(V, device, tdt, bt, 12)
        q = 0.3 * torch.randn(len(qpos), H, dk, generator=g)
        q[:, 0] = 20.0 * u / scale / 6.0      # head 0 (kv head 0): score 20 on the hot key
        q = q.to(tdt)
        want = o_attention(q.float(), KK, V, scale, chunk, True, pos) * 0.75
        qd = q.reshape(len(qpos), H * dk).to(device)
        seq = torch.zeros(len(qpos), dtype=torch.int32, device=device)
        btd = dev(bt.view(1, -1))
        kw = dict(scale=scale, chunk=chunk, sink=0.0, factor=0.75)
        for name in ("row", "single"):
            row = torch.zeros(len(qpos), w8, dtype=tdt, device=device)
            out = row[:, 8:8 + H * dv]
            if name == "row":
                ops.softmax_attention(qd, kc, vc, btd, seq, dev(pos), H, G, dk, dv, out=out, **kw)
            else:
                ops.softmax_attention_rows(qd, kc, vc, btd, seq, dev(pos), H, G, dk, dv, max_ctx=512, out=out, **kw)
            close(out, want, dtype, f"{name} form, hot key {hot}")
            assert float(row[:, :8].abs().max()) == 0.0 and float(row[:, 8 + H * dv:].abs().max()) == 0.0
        for t, p in enumerate(qpos):
            seen = hot <= p and (not chunk or hot // chunk == p // chunk)
            hit = (out[t, :dv].double().cpu() - 0.75 * V[hot, 0].double()).abs().max().item() < 0.05
            assert hit == seen, f"query at {p}, hot key at {hot}: seen={hit}"
    # a portion that starts in the middle of a chunk and of a page
    lo, nq = 173, 460 - 173
    q = 0.3 * torch.randn(nq, H, dk, generator=g)
    q[:, H - 1] = 20.0 * u / scale / 6.0
    q = q.to(tdt)
    KK = K.clone()
    KK[250, G - 1] = (6.0 * u).to(tdt).float()
    kc, vc = _pages(KK, device, tdt, bt, 12), _pages(V, device, tdt, bt, 12)
    want = o_attention(q.float(), KK, V, scale, chunk, True, torch.arange(lo, 460))
    row = torch.zeros(nq, w8, dtype=tdt, device=device)
    out = row[:, 8:8 + H * dv]
    ops.softmax_attention_prefill(dev(q.reshape(nq, H * dk)), kc, vc, dev(bt.view(1, -1)), i32(0, nq, device=device),
                                  i32(460, device=device), nq, H, G, dk, dv, scale=scale, chunk=chunk, sink=0.0, out=out)
    close(out, want, dtype, "portion")
    for p in (249, 250, 251, 299, 300, 383, 384, 399, 400, 459):
        seen = p >= 250 and (not chunk or 250 // chunk == p // chunk)
        hit = (out[p - lo, (H - 1) * dv:].double().cpu() - V[250, G - 1].double()).abs().max().item() < 0.05
        assert hit == seen, f"portion: query at {p}"


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_sink_score(device, dtype):
    """A sink of other scores than 0, none, and scores far below it (the output fades away)."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(12)
    for (H, G, dk, dv) in ((3, 1, 10, 6), (4, 2, 64, 32)):
        K, V = torch.randn(100, G, dk, generator=g).to(tdt).float(), torch.randn(100, G, dv, generator=g).to(tdt).float()
        q = torch.randn(2, H, dk, generator=g).to(tdt)
        bt = i32(1, 0)
        kc, vc = _pages(K, device, tdt, bt, 2), _pages(V, device, tdt, bt, 2)
        pos = i32(99, 40)
        for sink in (None, 2.5, -1.0, 12.0):
            for scale in (0.2, 2.0):
                want = torch.zeros(2, H, dv, dtype=torch.float64)
                for t in range(2):
                    for h in range(H):
                        s = K[:int(pos[t]) + 1, h // (H // G)].double() @ q[t, h].double() * scale
                        s2 = s if sink is None else torch.cat([s, torch.tensor([sink], dtype=torch.float64)])
                        want[t, h] = torch.softmax(s2, -1)[:s.numel()] @ V[:int(pos[t]) + 1, h // (H // G)].double()
                args = (q.reshape(2, -1).to(device), kc, vc, bt.view(1, -1).to(device))
                rows = (torch.zeros(2, dtype=torch.int32, device=device), pos.to(device), H, G, dk, dv)
                close(ops.softmax_attention(*args, *rows, scale=scale, sink=sink), want.reshape(2, -1), dtype, f"row, sink {sink}")
                close(ops.softmax_attention_rows(*args, *rows, scale=scale, max_ctx=128, sink=sink), want.reshape(2, -1), dtype,
                      f"single, sink {sink}")
                one = ops.softmax_attention_prefill(args[0][:1], *args[1:], i32(0, 1, device=device), i32(100, device=device), 1,
                                                    H, G, dk, dv, scale=scale, sink=sink)
                close(one, want[:1].reshape(1, -1), dtype, f"portion, sink {sink}")


def run_cuts(call, cuts, T):
    """Portions ``cuts`` (pairs of row ranges), then single rows to T."""
    got = [call(a, b, False) for a, b in zip(cuts, cuts[1:])]
    return torch.cat(got + [call(t, t + 1, True) for t in range(cuts[-1], T)])


@pytest.mark.parametrize("C,n", [(13, 3), (24, 4), (24, 2), (16, 1), (40, 7)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_short_convolution(device, dtype, C, n):
    """Portions down to one and two rows (shorter than the taps) and single rows against the whole
    sequence; a stale slot at position 0, a slot of -1, two segments in one launch."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(13)
    T = 60
    x = torch.randn(T, C + 8, generator=g).to(tdt)[:, :C]
    taps = torch.randn(C, n, generator=g)
    want = O.short_conv(x.double(), taps)
    state = torch.full((3, n - 1, C), 7.0, dtype=tdt, device=device)
    xd = torch.zeros(T, C + 8, dtype=tdt, device=device)
    xd[:, :C] = x.to(device)
    xd, td = xd[:, :C], taps.t().contiguous().to(device)

    def call(a, b, single, slot=1):
        pos = torch.arange(a, b, dtype=torch.int32, device=device)
        cu = None if single else i32(0, b - a, device=device)
        return ops.short_conv(xd[a:b], td, state, cu, i32(slot, device=device), torch.zeros_like(pos), pos)

    close(run_cuts(call, [0, 1, 3, 5, 22, 24, 25, 41, 43], T), want, dtype, "portions, then single rows")
    close(torch.cat([call(t, t + 1, True) for t in range(T)]), want, dtype, "single rows into the stale slot of the run before")
    if n > 1:
        assert torch.equal(state[1].cpu(), x[T - n + 1:]), "the slot holds the last inputs"
        assert float((state[0] - 7.0).abs().max()) == 0.0 and float((state[2] - 7.0).abs().max()) == 0.0
    keep = state.clone()
    close(call(0, 30, False, slot=-1), want[:30], dtype, "no slot")
    assert torch.equal(keep, state)
    call(0, 40, False, slot=2)
    rows = torch.cat([xd[40:60], xd[:2]])
    pos = torch.cat([torch.arange(40, 60), torch.arange(2)]).to(torch.int32).to(device)
    seq = torch.tensor([0] * 20 + [1] * 2, dtype=torch.int32, device=device)
    out = ops.short_conv(rows, td, state, i32(0, 20, 22, device=device), i32(2, 0, device=device), seq, pos)
    close(out, torch.cat([want[40:], want[:2]]), dtype, "two segments")
    if n > 2:
        pad = torch.cat([torch.zeros(n - 1, C, dtype=tdt), x[:2]])[-(n - 1):]
        assert torch.equal(state[0].cpu(), pad), "a short first portion leaves zeros in front of its rows"


def gated_inputs(T, H, G, d, dv, tdt, g, decay=2.0):
    x = torch.randn(T, 2 * G * d + H * dv, generator=g).to(tdt)
    ba = (decay * torch.randn(T, 2 * H, generator=g)).to(tdt)
    return x, ba, torch.randn(H, generator=g), torch.randn(H, generator=g)


def o_gated(x, ba, a_log, dt_bias, H, G, d, dv):
    T = x.shape[0]
    xd = x.double()
    q = O.unit_vector(xd[:, :G * d].reshape(T, G, d)) * d ** -0.5
    k, v = O.unit_vector(xd[:, G * d:2 * G * d].reshape(T, G, d)), xd[:, 2 * G * d:].reshape(T, H, dv)
    beta = torch.sigmoid(ba[:, :H].double())
    dec = torch.exp(-torch.exp(a_log.double()) * torch.nn.functional.softplus(ba[:, H:].double() + dt_bias.double()))
    return torch.stack([O.gated_delta_cell(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], beta[:, h], dec[:, h])
                        for h in range(H)], 1).reshape(T, H * dv)


def check_scan(call, want, dtype, state, sp, device):
    """Portions of many sizes, single rows, slots, two segments with single rows in front."""
    T = want.shape[0]
    close(run_cuts(lambda a, b, s: call([(a, b)], [1], single=s), [0, 1, 20, 22, 27, 43, 44, 60], T), want, dtype,
          "portions, then single rows")
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


@pytest.mark.parametrize("shape", [(6, 2, 10, 7), (3, 3, 5, 11), (4, 2, 64, 64), (1, 1, 1, 1), (2, 1, 130, 20), (2, 2, 48, 100),
                                   (3, 1, 200, 36)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_gated_delta_scan_portions_and_slots(device, dtype, shape):
    """The scan in portions and as single rows against the whole-sequence cell. Some heads forget
    nearly everything per row (decays that vanish over a block), some nearly nothing."""
    H, G, d, dv = shape
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(17)
    T = 83
    x, ba, a_log, dt_bias = gated_inputs(T, H, G, d, dv, tdt, g, 3.0)
    a_log[0], dt_bias[0] = 3.5, 1.0               # decays down to exp(-100)
    if H > 1:
        a_log[1], dt_bias[1] = -6.0, -3.0         # next to no decay
    want = o_gated(x, ba, a_log, dt_bias, H, G, d, dv)
    state = torch.full((5, H, d, dv), 7.0, device=device)
    xd, bd, al, db = (t.to(device) for t in (x, ba, a_log, dt_bias))

    def call(segs, slots, single=False, n_single=0):
        rows = torch.cat([torch.arange(a, b) for a, b in segs]).to(device)
        cu = None if single else torch.tensor([0] + [b - a for a, b in segs]).cumsum(0).to(torch.int32).to(device)
        return ops.gated_delta_scan(xd[rows], bd[rows], al, db, state, H, G, d, dv, cu, i32(*slots, device=device),
                                    rows.to(torch.int32), n_single=n_single, max_q=max(b - a for a, b in segs))

    check_scan(call, want, dtype, state, 7.0, device)


@pytest.mark.parametrize("shape", [(3, 9, 9), (2, 17, 17), (4, 32, 32), (1, 1, 1), (2, 48, 48), (2, 130, 24), (1, 256, 40)])
@pytest.mark.parametrize("device,dtype", DTYPES)
def test_channel_delta_scan_portions_and_slots(device, dtype, shape):
    """As above for the rule with a decay and a removal rate per channel: rates near 1 and near 0,
    decay pre-activations wide enough for both ends, key lengths far from one, and very short keys (the
    floor of the unit norm)."""
    H, d, dv = shape
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(19)
    T, decay = 83, math.exp(-0.5)
    r, k, a, w = (torch.randn(T, H * d, generator=g) for _ in range(4))
    k = k * (0.2 + 2.0 * torch.rand(T, 1, generator=g))
    k[5] *= 1e-4
    v = torch.randn(T, H * dv, generator=g)
    a, w = 3.0 * a, 4.0 * w
    ab, wb = torch.randn(H * d, generator=g), torch.randn(H * d, generator=g)
    r, k, v, a, w = (t.to(tdt) for t in (r, k, v, a, w))

    def heads(t, n):
        return t.double().view(T, H, n)

    dec = O.decay_of(heads(w.double() + wb.double(), d))
    rate = torch.sigmoid(heads(a.double() + ab.double(), d))
    want = torch.stack([O.generalized_delta_cell(heads(r, d)[:, h], dec[:, h], heads(k, d)[:, h], heads(v, dv)[:, h], rate[:, h])
                        for h in range(H)], 1).reshape(T, H * dv)
    state = torch.full((5, H, d, dv), -3.0, device=device)
    row = torch.cat([r, k, v, a], 1).to(device)          # columns of one row, as the projection leaves them
    wd, abd, wbd = w.to(device), ab.to(device), wb.to(device)
    c = [0, H * d, 2 * H * d, 2 * H * d + H * dv, 3 * H * d + H * dv]

    def call(segs, slots, single=False, n_single=0):
        rows = torch.cat([torch.arange(x, y) for x, y in segs]).to(device)
        cu = None if single else torch.tensor([0] + [y - x for x, y in segs]).cumsum(0).to(torch.int32).to(device)
        p = row[rows]
        return ops.channel_delta_scan(*(p[:, c[i]:c[i + 1]] for i in range(4)), wd[rows], abd, wbd, state, H, d, dv, decay, cu,
                                      i32(*slots, device=device), rows.to(torch.int32), n_single=n_single,
                                      max_q=max(y - x for x, y in segs))

    check_scan(call, want, dtype, state, -3.0, device)


@pytest.mark.parametrize("device", DEVICES)
def test_one_write_is_found_again_far_back(device):
    """A value written under a key that no later key touches is read back hundreds of rows later, and
    is gone once the same key is written again (the delta rule removes what it held)."""
    H, d, dv, T = 1, 16, 8, 300
    g = torch.Generator().manual_seed(23)
    key, val, val2 = torch.zeros(d), torch.randn(dv, generator=g), torch.randn(dv, generator=g)
    key[3] = 2.0
    k = torch.randn(T, d, generator=g)
    k[:, 3] = 0.0
    v = torch.randn(T, dv, generator=g)
    k[7], v[7] = key, val
    k[250], v[250] = key, val2
    q = torch.randn(T, d, generator=g)
    q[[200, 249, 250, 299]] = key
    x = torch.cat([q, k, v], 1).to(device)
    ba = torch.tensor([[30.0, -30.0]]).repeat(T, 1).to(device)     # step size 1, no decay
    state = torch.zeros(1, H, d, dv, device=device)
    a_log, bias = torch.zeros(1, device=device), torch.zeros(1, device=device)
    out = ops.gated_delta_scan(x, ba, a_log, bias, state, H, 1, d, dv, i32(0, T, device=device), i32(0, device=device),
                               torch.arange(T, dtype=torch.int32, device=device), max_q=T).cpu() * d ** 0.5
    assert (out[200] - val).abs().max() < 1e-3 and (out[249] - val).abs().max() < 1e-3
    assert (out[250] - val2).abs().max() < 1e-3 and (out[299] - val2).abs().max() < 1e-3


@pytest.mark.parametrize("device", DEVICES)
def test_routing_without_correction(device):
    g = torch.Generator().manual_seed(7)
    for (T, E, k, scale) in ((50, 6, 3, 1.7), (33, 20, 4, 2.0), (20, 8, 8, 1.0), (9, 1, 1, 3.0), (25, 64, 6, 0.5)):
        z = 2.0 * torch.randn(T, E, generator=g)
        z[0, :] = 0.25                                        # all tied: the lowest indices
        want = O.route(z.double(), {"top": k, "scale": scale})
        ids, wts = ops.moe_route_grouped(z.to(device), None, k, 1, 1, scale)
        for t in range(T):
            assert ids[t].tolist() == [e for e, _ in want[t]], f"row {t}: experts chosen"
            close(wts[t], torch.tensor([w for _, w in want[t]]), "float32", "weights")


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_router_of_few_and_many_rows(device, dtype):
    """The router product with the choice behind it: few rows (one launch) and more than that form takes,
    widths that are no multiple of 4, tied experts (equal router rows: the lower index), all chosen."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(8)
    for (T, H, E, k, scale) in ((7, 40, 5, 3, 1.7), (64, 1024, 32, 4, 2.0), (3, 33, 70, 9, 1.0), (5, 16, 1, 1, 3.0), (700, 64, 8, 2, 1.0),
                                (9, 24, 6, 6, 0.5), (4, 256, 512, 8, 1.0)):
        x = torch.randn(T, H, generator=g).to(tdt)
        r = torch.randn(E, H, generator=g) * (3.0 / H ** 0.5)
        if E == 5:
            r[3], r[4] = r[1], r[1]
        want = O.route(x.double() @ r.double().T, {"top": k, "scale": scale})
        ids, wts = ops.moe_router(x.to(device), r.to(device), k, scale)
        for t in range(T):
            assert ids[t].tolist() == [e for e, _ in want[t]], f"{T} x {H}, {E} experts, row {t}"
            close(wts[t], torch.tensor([w for _, w in want[t]]), "float32", "weights")


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_gelu_experts(device, dtype):
    """Small experts on the tiled form; sizes the MFMA form takes (a partial last block of features,
    more than one block, more rows than one tile)."""
    tdt = tdtype(dtype)
    g = torch.Generator().manual_seed(9)
    for (T, H, E, k, F) in ((33, 40, 5, 3, 14), (70, 24, 3, 2, 7), (150, 256, 4, 2, 64), (300, 256, 3, 2, 320), (12, 16, 1, 1, 8)):
        x = torch.randn(T, H, generator=g).to(tdt)
        ids, wts = ops.moe_route_grouped(torch.randn(T, E, generator=g).to(device), None, k, 1, 1, 1.3)
        w1 = (torch.randn(E, F, H, generator=g) * H ** -0.5).to(tdt)
        w2 = (torch.randn(E, H, F, generator=g) * F ** -0.5).to(tdt)
        got = ops.moe_plain_experts(x.to(device), ids, wts, w1.to(device), w2.to(device))
        want = torch.zeros(T, H, dtype=torch.float64)
        for t in range(T):
            for e, s in zip(ids[t].tolist(), wts[t].tolist()):
                want[t] += s * (O.gelu_erf(x[t].double() @ w1[e].double().T) @ w2[e].double().T)
        close(got, want, dtype, f"experts {E}, top {k}, ff {F}")
        x0, nw = torch.randn(T, H, generator=g), 1 + 0.1 * torch.randn(H, generator=g)
        args = (x.to(device), ids, wts, w1.to(device), w2.to(device))
        for mode in ("norm", "copy", "sum"):       # summed straight into the stream
            xs = x0.clone().to(device)
            out = ops.residual_plain_experts_(xs, *args, nw.to(device) if mode == "norm" else None, 1e-5, tdt, copy=mode == "copy")
            xw = x0.double() + want
            close(xs, xw, dtype, "stream")
            if mode == "sum":
                assert out is None
            else:
                close(out, xw if mode == "copy" else O.unit_rms(xw, 1e-5) * nw.double(), dtype, mode)


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
    assert len(tap) == len(runs) == len(cd["layers"])
    for i, (a, b) in enumerate(zip(tap, runs)):
        close_rows(a, b, dtype, f"residual stream after layer {i}")
    close_rows(got, want, dtype, "logits")
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
    """One head, q / k heads as many as heads and one for all, one expert with top 1, all experts
    chosen, a rotation of one pair and of the whole head, vdim = dim, one tap, a chunk of one token and none,
    scales of 1, no bigram, no token input, no feed-forward, a rank of one, a width that is no
    multiple of 8, one layer. (A head of one value column is brought to plus or minus one by its
    norm, so a rounding can turn its sign: heads of one column in float32 only.)"""
    one = 1 if dtype == "float32" else 4
    a = [par(heads=1, kv=1, dim=2, vdim=3, dims=2, chunk=1, rheads=1, rdim=one, rank=1, left_scale=1.0, right_scale=1.0),
         delta(heads=1, kv=1, dim=one, vdim=one, conv=1, mlp=moe(1, 1, 8, 1.0)),
         delta(heads=4, kv=4, dim=6, vdim=6, conv=2, mlp=moe(3, 3, 5, 0.7)),
         par(heads=6, kv=6, dim=4, vdim=4, dims=4, chunk=0, scaling=None, rheads=2, rdim=4, rank=8, mlp=moe(2, 1, 6))]
    toks = tokens(140, vocab=61, seed=9)
    for layers, bigram, side in ((a, (1, 0, 5), 1), (a, None, 0), (a[2:3], (7, 3, 0), 0), (a[3:], None, 5)):
        eng, cd, W = build(device, dtype, cd=cfg_dict(layers, width=36, vocab=61, bigram=bigram, side=side))
        close_rows(replay_cuts(eng, toks, [66, 5]), O.forward(cd, W, toks), dtype, f"bigram {bigram}, side {side}")


@pytest.mark.parametrize("device,dtype", DTYPES)
def test_long_decoding(device, dtype):
    """300 tokens decoded one by one after a short prompt: recurrent states carried through hundreds of
    single-row steps, chunk and page borders crossed by decoded tokens only."""
    eng, cd, W = build(device, dtype, cd=cfg_dict([delta(mlp=moe()), par(chunk=70)]))
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
    """Pipelined steps gather the ids of the step in flight on the device: the bigram embedding must
    read them from there and from the slots, not from the host."""
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


def test_model_folder_roundtrip(tmp_path):
    """config.json + safetensors -> registry -> engine (EngineConfig.model as a folder)."""
    from nv_genai_amd.models.registry import read_config
    from nv_genai_amd.utils.checkpoint import save_weights

    cd = cfg_odd()
    cfg = VivesunConfig.from_dict(cd)
    assert cfg.to_json_dict() == cd
    assert cfg.is_moe and cfg.experts_per_tok == 3 and cfg.num_experts == 5
    w = random_weights(cfg, 3, torch.bfloat16)
    save_weights(w, str(tmp_path))
    for b in cd["layers"]:      # the rank of the decay may also come from the tensors alone
        if b["type"] == "parallel":
            del b["mixer"]["right"]["decay_rank"]
    (tmp_path / "config.json").write_text(json.dumps(cd))
    got, cls = read_config(str(tmp_path))
    assert cls is VivesunModel and got == VivesunConfig.from_dict(cd)
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
        VivesunConfig.from_dict(bad)
    for layer in (delta(mlp=moe(3, 5)), par(dim=4, dims=6), par(heads=5, kv=2), delta(heads=5, kv=2),
                  delta(mlp={"kind": "dense", "ff": 4}), par(rdim=0), delta(conv=0)):
        with pytest.raises(ValueError):
            VivesunConfig.from_dict(cfg_dict([layer]))
    cfg = VivesunConfig.from_dict(cfg_odd())
    w = random_weights(cfg, 0)
    w["l0.mix.norm"] = w["l0.mix.norm"][:-1]
    with pytest.raises(ValueError):
        VivesunModel(cfg, "cpu", torch.float32, weights=w)
    c = vivesun_layers(["delta", "parallel", "delta"], 64, 4, 2, 16, 8, chunk=128, delta_heads=4, delta_kv_heads=2, delta_dim=8,
                       delta_vdim=16, right_heads=2, right_dim=8, experts=4, top=2, expert_ff=16, route_scale=2.0, rot_dims=8,
                       bands=(4.0, 1.0, 4.0, 64), bigram=(31, 3, 5), side_dim=8, left_scale=1.5)
    assert VivesunConfig.from_dict(c.to_json_dict()) == c
    assert c.blocks[1].mixer.left.chunk == 128 and c.blocks[0].mixer.kv_heads == 2


@pytest.mark.gpu
def test_mfma_forms_run_and_agree_with_the_plain_kernels():
    """At layer sizes (bf16): chunked attention with a sink on the MFMA prompt and single-token kernels
    against the row kernel, the gelu expert GEMMs on MFMA tiles against the tiled ones, and the
    block form of both scans against their single-row form."""
    dev = "cuda"
    g = torch.Generator().manual_seed(2)
    H, G, dk, dv, npg, chunk = 8, 2, 128, 128, 40, 300
    kc = (0.5 * torch.randn(npg, G, 64, dk, generator=g)).bfloat16().to(dev)
    vc = torch.randn(npg, G, 64, dv, generator=g).bfloat16().to(dev)
    bt = torch.randperm(npg, generator=g).to(torch.int32).view(2, 20).to(dev)
    cu, ctx = i32(0, 301, 370, device=dev), i32(1000, 69, device=dev)
    qq = (2.0 * torch.randn(370, H * dk, generator=g)).bfloat16().to(dev)
    assert ops.softmax_attention_mfma_ok(qq, dk, dv, 4, 1)
    seq, pos = ops._rows_of_portions(cu, ctx, 370, dev)
    kw = dict(scale=dk ** -0.5, chunk=chunk, sink=0.0)
    want = ops.softmax_attention(qq, kc, vc, bt, seq, pos, H, G, dk, dv, **kw).float()
    free = ops.softmax_attention(qq, kc, vc, bt, seq, pos, H, G, dk, dv, scale=dk ** -0.5, sink=0.0).float()
    assert (want - free).abs().max().item() > 0.1, "the chunk changes the result"
    for got in (ops.softmax_attention_prefill(qq, kc, vc, bt, cu, ctx, 301, H, G, dk, dv, **kw),
                ops.softmax_attention_rows(qq, kc, vc, bt, seq, pos, H, G, dk, dv, max_ctx=1024, **kw)):
        assert (got.float() - want).abs().max().item() < 0.03 * max(1.0, want.abs().max().item())
    T, W, E, k, F = 700, 512, 8, 3, 448
    x = torch.randn(T, W, generator=g).bfloat16().to(dev)
    w1 = (torch.randn(E, F, W, generator=g) * W ** -0.5).bfloat16().to(dev)
    w2 = (torch.randn(E, W, F, generator=g) * F ** -0.5).bfloat16().to(dev)
    ids, wts = ops.moe_route_grouped(torch.randn(T, E, generator=g).to(dev), None, k, 1, 1, 2.0)
    assert ops.moe_plain_mfma_ok(x, F)
    a = ops.moe_plain_experts(x, ids, wts, w1, w2).float()
    b = ops.moe_plain_experts(x.float(), ids, wts, w1.float(), w2.float())
    assert (a - b).abs().max().item() < 0.03 * max(1.0, b.abs().max().item())
    T, H, d, dv = 200, 4, 128, 128
    x, ba, al, db = gated_inputs(T, H, 2, d, dv, torch.bfloat16, g)
    x, ba, al, db = x.to(dev), ba.to(dev), al.to(dev), db.to(dev)
    s1, s2 = (torch.zeros(1, H, d, dv, device=dev) for _ in range(2))
    p = torch.arange(T, dtype=torch.int32, device=dev)
    slot = i32(0, device=dev)
    a = ops.gated_delta_scan(x, ba, al, db, s1, H, 2, d, dv, i32(0, T, device=dev), slot, p, max_q=T)
    b = torch.cat([ops.gated_delta_scan(x[t:t + 1], ba[t:t + 1], al, db, s2, H, 2, d, dv, None, slot, p[t:t + 1]) for t in range(T)])
    assert (a - b).abs().max().item() < 1e-4 * max(1.0, b.abs().max().item())
    assert (s1 - s2).abs().max().item() < 1e-4 * max(1.0, s2.abs().max().item())


@pytest.mark.gpu
@pytest.mark.parametrize("n", [3, 4])
def test_convolution_of_many_rows(n):
    """The form with the window of inputs in registers (bf16, hundreds of rows): segments of one, two and
    many rows whose borders fall anywhere in a thread's run of rows, fresh and going on from slots."""
    dev = "cuda"
    g = torch.Generator().manual_seed(31)
    C, lens = 72, [300, 1, 2, 5, 8, 250, 3, 17]
    T = 400
    xs = [torch.randn(T, C, generator=g).bfloat16() for _ in lens]
    taps = torch.randn(C, n, generator=g)
    want = [O.short_conv(x.double(), taps) for x in xs]
    td = taps.t().contiguous().to(dev)
    state = torch.full((len(lens), n - 1, C), 9.0, dtype=torch.bfloat16, device=dev)
    start = [0, 40, 1, 0, 2, 100, 0, 7]            # rows of the sequence already seen
    for i, s in enumerate(start):
        if s:
            pos = torch.arange(s, dtype=torch.int32, device=dev)
            ops.short_conv(xs[i][:s].to(dev), td, state, i32(0, s, device=dev), i32(i, device=dev), torch.zeros_like(pos), pos)
    wide = torch.zeros(sum(lens), C + 8, dtype=torch.bfloat16, device=dev)
    x = wide[:, :C]
    x.copy_(torch.cat([xs[i][s:s + k] for i, (s, k) in enumerate(zip(start, lens))]))
    pos = torch.cat([torch.arange(s, s + k) for s, k in zip(start, lens)]).to(torch.int32).to(dev)
    seq = torch.cat([torch.full((k,), i) for i, k in enumerate(lens)]).to(torch.int32).to(dev)
    cu = torch.tensor([0] + lens).cumsum(0).to(torch.int32).to(dev)
    assert sum(lens) >= 512
    got = ops.short_conv(x, td, state, cu, torch.arange(len(lens), dtype=torch.int32, device=dev), seq, pos)
    close(got, torch.cat([want[i][s:s + k] for i, (s, k) in enumerate(zip(start, lens))]), "bfloat16", "many rows")
    for i, (s, k) in enumerate(zip(start, lens)):
        pad = torch.cat([torch.zeros(n - 1, C).bfloat16(), xs[i][:s + k]])[-(n - 1):]
        assert torch.equal(state[i].cpu(), pad), f"inputs left in slot {i}"


@pytest.mark.gpu
@pytest.mark.parametrize("T,H", [(5000, 256), (4097, 1024), (4100, 3000), (37, 1024), (40, 5120), (33, 30)])
def test_residual_steps_of_many_rows(T, H):
    """The residual steps with the row in registers (one wave per row, one workgroup per row) and the
    scalar form: sum, copy, norm of the sum, norm of the sub-layer's output in front of the sum."""
    dev = "cuda"
    g = torch.Generator().manual_seed(37)
    x0, y = 3.0 * torch.randn(T, H, generator=g), torch.randn(T, H, generator=g).bfloat16()
    w, nw = 1 + 0.2 * torch.randn(H, generator=g), 1 + 0.2 * torch.randn(H, generator=g)
    xd, yd = x0.double(), y.double()
    eps = 1e-3
    x = x0.to(dev)
    h = ops.residual_add_rmsnorm_(x, y.to(dev), nw.to(dev), eps, torch.bfloat16)
    close(x, xd + yd, "float32", "sum")
    close(h, O.unit_rms(xd + yd, eps) * nw.double(), "bfloat16", "norm of the sum")
    assert ops.residual_add_rmsnorm_(x, y.to(dev), None, eps, torch.bfloat16) is None
    close(x, xd + 2 * yd, "float32", "sum alone")
    x = x0.to(dev)
    close(ops.residual_add_cast_(x, y.to(dev), torch.bfloat16), xd + yd, "bfloat16", "copy")
    x = x0.to(dev)
    h = ops.rmsnorm_residual_next_(x, y.to(dev), w.to(dev), eps, nw.to(dev), torch.bfloat16)
    xs = xd + O.unit_rms(yd, eps) * w.double()
    close(x, xs, "float32", "sum of the normed output")
    close(h, O.unit_rms(xs, eps) * nw.double(), "bfloat16", "next norm")


@pytest.mark.gpu
def test_captured_decode_graph_replays():
    """Decode steps from the captured graph, several in a row with eager steps of other sequences in
    between, against eager decoding of the same tokens: state, convolution inputs and previous
    tokens are written by the replays."""
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


@pytest.mark.parametrize("device", DEVICES)
def test_trace_runner_replays_a_schedule(device, tmp_path, monkeypatch, capsys):
    """The trace runner on a model folder: steps as JSON lines on standard input (a prompt in two
    portions, a second request beside single tokens of the first, requests ended and their names
    used again), logits files of the wanted places, a ``done`` line per step."""
    import io

    import numpy as np

    from nv_genai_amd.tools import trace_run
    from nv_genai_amd.utils.checkpoint import save_weights

    cd = cfg_dict([delta(mlp=moe()), par(chunk=33)])
    cfg = VivesunConfig.from_dict(cd)
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
