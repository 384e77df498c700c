"""Plain float64 implementation of the Vivesun design, written from its equations: one function
per mechanism, whole sequences, no cache, no batching. It imports nothing from the package and
is what the tests compare the serving path with.

``cfg`` is the config.json dict, ``w`` a dict of tensors under the checkpoint's names.
"""
import math

import torch

F64 = torch.float64
UNIT_EPS = 1e-6        # under the root of the unit vectors (keys, queries)
WEIGHT_FLOOR = 1e-20   # added to the sum of the chosen experts' scores


# ----------------------------------------------------------------------------- small pieces
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def norm(x, weight, eps):
    """RMS norm whose weight is stored around zero."""
    return unit_rms(x, eps) * (1.0 + weight.to(F64))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def silu(z):
    return z * torch.sigmoid(z)


def lin(x, w):
    return x @ w.to(F64).t()


# ----------------------------------------------------------------------------- embedding
def bigram_rows(tokens, bg):
    """Row of the bigram table per token: the pair's hash, the last row for a first token."""
    out = []
    for i, t in enumerate(tokens):
        if i == 0:
            out.append(int(bg["buckets"]))
        else:
            out.append((int(tokens[i - 1]) * int(bg["mul_prev"]) + int(t) * int(bg["mul_cur"])) % int(bg["buckets"]))
    return out


def embedding(cfg, w, tokens):
    x = w["embed"][torch.tensor(tokens)].to(F64)
    bg = (cfg.get("embedding") or {}).get("bigram")
    if bg:
        x = x + w["bigram"][torch.tensor(bigram_rows(tokens, bg))].to(F64)
    return x


def token_side(x, tokens, w, p, layer, dim, eps):
    """Per-layer token input: a gate of the stream on the token's own vector for this layer."""
    e = w["side.embed"][torch.tensor(tokens)][:, layer * dim:(layer + 1) * dim].to(F64)
    y = lin(gelu_tanh(lin(x, w[p + "side.gate"])) * e, w[p + "side.proj"])
    return x + unit_rms(y, eps) * w[p + "side.norm"].to(F64)


# ----------------------------------------------------------------------------- rotary positions
def rotary_frequencies(rot):
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F64)
    factor, low, high, orig = (float(sc[k]) for k in ("factor", "low", "high", "original"))
    out = []
    for v in f:
        wave = 2.0 * math.pi / v
        if wave < orig / high:
            out.append(v)
        elif wave > orig / low:
            out.append(v / factor)
        else:
            s = (orig / wave - low) / (high - low)
            out.append((1.0 - s) * v / factor + s * v)
    return torch.tensor(out, dtype=F64)


def rotate(x, rot, first_pos=0):
    """x [T, heads, d]: element i of the first ``dims`` is paired with element i + dims / 2."""
    dims = int(rot["dims"])
    half = dims // 2
    pos = torch.arange(first_pos, first_pos + x.shape[0], dtype=F64)
    ang = pos[:, None] * rotary_frequencies(rot)[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    a, b = x[..., :half], x[..., half:dims]
    return torch.cat([a * c - b * s, b * c + a * s, x[..., dims:]], dim=-1)


# ----------------------------------------------------------------------------- attention
def sink_weights(s):
    """exp(s) / (1 + sum exp(s)) over the last dimension (-inf: not seen)."""
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def chunk_mask(T, size, first_pos=0):
    """mask[i, j]: position i sees position j (same chunk of ``size``, counted from 0; not later)."""
    i = torch.arange(first_pos, first_pos + T)
    seen = i[:, None] >= i[None, :]
    if size:
        seen &= (i[:, None] // size) == (i[None, :] // size)
    return seen


def chunked_attention(q, k, v, scale, size=0):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; query head h reads kv head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    seen = chunk_mask(T, size)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].t()) * scale).masked_fill(~seen, float("-inf"))
        out[:, h] = sink_weights(s) @ v[:, g]
    return out


def mix_left(h, m, w, p):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate(lin(h, w[p + "q"]).view(T, H, d), m["rot"])
    k = rotate(lin(h, w[p + "k"]).view(T, G, d), m["rot"])
    v = lin(h, w[p + "v"]).view(T, G, dv)
    a = chunked_attention(q, k, v, float(m["scale"]), int((m.get("mask") or {}).get("size") or 0))
    return lin(a.reshape(T, H * dv), w[p + "o"])


# ----------------------------------------------------------------------------- delta rules
def generalized_delta_cell(r, w, k, v, a):
    """One head. r, k, a, w [T, d], v [T, dv]: S <- diag(w) S - (a u)(u^T S) + k v^T with u the unit
    key and both terms on the old state; o = S^T r."""
    T, d = k.shape
    S = torch.zeros(d, v.shape[1], dtype=F64)
    out = torch.zeros(T, v.shape[1], dtype=F64)
    for t in range(T):
        u = unit_vector(k[t])
        S = w[t][:, None] * S - torch.outer(a[t] * u, u @ S) + torch.outer(k[t], v[t])
        out[t] = r[t] @ S
    return out


def decay_of(z):
    """Decay of a pre-activation: exp(-exp(-1/2) sigmoid(z))."""
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(z))


def mix_right(h, m, w, p, eps):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    r, k, v = (lin(h, w[p + n]).view(T, H, d) for n in ("r", "k", "v"))
    dec = decay_of(lin(torch.tanh(lin(h, w[p + "w1"])), w[p + "w2"]) + w[p + "w0"].to(F64)).view(T, H, d)
    a = torch.sigmoid(lin(h, w[p + "a"]) + w[p + "a.b"].to(F64)).view(T, H, d)
    o = torch.stack([generalized_delta_cell(r[:, i], dec[:, i], k[:, i], v[:, i], a[:, i]) for i in range(H)], dim=1)
    o = unit_rms(o, eps).reshape(T, H * d) * w[p + "norm"].to(F64) * torch.sigmoid(lin(h, w[p + "g"]))
    return lin(o, w[p + "o"])


def mix_parallel(h, m, w, p, eps):
    return (float(m["left_scale"]) * mix_left(h, m["left"], w, p + "left.")
            + float(m["right_scale"]) * mix_right(h, m["right"], w, p + "right.", eps))


def short_conv(x, taps):
    """Causal convolution per channel (last column of ``taps`` is the current token's), then silu."""
    T, n = x.shape[0], taps.shape[1]
    pad = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=F64), x])
    y = sum(pad[j:j + T] * taps[:, j].to(F64)[None, :] for j in range(n))
    return silu(y)


def gated_delta_cell(q, k, v, beta, g):
    """One head, unit k, unit and scaled q: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, d = k.shape
    S = torch.zeros(d, v.shape[1], dtype=F64)
    out = torch.zeros(T, v.shape[1], dtype=F64)
    for t in range(T):
        S = g[t] * S
        S = S + torch.outer(k[t], beta[t] * (v[t] - k[t] @ S))
        out[t] = q[t] @ S
    return out


def mix_delta(h, m, w, p, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(lin(h, w[p + n]), w[p + n + ".conv"]) for n in ("q", "k", "v"))
    q = unit_vector(q.view(T, G, d)) * d ** -0.5
    k = unit_vector(k.view(T, G, d))
    v = v.view(T, H, dv)
    beta = torch.sigmoid(lin(h, w[p + "b"]))
    g = torch.exp(-torch.exp(w[p + "A_log"].to(F64))
                  * torch.nn.functional.softplus(lin(h, w[p + "a"]) + w[p + "dt_bias"].to(F64)))
    o = torch.stack([gated_delta_cell(q[:, i // (H // G)], k[:, i // (H // G)], v[:, i], beta[:, i], g[:, i])
                     for i in range(H)], dim=1)
    o = unit_rms(o, eps) * w[p + "norm"].to(F64) * silu(lin(h, w[p + "g"])).view(T, H, dv)
    return lin(o.reshape(T, H * dv), w[p + "o"])


# ----------------------------------------------------------------------------- feed-forward
def route(z, r):
    """Router logits [T, E] -> per row [(expert, weight), ...] in order of falling score."""
    s = torch.softmax(z.to(F64), dim=-1)
    out = []
    for row in s:
        ch = sorted(range(row.numel()), key=lambda e: (-float(row[e]), e))[:int(r["top"])]
        tot = sum(float(row[e]) for e in ch) + WEIGHT_FLOOR
        out.append([(e, float(row[e]) / tot * float(r.get("scale", 1.0))) for e in ch])
    return out


def moe_ff(h, m, w, p):
    out = torch.zeros_like(h)
    chosen = route(lin(h, w[p + "router"]), m["router"])
    for e in range(int(m["router"]["experts"])):
        rows = [(t, s) for t, ch in enumerate(chosen) for (x, s) in ch if x == e]
        if rows:
            idx = torch.tensor([t for t, _ in rows])
            y = lin(gelu_erf(lin(h[idx], w[f"{p}e{e}.up"])), w[f"{p}e{e}.down"])
            out[idx] += torch.tensor([s for _, s in rows], dtype=F64)[:, None] * y
    return out


# ----------------------------------------------------------------------------- the model
def forward(cfg, w, tokens, layer_runs_out=None):
    """Logits [T, vocab] of a whole sequence; ``layer_runs_out`` collects x after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = embedding(cfg, w, tokens)
    side = cfg.get("token_side")
    for i, b in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = norm(x, w[p + "norm1"], eps)
        if b["type"] == "delta":
            x = x + mix_delta(h, b["mixer"], w, p + "mix.", eps)
        elif b["type"] == "parallel":
            x = x + mix_parallel(h, b["mixer"], w, p + "mix.", eps)
        else:
            raise ValueError(b["type"])
        if b.get("mlp"):
            x = x + moe_ff(norm(x, w[p + "norm2"], eps), b["mlp"], w, p + "mlp.")
        if side:
            x = token_side(x, tokens, w, p, i, int(side["dim"]), eps)
        if layer_runs_out is not None:
            layer_runs_out.append(x.clone())
    return lin(norm(x, w["final.norm"], eps), w["embed"])


def greedy(cfg, w, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, w, toks)[-1].argmax()))
    return toks[len(prompt):]
