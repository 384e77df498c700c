"""Plain float64 implementation of the Kevelorn design, written from its equations: one function
per mechanism, whole sequences, no cache, no batching. It imports nothing from the package and
is what the tests compare the serving path with.

``cfg`` is the config.json dict, ``w`` a dict of tensors under the checkpoint's names.
"""
import math

import torch

F64 = torch.float64


# ----------------------------------------------------------------------------- small pieces
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, weight, eps):
    """RMS norm whose weight is stored around zero."""
    return unit_rms(x, eps) * (1.0 + weight.to(F64))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def lin(x, w):
    return x @ w.to(F64).t()


# ----------------------------------------------------------------------------- rotary positions
def rotary_frequencies(rot):
    dims, base = int(rot["dims"]), float(rot["base"])
    factor = float((rot.get("scaling") or {}).get("factor", 1.0))
    return torch.tensor([base ** (-2.0 * i / dims) / factor for i in range(dims // 2)], dtype=F64)


def rotate(x, rot, first_pos=0):
    """x [T, heads, d]: neighbouring elements (2i, 2i + 1) of the first ``dims`` turn together."""
    dims = int(rot["dims"])
    pos = torch.arange(first_pos, first_pos + x.shape[0], dtype=F64)
    ang = pos[:, None] * rotary_frequencies(rot)[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    y = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    y[..., 0:dims:2] = u * c - v * s
    y[..., 1:dims:2] = v * c + u * s
    return y


# ----------------------------------------------------------------------------- attention
def window_mask(T, size, first_pos=0):
    """mask[i, j]: position i sees position j (not later, fewer than ``size`` back; 0: all earlier)."""
    i = torch.arange(first_pos, first_pos + T)
    back = i[:, None] - i[None, :]
    seen = back >= 0
    if size:
        seen &= back < size
    return seen


def window_attention(q, k, v, scale, size=0):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; query head h reads kv head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    seen = window_mask(T, size)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].t()) * scale).masked_fill(~seen, float("-inf"))
        out[:, h] = torch.softmax(s, dim=-1) @ v[:, g]
    return out


def mix_attention(h, m, w, p, eps):
    """Rotation, then unit RMS of every q and k head; window; sigmoid gate per output element."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms(rotate(lin(h, w[p + "q"]).view(T, H, d), m["rot"]), eps)
    k = unit_rms(rotate(lin(h, w[p + "k"]).view(T, G, d), m["rot"]), eps)
    v = lin(h, w[p + "v"]).view(T, G, dv)
    a = window_attention(q, k, v, float(m["scale"]), int((m.get("mask") or {}).get("size") or 0))
    return lin(a.reshape(T, H * dv) * torch.sigmoid(lin(h, w[p + "g"])), w[p + "o"])


# ----------------------------------------------------------------------------- linear recurrences
def linear_cell(q, k, v, decay):
    """One head. q, k [T, d], v [T, dv], decay [T, d] (one factor per key channel and row):
    S <- diag(decay) S + k v^T, o = S^T q."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=F64)
    out = torch.zeros(v.shape, dtype=F64)
    for t in range(k.shape[0]):
        S = decay[t][:, None] * S + k[t][:, None] * v[t][None, :]
        out[t] = q[t] @ S
    return out


def mix_lightning(h, m, w, p, eps):
    """One constant decay per head; silu on q, k, v; one norm over all heads together."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = silu(lin(h, w[p + "q"])).view(T, H, d)
    k = silu(lin(h, w[p + "k"])).view(T, H, d)
    v = silu(lin(h, w[p + "v"])).view(T, H, dv)
    o = torch.stack([linear_cell(q[:, i], k[:, i], v[:, i], torch.full((T, d), float(m["decay"][i]), dtype=F64))
                     for i in range(H)], dim=1).reshape(T, H * dv)
    o = unit_rms(o, eps) * w[p + "norm"].to(F64)
    return lin(o * torch.sigmoid(lin(h, w[p + "g"])), w[p + "o"])


def gla_decay(z, tau):
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def mix_gla(h, m, w, p, eps):
    """A decay per key channel and token from a low-rank projection; a norm per head."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = (lin(h, w[p + "q"]) * d ** -0.5).view(T, H, d)
    k = lin(h, w[p + "k"]).view(T, H, d)
    v = lin(h, w[p + "v"]).view(T, H, dv)
    z = lin(lin(h, w[p + "a1"]), w[p + "a2"]) + w[p + "a2.b"].to(F64)
    a = gla_decay(z, float(m["tau"])).view(T, H, d)
    o = torch.stack([linear_cell(q[:, i], k[:, i], v[:, i], a[:, i]) for i in range(H)], dim=1)
    o = (unit_rms(o, eps) * w[p + "norm"].to(F64)).reshape(T, H * dv)
    return lin(o * silu(lin(h, w[p + "g"])), w[p + "o"])


def mix_parallel(h, m, w, p, eps):
    left = mix_attention(h, m["left"], w, p + "left.", eps)
    right = mix_lightning(h, m["right"], w, p + "right.", eps)
    return 0.5 * (unit_rms(left, eps) * w[p + "left.out"].to(F64) + unit_rms(right, eps) * w[p + "right.out"].to(F64))


MIXERS = {"parallel": mix_parallel, "lightning": mix_lightning, "gla": mix_gla}


# ----------------------------------------------------------------------------- feed-forwards
def glu(x, w, p, act):
    return lin(act(lin(x, w[p + "gate"])) * lin(x, w[p + "up"]), w[p + "down"])


def route(z, top):
    """(ids, weights) of one token: the largest logits, weights = softmax over the chosen ones."""
    ids = sorted(range(len(z)), key=lambda e: (-float(z[e]), e))[:top]
    return ids, torch.softmax(torch.stack([z[e] for e in ids]), dim=0)


def moe_ff(x, f, w, p):
    z = lin(x, w[p + "router"])
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        ids, wts = route(z[t], int(f["router"]["top"]))
        for e, c in zip(ids, wts):
            out[t] += c * glu(x[t:t + 1], w, f"{p}e{e}.", silu)[0]
    if f.get("shared"):
        out = out + torch.sigmoid(lin(x, w[p + "shared.sg"])) * glu(x, w, p + "shared.", silu)
    return out


def feed_forward(x, f, w, p):
    return moe_ff(x, f, w, p) if f.get("kind", "dense") == "moe" else glu(x, w, p, gelu_tanh)


# ----------------------------------------------------------------------------- the model
def layer_runs(cfg):
    """(layer, t) in running order; t is the number of the pass that begins with this run, else None."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, None) for i in range(lp["stop"], n)]


def forward(cfg, w, tokens, layers=None):
    """Logits [T, vocab] of a whole sequence; ``layers`` (a list) receives the stream after every run."""
    eps, m = float(cfg["norm"]["eps"]), float(cfg.get("residual_mult", 1.0))
    x0 = w["embed"][torch.tensor(tokens)].to(F64)
    x = x0
    for i, t in layer_runs(cfg):
        b, p = cfg["layers"][i], f"l{i}."
        if t is not None:
            x = (x + x0 if t else x) + w["loop.step"][t].to(F64)
        x = x + m * MIXERS[b["type"]](norm(x, w[p + "norm1"], eps), b["mixer"], w, p + "mix.", eps)
        if b.get("mlp"):
            x = x + m * feed_forward(norm(x, w[p + "norm2"], eps), b["mlp"], w, p + "mlp.")
        if layers is not None:
            layers.append(x)
    return lin(norm(x, w["final.norm"], eps), w["head"])


def greedy(cfg, w, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, w, toks)[-1].argmax()))
    return toks[len(prompt):]
