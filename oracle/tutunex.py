"""Plain, slow torch-CPU statement of the Tutunex design (test infrastructure only; shares no code with umbrella_amd/).

One function per mechanism, float64 unless the caller passes other tensors.  Notation: n tokens, X a sublayer's input
[n, width]; linear weights are [out, in] and applied as X @ W.T.  Every mixer takes the state an earlier stretch of the same
sequence left (``None``: a sequence that starts) and returns the state it leaves, so a prompt can be fed in portions.
``forward`` strings the mechanisms together from a configuration dictionary (the keys of config.json) and a name -> tensor
dictionary (the checkpoint's names).
"""
from __future__ import annotations

import math

import torch

F = torch.float64


def silu(z):
    return z * torch.sigmoid(z)


def rms(x, eps):
    """x over its root mean square"""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def unit(x):
    """x as a unit vector"""
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


# ------------------------------------------------------------------ rotary positions
def rotary_table(rot: dict):
    """(frequencies [dims / 2], factor on cos and sin).  Unscaled: base^(-2 i / dims), 1.  With ``scaling`` (YaRN): feature
    pairs that turn more than ``fast`` times over ``original`` positions keep their frequency, those that turn less than
    ``slow`` times are slowed down by ``factor``, a linear ramp over the pair's index in between."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F), 1.0
    factor, orig = float(sc["factor"]), float(sc["original"])

    def index_of(turns):
        return dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index_of(float(sc["fast"]))), 0)
    hi = min(math.ceil(index_of(float(sc["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=F), 0.1 * math.log(factor) + 1.0


def rotary(x, pos, freqs, mult: float):
    """x [n, heads, d]; of every head the first 2 len(freqs) features turn by pos * f_i (feature i pairs with i + len(freqs)) and
    grow by ``mult``; the other features pass"""
    half = freqs.numel()
    out = x.clone()
    ang = pos.to(x.dtype)[:, None] * freqs.to(x.dtype)[None, :]
    c, s = mult * torch.cos(ang)[:, None, :], mult * torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    out[..., :half] = u * c - v * s
    out[..., half:2 * half] = v * c + u * s
    return out


# ------------------------------------------------------------------ attention
def softmax_attention(q, k, v, q_pos, scale: float, chunk: int = 0, one_more: bool = False):
    """q [n, H, D] at positions q_pos; k [m, G, D], v [m, G, E] of positions 0 .. m - 1; query head h reads key / value head
    h // (H / G).  Position i sees the j <= i, with ``chunk`` only those of its own run of ``chunk`` positions (counted from
    position 0).  ``one_more``: one is added to the softmax denominator.  Returns [n, H, E]."""
    n, H, _ = q.shape
    m_, G, E = v.shape
    kpos = torch.arange(m_)
    hidden = kpos[None, :] > q_pos[:, None]
    if chunk:
        hidden = hidden | (kpos[None, :] // chunk != q_pos[:, None] // chunk)
    out = torch.zeros(n, H, E, dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(hidden, -math.inf)
        if one_more:
            s = torch.cat([torch.zeros(n, 1, dtype=s.dtype), s], dim=1)          # a key of score 0 that carries no value
            p = torch.softmax(s, dim=-1)[:, 1:]
        else:
            p = torch.softmax(s, dim=-1)
        out[:, h] = p @ v[:, g]
    return out


def differential_lambda(w: dict, diff: float) -> float:
    return float(torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum())) + diff


def differential_attention(X, pos, m: dict, w: dict, eps: float, kv=None):
    """two softmax maps per head over the same values: o = a1 - lambda a2, every head's o over its root mean square, times
    1 - diff.  kv: (k [m, G, 2, D] rotated, v [m, G, E]) of the positions before -- or, where the layer has no key / value
    projections of its own, of all positions including these.  Returns (out, (k, v))."""
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    n, diff = X.shape[0], float(m["diff"])
    fr, mult = rotary_table(m["rot"]) if m.get("rot") else (torch.zeros(0, dtype=F), 1.0)
    q = rotary((X @ w["q"].T).view(n, H * 2, D), pos, fr, mult).view(n, H, 2, D)
    if "k" in w:
        k = rotary((X @ w["k"].T).view(n, G * 2, D), pos, fr, mult).view(n, G, 2, D)
        v = (X @ w["v"].T).view(n, G, E)
        if kv is not None:
            k, v = torch.cat([kv[0], k]), torch.cat([kv[1], v])
    else:
        k, v = kv
    chunk = int((m.get("mask") or {}).get("size", 0))
    a1 = softmax_attention(q[:, :, 0], k[:, :, 0], v, pos, float(m["scale"]), chunk)
    a2 = softmax_attention(q[:, :, 1], k[:, :, 1], v, pos, float(m["scale"]), chunk)
    o = rms(a1 - differential_lambda(w, diff) * a2, eps) * (1.0 - diff)
    return o.reshape(n, H * E) @ w["o"].T, (k, v)


def sink_attention(X, pos, m: dict, w: dict, eps: float, kv=None):
    """grouped-query causal attention without positions: q and k RMS-normed per head (one weight for all heads), one added to
    the softmax denominator"""
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    n = X.shape[0]
    q = rms((X @ w["q"].T).view(n, H, D), eps) * w["q.norm"]
    k = rms((X @ w["k"].T).view(n, G, D), eps) * w["k.norm"]
    v = (X @ w["v"].T).view(n, G, E)
    if kv is not None:
        k, v = torch.cat([kv[0], k]), torch.cat([kv[1], v])
    o = softmax_attention(q, k, v, pos, float(m["scale"]), one_more=True)
    return o.reshape(n, H * E) @ w["o"].T, (k, v)


# ------------------------------------------------------------------ gated delta rule
def causal_conv(U, taps_w, history=None):
    """U [n, channels]; taps_w [channels, taps]; y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the sequence's start.
    history: the last taps - 1 inputs of earlier stretches.  Returns (y, new history)."""
    taps = taps_w.shape[1]
    n, C = U.shape
    hist = torch.zeros(taps - 1, C, dtype=U.dtype) if history is None else history
    ext = torch.cat([hist, U], dim=0)
    y = torch.zeros_like(U)
    for j in range(taps):
        y = y + taps_w[:, j][None, :] * ext[j:j + n]
    return y, ext[ext.shape[0] - (taps - 1):].clone()


def delta_recurrence(q, k, v, g, beta, S):
    """q, k [n, H, D], v [n, H, E], g, beta [n, H], S [H, D, E]: per token S <- g S, u = beta (v - S^T k), S <- S + k u^T,
    o = S^T q.  Returns (o [n, H, E], S)."""
    o = torch.zeros(v.shape, dtype=v.dtype)
    S = S.clone()
    for t in range(q.shape[0]):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hde,hd->he", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = torch.einsum("hde,hd->he", S, q[t])
    return o, S


def gated_delta(X, m: dict, w: dict, eps: float, state=None):
    """q, k (kv_heads x dim) and v (heads x vdim) through a short causal convolution and silu, q and k as unit vectors per head
    (q times dim^-1/2), one decay and one step size per head, the delta rule, every head's read-out over its root mean square
    times a weight and silu of a gate, then W_o.  state: {"hist": inputs of q | k | v, "S": [heads, dim, vdim]}."""
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    n = X.shape[0]
    st = state or {}
    raw = torch.cat([X @ w["q"].T, X @ w["k"].T, X @ w["v"].T], dim=1)
    u, hist = causal_conv(raw, torch.cat([w["q.conv"], w["k.conv"], w["v.conv"]]), st.get("hist"))
    u = silu(u)
    q = unit(u[:, :G * D].reshape(n, G, D)) * D ** -0.5
    k = unit(u[:, G * D:2 * G * D].reshape(n, G, D))
    v = u[:, 2 * G * D:].reshape(n, H, E)
    rep = H // G
    q, k = q.repeat_interleave(rep, dim=1), k.repeat_interleave(rep, dim=1)
    beta = torch.sigmoid(X @ w["b"].T)
    z = X @ w["a"].T + w["dt_bias"]
    softplus = torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))
    g = torch.exp(-torch.exp(w["A_log"]) * softplus)
    S0 = torch.zeros(H, D, E, dtype=X.dtype) if st.get("S") is None else st["S"]
    o, S = delta_recurrence(q, k, v, g, beta, S0)
    y = rms(o, eps) * w["norm"] * silu(X @ w["g"].T).view(n, H, E)
    return y.reshape(n, H * E) @ w["o"].T, {"hist": hist, "S": S}


# ------------------------------------------------------------------ feed-forward
def capped_glu(X, w: dict, limit: float):
    g = torch.clamp(X @ w["gate"].T, max=limit)
    u = torch.clamp(X @ w["up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


# ------------------------------------------------------------------ the model
def _sub(sd: dict, prefix: str, dtype) -> dict:
    return {k[len(prefix):]: v.to(dtype) for k, v in sd.items() if k.startswith(prefix)}


def forward(cfg: dict, sd: dict, tokens, state=None, dtype=F):
    """tokens: the next ids of ONE sequence; state: what ``forward`` returned for the stretch before (None: the sequence
    starts).  Returns (logits [n, vocab], residual stream after every layer [layers, n, width], state)."""
    eps = float(cfg["norm"]["eps"])
    ids = torch.as_tensor(tokens, dtype=torch.long)
    n = ids.numel()
    state = state or {"len": 0, "layers": {}}
    pos = torch.arange(state["len"], state["len"] + n)
    x = sd["embed"].to(dtype)[ids] * float(cfg["embedding"]["scale"])
    trace, new = [], {}
    for i, ly in enumerate(cfg["layers"]):
        p, m = f"l{i}.", ly["mixer"]
        nw = {k: sd[p + k].to(dtype) for k in ("norm1", "norm1b", "norm2", "norm2b") if p + k in sd}
        h = rms(x, eps) * nw["norm1"]
        st = state["layers"].get(i)
        if ly["type"] == "attention":
            kv = new[int(m["kv_from"])] if m.get("kv_from") is not None else st
            y, new[i] = differential_attention(h, pos, m, _sub(sd, p + "mix.", dtype), eps, kv)
        elif ly["type"] == "parallel":
            st = st or (None, None)
            left, right = _sub(sd, p + "mix.left.", dtype), _sub(sd, p + "mix.right.", dtype)
            ya, sa = sink_attention(h, pos, m["left"], left, eps, st[0])
            yb, sb = gated_delta(h, m["right"], right, eps, st[1])
            y, new[i] = 0.5 * (rms(ya, eps) * left["out"] + rms(yb, eps) * right["out"]), (sa, sb)
        else:
            raise ValueError(ly["type"])
        x = x + rms(y, eps) * nw["norm1b"]
        if ly.get("mlp"):
            f = capped_glu(rms(x, eps) * nw["norm2"], _sub(sd, p + "mlp.", dtype), float(ly["mlp"]["limit"]))
            x = x + rms(f, eps) * nw["norm2b"]
        trace.append(x.clone())
    logits = (rms(x, eps) * sd["final.norm"].to(dtype)) @ sd["head"].to(dtype).T
    return logits, torch.stack(trace), {"len": state["len"] + n, "layers": new}
