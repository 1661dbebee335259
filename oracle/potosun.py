"""Plain, slow torch-CPU statement of the Potosun design (test infrastructure only; shares no code with umbrella_amd/).

One function per mechanism, float64 unless the caller passes other tensors.  Notation: n tokens, X a sublayer's input
[n, width]; linear weights are [out, in] and applied as X @ W.T.  Every mixer takes the rows an earlier stretch of the same
sequence left (``None``: a sequence that starts) and returns what it leaves, so a prompt can be fed in portions.
``forward`` strings the mechanisms together from a configuration dictionary (the keys of config.json) and a name -> tensor
dictionary (the checkpoint's names).
"""
from __future__ import annotations

import math

import torch

F = torch.float64


def rms(x, eps):
    """x over its root mean square"""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def gelu(z):
    """the tanh form of gelu"""
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z.pow(3))))


# ------------------------------------------------------------------ positions
def frequencies(rot: dict):
    """(angle per position of every feature pair, factor on cos and sin): base^(-2 i / dims), 1; with ``scaling`` (YaRN) the pairs
    that turn more than ``fast`` times over ``original`` positions keep it, those below ``slow`` turns get a ``factor``-th, with a
    linear ramp over the pair's index in between"""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F), 1.0
    factor, orig = float(sc["factor"]), float(sc["original"])
    at = lambda turns: dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))      # noqa: E731
    lo, hi = max(math.floor(at(float(sc["fast"]))), 0), min(math.ceil(at(float(sc["slow"]))), dims - 1)
    ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(len(f))]
    return torch.tensor([a / factor * r + a * (1.0 - r) for a, r in zip(f, ramp)], dtype=F), 0.1 * math.log(factor) + 1.0


def rotate(x, pos, rot, interleaved: bool):
    """x [n, heads, d]: the first rot["dims"] features turn, pairs (2i, 2i + 1) or (i, i + dims / 2); the others pass"""
    if not rot or not int(rot["dims"]):
        return x
    fr, mult = frequencies(rot)
    d, half = int(rot["dims"]), int(rot["dims"]) // 2
    a = pos.to(F)[:, None, None] * fr.to(x.dtype)
    c, s = mult * torch.cos(a), mult * torch.sin(a)
    out = x.clone()
    iu, iv = (slice(0, d, 2), slice(1, d, 2)) if interleaved else (slice(0, half), slice(half, d))
    u, v = x[..., iu], x[..., iv]
    out[..., iu] = u * c - v * s
    out[..., iv] = v * c + u * s
    return out


def distance_bucket(n: int, rows: int, far: float) -> int:
    """row of the bias table at distance n: the distance itself below rows // 2, then logarithmic steps, the last row from ``far`` on (a whole
    number of steps counts as that number although the quotient of two rounded logarithms may fall short of it)"""
    half = rows // 2
    if n < half:
        return n
    steps = math.log(n / half) / math.log(far / half) * (rows - half)
    whole = round(steps)
    return min(rows - 1, half + (whole if abs(steps - whole) < 1e-9 else math.floor(steps)))


# ------------------------------------------------------------------ which keys a position sees
def sees_window(i: int, j: int, size: int, keep_first: int = 0) -> bool:
    return j <= i and (i - j < size or j < keep_first)


def sees_chunk(i: int, j: int, size: int) -> bool:
    return j <= i and i // size == j // size


def visible(q_pos, m: int, sees):
    """[n, m] booleans"""
    return torch.tensor([[bool(sees(int(i), j)) for j in range(m)] for i in q_pos])


def softmax_over(scores, see, sink=None):
    """weights over the seen keys; a sink's exponential joins the denominator and carries nothing"""
    s = scores.masked_fill(~see, -math.inf)
    if sink is None:
        return torch.softmax(s, dim=-1)
    extra = torch.full((s.shape[0], 1), float(sink), dtype=s.dtype)
    return torch.softmax(torch.cat([s, extra], dim=1), dim=-1)[:, :-1]


# ------------------------------------------------------------------ mixers
def mix_values(v, lam: float, v_first):
    return (1.0 - lam) * v + lam * v_first


def attend(q, k, v, see, scale: float, sink=None, bias=None):
    """q [n, H, D], k [m, G, D], v [m, G, E]; query head h reads key / value head h // (H / G); bias [n, m, H] joins the scaled
    products.  Returns [n, H, E]."""
    n, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(n, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if bias is not None:
            s = s + bias[..., h]
        out[:, h] = softmax_over(s, see, None if sink is None else sink[h]) @ v[:, g]
    return out


def _project(X, m, w, v_first):
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    n = X.shape[0]
    q, k, v = (X @ w["q"].T).view(n, H, D), (X @ w["k"].T).view(n, G, D), (X @ w["v"].T).view(n, G, E)
    raw = v
    if m.get("v_mix") and v_first is not None:
        v = mix_values(v, float(w["vmix"]), v_first)
    return q, k, v, raw


def biased_attention(X, pos, m: dict, w: dict, eps: float, v_first=None, kv=None):
    """per-head normed q and k, no rotation, a learned bias by distance, a sliding window that keeps the first tokens, an element-wise
    sigmoid gate.  v_first: [n, G, E] of the first layer that mixes values (None: this is it, or the layer does not mix).
    Returns (out, the layer's own unmixed values, (k, v) rows)."""
    n = X.shape[0]
    q, k, v, raw = _project(X, m, w, v_first)
    q, k = rms(q, eps) * w["q.norm"], rms(k, eps) * w["k.norm"]
    if kv is not None:
        k, v = torch.cat([kv[0], k]), torch.cat([kv[1], v])
    size, keep = int(m["mask"]["size"]), int(m["mask"].get("keep_first", 0))
    see = visible(pos, k.shape[0], lambda i, j: sees_window(i, j, size, keep))
    rows = w["rel"].shape[0]
    row_of = torch.tensor([[distance_bucket(max(int(i) - j, 0), rows, float(m["bias_max"])) for j in range(k.shape[0])] for i in pos])
    o = attend(q, k, v, see, float(m["scale"]), bias=w["rel"][row_of])
    return (o.reshape(n, -1) * torch.sigmoid(X @ w["g"].T)) @ w["o"].T, raw, (k, v)


def chunked_attention(X, pos, m: dict, w: dict, eps: float, v_first=None, kv=None):
    """interleaved rotary positions, keys of the query's own chunk of positions, a sink; otherwise as above"""
    n = X.shape[0]
    q, k, v, raw = _project(X, m, w, v_first)
    q, k = rotate(q, pos, m.get("rot"), True), rotate(k, pos, m.get("rot"), True)
    if kv is not None:
        k, v = torch.cat([kv[0], k]), torch.cat([kv[1], v])
    size = int(m["mask"]["size"])
    see = visible(pos, k.shape[0], lambda i, j: sees_chunk(i, j, size))
    o = attend(q, k, v, see, float(m["scale"]), sink=w["sink"])
    return o.reshape(n, -1) @ w["o"].T, raw, (k, v)


def latent_attention(X, pos, m: dict, w: dict, eps: float, rows=None):
    """keys and values from one normed latent per token plus one rotated key part that all heads share; queries straight from the
    input; sliding window, sink, one sigmoid gate per head.  rows: (latents [m, r], rotated parts [m, R]) of earlier positions."""
    H, D, R, E, r = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    n = X.shape[0]
    q = (X @ w["q"].T).view(n, H, D + R)
    q_plain, q_rot = q[..., :D], rotate(q[..., D:], pos, m["rot"], False)
    down = X @ w["dkv"].T
    c = rms(down[:, :r], eps) * w["dkv.norm"]
    kr = rotate(down[:, None, r:], pos, m["rot"], False)[:, 0]
    if rows is not None:
        c, kr = torch.cat([rows[0], c]), torch.cat([rows[1], kr])
    k = (c @ w["uk"].T).view(-1, H, D)
    v = (c @ w["uv"].T).view(-1, H, E)
    size = int(m["mask"]["size"])
    see = visible(pos, c.shape[0], lambda i, j: sees_window(i, j, size))
    gate = torch.sigmoid(X @ w["g"].T)
    out = torch.zeros(n, H, E, dtype=X.dtype)
    for h in range(H):
        s = (q_plain[:, h] @ k[:, h].T + q_rot[:, h] @ kr.T) * float(m["scale"])
        out[:, h] = (softmax_over(s, see, w["sink"][h]) @ v[:, h]) * gate[:, h:h + 1]
    return out.reshape(n, -1) @ w["o"].T, (c, kr)


def gated_ff(X, w: dict):
    return (gelu(X @ w["gate"].T) * (X @ w["up"].T)) @ w["down"].T


def cap(logits, limit: float):
    return limit * torch.tanh(logits / limit)


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
    trace, new, v_first = [], {}, None
    for i, ly in enumerate(cfg["layers"]):
        p, m, st = f"l{i}.", ly["mixer"], state["layers"].get(i)
        w = _sub(sd, p + "mix.", dtype)
        h = rms(x, eps) * sd[p + "norm1"].to(dtype)
        if ly["type"] == "latent_attention":
            y, new[i] = latent_attention(h, pos, m, w, eps, st)
        else:
            mixer = {"attention": biased_attention, "attention_2": chunked_attention}[ly["type"]]
            y, raw, new[i] = mixer(h, pos, m, w, eps, v_first, st)
            if m.get("v_mix") and v_first is None:
                v_first = raw
        x = x + y
        if ly.get("mlp"):
            x = x + gated_ff(rms(x, eps) * sd[p + "norm2"].to(dtype), _sub(sd, p + "mlp.", dtype))
        trace.append(x.clone())
    logits = (rms(x, eps) * sd["final.norm"].to(dtype)) @ sd["head"].to(dtype).T
    return cap(logits, float(cfg["logit_softcap"])), torch.stack(trace), {"len": state["len"] + n, "layers": new}
