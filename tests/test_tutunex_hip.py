"""The Tutunex design on the HIP path against the plain oracle (oracle/tutunex.py): its mechanisms alone through their own entry
points of libumbrella_seq.so (rotary prep of both maps, differential attention over chunks with own and with shared keys, sink
attention, the gated delta rule token by token and in chunks, the seam behind two mixers), then whole models through the runtime,
the cache manager, the batch engine and the trace replay command.

fp32 runs are the sharp ones (every comparison to ~1e-5: one key too many, a lost state or a tap from the wrong position is a
thousand times that); bf16 runs use inputs built so that a fault still shows."""
import json
import os
import subprocess
import sys

import pytest
import torch

pytestmark = pytest.mark.gpu

ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))
sys.path.insert(0, os.path.dirname(__file__))
F32_TOL = 2e-5
BF16_TOL = 4e-2


@pytest.fixture(scope="module")
def lib():
    import __graft_entry__ as ge
    from umbrella_amd import _lib
    if not os.path.exists(_lib.SEQ_LIB_PATH):
        ge.build_seq()
    return _lib.load_seq()


def code(dtype):
    from umbrella_amd import _lib
    return _lib.seq_dtype_code(dtype)


def call(name, *a):
    from umbrella_amd import _lib
    return _lib.seq_call(name, *a)


def form(maps=1, chunk=0, sink=None, lam=0.0, eps=0.0):
    from umbrella_amd import _lib
    f = _lib.UmbAttnForm()
    f.maps, f.chunk, f.sink, f.lambda_, f.eps = maps, chunk, (sink.data_ptr() if sink is not None else None), lam, eps
    return f


def tol_of(dtype):
    return F32_TOL if dtype == torch.float32 else BF16_TOL


# ------------------------------------------------------------------ embedding and seams
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W,T,scale", [(40, 3, 1.0), (300, 5, 2.5), (1500, 2, 0.3)])
def test_scaled_embedding_and_first_norm(lib, dtype, W, T, scale):
    from oracle import tutunex as O
    from tutunex_helpers import close, dev, i32, rnd, tokens, zeros
    emb, w, tk = rnd((17, W), 1).to(dtype), (1 + rnd((W,), 2, 0.2)).to(dtype), tokens(T, 17, 3)
    x, h = zeros(T, W), zeros(T, W, dtype=dtype)
    call("umb_seq_embed_norm", x, h, dev(emb), i32(tk), scale, dev(w), T, W, 17, 1, 1e-2, code(dtype))
    want = emb[tk].double() * scale
    assert close(x, want, 1e-6) and close(h, O.rms(want, 1e-2) * w.double(), 1e-6 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W,T", [(40, 3), (300, 5), (512, 2), (1500, 2), (4000, 2), (5000, 3)])
def test_seam_behind_two_mixers(lib, dtype, W, T):
    from oracle import tutunex as O
    from tutunex_helpers import close, dev, rnd, zeros
    eps = 3e-2                                            # large: where it stands in the root shows
    x0, y1, y2 = rnd((T, W), 1), rnd((T, W), 2, 0.2), rnd((T, W), 3, 7.0)
    w1, w2, wp, wn = ((1 + rnd((W,), 4 + k, 0.3)).to(dtype) for k in range(4))
    want_m = 0.5 * (O.rms(y1.double(), eps) * w1.double() + O.rms(y2.double(), eps) * w2.double())
    want = x0.double() + O.rms(want_m, eps) * wp.double()
    for nxt in (True, False):
        x, h = dev(x0.clone()), zeros(T, W, dtype=dtype)
        call("umb_seq_pair_resid_norm", x, h, dev(y1), dev(y2), dev(w1), dev(w2), 0.5, dev(wp), dev(wn) if nxt else None, T, W, eps, code(dtype))
        assert close(x, want, 1e-6)
        if nxt:
            assert close(h, O.rms(want, eps) * wn.double(), 1e-6 if dtype == torch.float32 else 1e-2)
        else:
            assert float(h.float().abs().max()) == 0.0


# ------------------------------------------------------------------ attention
def _cache(G, DK, E, dtype, page, seqs=3, max_tokens=2048):
    from umbrella_amd.attn.cache import PagedSeqCache
    c = PagedSeqCache([(G, DK, 0, E)], [], max_tokens, seqs, "cuda:0", dtype, page=page)
    for z in (c.kv[0]["k"], c.kv[0]["v"]):
        z.fill_(9.0)                                      # what a page held before must not matter
    return c


def _attend(lib, out, ldo, q, kv, st, H, G, D, E, scale, out_scale, f, dtype, split):
    from tutunex_helpers import zeros
    if st.max_len >= 16 and lib.umb_bsa_attend_tiled_ok(H, G, D, E, code(dtype)):
        call("umb_attn_attend_tiled", out, ldo, q, kv, None, 0, -1, None, 0, *st.seqs, st.B, st.max_len, H, G, D, E, 2 ** 30, scale, out_scale,
             0.0, f, code(dtype))
    else:
        scratch = zeros(st.T * H * f.maps * 16 * (E + 2)) if split else None
        call("umb_attn_attend", out, ldo, q, kv, None, 0, -1, None, 0, st.d["pos"], st.d["slot"], st.T, H, G, D, E, 2 ** 30, scale, out_scale, 0.0,
             f, scratch, scratch.numel() if split else 0, code(dtype))


def _run_diff(lib, m, w, X, splits, dtype, page=4, cache=None, seq="s", split=True, readers=()):
    """the attention through prep / append / attend, the output projection left out (w["o"] is the identity).  readers: further
    (m, w) that attend over the same store with queries of their own -> list of outputs"""
    from oracle import tutunex as O
    from umbrella_amd.models.config import rotary_table
    from tutunex_helpers import Steps, dev, zeros
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    freq, mult = rotary_table(rot["base"], rot["dims"], rot.get("scaling")) if rot["dims"] else (None, 1.0)
    fr = dev(freq) if freq is not None else None
    Xd = X.double()
    proj_all = torch.cat([Xd @ w["q"].double().T, Xd @ w["k"].double().T, Xd @ w["v"].double().T], dim=1).float()
    ld = proj_all.shape[1]
    cache = cache or _cache(G, 2 * D, E, dtype, page)
    cache.open(seq)
    kv = cache.struct(0)
    outs, at = [[] for _ in range(1 + len(readers))], 0
    for cnt in splits:
        p0 = cache.extend(seq, cnt)
        st = Steps([cnt], [p0], [cache.slot(seq)])
        for n, (mm, ww) in enumerate([(m, w)] + list(readers)):
            proj = dev(proj_all[at:at + cnt]) if n == 0 else dev((Xd[at:at + cnt] @ ww["q"].double().T).float())
            q, out = zeros(cnt, 2 * H * D), zeros(cnt, H * E + 3, dtype=dtype)
            call("umb_attn_prep", q, kv, proj, proj.shape[1], int(n == 0), None, None, 0, 0, st.d["pos"], st.d["slot"], fr, rot["dims"], 0, mult, cnt,
                 H, G, D, E, 2, 0.0, 0, 1e-5, code(dtype))
            lam = O.differential_lambda({k: v.double() for k, v in ww.items()}, mm["diff"])
            f = form(2, (mm.get("mask") or {}).get("size", 0), None, lam, 1e-5)
            _attend(lib, out, H * E + 3, q, kv, st, H, G, D, E, mm["scale"], 1.0 - mm["diff"], f, dtype, split)
            assert float(out[:, H * E:].float().abs().max()) == 0.0
            outs[n].append(out[:, :H * E].clone())
        at += cnt
    outs = [torch.cat(o) for o in outs]
    return (outs if readers else outs[0]), cache


def _diff_case(H, G, D, E, chunk, dims, seed, W=24, scaling=True, diff=0.4):
    from tutunex_helpers import YARN, attention, rnd
    _, m = attention(H, G, D, E, diff=diff, chunk=chunk, rot_dims=dims, scaling=YARN if scaling else None)
    w = {"q": 1.5 * rnd((H * 2 * D, W), seed) / W ** 0.5, "k": 1.5 * rnd((G * 2 * D, W), seed + 1) / W ** 0.5, "v": rnd((G * E, W), seed + 2) / W ** 0.5,
         "o": torch.eye(H * E), **{n: rnd((D,), seed + 3 + k, 0.6 / D ** 0.25) for k, n in enumerate(("lq1", "lk1", "lq2", "lk2"))}}
    return m, w


DIFF_SHAPES = [(4, 2, 8, 12, 10, 6, [19]), (3, 1, 7, 5, 0, 0, [1] * 12), (2, 2, 16, 16, 8, 16, [2, 9, 1, 1, 17, 3]), (4, 4, 16, 32, 33, 8, [40, 1, 1, 30, 2, 2]),
               (8, 2, 40, 80, 64, 20, [70, 1, 64, 3, 62]), (6, 1, 24, 48, 1, 24, [20, 1, 1]), (8, 1, 72, 144, 50, 72, [33, 20, 1, 48]),
               (2, 1, 136, 272, 30, 10, [17, 2, 16])]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,E,chunk,dims,splits", DIFF_SHAPES)
def test_differential_attention_prompt_portions_and_single_tokens(lib, dtype, H, G, D, E, chunk, dims, splits):
    from oracle import tutunex as O
    from tutunex_helpers import close, rnd
    n = sum(splits)
    m, w = _diff_case(H, G, D, E, chunk, dims, 1)
    X = rnd((n, 24), 9)
    want, _ = O.differential_attention(X.double(), torch.arange(n), m, {k: v.double() for k, v in w.items()}, 1e-5)
    got, cache = _run_diff(lib, m, w, X, splits, dtype)
    assert close(got, want, tol_of(dtype))
    one, _ = _run_diff(lib, m, w, X, splits, dtype, page=16, split=False)
    assert close(one, want, tol_of(dtype))
    cache.close("s")                                      # pages and slot go back and are used again by a sequence that starts at 0
    again, _ = _run_diff(lib, m, w, X[:9], [4, 1, 4], dtype, cache=cache, seq="t")
    assert close(again, want[:9], tol_of(dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_layers_that_read_another_layers_keys(lib, dtype):
    """two readers with queries, masks, scales and constants of their own over one store"""
    from oracle import tutunex as O
    from tutunex_helpers import close, rnd
    m, w = _diff_case(4, 2, 16, 32, 10, 8, 1)
    readers = []
    for seed, (chunk, diff, scale) in ((30, (7, 0.7, 0.2)), (40, (0, 0.1, 0.4))):
        m2, w2 = _diff_case(4, 2, 16, 32, chunk, 8, seed, diff=diff)
        m2["scale"] = scale
        readers.append((m2, {k: v for k, v in w2.items() if k not in ("k", "v")}))
    splits = [21, 1, 1, 2, 18, 1]
    n = sum(splits)
    X = rnd((n, 24), 9)
    dbl = lambda d: {k: v.double() for k, v in d.items()}                                                # noqa: E731
    want, kv = O.differential_attention(X.double(), torch.arange(n), m, dbl(w), 1e-5)
    outs, _ = _run_diff(lib, m, w, X, splits, dtype, readers=readers)
    assert close(outs[0], want, tol_of(dtype))
    for got, (m2, w2) in zip(outs[1:], readers):
        assert close(got, O.differential_attention(X.double(), torch.arange(n), m2, dbl(w2), 1e-5, kv)[0], tol_of(dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("page", [4, 16])
def test_chunk_edges_of_one_outstanding_key(lib, dtype, page):
    """map 1 finds one key (score far above all others) whose value row carries a mark, map 2 sees everything evenly: the positions
    of the key's own chunk from the key on read the mark, the first position of the next chunk and everything before the key do
    not -- for keys at the first, a middle and the last place of a chunk, in prompts (matrix pipe in 16 bits), portions cut at
    and beside the edge, and tokens decoded one by one across it"""
    from tutunex_helpers import Steps, close, dev, rnd, zeros
    from oracle import tutunex as O
    H, G, D, E, n, chunk, lam = 4, 2, 16, 16, 130, 30, 0.3
    for far in (30, 47, 59):
        q = 0.02 * rnd((n, H, 2, D), 1)
        k = 0.02 * rnd((n, G, 2, D), 2)
        v = 0.3 * rnd((n, G, E), 3)
        q[:, :, 0, 0] = 4.0
        k[far, :, 0, 0] = 4.0
        v[far] = torch.linspace(3.0, 8.0, E)
        ref1 = O.softmax_attention(q[:, :, 0].double(), k[:, :, 0].double(), v.double(), torch.arange(n), 1.0, chunk)
        ref2 = O.softmax_attention(q[:, :, 1].double(), k[:, :, 1].double(), v.double(), torch.arange(n), 1.0, chunk)
        ref = (O.rms(ref1 - lam * ref2, 1e-5) * 0.6).reshape(n, H * E)
        mark = torch.linspace(3.0, 8.0, E).double()
        mark = mark / mark.pow(2).mean().sqrt()
        proj_all = torch.cat([q.reshape(n, -1), k.reshape(n, -1), v.reshape(n, -1)], dim=1)
        f = form(2, chunk, None, lam, 1e-5)
        for splits in ([n], [far + 1] + [1] * (n - far - 1), [60, 2, 1, 27, 40], [59, 1, 1, 29, 40]):
            cache = _cache(G, 2 * D, E, dtype, page)
            cache.open("s")
            kv, at, rows = cache.struct(0), 0, []
            for cnt in splits:
                st = Steps([cnt], [cache.extend("s", cnt)], [cache.slot("s")])
                proj, qq, out = dev(proj_all[at:at + cnt]), zeros(cnt, 2 * H * D), zeros(cnt, H * E, dtype=dtype)
                call("umb_attn_prep", qq, kv, proj, proj.shape[1], 1, None, None, 0, 0, st.d["pos"], st.d["slot"], None, 0, 0, 1.0, cnt, H, G, D, E, 2,
                     0.0, 0, 1e-5, code(dtype))
                _attend(lib, out, H * E, qq, kv, st, H, G, D, E, 1.0, 0.6, f, dtype, True)
                rows.append(out)
                at += cnt
            got = torch.cat(rows)
            assert close(got, ref, 3e-5 if dtype == torch.float32 else BF16_TOL), (far, splits[:3])
            like = (got.double().cpu().view(n, H, E) / 0.6 * mark).mean(-1).mean(-1)          # 1 where the head holds the mark
            inside = list(range(far, (far // chunk + 1) * chunk))
            assert float(like[inside].min()) > 0.95
            out_ = [i for i in range(n) if i not in inside and i % chunk > 3]
            assert float(like[out_].max()) < 0.8 and float(like[(far // chunk + 1) * chunk]) < 0.95


def _sink_case(H, G, D, E, seed, W=24):
    from tutunex_helpers import parallel, rnd
    m = parallel(H, G, D, E)[1]["left"]
    w = {"q": rnd((H * D, W), seed) / W ** 0.5, "k": rnd((G * D, W), seed + 1) / W ** 0.5, "v": rnd((G * E, W), seed + 2) / W ** 0.5,
         "q.norm": 1 + rnd((D,), seed + 3, 0.3), "k.norm": 1 + rnd((D,), seed + 4, 0.3), "o": torch.eye(H * E)}
    return m, w


def _run_sink(lib, m, w, X, splits, dtype, page=4, cache=None, seq="s", split=True):
    from tutunex_helpers import Steps, dev, zeros
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    Xd = X.double()
    proj_all = torch.cat([Xd @ w["q"].double().T, Xd @ w["k"].double().T, Xd @ w["v"].double().T], dim=1).float()
    ld = proj_all.shape[1]
    cache = cache or _cache(G, D, E, dtype, page)
    cache.open(seq)
    kv, sink, outs, at = cache.struct(0), zeros(H), [], 0
    for cnt in splits:
        st = Steps([cnt], [cache.extend(seq, cnt)], [cache.slot(seq)])
        proj, q, out = dev(proj_all[at:at + cnt]), zeros(cnt, H * D), zeros(cnt, H * E + 2, dtype=dtype)
        call("umb_attn_prep", q, kv, proj, ld, 1, dev(w["q.norm"], dtype), dev(w["k.norm"], dtype), 1, 0, st.d["pos"], st.d["slot"], None, 0, 0, 1.0,
             cnt, H, G, D, E, 1, 0.0, 0, 1e-5, code(dtype))
        _attend(lib, out, H * E + 2, q, kv, st, H, G, D, E, m["scale"], 1.0, form(1, 0, sink), dtype, split)
        outs.append(out[:, :H * E].clone())
        at += cnt
    return torch.cat(outs), cache


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("scale", [0.3, 3.0, -6.0])
@pytest.mark.parametrize("H,G,D,E,splits", [(4, 2, 8, 12, [19]), (3, 1, 7, 5, [1] * 12), (10, 2, 32, 48, [40, 1, 1, 17, 2]), (2, 2, 136, 160, [20, 1, 3])])
def test_sink_attention_prompt_portions_and_single_tokens(lib, dtype, scale, H, G, D, E, splits):
    """with a negative scale and keys that follow the queries most scores are far below 0: the added one rules the denominator"""
    from oracle import tutunex as O
    from tutunex_helpers import close, rnd
    n = sum(splits)
    m, w = _sink_case(H, G, D, E, 1)
    m["scale"] = scale / D ** 0.5
    if scale < 0:
        w["k"] = torch.cat([w["q"][g * (H // G) * D:(g * (H // G) + 1) * D] for g in range(G)])
    X = rnd((n, 24), 9)
    if scale < 0:
        X = X[:1] + 0.2 * X                               # tokens alike: q . k is large for all of them
    wd = {k: v.to(dtype).double() if k.endswith("norm") else v.double() for k, v in w.items()}
    want, _ = O.sink_attention(X.double(), torch.arange(n), m, wd, 1e-5)
    got, cache = _run_sink(lib, m, w, X, splits, dtype)
    assert close(got, want, tol_of(dtype))
    cache.close("s")
    again, _ = _run_sink(lib, m, w, X[:7], [3, 1, 3], dtype, cache=cache, seq="t", split=False)
    assert close(again, want[:7], tol_of(dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("kind", ["sink", "diff"])
def test_long_context_keys_dealt_to_several_workgroups(lib, dtype, kind):
    """single tokens behind 900 keys: the keys are dealt to several workgroups and merged"""
    from oracle import tutunex as O
    from tutunex_helpers import close, rnd
    splits = [900, 1, 1, 3, 1]
    n = sum(splits)
    X = rnd((n, 24), 9)
    if kind == "sink":
        m, w = _sink_case(6, 3, 16, 24, 1)
        want, _ = O.sink_attention(X.double(), torch.arange(n), m, {k: v.to(dtype).double() if k.endswith("norm") else v.double() for k, v in w.items()}, 1e-5)
        got, _ = _run_sink(lib, m, w, X, splits, dtype, page=64)
    else:
        m, w = _diff_case(4, 1, 16, 80, 800, 16, 1)
        want, _ = O.differential_attention(X.double(), torch.arange(n), m, {k: v.double() for k, v in w.items()}, 1e-5)
        got, _ = _run_diff(lib, m, w, X, splits, dtype, page=64)
        m["mask"]["size"] = 2000
        want2, _ = O.differential_attention(X.double(), torch.arange(n), m, {k: v.double() for k, v in w.items()}, 1e-5)
        got2, _ = _run_diff(lib, m, w, X, splits, dtype, page=64)
        assert close(got2, want2, 5e-5 if dtype == torch.float32 else BF16_TOL)
    assert close(got, want, 5e-5 if dtype == torch.float32 else BF16_TOL)          # fp32 angles at position 900


# ------------------------------------------------------------------ gated delta rule
def _delta_case(H, Hk, D, E, taps, seed, W=24, a_gain=2.0):
    from tutunex_helpers import parallel, rnd
    m = parallel(r_heads=H, r_kv=Hk, r_dim=D, r_vdim=E, conv=taps)[1]["right"]
    w = {"q": rnd((Hk * D, W), seed) / W ** 0.5, "k": rnd((Hk * D, W), seed + 1) / W ** 0.5, "v": rnd((H * E, W), seed + 2) / W ** 0.5,
         "q.conv": rnd((Hk * D, taps), seed + 3, 0.6), "k.conv": rnd((Hk * D, taps), seed + 4, 0.6), "v.conv": rnd((H * E, taps), seed + 5, 0.6),
         "b": 3 * rnd((H, W), seed + 6) / W ** 0.5, "a": a_gain * rnd((H, W), seed + 7) / W ** 0.5, "A_log": rnd((H,), seed + 8) - 1.0,
         "dt_bias": rnd((H,), seed + 9) - 1.0, "norm": 1 + rnd((E,), seed + 10, 0.2), "g": rnd((H * E, W), seed + 11) / W ** 0.5, "o": torch.eye(H * E)}
    return m, w


def _run_delta(lib, m, w, X, splits, dtype, slot=1, state=None, at=0):
    from tutunex_helpers import Steps, dev, zeros
    H, Hk, D, E, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    C, col0, Dp = 2 * Hk * D + H * E, 3, (D + 15) // 16 * 16
    Xd = X.double()
    proj_all = torch.cat([torch.full((X.shape[0], col0), 7.0).double()] + [Xd @ w[k].double().T for k in ("q", "k", "v", "g", "b", "a")], dim=1).float()
    ld = proj_all.shape[1]
    if state is None:
        state = (zeros(3, H, D, E) + 3.0, zeros(3, taps, C) + 5.0)          # a fresh sequence must not read what the slot holds
    S, ring = state
    conv = dev(torch.cat([w["q.conv"], w["k.conv"], w["v.conv"]]), dtype)
    alog, dtb = dev(w["A_log"]), dev(w["dt_bias"])
    outs, row = [], 0
    for cnt in splits:
        st = Steps([cnt], [at], [slot])
        proj, o, out = dev(proj_all[row:row + cnt]), zeros(cnt, H * E), zeros(cnt, H * E + 2, dtype=dtype)
        if cnt == 1:
            call("umb_delta_step", o, S, proj, ld, col0, conv, ring, dtb, alog, st.d["pos"], st.d["slot"], 1, Hk, H, D, E, taps, code(dtype))
        else:
            q, k, v = zeros(cnt, Hk * Dp) + 8.0, zeros(cnt, Hk * Dp) + 8.0, zeros(cnt, H * E)
            beta, lg = zeros(cnt, H), zeros(cnt, H)
            scratch = zeros(lib.umb_delta_scan_floats(cnt, H, D, E)) + 6.0
            call("umb_delta_prep", q, k, Hk * Dp, v, beta, lg, proj, ld, col0, conv, ring, dtb, alog, st.d["pos"], st.d["slot"], cnt, Hk, H, D, E, taps,
                 code(dtype))
            call("umb_ssd_conv_update", ring, proj, ld, col0, *st.seqs, 1, C, taps + 1)
            call("umb_delta_scan", o, S, q, k, Hk * Dp, v, beta, lg, *st.seqs, cnt, 1, cnt, Hk, H, D, E, scratch, scratch.numel())
        call("umb_head_gate", out, H * E + 2, o, E, -1, None, proj, ld, col0 + C, dev(w["norm"], dtype), 0, 0, cnt, H, E, 1e-5, 1.0, code(dtype))
        outs.append(out[:, :H * E].clone())
        at += cnt
        row += cnt
    return torch.cat(outs), (S, ring)


DELTA_SHAPES = [(4, 2, 10, 7, 3, [19]), (3, 3, 5, 9, 1, [1] * 12), (2, 1, 16, 32, 4, [2, 9, 1, 1, 17, 3]), (5, 1, 3, 3, 5, [2, 2, 2, 1, 1, 1, 6]),
                (4, 2, 72, 40, 2, [40, 1, 1]), (2, 2, 130, 50, 4, [30, 1, 2]), (2, 1, 256, 33, 9, [12, 1, 1, 5])]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,Hk,D,E,taps,splits", DELTA_SHAPES)
def test_delta_rule_prompt_portions_and_single_tokens(lib, dtype, H, Hk, D, E, taps, splits):
    from oracle import tutunex as O
    from tutunex_helpers import close, rnd
    n = sum(splits)
    m, w = _delta_case(H, Hk, D, E, taps, 1)
    X = rnd((n, 24), 20)
    rounded = {k: v.to(dtype).double() if k == "norm" or k.endswith("conv") else v.double() for k, v in w.items()}
    want, st = O.gated_delta(X.double(), m, rounded, 1e-5)
    got, (S, ring) = _run_delta(lib, m, w, X, splits, dtype)
    assert close(got, want, F32_TOL if dtype == torch.float32 else 1e-2)
    assert close(S[1], st["S"], F32_TOL) and float((S[0] - 3.0).abs().max()) == 0.0 and float((ring[0] - 5.0).abs().max()) == 0.0
    for p in range(max(n - taps + 1, 0), n):              # the ring holds the last inputs, position p in row p % taps
        if taps > 1:
            raw = torch.cat([X[p].double() @ w[k].double().T for k in ("q", "k", "v")])
            assert close(ring[1, p % taps], raw, 1e-5)


@pytest.mark.parametrize("H,Hk,D,E,taps,a_gain,splits", [(4, 2, 10, 7, 3, 2.0, [150]), (2, 1, 32, 20, 4, 2.0, [70, 1, 1, 64, 3, 130]),
                                                         (2, 2, 130, 17, 2, 0.1, [64, 65]), (3, 1, 48, 16, 4, 30.0, [63, 2, 128, 1, 61]),
                                                         (1, 1, 256, 16, 3, 1.0, [129, 2])])
def test_delta_rule_long_stretches_in_chunks(lib, H, Hk, D, E, taps, a_gain, splits):
    """stretches over many chunks, cut at and beside their edges; decays near 1 and (a_gain 30) down to e^-30 in one step; keys that
    repeat, so that the triangular systems are far from the identity"""
    from oracle import tutunex as O
    from tutunex_helpers import close, rnd
    n = sum(splits)
    m, w = _delta_case(H, Hk, D, E, taps, 1, a_gain=a_gain)
    w["A_log"][0], w["dt_bias"][0] = -6.0, -6.0           # nearly nothing is forgotten: the first token still counts at the end
    X = rnd((n, 24), 20)
    X[5::7] = X[5] + 0.05 * X[5::7]
    wd = {k: v.double() for k, v in w.items()}
    want, st = O.gated_delta(X.double(), m, wd, 1e-5)
    got, state = _run_delta(lib, m, w, X, splits, torch.float32)
    assert close(got, want, 3e-5) and close(state[0][1], st["S"], 3e-5)
    again, _ = _run_delta(lib, m, w, X, [30, 1, 1], torch.float32, state=state)         # the slot is used again from position 0
    assert close(again, want[:32], 3e-5)


def test_delta_rule_chunks_of_an_unequal_batch(lib):
    """three sequences of different lengths and ages in one launch, slots out of order, against each alone"""
    from oracle import tutunex as O
    from tutunex_helpers import Steps, close, dev, rnd, zeros
    H, Hk, D, E = 4, 2, 20, 24
    Dp = 32
    counts, pos0, slots = [70, 3, 130], [0, 12, 0], [3, 0, 2]
    st = Steps(counts, pos0, slots)
    T = st.T
    q, k = rnd((T, Hk, D), 1), rnd((T, Hk, D), 2)
    q, k = q / q.norm(dim=-1, keepdim=True), k / k.norm(dim=-1, keepdim=True)
    v, beta, lg = rnd((T, H, E), 3), torch.sigmoid(rnd((T, H), 4)), -torch.rand((T, H), generator=torch.Generator().manual_seed(5)) * 0.3
    S0 = rnd((4, H, D, E), 6)
    S, o = dev(S0.clone()), zeros(T, H * E)
    pad = lambda z: dev(torch.nn.functional.pad(z, (0, Dp - D)).reshape(T, Hk * Dp))                     # noqa: E731
    scratch = zeros(lib.umb_delta_scan_floats(T, H, D, E))
    call("umb_delta_scan", o, S, pad(q), pad(k), Hk * Dp, dev(v.reshape(T, -1)), dev(beta), dev(lg), *st.seqs, T, 3, 130, Hk, H, D, E, scratch,
         scratch.numel())
    at = 0
    for c, p, s in zip(counts, pos0, slots):
        sl = slice(at, at + c)
        rep = lambda z: z[sl].double().repeat_interleave(H // Hk, dim=1)                                 # noqa: E731
        want, Sw = O.delta_recurrence(rep(q), rep(k), v[sl].double(), torch.exp(lg[sl].double()), beta[sl].double(),
                                      S0[s].double() if p else torch.zeros(H, D, E, dtype=torch.float64))
        assert close(o[sl].view(c, H, E), want, F32_TOL) and close(S[s], Sw, F32_TOL)
        at += c
    assert torch.equal(S[1].cpu(), S0[1])


def test_shapes_the_kernels_do_not_cover_are_refused(lib):
    from umbrella_amd import _lib
    from tutunex_helpers import Steps, i32, zeros
    assert lib.umb_delta_scan_floats(4, 2, 257, 8) == 0 and lib.umb_delta_scan_floats(4, 2, 256, 8) > 0
    z, st = zeros(4096), Steps([4], [0], [0])
    with pytest.raises(_lib.UmbError):                    # not enough scratch
        call("umb_delta_scan", z, z, z, z, 32, z, z, z, *st.seqs, 4, 1, 4, 1, 1, 16, 16, z, 16)
    with pytest.raises(_lib.UmbError):                    # heads that do not divide
        call("umb_delta_step", z, z, z, 4096, 0, z, z, z, z, i32([0]), i32([0]), 1, 2, 3, 8, 8, 2, 2)
    with pytest.raises(_lib.UmbError):                    # three maps
        call("umb_attn_attend", z, 4096, z, _cache(1, 8, 8, torch.float32, 4).struct(0), None, 0, -1, None, 0, i32([0]), i32([0]), 1, 1, 1, 8, 8, 8, 1.0,
             1.0, 0.0, form(3), None, 0, 2)


# ------------------------------------------------------------------ whole models
def _oracle_logits(cfgd, sd, toks):
    from oracle import tutunex as O
    return O.forward(cfgd, sd, toks)[0]


@pytest.mark.parametrize("name", ["mixed", "odd", "plain", "wide"])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_model_prefill_decode_portions_against_oracle(lib, name, dtype):
    from oracle import tutunex as O
    from tutunex_helpers import CONFIGS, build, close, rel_err, tokens
    cfgd = CONFIGS[name]
    m, sd = build(cfgd, dtype, seed=11, page=4)
    n = 41
    toks = tokens(n, cfgd["vocab"], 5)
    want, lo, _ = O.forward(cfgd, sd, toks)
    tol = F32_TOL if dtype == torch.float32 else BF16_TOL
    m.open("w")
    whole, layers = m.forward_batch([("w", toks)], want=[list(range(n))], trace=True)
    whole = whole.clone()
    if dtype == torch.float32:
        assert close(layers, lo, F32_TOL)
    assert rel_err(whole, want) < tol
    same = F32_TOL if dtype == torch.float32 else 3e-2          # the model against itself under another schedule
    for sid, splits in (("d", [1] * n), ("p", [2, 2, 7, 1, 16, 3, 10]), ("q", [30] + [1] * 11), ("r", [17, 2, 2, 20]), ("t", [2] * 20 + [1])):
        m.open(sid)
        rows, at = [], 0
        for k in splits:
            rows.append(m.forward_batch([(sid, toks[at:at + k])], want=[list(range(k))]).clone())
            at += k
        got = torch.cat(rows)
        assert rel_err(got, want) < tol, (sid, "against the oracle")
        assert rel_err(got, whole) < same, (sid, "against the whole prompt")
        m.close(sid)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_model_unequal_batch_equals_each_alone(lib, dtype):
    """three requests of different lengths prefilled in one step and decoded together, the shortest ending first, against
    each of them alone; then a new request in the slot and pages the shortest one gave back"""
    from tutunex_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS["mixed"]
    m, _ = build(cfgd, dtype, seed=3, page=4, batch=3)
    V = cfgd["vocab"]
    seqs = {"a": tokens(33, V, 1), "b": tokens(9, V, 2), "c": tokens(21, V, 3)}
    pre = {"a": 20, "b": 1, "c": 13}
    alone = {}
    for k, t in list(seqs.items()) + [("d", tokens(17, V, 4))]:
        m.open(k)
        alone[k] = m.forward_batch([(k, t)], want=[list(range(len(t)))]).clone()
        m.close(k)
    got = {k: [] for k in seqs}
    for k in seqs:
        m.open(k)
    out = m.forward_batch([(k, seqs[k][:pre[k]]) for k in seqs], want=[list(range(pre[k])) for k in seqs]).clone()
    at = 0
    for k in seqs:
        got[k].append(out[at:at + pre[k]])
        at += pre[k]
    done, live = dict(pre), list(seqs)
    while live:
        out = m.forward_batch([(k, [seqs[k][done[k]]]) for k in live], want=[[0]] * len(live)).clone()
        for i, k in enumerate(live):
            got[k].append(out[i:i + 1])
            done[k] += 1
        for k in [k for k in live if done[k] == len(seqs[k])]:
            m.close(k)
            live.remove(k)
            if k == "b":                              # its slot and pages are handed to a new request at once
                m.open("d")
                got["d"] = [m.forward_batch([("d", tokens(17, V, 4))], want=[list(range(17))]).clone()]
                m.close("d")
    for k in got:
        assert rel_err(torch.cat(got[k]), alone[k]) < (F32_TOL if dtype == torch.float32 else 3e-2), k


def test_model_mixed_step_of_prompt_and_single_tokens(lib):
    """one step that brings a long stretch of one sequence and one token of another: the same numbers as apart"""
    from tutunex_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS["plain"]
    m, sd = build(cfgd, torch.float32, seed=3, page=4, batch=3)
    a, b = tokens(80, cfgd["vocab"], 1), tokens(30, cfgd["vocab"], 2)
    m.open("a"), m.open("b")
    m.forward_batch([("b", b[:29])])
    out = m.forward_batch([("a", a), ("b", b[29:])], want=[list(range(80)), [0]]).clone()
    assert rel_err(out[:80], _oracle_logits(cfgd, sd, a)) < F32_TOL and rel_err(out[80:], _oracle_logits(cfgd, sd, b)[29:]) < F32_TOL


def test_model_long_decoding_and_first_tokens(lib):
    """fp32: 150 tokens decoded one by one after a two-token prompt (pages of 4 tokens used up and down the table, chunk edges of
    three masks crossed many times, the ring going round) against the oracle's whole-sequence pass"""
    from tutunex_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS["mixed"]
    m, sd = build(cfgd, torch.float32, seed=7, page=4, batch=2, max_tokens=400)
    toks = tokens(152, cfgd["vocab"], seed=9)
    want = _oracle_logits(cfgd, sd, toks)
    m.open("x")
    rows = [m.forward_batch([("x", toks[:2])], want=[[0, 1]]).clone()]
    for t in toks[2:]:
        rows.append(m.forward_batch([("x", [t])], want=[[0]]).clone())
    got = torch.cat(rows)
    assert rel_err(got, want) < F32_TOL and rel_err(got[:3], want[:3]) < F32_TOL


@pytest.mark.parametrize("name", ["mixed", "wide"])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_model_long_prompt_in_one_step_and_in_portions(lib, name, dtype):
    """several delta-rule chunks and matrix-pipe attention, cut at and beside chunk and page borders"""
    from tutunex_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS[name]
    m, sd = build(cfgd, dtype, seed=5, page=16, batch=2, max_length=320, max_tokens=700)
    n = 200
    toks = tokens(n, cfgd["vocab"], 40)
    want = _oracle_logits(cfgd, sd, toks)
    tol = F32_TOL if dtype == torch.float32 else 8e-2
    m.open("w")
    whole = m.forward_batch([("w", toks)], want=[list(range(n))]).clone()
    assert rel_err(whole, want) < tol
    for sid, splits in (("p", [64, 65, 1, 1, 69]), ("q", [127, 2, 71]), ("r", [48, 52, 1, 99])):
        m.open(sid)
        rows, at = [], 0
        for k in splits:
            rows.append(m.forward_batch([(sid, toks[at:at + k])], want=[list(range(k))]).clone())
            at += k
        assert rel_err(torch.cat(rows), want) < tol, sid
        m.close(sid)


def test_model_refuses_a_reader_without_a_source(lib):
    from tutunex_helpers import attention, build, config, layer
    with pytest.raises(ValueError):
        build(config([layer(attention(kv_from=0)), layer(attention())]), torch.float32)
    with pytest.raises(ValueError):
        build(config([layer(attention()), layer(attention(kv_from=0)), layer(attention(kv_from=1))]), torch.float32)


def test_shared_keys_take_no_cache_of_their_own(lib):
    from tutunex_helpers import CONFIGS, build
    m, _ = build(CONFIGS["mixed"], torch.bfloat16)
    assert [(e["G"], e["D"], e["E"]) for e in m.kv_cache.kv] == [(3, 8, 6), (2, 16, 12), (2, 8, 6)]      # two readers, no store of theirs
    assert [tuple(s.shape[1:]) for s in m.kv_cache.state] == [(4, 10, 7), (3, 5, 9)]


def test_model_decode_steps_replayed_as_graphs_equal_eager_launches(lib):
    from tutunex_helpers import CONFIGS, build, tokens
    cfgd = CONFIGS["mixed"]
    V = cfgd["vocab"]
    seqs = {"a": tokens(30, V, 1), "b": tokens(24, V, 2)}
    outs = {}
    for graph in (False, True):
        m, _ = build(cfgd, torch.float32, seed=3, page=4, batch=2, hip_graph=graph)
        for k in seqs:
            m.open(k)
        rows = [m.forward_batch([(k, seqs[k][:10]) for k in seqs], want=[[9], [9]]).clone()]
        for i in range(10, 24):
            rows.append(m.forward_batch([(k, [seqs[k][i]]) for k in seqs], want=[[0], [0]]).clone())
            torch.cuda.synchronize()
        outs[graph] = torch.cat(rows)
    assert torch.equal(outs[False], outs[True])


# ------------------------------------------------------------------ engine and trace replay
def _engine(cfgd, dtype, sd=None, **kw):
    from tutunex_helpers import build
    from umbrella_amd.speculation.auto_engine import AutoEngine
    from umbrella_amd.speculation.speculation_utils import IdTokenizer
    m, sd = build(cfgd, dtype, seed=21, page=4, batch=kw.pop("batch", 3), max_length=96, max_tokens=kw.pop("max_tokens", 512), sd=sd)
    e = AutoEngine.from_config("cuda:0", engine="batch", model="tiny", dtype=dtype, target_model_obj=m, tokenizer=IdTokenizer(), **kw)
    e.initialize()
    return e, sd


def test_engine_greedy_generation_matches_oracle(lib):
    """five queued requests through the scheduler (three slots: two batches), greedy, fp32: the oracle's tokens"""
    from tutunex_helpers import CONFIGS, tokens
    cfgd = CONFIGS["mixed"]
    e, sd = _engine(cfgd, torch.float32)
    prompts = [tokens(n, cfgd["vocab"], seed=n) for n in (7, 1, 12, 3, 9)]
    outs = e.generate_batch(prompts, max_new_tokens=10)
    for p, got in zip(prompts, outs):
        toks, margins = list(p), []
        for _ in range(10):
            row = _oracle_logits(cfgd, sd, toks)[-1]
            top = torch.topk(row, 2).values
            margins.append(float(top[0] - top[1]))
            toks.append(int(row.argmax()))
        want = toks[len(p):]
        k = next((i for i, (a, b) in enumerate(zip(got, want)) if a != b), None)
        assert k is None or margins[k] < 1e-4, (got, want, margins)
    assert not e.target_model.kv_cache.seqs and len(e.target_model.kv_cache.free_slots) == 3
    assert e.generate(input_ids=prompts[2], max_new_tokens=10)["generated_tokens"] == outs[2]


def test_engine_sampling_is_seeded_and_in_range(lib):
    from tutunex_helpers import CONFIGS, tokens
    cfgd = CONFIGS["odd"]
    e, _ = _engine(cfgd, torch.bfloat16, temperature=0.8, topk=8, topp=0.9, repetition_penalty=1.2, seed=5)
    prompts = [tokens(6, cfgd["vocab"], seed=1), tokens(11, cfgd["vocab"], seed=2)]
    a = e.generate_batch(prompts, max_new_tokens=12)
    e.reset()
    e.manual_seed(5)
    e.step_count.zero_()
    b = e.generate_batch(prompts, max_new_tokens=12)
    assert a == b and all(0 <= t < cfgd["vocab"] for o in a for t in o) and all(len(o) == 12 for o in a)


def test_trace_replay_command(lib, tmp_path):
    """bin/trace_run on a checkpoint directory: a mixed batch prefilled, decoded together, one request ending early"""
    import numpy as np
    from safetensors.torch import save_file
    from tutunex_helpers import CONFIGS, checkpoint, rel_err, tokens
    cfgd = CONFIGS["mixed"]
    _, sd = checkpoint(cfgd, seed=4)
    sd = {k: v.to(torch.bfloat16) for k, v in sd.items()}
    mdir, out = tmp_path / "model", tmp_path / "out"
    mdir.mkdir()
    save_file({k: v.contiguous() for k, v in sd.items()}, str(mdir / "model.safetensors"))
    (mdir / "config.json").write_text(json.dumps(cfgd))
    V = cfgd["vocab"]
    a, b = tokens(26, V, 1), tokens(8, V, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:5], "want": [4]}],
              "end": []}]
    for i in range(6):
        ent = [{"id": "a", "tokens": [a[20 + i]], "want": [0]}]
        if 5 + i < len(b):
            ent.append({"id": "b", "tokens": [b[5 + i]], "want": [] if i == 1 else [0]})
        steps.append({"step": i + 1, "entries": ent, "end": (["b"] if 5 + i == len(b) - 1 else []) + (["a"] if i == 5 else [])})
    f32 = {k: v.float() for k, v in sd.items()}
    wa, wb = (_oracle_logits(cfgd, f32, t) for t in (a, b))
    for dt, tol in (("float32", F32_TOL), ("bfloat16", BF16_TOL)):
        p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(mdir), "--dtype", dt, "--out",
                            str(out), "--max-tokens", "64", "--page-size", "4"], input="\n".join(json.dumps(s) for s in steps),
                           capture_output=True, text=True, timeout=300)
        assert p.returncode == 0, p.stderr[-2000:]
        assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(7)]
        read = lambda s, n: torch.from_numpy(np.fromfile(out / f"{s}.f32", dtype="<f4").reshape(n, V))        # noqa: E731
        assert rel_err(read(0, 3), torch.stack([wa[0], wa[19], wb[4]])) < tol
        assert rel_err(read(2, 1), wa[21:22]) < tol                                                        # b wanted nothing in step 2
        assert rel_err(read(3, 2), torch.stack([wa[22], wb[7]])) < tol
        assert rel_err(read(6, 1), wa[25:26]) < tol
