"""The Potosun design on the HIP path against the plain oracle (oracle/potosun.py): its mechanisms alone through their own entry points
of libumbrella_seq.so (biased attention over a window with kept first tokens, chunked attention with a sink, values mixed over
layers, latent attention with direct queries, the gelu, gate and cap epilogues, the plain residual), then whole models through the
runtime, the cache manager, the batch engine and the trace replay command.

fp32 runs are the sharp ones (every comparison to ~1e-5: one key too many or a wrong distance is a thousand times that); bf16 runs
use inputs built so that a fault still shows."""
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
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])


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


def form(chunk=0, sink=None, keep=0, gate_elem=0, maps=1, lam=0.0, eps=0.0):
    from umbrella_amd import _lib
    f = _lib.UmbAttnForm()
    f.maps, f.chunk, f.sink, f.lambda_, f.eps = maps, chunk, (sink.data_ptr() if sink is not None else None), lam, eps
    f.keep_first, f.gate_elem = keep, gate_elem
    return f


def tol_of(dtype):
    return F32_TOL if dtype == torch.float32 else BF16_TOL


def dbl(w):
    return {k: v.double() for k, v in w.items()}


# ------------------------------------------------------------------ products with an epilogue, the plain residual
@BOTH
@pytest.mark.parametrize("T,F,K", [(1, 24, 40), (5, 33, 17), (20, 96, 64), (40, 50, 72), (100, 80, 64), (300, 160, 136)])
def test_gelu_gated_product(lib, dtype, T, F, K):
    from oracle import potosun as O
    from potosun_helpers import close, dev, rnd, zeros
    x, w = rnd((T, K), 1).to(dtype), (2.0 * rnd((2 * F, K), 2) / K ** 0.5).to(dtype)
    out = zeros(T, F, dtype=dtype)
    call("umb_seq_linear", out, dev(x), dev(w), None, T, 2 * F, K, 6, code(dtype))
    xd, wd = x.double(), w.double()
    assert close(out, O.gelu(xd @ wd[:F].T) * (xd @ wd[F:].T), 3e-6 if dtype == torch.float32 else 1e-2)


def test_gelu_far_from_zero(lib):
    """gate values from -30 to 30: no overflow, exactly zero and exactly z at the ends"""
    from oracle import potosun as O
    from potosun_helpers import close, dev, zeros
    z = torch.linspace(-30, 30, 61)
    x = torch.stack([z, torch.ones(61)], dim=1)
    w = torch.tensor([[1.0, 0.0], [0.0, 1.0]])
    out = zeros(61, 1)
    call("umb_seq_linear", out, dev(x), dev(w), None, 61, 2, 2, 6, 2)
    assert close(out[:, 0], O.gelu(z.double()), 1e-6) and float(out[0]) == 0.0 and float(out[-1]) == 30.0


@BOTH
@pytest.mark.parametrize("T,N,K", [(1, 75, 36), (3, 130, 64), (40, 90, 40), (100, 200, 64), (300, 260, 72)])
@pytest.mark.parametrize("cap", [0.7, 20.0])
def test_capped_product(lib, dtype, T, N, K, cap):
    from oracle import potosun as O
    from potosun_helpers import close, dev, rnd, zeros
    x, w = rnd((T, K), 1).to(dtype), (3.0 * rnd((N, K), 2) / K ** 0.5).to(dtype)
    out = zeros(T, N)
    call("umb_seq_linear_cap", out, dev(x), dev(w), None, T, N, K, cap, code(dtype))
    assert close(out, O.cap(x.double() @ w.double().T, cap), 3e-6)


@BOTH
@pytest.mark.parametrize("T", [1, 3, 20, 70, 300])
def test_batched_product_with_one_gate_per_row(lib, dtype, T):
    from potosun_helpers import close, dev, rnd, zeros
    H, N, K, ldg, col = 5, 72, 24, 11, 4
    x, w, g = rnd((T, H, K), 1).to(dtype), (rnd((H, N, K), 2) / K ** 0.5).to(dtype), 3 * rnd((T, ldg), 3)
    out, gate = zeros(T, H, N, dtype=dtype), dev(g)
    call("umb_seq_linear_batched", out, dev(x), dev(w), T, N, K, H * K, H * N, H, K, N * K, N, 7, gate[:, col:], ldg, 1, code(dtype))
    want = torch.stack([(x[:, h].double() @ w[h].double().T) * torch.sigmoid(g[:, col + h:col + h + 1].double()) for h in range(H)], dim=1)
    assert close(out, want, 3e-6 if dtype == torch.float32 else 1e-2)


@BOTH
@pytest.mark.parametrize("W,T", [(40, 3), (320, 2), (1500, 2), (5000, 3)])
def test_plain_residual_and_next_norm(lib, dtype, W, T):
    from oracle import potosun as O
    from potosun_helpers import close, dev, i32, rnd, tokens, zeros
    eps = 3e-2                                            # large: where it stands in the root shows
    emb, w, tk = rnd((17, W), 1).to(dtype), (1 + rnd((W,), 2, 0.3)).to(dtype), tokens(T, 17, 3)
    x, h, y = zeros(T, W), zeros(T, W, dtype=dtype), rnd((T, W), 4)
    call("umb_hc_embed", x, h, dev(emb), i32(tk), 2.5, None, dev(w), 0.0, T, W, 17, 1, eps, code(dtype))
    x0 = emb[tk].double() * 2.5
    tol = 1e-6 if dtype == torch.float32 else 1e-2
    assert close(x, x0, 1e-6) and close(h, O.rms(x0, eps) * w.double(), tol)
    call("umb_hc_seam", x, h, dev(y), None, None, 1.0, None, dev(w), 0.0, T, W, 1, eps, code(dtype))
    assert close(x, x0 + y.double(), 1e-6) and close(h, O.rms(x0 + y.double(), eps) * w.double(), tol)


# ------------------------------------------------------------------ grouped-query attention by form
def _cache(G, D, E, dtype, page, seqs=3, max_tokens=2048):
    from umbrella_amd.attn.cache import PagedSeqCache
    c = PagedSeqCache([(G, D, 0, E)], [], max_tokens, seqs, "cuda:0", dtype, page=page)
    for z in (c.kv[0]["k"], c.kv[0]["v"]):
        z.fill_(9.0)                                      # what a page held before must not matter
    return c


def _attend(lib, out, ldo, q, kv, st, H, G, D, E, window, scale, f, dtype, split, proj=None, ld=0, gate_col=-1, bias=None):
    from potosun_helpers import zeros
    nd = bias.shape[1] if bias is not None else 0
    if st.max_len >= 16 and lib.umb_bsa_attend_tiled_ok(H, G, D, E, code(dtype)):
        call("umb_attn_attend_tiled", out, ldo, q, kv, proj, ld, gate_col, bias, nd, *st.seqs, st.B, st.max_len, H, G, D, E, window, scale, 1.0, 0.0, f,
             code(dtype))
    else:
        scratch = zeros(st.T * H * 16 * (E + 2)) if split else None
        call("umb_attn_attend", out, ldo, q, kv, proj, ld, gate_col, bias, nd, st.d["pos"], st.d["slot"], st.T, H, G, D, E, window, scale, 1.0, 0.0, f,
             scratch, scratch.numel() if split else 0, code(dtype))


def _run(lib, kind, m, w, X, splits, dtype, page=4, cache=None, seq="s", split=True, v_first=None):
    """one mixer through prep / append / attend, the output projection left out (w["o"] is the identity).  v_first [n, G E]: values to
    mix in (None: the layer keeps its own).  Returns (outputs, the kept values or None, cache)."""
    from umbrella_amd import _lib
    from umbrella_amd.models.config import bias_by_distance, rotary_table
    from potosun_helpers import Steps, dev, zeros
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    Xd, n = X.double(), X.shape[0]
    names = ["q", "k", "v"] + (["g"] if kind == "attention" else [])
    proj_all = torch.cat([Xd @ w[k].double().T for k in names], dim=1).float()
    ld, gate_col = proj_all.shape[1], H * D + G * (D + E)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    freq, mult = rotary_table(rot["base"], rot["dims"], rot.get("scaling")) if rot["dims"] else (None, 1.0)
    fr = dev(freq) if freq is not None else None
    bias = dev(bias_by_distance(w["rel"], float(m["bias_max"]), 4096)) if kind == "attention" else None
    sink = dev(w["sink"]) if kind == "attention_2" else None
    qn, kn = (dev(w["q.norm"], dtype), dev(w["k.norm"], dtype)) if kind == "attention" else (None, None)
    window = m["mask"]["size"] if kind == "attention" else 2 ** 30
    f = form(0, None, m["mask"].get("keep_first", 0), 1) if kind == "attention" else form(m["mask"]["size"], sink)
    cache = cache or _cache(G, D, E, dtype, page)
    if seq not in cache.seqs:
        cache.open(seq)
    kv, outs, kept, at = cache.struct(0), [], [], 0
    for cnt in splits:
        st = Steps([cnt], [cache.extend(seq, cnt)], [cache.slot(seq)])
        proj, q, out = dev(proj_all[at:at + cnt]), zeros(cnt, H * D), zeros(cnt, H * E + 3, dtype=dtype)
        keep, first = zeros(cnt, G * E), (dev(v_first[at:at + cnt]) if v_first is not None else None)
        mix = _lib.UmbValueMix()
        mix.keep, mix.first, mix.lambda_ = keep.data_ptr(), (first.data_ptr() if first is not None else None), float(w.get("vmix", 0.0))
        call("umb_attn_prep_mix", q, kv, proj, ld, 1, qn, kn, int(qn is not None), 0, st.d["pos"], st.d["slot"], fr, rot["dims"], 1, mult, cnt, H, G, D,
             E, 1, 0.0, 0, 1e-5, mix, code(dtype))
        _attend(lib, out, H * E + 3, q, kv, st, H, G, D, E, window, m["scale"], f, dtype, split, proj, ld, gate_col if kind == "attention" else -1, bias)
        assert float(out[:, H * E:].float().abs().max()) == 0.0
        outs.append(out[:, :H * E].clone())
        kept.append(keep)
        at += cnt
    assert at == n
    return torch.cat(outs), torch.cat(kept), cache


def _oracle(kind, m, w, X, dtype, v_first=None):
    from oracle import potosun as O
    G, E = m["kv_heads"], m["vdim"]
    wd = {k: v.to(dtype).double() if k.endswith("norm") else v.double() for k, v in w.items()}
    vf = v_first.double().view(-1, G, E) if v_first is not None else None
    fn = O.biased_attention if kind == "attention" else O.chunked_attention
    return fn(X.double(), torch.arange(X.shape[0]), m, wd, 1e-5, vf)[0]


def _case(kind, seed, W=24, rows=8, **kw):
    from potosun_helpers import biased, chunked, rnd
    _, m = (biased if kind == "attention" else chunked)(**kw)
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    w = {"q": 1.5 * rnd((H * D, W), seed) / W ** 0.5, "k": 1.5 * rnd((G * D, W), seed + 1) / W ** 0.5, "v": rnd((G * E, W), seed + 2) / W ** 0.5,
         "o": torch.eye(H * E), "vmix": torch.tensor(0.35)}
    if kind == "attention":
        w.update({"q.norm": 1 + rnd((D,), seed + 3, 0.3), "k.norm": 1 + rnd((D,), seed + 4, 0.3), "rel": 1.5 * rnd((rows, H), seed + 5),
                  "g": 2 * rnd((H * E, W), seed + 6) / W ** 0.5})
    else:
        w["sink"] = 1.5 * rnd((H,), seed + 3)
    return m, w


BIASED = [((4, 2, 8, 12), (9, 3, 14), 8, [19]), ((3, 1, 7, 5), (1, 0, 9), 6, [1] * 12), ((3, 1, 7, 5), (5, 1, 30), 16, [2, 9, 1, 1, 17, 3]),
          ((2, 2, 16, 16), (8, 11, 20), 8, [40, 1, 1, 30, 2, 2]), ((10, 2, 40, 80), (33, 16, 60), 12, [70, 1, 64, 3, 62]),
          ((8, 1, 72, 144), (50, 6, 45), 32, [33, 20, 1, 48]), ((2, 1, 136, 272), (12, 2, 90), 8, [17, 2, 16]), ((4, 4, 24, 48), (20, 70, 25), 4, [64, 1, 1, 31]),
          ((12, 2, 56, 64), (21, 5, 40), 8, [50, 1, 2, 17])]


@BOTH
@pytest.mark.parametrize("shape,mask,rows,splits", BIASED)
def test_biased_window_attention_prompt_portions_and_single_tokens(lib, dtype, shape, mask, rows, splits):
    from potosun_helpers import close, rnd
    (H, G, D, E), (window, keep, far), n = shape, mask, sum(splits)
    m, w = _case("attention", 1, rows=rows, heads=H, kv_heads=G, dim=D, vdim=E, window=window, keep=keep, bias_max=far)
    X, vf = rnd((n, 24), 9), rnd((n, G * E), 30)
    want, mixed = _oracle("attention", m, w, X, dtype), _oracle("attention", m, w, X, dtype, vf)
    got, kept, cache = _run(lib, "attention", m, w, X, splits, dtype)
    assert close(got, want, tol_of(dtype)) and close(kept, X.double() @ w["v"].double().T, 1e-6)
    one, _, _ = _run(lib, "attention", m, w, X, splits, dtype, page=16, split=False, v_first=vf)
    assert close(one, mixed, tol_of(dtype))
    cache.close("s")                                      # pages and slot go back and are used again by a sequence that starts at 0
    again, _, _ = _run(lib, "attention", m, w, X[:9], [4, 1, 4], dtype, cache=cache, seq="t")
    assert close(again, want[:9], tol_of(dtype))


CHUNKED = [((6, 2, 10, 12), (7, 6), [19]), ((3, 1, 7, 5), (1, 4), [1] * 12), ((2, 2, 16, 16), (8, 16), [2, 9, 1, 1, 17, 3]),
           ((4, 4, 16, 32), (33, 8), [40, 1, 1, 30, 2, 2]), ((10, 2, 40, 80), (64, 20), [70, 1, 64, 3, 62]), ((8, 1, 72, 144), (50, 72), [33, 20, 1, 48]),
           ((2, 1, 136, 272), (30, 0), [17, 2, 16])]


@BOTH
@pytest.mark.parametrize("shape,mask,splits", CHUNKED)
def test_chunked_sink_attention_prompt_portions_and_single_tokens(lib, dtype, shape, mask, splits):
    from potosun_helpers import close, rnd
    (H, G, D, E), (chunk, dims), n = shape, mask, sum(splits)
    m, w = _case("attention_2", 1, heads=H, kv_heads=G, dim=D, vdim=E, chunk=chunk, rot_dims=dims)
    X, vf = rnd((n, 24), 9), rnd((n, G * E), 30)
    want, mixed = _oracle("attention_2", m, w, X, dtype), _oracle("attention_2", m, w, X, dtype, vf)
    got, kept, cache = _run(lib, "attention_2", m, w, X, splits, dtype)
    assert close(got, want, tol_of(dtype)) and close(kept, X.double() @ w["v"].double().T, 1e-6)
    one, _, _ = _run(lib, "attention_2", m, w, X, splits, dtype, page=16, split=False, v_first=vf)
    assert close(one, mixed, tol_of(dtype))
    cache.close("s")
    again, _, _ = _run(lib, "attention_2", m, w, X[:9], [4, 1, 4], dtype, cache=cache, seq="t")
    assert close(again, want[:9], tol_of(dtype))


@BOTH
@pytest.mark.parametrize("page", [4, 16])
@pytest.mark.parametrize("mask", ["window", "chunk"])
def test_edges_of_one_outstanding_key(lib, dtype, page, mask):
    """one key's score is far above all others and its value row carries a mark: exactly the positions that see the key read the mark --
    keys at page borders, the last kept and the first not kept token, the first, a middle and the last place of a chunk; in prompts
    (matrix pipe in 16 bits), portions cut at and beside the edge, and tokens decoded one by one across it"""
    from oracle import potosun as O
    from potosun_helpers import Steps, close, dev, rnd, zeros
    H, G, D, E, n, size, keep = 4, 2, 16, 16, 130, 30, 19
    far_keys = (0, keep - 1, keep, 47, 63, 64) if mask == "window" else (30, 47, 59)
    for far in far_keys:
        q, k, v = 0.02 * rnd((n, H, D), 1), 0.02 * rnd((n, G, D), 2), 0.3 * rnd((n, G, E), 3)
        q[..., 0] = 4.0
        k[far, :, 0] = 4.0
        v[far] = torch.linspace(3.0, 8.0, E)
        sees = (lambda i, j: O.sees_window(i, j, size, keep)) if mask == "window" else (lambda i, j: O.sees_chunk(i, j, size))
        ref = O.attend(q.double(), k.double(), v.double(), O.visible(torch.arange(n), n, sees), 1.0)
        inside = [i for i in range(n) if sees(i, far)]
        f = form(0, None, keep) if mask == "window" else form(size)
        proj_all = torch.cat([q.reshape(n, -1), k.reshape(n, -1), v.reshape(n, -1)], dim=1)
        for splits in ([n], [far + 1] + [1] * (n - far - 1), [60, 2, 1, 27, 40], [59, 1, 1, 29, 40]):
            cache = _cache(G, D, E, dtype, page)
            cache.open("s")
            kv, at, rows = cache.struct(0), 0, []
            for cnt in splits:
                st = Steps([cnt], [cache.extend("s", cnt)], [cache.slot("s")])
                proj, qq, out = dev(proj_all[at:at + cnt]), zeros(cnt, H * D), zeros(cnt, H * E, dtype=dtype)
                call("umb_attn_prep", qq, kv, proj, proj.shape[1], 1, None, None, 0, 0, st.d["pos"], st.d["slot"], None, 0, 0, 1.0, cnt, H, G, D, E, 1,
                     0.0, 0, 1e-5, code(dtype))
                _attend(lib, out, H * E, qq, kv, st, H, G, D, E, size if mask == "window" else 2 ** 30, 1.0, f, dtype, True)
                rows.append(out)
                at += cnt
            got = torch.cat(rows)
            assert close(got, ref.reshape(n, -1), 3e-5 if dtype == torch.float32 else BF16_TOL), (far, splits[:3])
            like = (got.double().cpu().view(n, H, E) / torch.linspace(3.0, 8.0, E).double()).mean(-1).mean(-1)       # 1 where the mark was read
            outside = [i for i in range(n) if i not in inside]
            assert float(like[inside].min()) > 0.95 and (not outside or float(like[outside].abs().max()) < 0.5), (far, splits[:3])


@pytest.mark.parametrize("mask", ["window", "chunk"])
@pytest.mark.parametrize("n,H,G", [(330, 16, 16), (700, 24, 8)])
def test_prompt_tiles_dealt_from_both_ends(lib, mask, n, H, G):
    """enough head blocks that some of them walk the prompt's tiles from the far end: two sequences of unequal length in one launch"""
    from oracle import potosun as O
    from potosun_helpers import Steps, close, dev, rnd, zeros
    D, E, size, keep, dtype = 16, 16, 45, 6, torch.bfloat16
    counts = [n, 61]
    T = sum(counts)
    q, k, v = 2 * rnd((T, H, D), 1), rnd((T, G, D), 2), rnd((T, G, E), 3)
    cache = _cache(G, D, E, dtype, 16)
    slots = [cache.open("a"), cache.open("b")]
    st = Steps(counts, [cache.extend("a", n), cache.extend("b", 61)], slots)
    proj, qq, out = dev(torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], dim=1)), zeros(T, H * D), zeros(T, H * E, dtype=dtype)
    call("umb_attn_prep", qq, cache.struct(0), proj, proj.shape[1], 1, None, None, 0, 0, st.d["pos"], st.d["slot"], None, 0, 0, 1.0, T, H, G, D, E, 1, 0.0,
         0, 1e-5, code(dtype))
    f = form(0, None, keep) if mask == "window" else form(size)
    _attend(lib, out, H * E, qq, cache.struct(0), st, H, G, D, E, size if mask == "window" else 2 ** 30, 0.4, f, dtype, False)
    sees = (lambda i, j: O.sees_window(i, j, size, keep)) if mask == "window" else (lambda i, j: O.sees_chunk(i, j, size))
    at = 0
    for c in counts:
        z = slice(at, at + c)
        want = O.attend(q[z].double(), k[z].double(), v[z].double(), O.visible(torch.arange(c), c, sees), 0.4)
        assert close(out[z], want.reshape(c, -1), BF16_TOL)
        at += c


@BOTH
def test_bias_stands_at_the_true_distance_of_kept_tokens(lib, dtype):
    """equal scores, a table that is loud in one bucket only: position i reads the mark of the kept token exactly where i - j falls in it"""
    from oracle import potosun as O
    from potosun_helpers import close, rnd
    n, rows, far, window, keep = 90, 8, 60, 12, 3
    m, w = _case("attention", 1, rows=rows, heads=2, kv_heads=1, dim=16, vdim=16, window=window, keep=keep, bias_max=far)
    w["q"], w["k"] = 0 * w["q"], 0 * w["k"]
    for bucket in (1, 4, 6, 7):
        w["rel"] = torch.zeros(rows, 2)
        w["rel"][bucket] = 9.0
        X = rnd((n, 24), 9)
        want = _oracle("attention", m, w, X, dtype)
        loud = [i for i in range(n) if any(O.sees_window(i, j, window, keep) and O.distance_bucket(i - j, rows, far) == bucket for j in range(i + 1))]
        assert loud
        for splits in ([n], [20] + [1] * 70):
            got, _, _ = _run(lib, "attention", m, w, X, splits, dtype)
            assert close(got, want, tol_of(dtype)), bucket


@BOTH
@pytest.mark.parametrize("level", [-20.0, 0.0, 12.0])
def test_sinks_alone_and_above_all_scores(lib, dtype, level):
    """the first token of a chunk meets one key and the sink: its share is e^s / (e^s + e^sink), whatever the level"""
    from potosun_helpers import close, rnd
    m, w = _case("attention_2", 1, heads=4, kv_heads=2, dim=16, vdim=16, chunk=5, rot_dims=16)
    w["sink"] = torch.tensor([level, level + 1, level - 2, 0.0])
    X = rnd((43, 24), 9)
    want = _oracle("attention_2", m, w, X, dtype)
    for splits in ([43], [20] + [1] * 23):
        got, _, _ = _run(lib, "attention_2", m, w, X, splits, dtype)
        assert close(got, want, tol_of(dtype))


@BOTH
@pytest.mark.parametrize("window,keep", [(400, 30), (2 ** 20, 0), (300, 200)])
def test_long_context_keys_dealt_to_several_workgroups(lib, dtype, window, keep):
    """single tokens behind 500 keys: the keys, kept ones first, are dealt to several workgroups and merged; the gate per feature is
    applied by the merge"""
    from potosun_helpers import close, rnd
    splits = [500, 1, 1, 3, 1]
    X = rnd((sum(splits), 24), 9)
    m, w = _case("attention", 1, rows=16, heads=6, kv_heads=3, dim=16, vdim=24, window=window, keep=keep, bias_max=450)
    want = _oracle("attention", m, w, X, dtype)
    got, _, _ = _run(lib, "attention", m, w, X, splits, dtype, page=64)
    assert close(got, want, 3e-5 if dtype == torch.float32 else BF16_TOL)
    assert close(got[500:], want[500:], 3e-5 if dtype == torch.float32 else BF16_TOL)


@BOTH
def test_differential_maps_with_kept_tokens_and_a_gate_per_feature(lib, dtype):
    """the same parts in the two-map form of the kernels (no model uses them together yet): vector pipe, merge and matrix pipe"""
    from oracle import potosun as O
    from potosun_helpers import Steps, close, dev, rnd, zeros
    H, G, D, E, n, window, keep, lam, eps = 4, 2, 16, 32, 60, 11, 7, 0.4, 1e-3
    q, k, v, g = rnd((n, H, 2, D), 1), rnd((n, G, 2, D), 2), rnd((n, G, E), 3), rnd((n, H * E), 4)
    see = O.visible(torch.arange(n), n, lambda i, j: O.sees_window(i, j, window, keep))
    a1, a2 = (O.attend(q[:, :, z].double(), k[:, :, z].double(), v.double(), see, 0.3) for z in (0, 1))
    want = (O.rms(a1 - lam * a2, eps)).reshape(n, -1) * torch.sigmoid(g.double())
    proj_all = torch.cat([q.reshape(n, -1), k.reshape(n, -1), v.reshape(n, -1), g], dim=1)
    ld, gate_col = proj_all.shape[1], 2 * H * D + 2 * G * D + G * E
    for splits in ([n], [20] + [1] * 40):
        cache = _cache(G, 2 * D, E, dtype, 4)
        cache.open("s")
        at, rows = 0, []
        for cnt in splits:
            st = Steps([cnt], [cache.extend("s", cnt)], [cache.slot("s")])
            proj, qq, out = dev(proj_all[at:at + cnt]), zeros(cnt, 2 * H * D), zeros(cnt, H * E, dtype=dtype)
            call("umb_attn_prep", qq, cache.struct(0), proj, ld, 1, None, None, 0, 0, st.d["pos"], st.d["slot"], None, 0, 0, 1.0, cnt, H, G, D, E, 2, 0.0,
                 0, eps, code(dtype))
            f = form(0, None, keep, 1, 2, lam, eps)
            if cnt >= 16 and dtype != torch.float32:
                call("umb_attn_attend_tiled", out, H * E, qq, cache.struct(0), proj, ld, gate_col, None, 0, *st.seqs, 1, cnt, H, G, D, E, window, 0.3, 1.0,
                     0.0, f, code(dtype))
            else:
                call("umb_attn_attend", out, H * E, qq, cache.struct(0), proj, ld, gate_col, None, 0, st.d["pos"], st.d["slot"], cnt, H, G, D, E, window, 0.3,
                     1.0, 0.0, f, None, 0, code(dtype))
            rows.append(out)
            at += cnt
        assert close(torch.cat(rows), want, tol_of(dtype))


# ------------------------------------------------------------------ latent attention with direct queries
def _latent_case(H, D, R, E, r, window, seed, W=24, scaling=True):
    from potosun_helpers import YARN, latent, rnd
    _, m = latent(H, D, R, E, r, window, scaling=YARN if scaling else None)
    w = {"q": 1.5 * rnd((H * (D + R), W), seed) / W ** 0.5, "dkv": rnd((r + R, W), seed + 1) / W ** 0.5, "dkv.norm": 1 + rnd((r,), seed + 2, 0.3),
         "uk": rnd((H * D, r), seed + 3) / r ** 0.5, "uv": rnd((H * E, r), seed + 4) / r ** 0.5, "sink": 1.5 * rnd((H,), seed + 5),
         "g": 2 * rnd((H, W), seed + 6) / W ** 0.5, "o": torch.eye(H * E)}
    return m, w


def _latent_cache(Dk, dtype, page, max_tokens=2048):
    from umbrella_amd.attn.cache import PagedSeqCache
    c = PagedSeqCache([], [], max_tokens, 3, "cuda:0", dtype, page=page, latent_layers=[Dk])
    c.latent[0].fill_(9.0)
    return c


def _run_latent(lib, m, w, X, splits, dtype, page=4, cache=None, seq="s", layout=0):
    from umbrella_amd.models.config import rotary_table
    from potosun_helpers import Steps, dev, zeros
    H, D, R, E, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    freq, mult = rotary_table(m["rot"]["base"], m["rot"]["dims"], m["rot"].get("scaling"))
    fr, Xd = dev(freq), X.double()
    proj_all = torch.cat([Xd @ w[k].double().T for k in ("q", "dkv", "g")], dim=1).float()
    ld, kv_col = proj_all.shape[1], H * (D + R)
    uk_t, uv = dev(w["uk"].view(H, D, r).transpose(1, 2), dtype), dev(w["uv"], dtype)
    cache = cache or _latent_cache(r + R, dtype, page)
    cache.open(seq)
    kv, sink, outs, at = cache.latent_struct(0), dev(w["sink"], dtype), [], 0
    for cnt in splits:
        st = Steps([cnt], [cache.extend(seq, cnt)], [cache.slot(seq)])
        proj, qn, qa = dev(proj_all[at:at + cnt]), zeros(cnt, H * D, dtype=dtype), zeros(cnt, H, r + R)
        lat, out = zeros(cnt, H * r, dtype=dtype), zeros(cnt, H * E, dtype=dtype)
        call("umb_lat_front", qn, qa, kv, proj, ld, 0, kv_col, dev(w["dkv.norm"], dtype), st.d["pos"], st.d["slot"], fr, cnt, H, D, R, r, m["rot"]["dims"],
             layout, mult, 1e-5, code(dtype))
        call("umb_seq_linear_batched", qa, qn, uk_t, cnt, r, D, H * D, H * (r + R), H, D, r * D, r + R, 0, None, 0, 0, code(dtype))
        if cnt >= 16 and lib.umb_lat_attend_tiled_ok(H, r, R, code(dtype)):
            call("umb_lat_attend_tiled", lat, qa, kv, sink, *st.seqs, 1, cnt, H, r, R, m["mask"]["size"], m["scale"], code(dtype))
        else:
            call("umb_lat_attend", lat, qa, kv, sink, st.d["pos"], st.d["slot"], cnt, H, r, R, m["mask"]["size"], m["scale"], code(dtype))
        call("umb_seq_linear_batched", out, lat, uv, cnt, E, r, H * r, H * E, H, r, E * r, E, 7, proj[:, kv_col + r + R:], ld, 1, code(dtype))
        outs.append(out)
        at += cnt
    return torch.cat(outs), cache


LATENT = [(3, 6, 8, 10, 11, 6, [19]), (1, 3, 2, 5, 9, 1, [1] * 12), (5, 9, 4, 3, 16, 11, [2, 9, 1, 1, 17, 3]), (8, 24, 8, 16, 32, 21, [40, 1, 1, 30, 2, 2]),
          (5, 32, 16, 40, 80, 70, [70, 1, 64, 3, 62]), (16, 40, 24, 24, 144, 50, [33, 20, 1, 48]), (4, 130, 32, 20, 320, 9, [17, 2, 16])]


@BOTH
@pytest.mark.parametrize("H,D,R,E,r,window,splits", LATENT)
def test_latent_attention_prompt_portions_and_single_tokens(lib, dtype, H, D, R, E, r, window, splits):
    from oracle import potosun as O
    from potosun_helpers import close, rnd
    n = sum(splits)
    m, w = _latent_case(H, D, R, E, r, window, 1, scaling=H != 5)
    X = rnd((n, 24), 9)
    wd = {k: v.to(dtype).double() if k in ("dkv.norm", "uk", "uv", "sink") else v.double() for k, v in w.items()}
    want, rows = O.latent_attention(X.double(), torch.arange(n), m, wd, 1e-5)
    got, cache = _run_latent(lib, m, w, X, splits, dtype)
    assert close(got, want, tol_of(dtype))
    stored = cache.latent_rows(0, "s", list(range(n)))
    assert close(stored, torch.cat(rows, dim=1), 1e-5 if dtype == torch.float32 else 1e-2)
    cache.close("s")
    again, _ = _run_latent(lib, m, w, X[:9], [4, 1, 4], dtype, cache=cache, seq="t")
    assert close(again, want[:9], tol_of(dtype))


@BOTH
def test_latent_window_edge_of_one_outstanding_key(lib, dtype):
    """one token's rotated key part towers over all others: the positions less than a window behind it read its latent, no other"""
    from oracle import potosun as O
    from potosun_helpers import close, rnd
    m, w = _latent_case(4, 16, 8, 16, 32, 20, 1, scaling=False)
    m["rot"]["base"] = 1e12                               # the last pairs hardly turn: a key part that stays aligned
    n, W = 90, 24
    for far in (0, 15, 16, 33):
        X = rnd((n, W), 9)
        X[:, 0], X[:, 1] = 1.0, 0.0
        X[far, 1] = 30.0
        w["q"][:, :2] = 0
        w["q"].view(4, 24, W)[:, 16 + 3, 0] = 6.0          # every query's rotated feature 3 (a pair that hardly turns)
        w["dkv"][:, 1] = 0
        w["dkv"][32 + 3, 1] = 3.0
        w["sink"] = torch.zeros(4)
        wd = {k: v.to(dtype).double() if k in ("dkv.norm", "uk", "uv") else v.double() for k, v in w.items()}
        want, (c, _) = O.latent_attention(X.double(), torch.arange(n), m, wd, 1e-5)
        got = None
        for splits in ([n], [far + 2] + [1] * (n - far - 2), [40, 2, 1, 47]):
            got, _ = _run_latent(lib, m, w, X, splits, dtype, page=16)
            assert close(got, want, tol_of(dtype)), (far, splits[:3])
        gate = torch.sigmoid(X.double() @ w["g"].double().T)
        mark = (c[far] @ wd["uv"].T).view(4, 16)
        like = ((got.double().cpu().view(n, 4, 16) / gate[..., None] - mark).pow(2).mean((1, 2)) / mark.pow(2).mean()).sqrt()
        inside = list(range(far, min(far + 20, n)))
        assert float(like[inside].max()) < 0.02 and float(like[[i for i in range(n) if i not in inside]].min()) > 0.3, far


@pytest.mark.parametrize("layout,R,dims", [(0, 8, 8), (1, 8, 8), (0, 8, 4), (1, 9, 6), (0, 7, 4), (0, 3, 0)])
def test_latent_front_both_layouts_and_features_that_pass(lib, layout, R, dims):
    from oracle import potosun as O
    from potosun_helpers import YARN, Steps, close, dev, rnd, zeros
    from umbrella_amd.models.config import rotary_table
    T, H, D, r, off = 5, 3, 6, 10, 2
    rot = {"dims": dims, "base": 50.0, "scaling": YARN} if dims else None
    freq, mult = rotary_table(50.0, dims, YARN) if dims else (None, 1.0)
    ld = off + H * (D + R) + 1 + r + R
    proj, wn = rnd((T, ld), 1), 1 + rnd((r,), 2, 0.3)
    cache = _latent_cache(r + R, torch.float32, 4)
    cache.open("s")
    cache.extend("s", 13)
    st = Steps([T], [cache.extend("s", T)], [cache.slot("s")])
    qn, qa = zeros(T, H * D), zeros(T, H, r + R) + 7
    call("umb_lat_front", qn, qa, cache.latent_struct(0), dev(proj), ld, off, off + H * (D + R) + 1, dev(wn), st.d["pos"], st.d["slot"],
         dev(freq) if dims else None, T, H, D, R, r, dims, layout, mult, 1e-3, 2)
    q, pos = proj[:, off:off + H * (D + R)].double().view(T, H, D + R), torch.arange(13, 13 + T)
    down = proj[:, off + H * (D + R) + 1:].double()
    assert close(qn, q[..., :D].reshape(T, -1), 1e-6) and close(qa[..., r:], O.rotate(q[..., D:], pos, rot, layout == 1), 1e-6)
    assert float((qa[..., :r] - 7).abs().max()) == 0.0
    rows = cache.latent_rows(0, "s", list(range(13, 13 + T)))
    assert close(rows[:, :r], O.rms(down[:, :r], 1e-3) * wn.double(), 1e-6)
    assert close(rows[:, r:], O.rotate(down[:, None, r:], pos, rot, layout == 1)[:, 0], 1e-6)


def test_shapes_the_kernels_do_not_cover_are_refused(lib):
    from umbrella_amd import _lib
    from potosun_helpers import i32, zeros
    z, c = zeros(4096), _cache(1, 8, 8, torch.float32, 4)
    with pytest.raises(_lib.UmbError):                    # gate columns beyond the row
        call("umb_attn_attend", z, 16, z, c.struct(0), z, 20, 10, None, 0, i32([0]), i32([0]), 1, 2, 1, 8, 8, 8, 1.0, 1.0, 0.0, form(0, None, 0, 1), None, 0, 2)
    with pytest.raises(_lib.UmbError):
        call("umb_attn_attend", z, 16, z, c.struct(0), z, 99, -1, None, 0, i32([0]), i32([0]), 1, 2, 1, 8, 8, 8, 1.0, 1.0, 0.0, form(0, None, -1), None, 0, 2)
    with pytest.raises(_lib.UmbError):                    # no cap
        call("umb_seq_linear_cap", z, z, z, None, 1, 4, 4, 0.0, 2)
    with pytest.raises(_lib.UmbError):                    # queries that do not fit the row
        call("umb_lat_front", z, z, _latent_cache(12, torch.float32, 4).latent_struct(0), z, 30, 0, 20, z, i32([0]), i32([0]), z, 1, 2, 8, 4, 8, 4, 0, 1.0, 1e-5, 2)


# ------------------------------------------------------------------ whole models
def _oracle_logits(cfgd, sd, toks):
    from oracle import potosun as O
    return O.forward(cfgd, sd, toks)[0]


@pytest.mark.parametrize("name", ["mixed", "odd", "plain", "wide"])
@BOTH
def test_model_prefill_decode_portions_against_oracle(lib, name, dtype):
    from oracle import potosun as O
    from potosun_helpers import CONFIGS, build, close, rel_err, tokens
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


@BOTH
def test_model_unequal_batch_equals_each_alone(lib, dtype):
    """three requests of different lengths prefilled in one step and decoded together, the shortest ending first, against
    each of them alone; then a new request in the slot and pages the shortest one gave back"""
    from potosun_helpers import CONFIGS, build, rel_err, tokens
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
    from potosun_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS["plain"]
    m, sd = build(cfgd, torch.float32, seed=3, page=4, batch=3)
    a, b = tokens(80, cfgd["vocab"], 1), tokens(30, cfgd["vocab"], 2)
    m.open("a"), m.open("b")
    m.forward_batch([("b", b[:29])])
    out = m.forward_batch([("a", a), ("b", b[29:])], want=[list(range(80)), [0]]).clone()
    assert rel_err(out[:80], _oracle_logits(cfgd, sd, a)) < F32_TOL and rel_err(out[80:], _oracle_logits(cfgd, sd, b)[29:]) < F32_TOL


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_model_long_decoding_and_first_tokens(lib, name):
    """fp32: 150 tokens decoded one by one after a two-token prompt (pages of 4 tokens used up and down the table, windows passing over
    decoded tokens, chunk edges crossed many times) against the oracle's whole-sequence pass"""
    from potosun_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS[name]
    m, sd = build(cfgd, torch.float32, seed=7, page=4, batch=2, max_tokens=400)
    toks = tokens(152, cfgd["vocab"], seed=9)
    want = _oracle_logits(cfgd, sd, toks)
    m.open("x")
    rows = [m.forward_batch([("x", toks[:2])], want=[[0, 1]]).clone()]
    for t in toks[2:]:
        rows.append(m.forward_batch([("x", [t])], want=[[0]]).clone())
    got = torch.cat(rows)
    assert rel_err(got, want) < 3e-5 and rel_err(got[:3], want[:3]) < F32_TOL


@pytest.mark.parametrize("name", ["mixed", "plain", "wide"])
@BOTH
def test_model_long_prompt_in_one_step_and_in_portions(lib, name, dtype):
    """matrix-pipe attention, cut at and beside chunk, window and page borders"""
    from potosun_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS[name]
    m, sd = build(cfgd, dtype, seed=5, page=16, batch=2, max_length=320, max_tokens=700)
    n = 200
    toks = tokens(n, cfgd["vocab"], 40)
    want = _oracle_logits(cfgd, sd, toks)
    tol = 3e-5 if dtype == torch.float32 else 6e-2
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


def test_model_many_single_tokens_in_one_step(lib):
    """sixty sequences decoding together (no split keys, sixteen heads of a token as one latent query tile) against the oracle"""
    from potosun_helpers import CONFIGS, build, rel_err, tokens
    cfgd = CONFIGS["plain"]
    for dtype, tol in ((torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)):
        m, sd = build(cfgd, dtype, seed=3, page=4, batch=60, max_length=64, max_tokens=60 * 40)
        seqs = [tokens(20 + i % 7, cfgd["vocab"], i) for i in range(60)]
        for i, t in enumerate(seqs):
            m.open(i)
        m.forward_batch([(i, t[:-1]) for i, t in enumerate(seqs)])
        out = m.forward_batch([(i, t[-1:]) for i, t in enumerate(seqs)], want=[[0]] * 60).clone()
        for i in (0, 13, 59):
            assert rel_err(out[i:i + 1], _oracle_logits(cfgd, sd, seqs[i])[-1:]) < tol, i


def test_model_refuses_values_that_do_not_fit(lib):
    from potosun_helpers import biased, build, chunked, config, layer
    with pytest.raises(ValueError):
        build(config([layer(biased(kv_heads=2, vdim=12)), layer(chunked(kv_heads=2, vdim=6))]), torch.float32)
    with pytest.raises(ValueError):
        build(config([layer(biased(kv_heads=4, vdim=6)), layer(chunked(heads=6, kv_heads=2, vdim=12))]), torch.float32)
    m, _ = build(config([layer(biased(kv_heads=2, vdim=12)), layer(chunked(kv_heads=2, vdim=6, v_mix=False))]), torch.float32)
    assert [int(s.v_mix) for s in m._layer_structs] == [1, 0] and m._bufs["v_first"].shape[1] == 24


def test_caches_of_the_layers(lib):
    from potosun_helpers import CONFIGS, build
    m, _ = build(CONFIGS["mixed"], torch.bfloat16)
    assert [(e["G"], e["D"], e["E"], e["pool"]) for e in m.kv_cache.kv] == [(2, 8, 12, 0), (2, 10, 12, 0), (2, 8, 12, 0), (2, 7, 12, 0), (2, 8, 12, 0)]
    assert [tuple(z.shape[1:]) for z in m.kv_cache.latent] == [(4, 19), (4, 20)] and not m.kv_cache.state
    assert [int(s.v_mix) for s in m._layer_structs] == [0, 1, 0, 2, 0, 2, 2]


def test_model_decode_steps_replayed_as_graphs_equal_eager_launches(lib):
    from potosun_helpers import CONFIGS, build, tokens
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
    from potosun_helpers import build
    from umbrella_amd.speculation.auto_engine import AutoEngine
    from umbrella_amd.speculation.speculation_utils import IdTokenizer
    m, sd = build(cfgd, dtype, seed=21, page=4, batch=kw.pop("batch", 3), max_length=96, max_tokens=kw.pop("max_tokens", 512), sd=sd)
    e = AutoEngine.from_config("cuda:0", engine="batch", model="tiny", dtype=dtype, target_model_obj=m, tokenizer=IdTokenizer(), **kw)
    e.initialize()
    return e, sd


def test_engine_greedy_generation_matches_oracle(lib):
    """five queued requests through the scheduler (three slots: two batches), greedy, fp32: the oracle's tokens"""
    from potosun_helpers import CONFIGS, tokens
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
    from potosun_helpers import CONFIGS, tokens
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
    from potosun_helpers import CONFIGS, checkpoint, rel_err, tokens
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
