"""Tutunex: a decoder stack whose layers are chosen by the checkpoint's config.json:

* every sublayer is normed before and after: ``x <- x + norm1b(mixer(norm1(x)))``, then ``x <- x + norm2b(ff(norm2(x)))`` (RMS norms
  with plain weights); the embedding row is multiplied by a constant, the head is a matrix of its own;
* ``attention`` -- differential attention: two query / key maps per head over the same values, ``a1 - lambda a2`` over its root mean
  square times ``1 - diff``; keys only of the query's own run of ``mask.size`` positions; rotary positions (half layout, YaRN
  frequencies) on the first ``rot.dims`` features of every map; with ``kv_from`` the keys and values of an earlier layer;
* ``parallel`` -- two mixers reading the same input: causal grouped-query attention without positions (q / k RMS norm per head, one
  added to the softmax denominator) and a gated delta rule (short convolutions with silu, unit-vector q and k, one decay and one
  step size per head, gated per-head RMS norm); half the sum of the two outputs, each RMS-normed over the width;
* feed-forwards of the capped gated form ``g sigmoid(1.702 g) (u + 1)``.

This file only TRANSLATES the design -- config.json keys, tensor names, how matrices are fused -- into the generic
sequence-mixer runtime (models/seqmix.py); every mechanism lives there and in csrc/seq_*.hip with its constants as parameters.
"""
from __future__ import annotations

import json
import os

import torch

from .config import AttnDeltaCfg, DiffAttnCfg, SeqLayerCfg, SeqMixCfg
from .seqmix import SeqMixLM

ARCHITECTURE = "Tutunex"
GLU_ALPHA = 1.702          # the design fixes the sigmoid's factor of its feed-forwards
PAIR_COEF = 0.5            # and the weight of a parallel layer's two normed outputs


def _mixer(kind: str, m: dict):
    if kind == "attention":
        rot = m.get("rot") or {}
        return DiffAttnCfg(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=int(m["dim"]),
                           vdim=int(m.get("vdim", m["dim"])), scale=float(m["scale"]), diff=float(m["diff"]),
                           chunk=int((m.get("mask") or {}).get("size", 0)), rot_dims=int(rot.get("dims", 0)),
                           rot_base=float(rot.get("base", 10000.0)), rot_scaling=dict(rot["scaling"]) if rot.get("scaling") else None,
                           kv_from=int(m["kv_from"]) if m.get("kv_from") is not None else None)
    if kind == "parallel":
        a, b = m["left"], m["right"]
        return AttnDeltaCfg(heads=int(a["heads"]), kv_heads=int(a.get("kv_heads", a["heads"])), dim=int(a["dim"]),
                            vdim=int(a.get("vdim", a["dim"])), scale=float(a["scale"]), s_heads=int(b["heads"]),
                            s_groups=int(b.get("kv_heads", b["heads"])), s_state=int(b["dim"]), s_vdim=int(b.get("vdim", b["dim"])),
                            s_taps=int(b.get("conv", 1)), pair_coef=PAIR_COEF)
    raise ValueError(f"{ARCHITECTURE}: unknown layer type '{kind}'")


def _layer(entry: dict) -> SeqLayerCfg:
    mixer, mlp = _mixer(entry["type"], entry["mixer"]), entry.get("mlp")
    if mlp is None:
        return SeqLayerCfg(mixer=mixer, ff=0)
    if mlp.get("kind", "dense") != "dense":
        raise ValueError(f"{ARCHITECTURE}: unknown feed-forward kind '{mlp.get('kind')}'")
    return SeqLayerCfg(mixer=mixer, ff=int(mlp["ff"]), act="clamp_glu", act_limit=float(mlp["limit"]), act_alpha=GLU_ALPHA)


def config_from_dict(c: dict, name: str = "tutunex") -> SeqMixCfg:
    return SeqMixCfg(vocab_size=int(c["vocab"]), width=int(c["width"]), norm_eps=float(c["norm"]["eps"]), norm_groups=1,
                     layers=[_layer(e) for e in c["layers"]], name=name, architecture=ARCHITECTURE,
                     embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)))


def config_from_dir(path: str) -> SeqMixCfg:
    with open(os.path.join(path, "config.json")) as f:
        return config_from_dict(json.load(f), name=os.path.basename(os.path.normpath(path)))


def tensor_shapes(cfg: SeqMixCfg) -> dict:
    """checkpoint tensor name -> shape (linear weights are [out, in])"""
    W = cfg.width
    sh = {"embed": (cfg.vocab_size, W), "final.norm": (W,), "head": (cfg.vocab_size, W)}
    for i, ly in enumerate(cfg.layers):
        p, m = f"l{i}.", ly.mixer
        sh.update({p + "norm1": (W,), p + "norm1b": (W,)})
        if m.kind == "diff_attention":
            a = p + "mix."
            sh[a + "q"] = (m.heads * 2 * m.dim, W)
            if m.kv_from is None:
                sh.update({a + "k": (m.kv_heads * 2 * m.dim, W), a + "v": (m.kv_heads * m.vdim, W)})
            sh.update({a + n: (m.dim,) for n in ("lq1", "lk1", "lq2", "lk2")})
            sh[a + "o"] = (W, m.heads * m.vdim)
        else:
            a, b = p + "mix.left.", p + "mix.right."
            qk, inner = m.s_groups * m.s_state, m.s_heads * m.s_vdim
            sh.update({a + "q": (m.heads * m.dim, W), a + "k": (m.kv_heads * m.dim, W), a + "v": (m.kv_heads * m.vdim, W),
                       a + "q.norm": (m.dim,), a + "k.norm": (m.dim,), a + "o": (W, m.heads * m.vdim), a + "out": (W,),
                       b + "q": (qk, W), b + "k": (qk, W), b + "v": (inner, W), b + "q.conv": (qk, m.s_taps),
                       b + "k.conv": (qk, m.s_taps), b + "v.conv": (inner, m.s_taps), b + "b": (m.s_heads, W), b + "a": (m.s_heads, W),
                       b + "A_log": (m.s_heads,), b + "dt_bias": (m.s_heads,), b + "norm": (m.s_vdim,), b + "g": (inner, W),
                       b + "o": (W, inner), b + "out": (W,)})
        if ly.has_ff:
            sh.update({p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.gate": (ly.ff, W), p + "mlp.up": (ly.ff, W),
                       p + "mlp.down": (W, ly.ff)})
    return sh


def synth_state(cfg: SeqMixCfg, seed: int = 0) -> dict:
    """Seeded random fp32 checkpoint of the design (tests, benchmarks): name -> tensor."""
    g = torch.Generator().manual_seed(seed)
    sd = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g)
        if "norm" in leaf or leaf == "out":
            t = 1.0 + 0.1 * r
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.7 * r / shape[0] ** 0.25                      # products of unit size: lambda moves away from its constant
        elif leaf == "embed":
            t = r
        elif leaf == "conv":
            t = 0.6 * r
        elif leaf in ("A_log", "dt_bias"):
            t = r - 1.0
        elif leaf in ("a", "b"):
            t = 2.0 * r / shape[1] ** 0.5
        else:
            t = r / shape[1] ** 0.5
        sd[name] = t
    return sd


class Tutunex(SeqMixLM):
    """``AutoModelLM`` resolves a directory whose config.json says ``"architecture": "Tutunex"`` to this class."""

    @staticmethod
    def read_config(path: str) -> SeqMixCfg:
        return config_from_dir(path)

    def layer_tensors(self, i: int, ly: SeqLayerCfg, get):
        """The design's tensor names -> the runtime's fused per-layer tensors.  ``get(name)`` fetches one checkpoint tensor
        in the storage dtype on the device."""
        p, m = f"l{i}.", ly.mixer
        t = {"norm1": get(p + "norm1"), "norm1b": get(p + "norm1b")}
        if m.kind == "diff_attention":
            a = p + "mix."
            t["proj_w"] = get(a + "q") if m.kv_from is not None else torch.cat([get(a + "q"), get(a + "k"), get(a + "v")], dim=0)
            t["out_w"] = get(a + "o")
            lq1, lk1, lq2, lk2 = (get(a + n).to(torch.float64) for n in ("lq1", "lk1", "lq2", "lk2"))
            t["diff_lambda"] = float(torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum())) + m.diff
            rows = 2 * m.heads * m.dim + (0 if m.kv_from is not None else m.kv_heads * (2 * m.dim + m.vdim))
            assert t["proj_w"].shape[0] == rows and t["out_w"].shape[1] == m.heads * m.vdim
        else:
            a, b = p + "mix.left.", p + "mix.right."
            # ONE input projection for both mixers; an output projection each (their outputs are normed apart)
            t["proj_w"] = torch.cat([get(a + "q"), get(a + "k"), get(a + "v"), get(b + "q"), get(b + "k"), get(b + "v"), get(b + "g"),
                                     get(b + "b"), get(b + "a")], dim=0)
            t["out_w"], t["out2_w"], t["out_norm_a"], t["out_norm_b"] = get(a + "o"), get(b + "o"), get(a + "out"), get(b + "out")
            t["q_norm"], t["k_norm"], t["s_norm"] = get(a + "q.norm"), get(a + "k.norm"), get(b + "norm")
            t["s_conv"] = torch.cat([get(b + "q.conv"), get(b + "k.conv"), get(b + "v.conv")], dim=0)
            t["s_a_log"], t["s_dt_bias"] = get(b + "A_log").to(torch.float32), get(b + "dt_bias").to(torch.float32)
            C = 2 * m.s_groups * m.s_state + m.s_heads * m.s_vdim
            assert tuple(t["s_conv"].shape) == (C, m.s_taps), tuple(t["s_conv"].shape)
            assert t["proj_w"].shape[0] == (m.heads + m.kv_heads) * m.dim + m.kv_heads * m.vdim + C + m.s_heads * (m.s_vdim + 2)
        if ly.has_ff:
            t["norm2"], t["norm2b"] = get(p + "norm2"), get(p + "norm2b")
            t["gu_w"] = torch.cat([get(p + "mlp.gate"), get(p + "mlp.up")], dim=0)
            t["down_w"] = get(p + "mlp.down")
        return t

    def top_tensors(self, get):
        return {"embed": get("embed"), "final_norm": get("final.norm"), "head": get("head")}
