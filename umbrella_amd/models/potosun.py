"""Potosun: a pre-norm decoder stack (``x <- x + mixer(norm1(x))``, ``x <- x + ff(norm2(x))``, plain RMS norms) whose layers are
chosen by the checkpoint's config.json:

* ``attention`` -- grouped-query softmax attention without rotation: q / k RMS norm per head, a learned bias per (distance bucket,
  head), a sliding window that keeps the sequence's first tokens, one sigmoid gate per output feature;
* ``attention_2`` -- grouped-query softmax attention with interleaved rotary positions, keys of the query's own chunk of positions
  only, a learned sink per head in the denominator;
* in both, layers marked ``v_mix`` cache ``(1 - lambda) v + lambda v_first`` with v_first the values of the first such layer;
* ``latent_attention`` -- keys and values from one normed latent per token plus one rotated key part shared by the heads (half
  layout, YaRN frequencies), queries straight from the input, a sliding window, a sink and one sigmoid gate per head;
* feed-forwards of the form ``W_down (gelu(W_gate h) * W_up h)`` (tanh form); the embedding row is multiplied by a constant, the
  head is a matrix of its own and its logits are capped.

This file only TRANSLATES the design -- config.json keys, tensor names, how matrices are fused -- into the generic
sequence-mixer runtime (models/seqmix.py); every mechanism lives there and in csrc/seq_*.hip with its constants as parameters.
"""
from __future__ import annotations

import json
import os

import torch

from .config import LatentAttnCfg, SeqLayerCfg, SeqMixCfg, SoftmaxAttnCfg, bias_by_distance
from .seqmix import SeqMixLM

ARCHITECTURE = "Potosun"


def _mixer(kind: str, m: dict):
    mask, rot = m.get("mask") or {}, m.get("rot") or {}
    rotary = dict(rot_base=float(rot.get("base", 10000.0)), rot_scaling=dict(rot["scaling"]) if rot.get("scaling") else None)
    if kind == "latent_attention":
        rot_dim = int(m["rot_dim"])
        cfg = LatentAttnCfg(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=rot_dim, vdim=int(m.get("vdim", m["dim"])), q_rank=0,
                            kv_rank=int(m["kv_rank"]), window=int(mask.get("size", 0)), rot_dims=int(rot.get("dims", rot_dim)),
                            scale=float(m["scale"]), rot_layout="half", gate="head", **rotary)
        if cfg.rot_dims > rot_dim or cfg.rot_dims % 2:
            raise ValueError(f"{ARCHITECTURE}: rot.dims must be even and at most rot_dim")
        return cfg
    sizes = dict(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=int(m["dim"]), vdim=int(m.get("vdim", m["dim"])),
                 scale=float(m["scale"]), v_mix=bool(m.get("v_mix", False)))
    if kind == "attention":
        return SoftmaxAttnCfg(**sizes, window=int(mask.get("size", 0)), keep_first=int(mask.get("keep_first", 0)), qk_norm=True,
                              bias_far=float(m["bias_max"]), gate=True)
    if kind == "attention_2":
        return SoftmaxAttnCfg(**sizes, **rotary, chunk=int(mask.get("size", 0)), rot_dims=int(rot.get("dims", 0)),
                              rot_layout="interleaved", sink=True)
    raise ValueError(f"{ARCHITECTURE}: unknown layer type '{kind}'")


def _layer(entry: dict) -> SeqLayerCfg:
    mixer, mlp = _mixer(entry["type"], entry["mixer"]), entry.get("mlp")
    if mlp is None:
        return SeqLayerCfg(mixer=mixer, ff=0)
    if mlp.get("kind", "dense") != "dense":
        raise ValueError(f"{ARCHITECTURE}: unknown feed-forward kind '{mlp.get('kind')}'")
    return SeqLayerCfg(mixer=mixer, ff=int(mlp["ff"]), act="gelu_gated")


def config_from_dict(c: dict, name: str = "potosun") -> SeqMixCfg:
    return SeqMixCfg(vocab_size=int(c["vocab"]), width=int(c["width"]), norm_eps=float(c["norm"]["eps"]), norm_groups=1,
                     layers=[_layer(e) for e in c["layers"]], name=name, architecture=ARCHITECTURE, streams=1,
                     embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)), logit_cap=float(c.get("logit_softcap") or 0.0))


def config_from_dir(path: str) -> SeqMixCfg:
    with open(os.path.join(path, "config.json")) as f:
        return config_from_dict(json.load(f), name=os.path.basename(os.path.normpath(path)))


def tensor_shapes(cfg: SeqMixCfg, bias_rows: int = 16) -> dict:
    """checkpoint tensor name -> shape (linear weights are [out, in])"""
    W = cfg.width
    sh = {"embed": (cfg.vocab_size, W), "final.norm": (W,), "head": (cfg.vocab_size, W)}
    for i, ly in enumerate(cfg.layers):
        p, m = f"l{i}.", ly.mixer
        a = p + "mix."
        sh[p + "norm1"] = (W,)
        if m.kind == "latent_attention":
            sh.update({a + "q": (m.heads * (m.dim + m.rot_dim), W), a + "dkv": (m.kv_rank + m.rot_dim, W), a + "dkv.norm": (m.kv_rank,),
                       a + "uk": (m.heads * m.dim, m.kv_rank), a + "uv": (m.heads * m.vdim, m.kv_rank), a + "sink": (m.heads,),
                       a + "g": (m.heads, W)})
        else:
            sh.update({a + "q": (m.heads * m.dim, W), a + "k": (m.kv_heads * m.dim, W), a + "v": (m.kv_heads * m.vdim, W)})
            if m.qk_norm:
                sh.update({a + "q.norm": (m.dim,), a + "k.norm": (m.dim,)})
            if m.bias_far:
                sh[a + "rel"] = (m.bias_rows or bias_rows, m.heads)
            if m.v_mix:
                sh[a + "vmix"] = ()
            if m.sink:
                sh[a + "sink"] = (m.heads,)
            if m.gate:
                sh[a + "g"] = (m.heads * m.vdim, W)
        sh[a + "o"] = (W, m.heads * m.vdim)
        if ly.has_ff:
            sh.update({p + "norm2": (W,), p + "mlp.gate": (ly.ff, W), p + "mlp.up": (ly.ff, W), p + "mlp.down": (W, ly.ff)})
    return sh


def synth_state(cfg: SeqMixCfg, seed: int = 0, bias_rows: int = 16) -> dict:
    """Seeded random fp32 checkpoint of the design (tests, benchmarks): name -> tensor."""
    g = torch.Generator().manual_seed(seed)
    sd = {}
    for name, shape in tensor_shapes(cfg, bias_rows).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g)
        if "norm" in leaf:
            t = 1.0 + 0.1 * r
        elif leaf in ("embed", "sink", "rel"):
            t = r
        elif leaf == "vmix":
            t = 0.5 + 0.2 * r
        else:
            t = r / shape[1] ** 0.5
        sd[name] = t
    return sd


class Potosun(SeqMixLM):
    """``AutoModelLM`` resolves a directory whose config.json says ``"architecture": "Potosun"`` to this class."""

    @staticmethod
    def read_config(path: str) -> SeqMixCfg:
        return config_from_dir(path)

    def layer_tensors(self, i: int, ly: SeqLayerCfg, get):
        """The design's tensor names -> the runtime's fused per-layer tensors.  ``get(name)`` fetches one checkpoint tensor
        in the storage dtype on the device."""
        p, m = f"l{i}.", ly.mixer
        a = p + "mix."
        t = {"norm1": get(p + "norm1"), "norm1b": None, "out_w": get(a + "o")}
        if m.kind == "latent_attention":
            t["proj_w"] = torch.cat([get(a + "q"), get(a + "dkv"), get(a + "g")], dim=0)                 # [q | dkv | gate]
            t["dkv_norm"], t["sink"], t["uv_w"] = get(a + "dkv.norm"), get(a + "sink"), get(a + "uv")
            # W_uk [heads dim][kv_rank] -> per head transposed [kv_rank][dim]: the weight of "carry the query into latent space"
            t["uk_t"] = get(a + "uk").view(m.heads, m.dim, m.kv_rank).transpose(1, 2).contiguous()
            assert t["proj_w"].shape[0] == m.heads * (m.dim + m.rot_dim + 1) + m.kv_rank + m.rot_dim
            assert tuple(t["uv_w"].shape) == (m.heads * m.vdim, m.kv_rank) and t["out_w"].shape[1] == m.heads * m.vdim
        else:
            parts = [get(a + "q"), get(a + "k"), get(a + "v")] + ([get(a + "g")] if m.gate else [])      # [q | k | v | gate]
            t["proj_w"] = torch.cat(parts, dim=0)
            if m.qk_norm:
                t["q_norm"], t["k_norm"] = get(a + "q.norm"), get(a + "k.norm")
            if m.bias_far:
                rel = get(a + "rel").to(torch.float32)
                m.bias_rows = rel.shape[0]
                t["dist_bias"] = bias_by_distance(rel, m.bias_far, self.max_length)
            if m.sink:
                t["attn_sink"] = get(a + "sink").to(torch.float32)
            if m.v_mix:
                t["v_lambda"] = float(get(a + "vmix"))
            assert t["out_w"].shape[1] == m.heads * m.vdim
            assert t["proj_w"].shape[0] == m.heads * m.dim + m.kv_heads * (m.dim + m.vdim) + (m.heads * m.vdim if m.gate else 0)
        if ly.has_ff:
            t["norm2"], t["norm2b"] = get(p + "norm2"), None
            t["gu_w"] = torch.cat([get(p + "mlp.gate"), get(p + "mlp.up")], dim=0)
            t["down_w"] = get(p + "mlp.down")
        return t

    def top_tensors(self, get):
        return {"embed": get("embed"), "final_norm": get("final.norm"), "head": get("head")}
