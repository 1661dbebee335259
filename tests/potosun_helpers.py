"""Tiny Potosun configurations, seeded checkpoints and comparison helpers for the tests of that design."""
import torch

from tutunex_helpers import Steps, close, dev, i32, rel_err, rnd, tokens, zeros          # noqa: F401  (shared with that design's tests)
from umbrella_amd.models import potosun

YARN = {"factor": 4.0, "fast": 8.0, "original": 96, "slow": 0.5}


def biased(heads=4, kv_heads=2, dim=8, vdim=12, window=9, keep=3, bias_max=14, scale=None, v_mix=True):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "bias_max": bias_max, "mask": {"size": window},
         "scale": 1.4 * dim ** -0.5 if scale is None else scale, "v_mix": v_mix}
    if keep is not None:
        m["mask"]["keep_first"] = keep
    return "attention", m


def chunked(heads=6, kv_heads=2, dim=10, vdim=12, chunk=7, rot_dims=6, base=300.0, scale=None, v_mix=True):
    return "attention_2", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
                           "rot": {"base": base, "dims": rot_dims}, "scale": 1.2 * dim ** -0.5 if scale is None else scale, "v_mix": v_mix}


def latent(heads=3, dim=6, rot_dim=8, vdim=10, kv_rank=11, window=6, base=200.0, scaling=YARN, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
         "rot": {"base": base, "dims": rot_dim}, "scale": 1.1 * (dim + rot_dim) ** -0.5 if scale is None else scale}
    if scaling:
        m["rot"]["scaling"] = dict(scaling)
    return "latent_attention", m


def layer(mixer, ff=28):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, vocab=90, width=40, eps=1e-5, embed_scale=1.7, cap=9.0):
    return {"architecture": "Potosun", "embedding": {"scale": embed_scale}, "layers": layers, "logit_softcap": cap, "norm": {"eps": eps},
            "vocab": vocab, "width": width}


# shapes that differ from one another in every size: layer order, the first layer that mixes values of either type and not the first
# of its type, layers that do not mix, odd sizes (nothing a multiple of 8), one key/value head and as many as query heads, value sizes
# above and below the key size, windows and chunks of 1, kept tokens none / one / more than a window, rotary on all or some features,
# a scaled and an unscaled table, layers without feed-forward, scale 1, a bias table whose last row lies inside and outside the window
CONFIGS = {
    "mixed": config([layer(biased(v_mix=False)), layer(chunked()), layer(latent()), layer(biased(keep=5, window=4, bias_max=30)),
                     layer(latent(heads=2, dim=9, rot_dim=4, vdim=3, kv_rank=16, window=11, scaling=None), ff=0),
                     layer(chunked(heads=2, dim=7, rot_dims=2, chunk=16), ff=14), layer(biased(kv_heads=2, window=13, keep=1))]),
    "odd": config([layer(latent(heads=5, dim=3, rot_dim=2, vdim=5, kv_rank=9, window=1), ff=0),
                   layer(biased(heads=3, kv_heads=1, dim=7, vdim=5, window=1, keep=0, bias_max=9, scale=1.0), ff=9),
                   layer(chunked(heads=3, kv_heads=1, dim=5, vdim=5, chunk=1, rot_dims=4), ff=15),
                   layer(biased(heads=7, kv_heads=1, dim=9, vdim=5, window=20, keep=None, bias_max=5), ff=0)],
                  vocab=75, width=36, eps=1e-3, embed_scale=1.0, cap=2.0),
    "plain": config([layer(chunked(heads=4, kv_heads=4, dim=16, vdim=32, chunk=40, rot_dims=16), ff=48),
                     layer(latent(heads=8, dim=24, rot_dim=8, vdim=16, kv_rank=32, window=21, base=5000.0), ff=48),
                     layer(biased(heads=8, kv_heads=4, dim=24, vdim=32, window=18, keep=33, bias_max=50), ff=48)],
                    vocab=130, width=64, embed_scale=0.5, cap=25.0),
    "wide": config([layer(biased(heads=10, kv_heads=2, dim=40, vdim=80, window=50, keep=6, bias_max=90), ff=96),
                    layer(latent(heads=5, dim=32, rot_dim=16, vdim=40, kv_rank=80, window=70, base=20.0), ff=96),
                    layer(chunked(heads=2, kv_heads=2, dim=136, vdim=80, chunk=48, rot_dims=20, base=9000.0), ff=0)],
                   vocab=110, width=128, cap=15.0),
}


def checkpoint(cfg_dict, seed=0, bias_rows=8):
    cfg = potosun.config_from_dict(cfg_dict)
    return cfg, potosun.synth_state(cfg, seed=seed, bias_rows=bias_rows)


def build(cfg_dict, dtype, seed=0, page=4, batch=4, max_length=256, max_tokens=1024, sd=None, bias_rows=8, **kw):
    """a served model on cuda:0 over a seeded checkpoint (weights rounded to `dtype`) + the state dict it was built from"""
    cfg = potosun.config_from_dict(cfg_dict)
    if sd is None:
        _, sd = checkpoint(cfg_dict, seed, bias_rows)
    sd = {k: v.to(dtype).to(torch.float32) for k, v in sd.items()}          # the oracle sees exactly the stored weights
    m = potosun.Potosun("tiny", batch_size=batch, max_length=max_length, max_tokens=max_tokens, device="cuda:0", dtype=dtype,
                        state_dict=sd, config=cfg, page_size=page, **kw)
    m.alloc()
    return m, sd
