"""Host-side tests of the Potosun design: configuration reading, registry, checkpoint names, the bias table by distance, the rotation
tables, and the plain oracle against itself in portions and against direct statements of what a position sees (no GPU)."""
import json
import math
import os
import sys

import pytest
import torch

ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))
sys.path.insert(0, ROOT)
sys.path.insert(0, os.path.dirname(__file__))


def test_config_reading():
    from potosun_helpers import CONFIGS
    from umbrella_amd.models import potosun
    cfg = potosun.config_from_dict(CONFIGS["mixed"])
    assert [ly.mixer.kind for ly in cfg.layers] == ["softmax_attention", "softmax_attention", "latent_attention", "softmax_attention",
                                                    "latent_attention", "softmax_attention", "softmax_attention"]
    assert cfg.embed_scale == 1.7 and cfg.logit_cap == 9.0 and cfg.streams == 1 and cfg.norm_offset == 0.0 and cfg.resid_mult == 1.0
    a, b, c = (cfg.layers[i].mixer for i in (3, 5, 2))
    assert (a.window, a.keep_first, a.chunk, a.bias_far, a.qk_norm, a.gate, a.sink, a.rot_dims, a.v_mix) == (4, 5, 0, 30.0, True, True, False, 0, True)
    assert (b.window, b.keep_first, b.chunk, b.bias_far, b.qk_norm, b.gate, b.sink, b.rot_dims, b.rot_layout) == (0, 0, 16, 0.0, False, False, True, 2,
                                                                                                               "interleaved")
    assert (c.q_rank, c.kv_rank, c.rot_dim, c.rot_dims, c.rot_layout, c.gate, c.window, c.rot_scaling["slow"]) == (0, 11, 8, 8, "half", "head", 6, 0.5)
    assert not cfg.layers[4].has_ff and cfg.layers[5].act == "gelu_gated" and not cfg.layers[0].mixer.v_mix
    assert potosun.config_from_dict(CONFIGS["odd"]).layers[3].mixer.keep_first == 0
    for bad in ({"type": "other", "mixer": {}, "mlp": None}, dict(CONFIGS["odd"]["layers"][1], mlp={"kind": "moe", "ff": 3})):
        with pytest.raises((ValueError, KeyError)):
            potosun.config_from_dict(dict(CONFIGS["mixed"], layers=[bad]))


def test_registry_resolves_the_architecture(tmp_path):
    from potosun_helpers import CONFIGS
    from umbrella_amd.models.auto_model import AutoModelLM
    from umbrella_amd.models.config import read_architecture
    from umbrella_amd.models.potosun import Potosun
    (tmp_path / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    assert read_architecture(str(tmp_path)) == "Potosun"
    m = AutoModelLM.from_pretrained(str(tmp_path), device="cpu")
    assert isinstance(m, Potosun) and len(m.config.layers) == 4


def test_synthetic_checkpoint_names_and_shapes():
    from potosun_helpers import CONFIGS, checkpoint
    _, sd = checkpoint(CONFIGS["mixed"])
    assert sd["l0.mix.q"].shape == (32, 40) and sd["l0.mix.k"].shape == (16, 40) and sd["l0.mix.v"].shape == (24, 40)
    assert sd["l0.mix.g"].shape == (48, 40) and sd["l0.mix.rel"].shape == (8, 4) and sd["l0.mix.k.norm"].shape == (8,) and "l0.mix.sink" not in sd
    assert "l0.mix.vmix" not in sd and sd["l1.mix.vmix"].shape == () and sd["l1.mix.sink"].shape == (6,) and "l1.mix.g" not in sd
    assert sd["l2.mix.q"].shape == (42, 40) and sd["l2.mix.dkv"].shape == (19, 40) and sd["l2.mix.dkv.norm"].shape == (11,)
    assert sd["l2.mix.uk"].shape == (18, 11) and sd["l2.mix.uv"].shape == (30, 11) and sd["l2.mix.g"].shape == (3, 40) and sd["l2.mix.o"].shape == (40, 30)
    assert "l4.norm2" not in sd and sd["l6.norm2"].shape == (40,) and sd["head"].shape == (90, 40)


@pytest.mark.parametrize("rows,far", [(8, 14), (8, 30.0), (16, 128), (16, 100), (32, 2048), (2, 40), (12, 7), (4, 3), (10, 160), (48, 81)])
def test_bias_table_by_distance_equals_the_bucket_function(rows, far):
    from oracle import potosun as O
    from umbrella_amd.models.config import bias_by_distance
    rel = torch.arange(rows, dtype=torch.float32)[:, None] + torch.tensor([0.0, 100.0])
    n = int(far) + 40
    tab = bias_by_distance(rel, float(far), max_len=n)
    for d in range(n):
        want = O.distance_bucket(d, rows, float(far))
        assert float(tab[0, min(d, tab.shape[1] - 1)]) == want and float(tab[1, min(d, tab.shape[1] - 1)]) == want + 100
    short = bias_by_distance(rel, float(far), max_len=3)                   # a table for short sequences only
    assert short.shape[1] <= 3 and torch.equal(short, tab[:, :short.shape[1]])


def test_distances_a_whole_number_of_steps_out():
    """far / half = 2^5 over 5 steps, 1.5^3 over 24: the distance half 2^k (half 1.5^k) opens its bucket"""
    from oracle import potosun as O
    from umbrella_amd.models.config import distance_buckets
    for rows, far, at in ((10, 160, {10: 6, 9: 5, 20: 7, 19: 6, 80: 9, 79: 8}), (48, 81, {36: 32, 35: 31, 54: 40, 53: 39})):
        b = distance_buckets(rows, float(far), far + 2)
        for n, want in at.items():
            assert int(b[n]) == want and O.distance_bucket(n, rows, float(far)) == want, (rows, n)


def test_rotation_tables_and_layouts():
    from oracle import potosun as O
    from potosun_helpers import YARN
    from umbrella_amd.models.config import rotary_table
    for rot in ({"dims": 8, "base": 200.0, "scaling": YARN}, {"dims": 24, "base": 5e5}, {"dims": 2, "base": 30.0, "scaling": dict(YARN, slow=0.4)}):
        want, mult = O.frequencies(rot)
        got, gm = rotary_table(rot["base"], rot["dims"], rot.get("scaling"))
        assert float(((got.double() - want) / want).abs().max()) < 1e-7 and abs(gm - mult) < 1e-12
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 7.0]]], dtype=torch.float64)
    pos, rot = torch.tensor([3]), {"dims": 4, "base": 100.0}
    c, s = [math.cos(3.0), math.cos(0.3)], [math.sin(3.0), math.sin(0.3)]
    inter = [1 * c[0] - 2 * s[0], 2 * c[0] + 1 * s[0], 3 * c[1] - 4 * s[1], 4 * c[1] + 3 * s[1], 7.0]
    half = [1 * c[0] - 3 * s[0], 2 * c[1] - 4 * s[1], 3 * c[0] + 1 * s[0], 4 * c[1] + 2 * s[1], 7.0]
    assert torch.allclose(O.rotate(x, pos, rot, True)[0, 0], torch.tensor(inter, dtype=torch.float64))
    assert torch.allclose(O.rotate(x, pos, rot, False)[0, 0], torch.tensor(half, dtype=torch.float64))


@pytest.mark.parametrize("name", ["mixed", "odd", "plain", "wide"])
def test_oracle_in_portions_equals_whole(name):
    from oracle import potosun as O
    from potosun_helpers import CONFIGS, checkpoint, tokens
    cfgd = CONFIGS[name]
    _, sd = checkpoint(cfgd, seed=3)
    toks = tokens(37, cfgd["vocab"], 1)
    whole, layers, _ = O.forward(cfgd, sd, toks)
    assert layers.shape == (len(cfgd["layers"]), 37, cfgd["width"]) and float(whole.abs().max()) < cfgd["logit_softcap"]
    rows, st, at = [], None, 0
    for k in (5, 1, 1, 9, 2, 19):
        lg, _, st = O.forward(cfgd, sd, toks[at:at + k], st)
        rows.append(lg)
        at += k
    assert float((torch.cat(rows) - whole).abs().max()) < 1e-9


def test_what_a_position_sees():
    from oracle import potosun as O
    assert [j for j in range(40) if O.sees_window(20, j, 5, 3)] == [0, 1, 2, 16, 17, 18, 19, 20]
    assert [j for j in range(40) if O.sees_window(2, j, 2, 9)] == [0, 1, 2]
    assert [j for j in range(40) if O.sees_window(7, j, 1)] == [7]
    assert [j for j in range(40) if O.sees_chunk(20, j, 8)] == [16, 17, 18, 19, 20] and [j for j in range(40) if O.sees_chunk(24, j, 8)] == [24]


def test_first_mixing_layer_keeps_its_own_values():
    """of two layers that mix, the first one's mixing number is not used, the second one's is"""
    from oracle import potosun as O
    from potosun_helpers import CONFIGS, checkpoint, tokens
    cfgd = CONFIGS["mixed"]
    _, sd = checkpoint(cfgd, seed=3)
    toks = tokens(9, cfgd["vocab"], 1)
    base = O.forward(cfgd, sd, toks)[0]
    same = O.forward(cfgd, dict(sd, **{"l1.mix.vmix": torch.tensor(5.0)}), toks)[0]
    other = O.forward(cfgd, dict(sd, **{"l3.mix.vmix": torch.tensor(0.9)}), toks)[0]
    assert torch.equal(base, same) and not torch.allclose(base, other)
