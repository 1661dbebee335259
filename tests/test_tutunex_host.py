"""Host-side tests of the Tutunex design: configuration reading, registry, checkpoint names, the YaRN frequency table, the cache
layout of layers that share keys, and the plain oracle against itself in portions (no GPU)."""
import json
import os
import sys

import pytest
import torch

ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))
sys.path.insert(0, ROOT)
sys.path.insert(0, os.path.dirname(__file__))


def test_config_reading():
    from tutunex_helpers import CONFIGS
    from umbrella_amd.models import tutunex
    cfg = tutunex.config_from_dict(CONFIGS["mixed"])
    assert [ly.mixer.kind for ly in cfg.layers] == ["attention_delta", "diff_attention", "diff_attention", "attention_delta", "diff_attention"]
    assert cfg.embed_scale == 1.7 and cfg.norm_groups == 1 and cfg.block == "sequential" and cfg.streams == 0
    a, b = cfg.layers[1].mixer, cfg.layers[2].mixer
    assert (a.chunk, a.diff, a.kv_from, a.rot_dims, a.rot_scaling["fast"]) == (10, 0.4, None, 6, 8.0)
    assert (b.chunk, b.diff, b.kv_from, b.scale) == (7, 0.65, 1, 0.5)
    p = cfg.layers[0].mixer
    assert (p.s_heads, p.s_groups, p.s_state, p.s_vdim, p.s_taps, p.pair_coef) == (4, 2, 10, 7, 3, 0.5)
    assert not cfg.layers[3].has_ff and cfg.layers[4].act == "clamp_glu" and cfg.layers[4].act_limit == 0.6 and cfg.layers[4].act_alpha == 1.702
    with pytest.raises(ValueError):
        tutunex.config_from_dict(dict(CONFIGS["mixed"], layers=[{"type": "other", "mixer": {}, "mlp": None}]))


def test_registry_resolves_the_architecture(tmp_path):
    from tutunex_helpers import CONFIGS
    from umbrella_amd.models.auto_model import AutoModelLM
    from umbrella_amd.models.config import read_architecture
    from umbrella_amd.models.tutunex import Tutunex
    (tmp_path / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    assert read_architecture(str(tmp_path)) == "Tutunex"
    m = AutoModelLM.from_pretrained(str(tmp_path), device="cpu")
    assert isinstance(m, Tutunex) and len(m.config.layers) == 3


def test_synthetic_checkpoint_names_and_shapes():
    from tutunex_helpers import CONFIGS, checkpoint
    _, sd = checkpoint(CONFIGS["mixed"])
    assert sd["l1.mix.q"].shape == (64, 40) and sd["l1.mix.k"].shape == (32, 40) and sd["l1.mix.v"].shape == (24, 40)
    assert "l2.mix.k" not in sd and "l2.mix.v" not in sd and sd["l2.mix.q"].shape == (64, 40) and sd["l2.mix.lq1"].shape == (8,)
    assert sd["l0.mix.right.q"].shape == (20, 40) and sd["l0.mix.right.v.conv"].shape == (28, 3) and sd["l0.mix.right.norm"].shape == (7,)
    assert sd["l0.mix.left.out"].shape == (40,) and sd["l0.mix.left.k.norm"].shape == (8,) and sd["l0.mix.right.A_log"].shape == (4,)
    assert "l3.norm2" not in sd and "l3.norm2b" not in sd and sd["l3.norm1b"].shape == (40,) and sd["head"].shape == (90, 40)


@pytest.mark.parametrize("scaling", [None, {"factor": 2.0, "original": 4096, "fast": 32.0, "slow": 1.0}, {"factor": 16.0, "original": 64, "fast": 4.0, "slow": 0.25},
                                     {"factor": 1.0, "original": 300, "fast": 2.0, "slow": 1.9}, {"factor": 3.0, "original": 8, "fast": 40.0, "slow": 20.0}])
def test_yarn_table_equals_the_scalar_statement(scaling):
    from oracle import tutunex as O
    from umbrella_amd.models.config import rotary_table
    kinds = set()
    for dims, base in ((24, 250000.0), (6, 50.0), (64, 10000.0), (2, 7.0)):
        rot = {"dims": dims, "base": base}
        if scaling:
            rot["scaling"] = scaling
        want, mult = O.rotary_table(rot)
        got, gm = rotary_table(base, dims, scaling)
        assert got.dtype == torch.float32 and float(((got.double() - want) / want).abs().max()) < 1e-7 and abs(gm - mult) < 1e-12
        f = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
        r = (want / f).tolist()
        kinds |= {"kept" if abs(x - 1) < 1e-12 else ("slowed" if scaling and abs(x * scaling["factor"] - 1) < 1e-12 else "blended") for x in r}
    if scaling and scaling["original"] == 4096:
        assert kinds == {"kept", "slowed", "blended"}


def test_other_frequency_scalings_keep_their_table():
    from umbrella_amd.models.config import rotary_frequencies, rotary_table
    sc = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}
    f, mult = rotary_table(100.0, 16, sc)
    assert mult == 1.0 and torch.equal(f, rotary_frequencies(100.0, 16, sc))


@pytest.mark.parametrize("name", ["mixed", "odd", "plain", "wide"])
def test_oracle_in_portions_equals_whole(name):
    from oracle import tutunex as O
    from tutunex_helpers import CONFIGS, checkpoint, tokens
    cfgd = CONFIGS[name]
    _, sd = checkpoint(cfgd, seed=3)
    toks = tokens(37, cfgd["vocab"], 1)
    whole, layers, _ = O.forward(cfgd, sd, toks)
    assert layers.shape == (len(cfgd["layers"]), 37, cfgd["width"])
    rows, st, at = [], None, 0
    for k in (5, 1, 1, 9, 2, 19):
        lg, _, st = O.forward(cfgd, sd, toks[at:at + k], st)
        rows.append(lg)
        at += k
    assert float((torch.cat(rows) - whole).abs().max()) < 1e-9


def test_chunk_borders_cut_what_a_position_sees():
    """the plain attention itself: a marked value is read inside its own run of positions only, counted from position 0"""
    from oracle import tutunex as O
    n, chunk, mark = 30, 8, 11
    q, k, v = torch.ones(n, 2, 4), torch.ones(n, 1, 4), torch.zeros(n, 1, 3)
    v[mark] = 5.0
    o = O.softmax_attention(q, k, v, torch.arange(n), 1.0, chunk=chunk)[:, :, 0]
    seen = [i for i in range(n) if float(o[i].abs().max()) > 0]
    assert seen == [11, 12, 13, 14, 15]
    late = O.softmax_attention(q[12:], k, v, torch.arange(12, n), 1.0, chunk=chunk)[:, :, 0]
    assert torch.equal(late, o[12:])
    one = O.softmax_attention(q, k, torch.ones_like(v), torch.arange(n), 0.0, one_more=True)[:, 0, 0]
    assert torch.allclose(one, torch.tensor([(i + 1) / (i + 2) for i in range(n)]))
