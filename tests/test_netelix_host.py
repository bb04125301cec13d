"""CPU: the host side of the Netelix integration — configuration reading, cache planes and state pieces, tensor names, the
model registry — and the float64 restatement's own mechanisms on cases worked out by hand."""
import json
import math

import pytest
import torch

import tests.netelix_oracle as oracle
from hydrainfer_amd.model.netelix import NetelixForCausalLM, NetelixShape, tensor_shapes

F = torch.float64


def _config(**over):
    cfg = {"architecture": "Netelix", "vocab": 33, "width": 24, "norm": {"eps": 1e-4}, "layers": [
        {"type": "lightning", "mixer": {"decay": [0.5, 0.9, 1.0], "dim": 5, "heads": 3, "vdim": 7}, "mlp": {"ff": 10, "kind": "dense"}},
        {"type": "attention", "mixer": {"dim": 8, "heads": 6, "kv_heads": 3, "scale": 0.25, "vdim": 12, "mask": {"size": 11},
                                        "rot": {"base": 500.0, "dims": 4}}, "mlp": None},
        {"type": "attention", "mixer": {"dim": 6, "heads": 2, "kv_heads": 2, "scale": 0.5, "vdim": 4, "v_mix": True, "mask": {"size": 3},
                                        "rot": {"base": 50.0, "dims": 6}}, "mlp": None},
        {"type": "retention", "mixer": {"decay": [0.75], "dim": 8, "heads": 1, "vdim": 3, "rot": {"base": 100.0, "dims": 8}}, "mlp": None},
        {"type": "attention", "mixer": {"dim": 4, "heads": 4, "kv_heads": 2, "scale": 0.5, "vdim": 4, "v_mix": True, "mask": {"size": 5},
                                        "rot": {"base": 50.0, "dims": 2}}, "mlp": {"ff": 6, "kind": "dense"}}]}
    cfg.update(over)
    return cfg


def test_shape_from_config_planes_pieces_and_names():
    sh = NetelixShape.from_config(_config())
    assert sh.cache_plane == {1: 0, 2: 1, 4: 2} and (sh.num_hidden_layers, sh.num_key_value_heads, sh.head_dim, sh.num_attention_heads) == (3, 3, 12, 6)
    assert sh.state_piece == {0: 0, 3: 108} and sh.state_floats == 108 + 24          # 3 x 5 x 7 rounded up to four floats
    m = sh.layers[1].mixer
    assert (m.window, m.rot.dims, m.rot.base, m.v_mix, m.scale) == (11, 4, 500.0, False, 0.25) and sh.layers[0].mixer.rot is None
    assert [l.ff for l in sh.layers] == [10, None, None, None, 6] and sh.norm_eps == 1e-4
    assert sh.to_config() == _config() and NetelixShape.from_config(sh.to_config()).to_config() == sh.to_config()
    names = tensor_shapes(sh)
    assert names["l0.mix.q"] == (15, 24) and names["l0.mix.v"] == names["l0.mix.g"] == (21, 24) and names["l0.mix.norm"] == (21,) and names["l0.mix.o"] == (24, 21)
    assert names["l1.mix.k"] == (24, 24) and names["l1.mix.v"] == (36, 24) and names["l1.mix.q.norm"] == (8,) and names["l1.mix.o"] == (24, 72)
    assert "l1.mix.vmix" not in names and names["l2.mix.vmix"] == names["l4.mix.vmix"] == () and "l3.mix.norm" not in names
    assert "l1.norm2" not in names and names["l4.norm2"] == names["l4.ls2"] == names["embed.norm"] == (24,) and names["l4.mlp.down"] == (24, 6)
    sd = NetelixForCausalLM.random_state_dict(sh, seed=1)
    assert set(sd) == set(names) and all(tuple(sd[k].shape) == v for k, v in names.items())


def test_configurations_without_attention_or_recurrence():
    cfg = _config()
    only = lambda *kinds: NetelixShape.from_config(_config(layers=[l for l in cfg["layers"] if l["type"] in kinds]))
    rec, att = only("lightning", "retention"), only("attention")
    assert rec.num_hidden_layers == 1 and rec.cache_plane == {} and rec.head_dim == 1 and rec.state_floats == 132
    assert att.state_floats == 0 and att.cache_plane == {0: 0, 1: 1, 2: 2}
    cfg["layers"][1]["mixer"].pop("mask"); cfg["layers"][1]["mixer"].pop("rot"); cfg["layers"][1]["mixer"].pop("kv_heads")
    m = NetelixShape.from_config(cfg).layers[1].mixer
    assert m.window is None and m.rot is None and m.kv_heads == 6


def test_configurations_that_cannot_be():
    with pytest.raises(ValueError):
        NetelixShape.from_config(_config(architecture="Other"))
    for change in (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), lambda c: c["layers"][0]["mixer"].update(decay=[0.5]),
                   lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10), lambda c: c["layers"][3]["mixer"]["rot"].update(dims=3),
                   lambda c: c["layers"][0].update(type="other"), lambda c: c["layers"][0]["mlp"].update(kind="moe"),
                   lambda c: c["layers"][4]["mixer"].update(vdim=8), lambda c: c["layers"][0]["mixer"].update(dim=257),
                   lambda c: c["layers"][3]["mixer"]["rot"].update(scaling={"factor": 2.0, "original": 64})):
        cfg = _config()
        change(cfg)
        with pytest.raises(ValueError):
            NetelixShape.from_config(cfg)


def test_registry_knows_the_design(tmp_path):
    from hydrainfer_amd.model.registry import architecture_of, registered
    (tmp_path / "config.json").write_text(json.dumps(_config()))
    assert architecture_of(str(tmp_path)) == "Netelix" and "Netelix" in registered()


def test_powers_of_decays():
    from hydrainfer_amd._C.kernel.decay_attn import CHUNK, decay_powers
    p = decay_powers([0.5, 0.0, 1.0, 1e-3], "cpu")
    assert p.shape == (4, CHUNK + 1) and p.dtype == torch.float32 and torch.all(p[:, 0] == 1.0)
    assert p[0, 5] == 0.5 ** 5 and torch.all(p[1, 1:] == 0.0) and torch.all(p[2] == 1.0) and p[3, CHUNK] == 0.0
    from hydrainfer_amd import _lib
    import os
    import re
    header = open(os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "include", "hydra_mix.h")).read()
    assert int(re.search(r"#define HXM_DECAY_CHUNK (\d+)", header).group(1)) == CHUNK
    assert int(re.search(r"#define HXM_ABI_VERSION (\d+)", header).group(1)) == _lib.HXM_ABI_VERSION


def test_restatement_rotations_and_decayed_sum_by_hand():
    quarter = torch.tensor([math.pi / 2], dtype=F)
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 9.0]]], dtype=F)
    assert torch.allclose(oracle.turned(x, quarter, 4, 1.0, False), torch.tensor([[[-3.0, -4.0, 1.0, 2.0, 9.0]]], dtype=F))
    assert torch.allclose(oracle.turned(x, quarter, 4, 1.0, True), torch.tensor([[[-2.0, 1.0, -4.0, 3.0, 9.0]]], dtype=F))
    assert torch.allclose(oracle.turned(x, quarter, 2, 1.0, True), torch.tensor([[[-2.0, 1.0, 3.0, 4.0, 9.0]]], dtype=F))
    one = torch.ones(3, 1, 1, dtype=F)
    o, S = oracle.decayed_sum(one, one * 2.0, torch.tensor([[[1.0]], [[10.0]], [[100.0]]], dtype=F), [0.5])
    assert torch.allclose(o[:, 0, 0], torch.tensor([2.0, 21.0, 210.5], dtype=F)) and S.item() == 210.5
    o2, _ = oracle.decayed_sum(one[:1], one[:1], one[:1], [0.5], S)
    assert o2.item() == 106.25


def test_restatement_window_norms_and_blend_by_hand():
    q = torch.zeros(3, 1, 2, dtype=F)
    v = torch.tensor([[[3.0]], [[9.0]], [[30.0]]], dtype=F)
    assert torch.allclose(oracle.attend(q, q, v, 1.0, None)[:, 0, 0], torch.tensor([3.0, 6.0, 14.0], dtype=F))
    assert torch.allclose(oracle.attend(q, q, v, 1.0, 2)[:, 0, 0], torch.tensor([3.0, 6.0, 19.5], dtype=F))
    assert torch.allclose(oracle.attend(q, q, v, 1.0, 1)[:, 0, 0], v[:, 0, 0])
    assert torch.allclose(oracle.over_rms(torch.tensor([3.0, 4.0], dtype=F), 0.0), torch.tensor([3.0, 4.0], dtype=F) / math.sqrt(12.5))
    assert oracle.mixed_values(torch.tensor(4.0), torch.tensor(8.0), torch.tensor(0.25)) == 5.0


def test_restatement_is_causal_and_blends_with_the_first_marked_layer():
    cfg = _config()
    sh = NetelixShape.from_config(cfg)
    W = {k: v.float() for k, v in NetelixForCausalLM.random_state_dict(sh, seed=2).items()}
    toks = [3, 1, 4, 1, 5, 9, 2, 6, 5, 3, 5, 8, 9, 7]
    trace = []
    logits = oracle.forward(cfg, W, toks, trace)
    assert logits.shape == (len(toks), 33) and len(trace) == 5 and torch.isfinite(logits).all()
    assert torch.allclose(oracle.forward(cfg, W, toks[:9]), logits[:9], atol=1e-12)
    assert torch.allclose(oracle.forward(cfg, dict(W, **{"l2.mix.vmix": torch.tensor(0.9)}), toks), logits, atol=1e-12)
    assert (oracle.forward(cfg, dict(W, **{"l4.mix.vmix": torch.tensor(0.9)}), toks) - logits).abs().max() > 1e-3
