"""The Nuzinex configuration and registry on the CPU: keys read from config.json, refusals, the tensors a configuration names,
shared caches and their windows, a model folder written and read back, and the plain implementation's own mechanisms on
small cases worked by hand."""

import copy
import math

import pytest
import torch

import plain_nuzinex as pn
from bitwise_amd.config.llama import ConfigError
from bitwise_amd.config.nuzinex import NuzinexConfig
from bitwise_amd.model import describe, model_spec, write_random_model
from bitwise_amd.models.nuzinex import TINY_NUZINEX
from bitwise_amd.registry import ARCHITECTURES, architecture_of, read_model_config
from bitwise_amd.weights import loader


def test_registry_and_round_trip():
    arch = architecture_of(TINY_NUZINEX)
    assert arch is ARCHITECTURES["Nuzinex"] and arch.tiny_config is TINY_NUZINEX
    cfg = NuzinexConfig.from_dict(TINY_NUZINEX)
    assert NuzinexConfig.from_dict(cfg.to_dict()) == cfg
    assert cfg.side_dim == 8 and cfg.eps == 1e-5 and cfg.layers[1].mlp is None and cfg.layers[0].mlp["ff"] == 56
    bare = copy.deepcopy(TINY_NUZINEX)
    bare.pop("max_positions")
    bare.pop("eos_token_id")
    cfg = NuzinexConfig.from_dict(bare)
    assert cfg.max_positions == 1 << 16 and cfg.eos_token_id == -1 and cfg.bos_token_id == -1


def test_spec_follows_the_configuration():
    spec = model_spec(TINY_NUZINEX)
    assert [(c.layer, c.cache, c.writes_cache) for c in spec.schedule] == [(0, 0, True), (1, 1, True), (2, 2, True), (3, 0, False)]
    a, r = spec.layers[0].mixer, spec.layers[3].mixer
    assert a.kind == r.kind == "gated_attention" and a.params["bias"] and not a.params["gate"] and a.params["position"].kind == "rope_pairs"
    # the reader looks further back than the layer that owns the cache: both keep the wider window, each attends through its own
    assert (a.params["window"], r.params["window"]) == (11, 19) and a.params["cache_window"] == r.params["cache_window"] == 19
    p = spec.layers[2].mixer
    assert p.kind == "side_by_side" and p.params["scales"] == [0.7, 0.4]
    (_, left), (_, right) = p.params["branches"]
    assert left.params["window"] is None and left.params["gate"] and left.params["position"].kind == "rope_halves" and "bias" not in left.params
    assert right.kind == "gated_delta" and right.params["kv_heads"] == 2 and right.params["unit_eps"] == 1e-6
    assert [l.parts["side_input"].params["offset"] for l in spec.layers] == [0, 8, 16, 24]
    assert all("feed_forward" in l.parts for l in (spec.layers[0], spec.layers[2])) and "ffn_norm" not in spec.layers[1].parts


@pytest.mark.parametrize("own,reader,kept", [(11, 19, 19), (19, 11, 19), (7, None, None), (None, 7, None), (5, 5, 5)])
def test_cache_windows_cover_every_reader(own, reader, kept):
    d = copy.deepcopy(TINY_NUZINEX)
    for i, w in ((0, own), (3, reader)):
        m = d["layers"][i]["mixer"]
        m.pop("mask")
        if w is not None:
            m["mask"] = {"size": w}
    spec = model_spec(d)
    assert [spec.layers[i].mixer.params["cache_window"] for i in (0, 3)] == [kept, kept]
    assert [spec.layers[i].mixer.params["window"] for i in (0, 3)] == [own, reader]
    from bitwise_amd.models.assembled import AssembledModel
    from bitwise_amd.runtime import Runtime
    model = AssembledModel(spec, Runtime("float32", device=None))
    assert model.calls[0].group == model.calls[3].group and model.group_specs[model.calls[0].group].window == kept


def test_tensor_names():
    t = describe(TINY_NUZINEX)
    assert t["embed"].shape == (93, 40) and t["head"].shape == (93, 40) and t["side.embed"].shape == (93, 32) and t["final.norm"].shape == (40,)
    for i in range(4):
        assert t[f"l{i}.norm1"].shape == t[f"l{i}.ls1"].shape == t[f"l{i}.side.norm"].shape == (40,)
        assert t[f"l{i}.side.gate"].shape == (8, 40) and t[f"l{i}.side.proj"].shape == (40, 8)
    assert "l1.norm2" not in t and "l1.ls2" not in t and t["l0.ls2"].shape == (40,)
    for n, rows in (("q", 64), ("k", 32), ("v", 16)):
        assert t[f"l0.mix.{n}"].shape == (rows, 40) and t[f"l0.mix.{n}.b"].shape == (rows,)
    assert t["l0.mix.q.norm"].shape == (64,) and t["l0.mix.k.norm"].shape == (32,) and t["l0.mix.o"].shape == (40, 32) and "l0.mix.g" not in t
    assert t["l3.mix.q.b"].shape == (96,) and not any(f"l3.mix.{n}" in t for n in ("k", "v", "k.b", "v.b", "k.norm"))
    left, right = "l2.mix.left.", "l2.mix.right."
    assert t[left + "g"].shape == (48, 40) and t[left + "o"].shape == (40, 48) and left + "q.b" not in t
    assert t[right + "q"].shape == t[right + "k"].shape == (16, 40) and t[right + "v"].shape == t[right + "g"].shape == (80, 40)
    assert t[right + "q.conv"].shape == (16, 3) and t[right + "v.conv"].shape == (80, 3) and t[right + "norm"].shape == (20,)
    assert all(t[right + n].shape == (4,) for n in ("A_log", "dt_bias")) and t[right + "a"].shape == t[right + "b"].shape == (4, 40)
    assert "l2.mix.left.out" not in t
    assert t["l1.mix.norm"].shape == (36,) and t["l1.mix.k"].shape == (24, 40) and t["l1.mix.g"].shape == (36, 40)
    assert t["l0.mlp.up"].shape == (56, 40) and t["l0.mlp.down"].shape == (40, 56) and "l0.mlp.gate" not in t


BROKEN = {
    "no architecture": lambda d: d.pop("architecture"),
    "no eps": lambda d: d["norm"].pop("eps"),
    "no side": lambda d: d.pop("token_side"),
    "side dim 0": lambda d: d["token_side"].update(dim=0),
    "no layers": lambda d: d.update(layers=[]),
    "unknown type": lambda d: d["layers"][0].update(type="mamba2"),
    "no mixer": lambda d: d["layers"][0].pop("mixer"),
    "heads not a multiple": lambda d: d["layers"][0]["mixer"].update(kv_heads=3),
    "odd rotation": lambda d: d["layers"][0]["mixer"]["rot"].update(dims=7),
    "rotation beyond the head": lambda d: d["layers"][0]["mixer"]["rot"].update(dims=18),
    "no scale": lambda d: d["layers"][0]["mixer"].pop("scale"),
    "scale 0": lambda d: d["layers"][0]["mixer"].update(scale=0.0),
    "window 0": lambda d: d["layers"][0]["mixer"]["mask"].update(size=0),
    "kv_from a later layer": lambda d: d["layers"][0]["mixer"].update(kv_from=3),
    "kv_from another kind": lambda d: d["layers"][3]["mixer"].update(kv_from=1),
    "kv_from other heads": lambda d: d["layers"][3]["mixer"].update(kv_heads=6),
    "no left": lambda d: d["layers"][2]["mixer"].pop("left"),
    "no right scale": lambda d: d["layers"][2]["mixer"].pop("right_scale"),
    "delta heads": lambda d: d["layers"][2]["mixer"]["right"].update(kv_heads=3),
    "no taps": lambda d: d["layers"][2]["mixer"]["right"].pop("conv"),
    "decay count": lambda d: d["layers"][1]["mixer"].update(decay=[0.5]),
    "decay beyond 1": lambda d: d["layers"][1]["mixer"].update(decay=[0.5, 0.6, 1.5]),
    "mlp kind": lambda d: d["layers"][0]["mlp"].update(kind="moe"),
    "no ff": lambda d: d["layers"][0]["mlp"].pop("ff"),
}


@pytest.mark.parametrize("what", list(BROKEN))
def test_refusals(what):
    d = copy.deepcopy(TINY_NUZINEX)
    BROKEN[what](d)
    with pytest.raises(ConfigError):
        NuzinexConfig.from_dict(d)


def test_a_reader_of_a_reader_is_refused():
    d = copy.deepcopy(TINY_NUZINEX)
    d["layers"].append(copy.deepcopy(d["layers"][3]))
    NuzinexConfig.from_dict(d)                        # two readers of one cache
    d["layers"][4]["mixer"]["kv_from"] = 3
    with pytest.raises(ConfigError):
        NuzinexConfig.from_dict(d)


def test_folder_round_trip(tmp_path):
    folder = write_random_model(tmp_path / "m", TINY_NUZINEX, 3, 0.1)
    raw = read_model_config(folder)
    assert NuzinexConfig.from_dict(raw) == NuzinexConfig.from_dict(TINY_NUZINEX)
    tensors = loader.load_folder(folder, describe(raw))
    assert set(tensors) == set(describe(TINY_NUZINEX)) and tensors["l2.mix.right.A_log"].dtype == torch.bfloat16
    toks = [5, 9, 0, 92, 17]
    lg = pn.forward(raw, pn.to64(tensors), toks)
    assert lg.shape == (5, 93) and torch.isfinite(lg).all()
    # causal: a later token does not move an earlier row
    assert torch.allclose(pn.forward(raw, pn.to64(tensors), toks[:3]), lg[:3], atol=1e-12)


# ----------------------------------------------------------------------------- the plain mechanisms by hand

def test_plain_delta_by_hand():
    D = lambda *x: torch.tensor(x, dtype=pn.F)
    # one head of one channel: S1 = b1 k1 v1; S2 = a2 S1 + k2 b2 (v2 - a2 S1 k2)
    q, k, v = D(1.0, 2.0).view(2, 1, 1), D(0.5, 0.25).view(2, 1, 1), D(3.0, -1.0).view(2, 1, 1)
    g, b = D(0.9, 0.5).view(2, 1), D(0.4, 0.6).view(2, 1)
    s1 = 0.5 * 0.4 * 3.0
    s2 = 0.5 * s1 + 0.25 * 0.6 * (-1.0 - 0.5 * s1 * 0.25)
    assert torch.allclose(pn.delta_recurrence(q, k, v, g, b).flatten(), D(s1, 2.0 * s2))
    # a step size of 1 and unit keys: what a key reads is exactly what was last written for it, whatever came before
    k = torch.eye(3, dtype=pn.F)[[0, 1, 0]].view(3, 1, 3)
    v = torch.randn(3, 1, 2, dtype=pn.F, generator=torch.Generator().manual_seed(0))
    one = torch.ones(3, 1, dtype=pn.F)
    assert torch.allclose(pn.delta_recurrence(k, k, v, one, one), v)


def test_plain_fading_rotation_and_activations_by_hand():
    D = lambda *x: torch.tensor(x, dtype=pn.F)
    out = pn.fading_recurrence(D(1.0, 1.0).view(2, 1, 1), D(2.0, 3.0).view(2, 1, 1), D(5.0, 7.0).view(2, 1, 1), [0.5])
    assert torch.allclose(out.flatten(), D(10.0, 26.0))
    x = D(1.0, 2.0, 3.0, 4.0, 5.0).view(1, 1, 5)
    a0, a1 = 2.0, 2.0 * 100.0 ** -0.5
    turn = lambda u, v, a: (u * math.cos(a) - v * math.sin(a), v * math.cos(a) + u * math.sin(a))
    (p, q), (r, s) = turn(1.0, 2.0, a0), turn(3.0, 4.0, a1)
    assert torch.allclose(pn.rotate(x, 2, {"base": 100.0, "dims": 4}, True).flatten(), D(p, q, r, s, 5.0))
    (p, r), (q, s) = turn(1.0, 3.0, a0), turn(2.0, 4.0, a1)
    assert torch.allclose(pn.rotate(x, 2, {"base": 100.0, "dims": 4}, False).flatten(), D(p, q, r, s, 5.0))
    z = D(-2.0, 0.0, 0.5)
    assert torch.allclose(pn.gelu_erf(z), torch.nn.functional.gelu(z)) and torch.allclose(pn.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert torch.allclose(pn.unit(D(3.0, 4.0)), D(0.6, 0.8), atol=1e-7)


def test_plain_window_by_hand():
    q = torch.zeros(4, 1, 1, dtype=pn.F)
    v = torch.tensor([1.0, 2.0, 4.0, 8.0], dtype=pn.F).view(4, 1, 1)
    mean = lambda w: pn.softmax_attention(q, q, v, 1.0, w).flatten().tolist()
    assert mean(None) == pytest.approx([1.0, 1.5, 7 / 3, 15 / 4]) and mean(2) == pytest.approx([1.0, 1.5, 3.0, 6.0]) and mean(1) == pytest.approx([1, 2, 4, 8])
