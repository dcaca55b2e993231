"""The Rasesun configuration and registry on the CPU: keys read from config.json, refusals, the tensors a configuration
names, the order in which looped layers run, a model folder written and read back with its expert tables, and the plain
implementation's own mechanisms on small cases worked by hand."""

import copy
import math

import pytest
import torch

import plain_rasesun as pr
from bitwise_amd.config.llama import ConfigError
from bitwise_amd.config.rasesun import RasesunConfig
from bitwise_amd.model import describe, model_spec, write_random_model
from bitwise_amd.models.rasesun import TINY_RASESUN
from bitwise_amd.registry import ARCHITECTURES, architecture_of, read_model_config
from bitwise_amd.weights import loader


def test_registry_and_round_trip():
    arch = architecture_of(TINY_RASESUN)
    assert arch is ARCHITECTURES["Rasesun"] and arch.tiny_config is TINY_RASESUN
    cfg = RasesunConfig.from_dict(TINY_RASESUN)
    assert RasesunConfig.from_dict(cfg.to_dict()) == cfg
    assert cfg.layers[2].mlp is None and cfg.loop == (1, 3, 3) and cfg.embedding_scale == 2.5 and cfg.logit_softcap == 12.0
    bare = copy.deepcopy(TINY_RASESUN)
    bare.pop("loop")
    bare.pop("logit_softcap")
    bare["layers"][1]["mixer"].pop("mask")
    cfg = RasesunConfig.from_dict(bare)
    assert cfg.loop == (0, 0, 1) and cfg.logit_softcap is None and RasesunConfig.from_dict(cfg.to_dict()) == cfg
    spec = model_spec(bare)
    assert spec.lm_head.kind == "lm_head" and spec.layers[1].mixer.params["window"] is None


def test_order_of_layer_runs():
    assert RasesunConfig.from_dict(TINY_RASESUN).layer_runs() == [0, 1, 2, 1, 2, 1, 2, 3] == pr.layer_runs(TINY_RASESUN)
    spec = model_spec(TINY_RASESUN)
    assert [(c.layer, c.cache, c.adds_embedding) for c in spec.schedule] == [(i, n, False) for n, i in enumerate([0, 1, 2, 1, 2, 1, 2, 3])]
    for loop, runs in (((2, 2, 5), [0, 1, 2, 3]), ((0, 4, 2), [0, 1, 2, 3, 0, 1, 2, 3]), ((3, 4, 3), [0, 1, 2, 3, 3, 3]), ((0, 1, 1), [0, 1, 2, 3])):
        other = dict(TINY_RASESUN, loop=dict(zip(("start", "stop", "times"), loop)))
        assert [c.layer for c in model_spec(other).schedule] == runs == pr.layer_runs(other)


def test_tensor_names_and_parts():
    spec, t = model_spec(TINY_RASESUN), describe(TINY_RASESUN)
    assert t["embed"].shape == (97, 40) and t["head"].shape == (97, 40) and t["final.norm"].shape == (40,)
    for n in ("norm1", "norm1b", "norm2", "norm2b"):
        assert t["l0." + n].shape == (40,)
    assert "l2.norm2" not in t and "l2.norm2b" not in t and "l2.norm1b" in t
    # 4 heads of 12, two groups of state 8: z and x of 48, B and C of 16, 4 step sizes
    assert t["l0.mix.in"].shape == (2 * 48 + 2 * 16 + 4, 40) and t["l0.mix.conv"].shape == (48 + 32, 3) and t["l0.mix.conv.b"].shape == (80,)
    assert all(t["l0.mix." + n].shape == (4,) for n in ("dt_bias", "A_log", "D")) and t["l0.mix.norm"].shape == (48,) and t["l0.mix.o"].shape == (40, 48)
    assert t["l1.mix.dq"].shape == (16, 40) and t["l1.mix.dq.norm"].shape == (16,) and t["l1.mix.uq"].shape == (36, 16)
    assert t["l1.mix.dkv"].shape == (24, 40) and t["l1.mix.dkv.norm"].shape == (20,) and t["l1.mix.uk"].shape == (24, 20)
    assert t["l1.mix.uv"].shape == (36, 20) and t["l1.mix.g"].shape == (3, 40) and t["l1.mix.o"].shape == (40, 36)
    assert "l1.mix.sink" not in t and "l1.mix.q" not in t
    assert t["l1.mlp.up"].shape == (56, 40) and t["l1.mlp.down"].shape == (40, 56) and t["l1.mlp.act"].shape == (2,) and "l1.mlp.gate" not in t
    assert t["l0.mlp.table"].shape == (97, 2) and t["l0.mlp.table"].kind == "int" and t["l0.mlp.table"].below == 6
    assert t["l0.mlp.e5.up"].shape == (24, 40) and t["l0.mlp.e5.down"].shape == (40, 24) and "l0.mlp.e0.gate" not in t and "l0.mlp.router" not in t
    assert all(l.block == "sandwich" for l in spec.layers)
    assert spec.lm_head.kind == "lm_head_softcap" and spec.lm_head.params["cap"] == 12.0 and spec.embedding.params["scale"] == 2.5
    m = spec.layers[1].mixer.params
    assert m["window"] == 21 and m["gate"] and not m["sink"] and m["q_rank"] == 16 and m["position"].kind == "rope_pairs"


@pytest.mark.parametrize("change, what", [
    (lambda c: c.pop("embedding"), "embedding"),
    (lambda c: c.update(logit_softcap=0), "logit_softcap"),
    (lambda c: c["loop"].update(stop=5), "loop"),
    (lambda c: c["loop"].update(times=0), "loop"),
    (lambda c: c["layers"][0].update(type="mamba"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("state"), "state"),
    (lambda c: c["layers"][0]["mixer"].update(groups=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=5), "norm_groups"),
    (lambda c: c["layers"][1]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=6), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "experts"),
    (lambda c: c["layers"][0]["mlp"].pop("router"), "experts"),
    (lambda c: c["layers"][1]["mlp"].update(kind="gated"), "kind"),
])
def test_refusals(change, what):
    cfg = copy.deepcopy(TINY_RASESUN)
    change(cfg)
    with pytest.raises(ConfigError) as e:
        RasesunConfig.from_dict(cfg)
    assert what in str(e.value)


def test_a_model_folder_comes_back_and_tables_are_checked(tmp_path):
    folder = write_random_model(tmp_path / "m", TINY_RASESUN, 5, 0.1)
    raw = read_model_config(folder)
    assert RasesunConfig.from_dict(raw) == RasesunConfig.from_dict(TINY_RASESUN)
    specs = describe(raw)
    w = loader.load_folder(folder, specs)
    table = w["l3.mlp.table"]
    assert table.dtype == torch.int32 and table.shape == (97, 3) and int(table.min()) >= 0 and int(table.max()) == 4
    assert all(len(set(row)) == 3 for row in table.tolist())
    for bad in (5, -1):
        broken = dict(w, **{"l3.mlp.table": table.clone()})
        broken["l3.mlp.table"][7, 1] = bad
        with pytest.raises(loader.WeightError, match="l3.mlp.table"):
            loader.check_and_convert(specs, broken)
    twice = dict(w, **{"l3.mlp.table": table.clone()})
    twice["l3.mlp.table"][7, 1] = twice["l3.mlp.table"][7, 2]
    with pytest.raises(loader.WeightError, match="twice"):
        loader.check_and_convert(specs, twice)


def test_the_plain_mechanisms_by_hand():
    F = pr.F
    # the convolution: the last tap is the current token's, nothing before the start, the bias on top
    out = pr.causal_convolution(torch.tensor([[2.0], [3.0], [5.0]], dtype=F), torch.tensor([[10.0, 1.0]], dtype=F), torch.tensor([0.5], dtype=F))
    assert out.flatten().tolist() == [2.5, 23.5, 35.5]
    # the memory is read behind the update; the second head shares the first one's B and C
    x = torch.tensor([[[1.0], [2.0]], [[3.0], [5.0]]], dtype=F)
    B, C = torch.tensor([[[2.0]], [[7.0]]], dtype=F), torch.tensor([[[1.0]], [[0.5]]], dtype=F)
    dt = torch.tensor([[0.5, 1.0], [0.25, 2.0]], dtype=F)
    out = pr.ssd_recurrence(x, B, C, dt, torch.tensor([0.0, math.log(2.0)], dtype=F), torch.tensor([0.0, 10.0], dtype=F))
    assert abs(float(out[0, 0]) - 0.5 * 2 * 1) < 1e-12 and abs(float(out[0, 1]) - (1.0 * 2 * 2 + 20)) < 1e-12
    assert abs(float(out[1, 0]) - 0.5 * (math.exp(-0.25) * 1.0 + 0.25 * 7 * 3)) < 1e-12
    assert abs(float(out[1, 1]) - (0.5 * (math.exp(-4.0) * 4.0 + 2.0 * 7 * 5) + 50)) < 1e-12
    # the gate comes before the norm, and each part has a root mean square of its own
    y, z = torch.tensor([[1.0, 1.0, 100.0, 100.0]], dtype=F), torch.tensor([[0.0, 3.0, 3.0, 3.0]], dtype=F)
    out = pr.gated_part_norm(y, z, torch.ones(4, dtype=F), 2, 0.0)
    assert torch.allclose(out, torch.tensor([[0.0, math.sqrt(2.0), 1.0, 1.0]], dtype=F))
    # a window of 2: the third token sees itself and the one before
    q = torch.zeros(3, 1, 1, dtype=F)
    v = torch.tensor([[[1.0]], [[3.0]], [[5.0]]], dtype=F)
    assert pr.window_attention(q, q, v, 1.0, 2).flatten().tolist() == [1.0, 2.0, 4.0]
    # neighbours are turned together, the first pair by the position itself; what lies behind passes
    y = pr.rotate_pairs(torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]], dtype=F), 3, {"base": 100.0, "dims": 4})
    assert float(y[0, 0, 4]) == 5.0 and abs(float(y[0, 0, 0]) - (math.cos(3.0) - 2.0 * math.sin(3.0))) < 1e-12
    assert abs(float(y[0, 0, 2]) - (3.0 * math.cos(0.3) - 4.0 * math.sin(0.3))) < 1e-12
    # the activations: continuous at zero with slope 1/2, and the two sides' own numbers
    act = torch.tensor([0.3, -0.4], dtype=F)
    p, q = math.log1p(math.exp(0.3)), math.log1p(math.exp(-0.4))
    got = pr.xielu(torch.tensor([2.0, 0.0, -1.0], dtype=F), act).tolist()
    assert abs(got[0] - (4 * p + 1)) < 1e-12 and got[1] == 0.0 and abs(got[2] - ((0.5 + q) * (math.exp(-1) - 1 + 1) - 0.5)) < 1e-12
    assert pr.squared_relu(torch.tensor([-2.0, 3.0], dtype=F)).tolist() == [0.0, 9.0]
    # the table's row names the experts, each weighs 1 / top
    w = {"e0.up": torch.tensor([[1.0]]), "e0.down": torch.tensor([[1.0]]), "e1.up": torch.tensor([[2.0]]), "e1.down": torch.tensor([[1.0]]),
         "e2.up": torch.tensor([[3.0]]), "e2.down": torch.tensor([[1.0]])}
    w = dict(pr.to64(w), table=torch.tensor([[0, 1], [2, 0]], dtype=torch.int32))
    out = pr.table_moe(torch.tensor([[1.0], [1.0]], dtype=F), [1, 0], w, "", {"router": {"experts": 3, "top": 2}})
    assert out.flatten().tolist() == [(9 + 1) / 2, (1 + 4) / 2]
