"""Zumizen without a device: the plain implementation pinned by what fixes it beside its own text, the configuration's
checks, the tensors the model declares, and what its layers keep."""
from __future__ import annotations

import copy
import json
import math

import pytest
import torch

from plain import zumizen as pz
from zumizen_cases import CASES, folder_of

F64 = torch.float64


# ------------------------------------------------------------------------------------------ the plain implementation
def test_the_rows_of_token_pairs_and_the_scaled_embedding():
    assert pz.pair_row(None, 7, 37, 11, 5) == 37 and pz.pair_row(3, 7, 37, 11, 5) == (33 + 35) % 37
    w = {"embed": torch.arange(12, dtype=F64).view(6, 2), "bigram": 100.0 * torch.arange(10, dtype=F64).view(5, 2)}
    cfg = {"embedding": {"scale": 2.0, "bigram": {"buckets": 4, "mul_prev": 3, "mul_cur": 1}}}
    x = pz.embed(cfg, w, [5, 2, 2])
    assert x[0].tolist() == [20.0 + 800.0, 22.0 + 900.0]            # the first token: the last row; the table of pairs is not scaled
    assert x[1].tolist() == [8.0 + 200.0, 10.0 + 300.0]              # (15 + 2) mod 4 = 1
    assert x[2].tolist() == [8.0 + 0.0, 10.0 + 100.0]                # (6 + 2) mod 4 = 0
    assert pz.embed({"embedding": {"scale": 2.0}}, w, [1])[0].tolist() == [4.0, 6.0]


def test_the_distance_bias_grows_from_head_to_head_and_the_sink_makes_it_matter():
    assert pz.slopes(8).tolist() == [2.0 ** -(h + 1) for h in range(8)]
    assert pz.slopes(3)[0] == pytest.approx(2.0 ** (-8 / 3))
    torch.manual_seed(1)
    q, k = torch.randn(6, 4, 5, dtype=F64), torch.randn(6, 2, 5, dtype=F64)
    s = pz.biased_scores(q, k, 0.3)
    assert float(s[3, 5, 2]) == pytest.approx(float(q[5, 3] @ k[2, 1]) * 0.3 - 2.0 ** -8 * 3)
    assert float(s[0, 4, 4]) == pytest.approx(float(q[4, 0] @ k[4, 0]) * 0.3)
    p = pz.softmax_plus_one(s, pz.visible(6, 4))
    for h in range(4):
        for i in range(6):
            first = i // 4 * 4
            e = torch.exp(s[h, i, first:i + 1])
            assert p[h, i, first:i + 1].tolist() == pytest.approx((e / (1.0 + e.sum())).tolist())
            assert float(p[h, i, :first].abs().sum() + p[h, i, i + 1:].abs().sum()) == 0.0
    # the same scores less a number a row: another share of the sink
    far = pz.softmax_plus_one(s - 3.0, pz.visible(6, 4))
    assert float((far.sum(-1) / p.sum(-1)).max()) < 0.9


def test_visibility_in_runs_counted_from_the_first_position():
    see = pz.visible(12, 5)
    assert see[9, 5] and not see[10, 9] and see[10, 10] and not see[9, 10] and pz.visible(12)[11, 0]


def test_the_delta_rule_replaces_what_a_key_holds():
    """With beta 1 and no decay, reading a unit key gives the value written last under it, whatever stood there."""
    T, dk, dv = 6, 4, 3
    torch.manual_seed(2)
    keys = torch.linalg.qr(torch.randn(dk, dk, dtype=F64))[0]
    k = keys[[0, 1, 0, 2, 1, 0]].view(T, 1, dk)
    v = torch.randn(T, 1, dv, dtype=F64)
    ones, all_ = torch.ones(T, 1, dtype=F64), torch.ones(T, 1, dk, dtype=F64)
    q = keys[[0, 0, 0, 1, 0, 1]].view(T, 1, dk)                      # what is read at each position
    got = pz.delta_rule(q, k, v, all_, ones)[:, 0]
    want = [v[0, 0], v[0, 0], v[2, 0], v[1, 0], v[2, 0], v[4, 0]]    # (the read-out sees the current token's write)
    for t in range(T):
        assert torch.allclose(got[t], want[t], atol=1e-12), t
    # a decay on key channels alone: what stands under a channel fades, and a write of beta b moves it by b of the way
    eye = torch.eye(2, dtype=F64)
    g = torch.tensor([[[1.0, 1.0]], [[0.5, 0.1]]], dtype=F64)
    got = pz.delta_rule(eye[[0, 1]].view(2, 1, 2), eye[[1, 1]].view(2, 1, 2), torch.tensor([[[8.0]], [[4.0]]], dtype=F64), g,
                        torch.tensor([[1.0], [0.25]], dtype=F64))
    assert got[:, 0, 0].tolist() == pytest.approx([0.0, 0.8 + 0.25 * (4.0 - 0.8)])


def test_the_delta_rule_in_chunks_by_hand():
    """The recurrence against its closed form over a stretch of tokens: u = (I + A)^-1 (beta v - (beta e^G k) S0), which the
    chunked kernels use."""
    torch.manual_seed(3)
    T, dk, dv = 9, 5, 4
    q, k = torch.randn(T, 1, dk, dtype=F64), pz.unit_length(torch.randn(T, 1, dk, dtype=F64))
    v, beta = torch.randn(T, 1, dv, dtype=F64), torch.rand(T, 1, dtype=F64)
    lg = -torch.rand(T, 1, dk, dtype=F64) * 3
    out = pz.delta_rule(q, k, v, torch.exp(lg), beta)[:, 0]
    G = lg[:, 0].cumsum(0)
    D = torch.exp(G[:, None] - G[None])                              # [i, j, channel]
    A = torch.tril((k[:, 0][:, None] * k[:, 0][None] * D).sum(-1) * beta, -1)
    u = torch.linalg.solve(torch.eye(T, dtype=F64) + A, beta * v[:, 0])
    P = torch.tril((q[:, 0][:, None] * k[:, 0][None] * D).sum(-1))
    assert torch.allclose(P @ u, out, atol=1e-10)


def test_the_decays_lie_between_nothing_and_everything():
    torch.manual_seed(4)
    h = torch.randn(7, 6, dtype=F64)
    w = {"x.A_log": torch.tensor([-2.0, 1.0], dtype=F64), "x.a": torch.randn(2, 6, dtype=F64), "x.dt_bias": torch.tensor([0.5, -0.5], dtype=F64),
         "y.A_log": torch.tensor([-2.0, 1.0], dtype=F64), "y.a1": torch.randn(3, 6, dtype=F64), "y.a2": torch.randn(8, 3, dtype=F64),
         "y.dt_bias": torch.randn(8, dtype=F64)}
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 3}
    g = pz.head_decay(w, "x.", m, h)
    z = float(w["x.a"][1] @ h[3]) - 0.5
    assert g.shape == (7, 2, 4) and g[3, 1].tolist() == pytest.approx([math.exp(-math.e * math.log1p(math.exp(z)))] * 4)
    c = pz.channel_decay(w, "y.", m, h)
    z = float(w["y.a2"][6] @ (w["y.a1"] @ h[2]) + w["y.dt_bias"][6])
    assert float(c[2, 1, 2]) == pytest.approx(math.exp(-math.e * math.log1p(math.exp(z))))
    assert 0.0 < float(c.min()) < float(c.max()) < 1.0
    assert float(pz.softplus(torch.tensor(800.0, dtype=F64))) == 800.0 and float(pz.softplus(torch.tensor(-800.0, dtype=F64))) == 0.0


def test_the_experts_weights_multiply_what_they_read():
    torch.manual_seed(5)
    d, E, ff = 6, 4, 5
    w = {f"m.e{e}.{n}": torch.randn(*s, dtype=F64) for e in range(E) for n, s in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff)))}
    w["m.router"] = torch.randn(E, d, dtype=F64)
    x = torch.randn(9, d, dtype=F64)
    got = pz.experts(w, "m.", {"router": {"experts": E, "top": 2}}, x)
    for t in range(9):
        s = torch.sigmoid(w["m.router"] @ x[t])
        want = torch.zeros(d, dtype=F64)
        for e in s.argsort(descending=True)[:2].tolist():
            h = float(s[e]) * x[t]
            want = want + w[f"m.e{e}.down"] @ (pz.silu(w[f"m.e{e}.gate"] @ h) * (w[f"m.e{e}.up"] @ h))
        assert torch.allclose(got[t], want, atol=1e-12)
    ids, wts = pz.route(torch.tensor([[3.0, -1.0, 2.0]], dtype=F64), 2)
    assert ids[0].tolist() == [0, 2] and wts[0].tolist() == pytest.approx([1 / (1 + math.exp(-3)), 1 / (1 + math.exp(-2))])
    assert float(pz.route_margin(torch.tensor([[3.0, -1.0, 2.0]], dtype=F64), 2)) == 3.0
    assert float(pz.capped(torch.tensor(1000.0, dtype=F64), 15.0)) == pytest.approx(15.0) and float(pz.capped(torch.tensor(7.0), None)) == 7.0


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = str(tmp_path_factory.mktemp("zumizen"))
    return {name: folder_of(base, name) for name in CASES}


@pytest.mark.parametrize("name", list(CASES))
def test_causality_and_every_tensors_influence(folders, name):
    """A changed token moves no logits before it; each tensor moves some."""
    cfg, w = pz.load_folder(folders[name])
    vocab = cfg["vocab"]
    torch.manual_seed(5)
    toks = torch.randint(0, vocab, (30,)).tolist()
    base = pz.forward(cfg, w, toks)
    other = list(toks)
    other[11] = (toks[11] + 1) % vocab
    moved = pz.forward(cfg, w, other)
    assert torch.allclose(moved[:11], base[:11], atol=1e-12) and not torch.allclose(moved[11], base[11], atol=1e-6)
    assert not torch.allclose(moved[-1], base[-1], atol=1e-9)          # (a state reaches to the end)
    for n in w:
        if ".mlp.e" in n or (n.startswith("l3.mix.left") and name == "D"):
            continue      # (an expert may serve no token; that layer's left factor is 0)
        changed = dict(w)
        changed[n] = w[n] + 0.5 * torch.randn(w[n].shape, generator=torch.Generator().manual_seed(1), dtype=F64)
        assert not torch.allclose(pz.forward(cfg, changed, toks), base, atol=1e-7), n


# ------------------------------------------------------------------------------------------ configuration and model
def test_the_configuration_keeps_the_nested_keys_and_refuses_what_the_design_has_not():
    from glassbox_amd.config import ConfigError, config_from_dict
    for raw in CASES.values():
        cfg = config_from_dict(raw)
        assert cfg.architecture == "Zumizen" and config_from_dict(cfg.to_dict()) == cfg
    cfg = config_from_dict(CASES["B"])
    assert cfg.bigram is None and cfg.logit_softcap == 0.0 and cfg.embedding_scale == 0.7

    def broken(change):
        raw = copy.deepcopy(CASES["A"])
        change(raw)
        with pytest.raises(ConfigError):
            config_from_dict(raw)
    broken(lambda r: r["layers"][0]["mixer"]["left"].update(kv_heads=3))
    broken(lambda r: r["layers"][0]["mixer"]["right"].update(kv_heads=3))
    broken(lambda r: r["layers"][0]["mixer"].pop("right"))
    broken(lambda r: r["layers"][1]["mixer"].pop("heads"))
    broken(lambda r: r["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda r: r["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda r: r["layers"][0].update(type="attention"))
    broken(lambda r: r.update(logit_softcap=0.0))
    broken(lambda r: r["embedding"]["bigram"].pop("buckets"))
    broken(lambda r: r.pop("norm"))


def test_the_model_declares_the_checkpoints_tensors_and_what_its_layers_keep(folders):
    from glassbox_amd import ops
    from glassbox_amd.config import config_from_dict
    from glassbox_amd.engine.engine import check_supported
    from glassbox_amd.weights import SafetensorsFile
    from glassbox_amd.weights.loader import build_model, checkpoint_layout
    for name in CASES:
        model = build_model(config_from_dict(CASES[name]))
        _, shapes = checkpoint_layout(model)
        f = SafetensorsFile(folders[name] + "/model.safetensors")
        assert set(shapes) == set(f.names())
        f.close()
        for layer, spec, state in zip(CASES[name]["layers"], model.cache_specs(), model.state_specs()):
            m = layer["mixer"]
            if layer["type"] == "parallel":
                run = (m["left"].get("mask") or {"size": 0})["size"]
                assert spec.num_kv_heads == m["left"]["kv_heads"] and (spec.kind, spec.window) == ((2, run) if run else (0, 0))
                m = m["right"]
            else:
                assert spec is None
            floats, ring_at = ops.delta_slot(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"])
            channels = 2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"]
            assert ring_at >= m["heads"] * m["dim"] * m["vdim"] and floats >= ring_at + (m["conv"] * channels if m["conv"] > 1 else 0)
            assert tuple(state.shape) == (floats,) and state.dtype == torch.float32
        assert (model.embedding_cache is not None) == ("bigram" in CASES[name]["embedding"])
        check_supported(model, torch.float32, 16)
        check_supported(model, torch.bfloat16, 16)
    names = set(checkpoint_layout(build_model(config_from_dict(CASES["A"])))[1])
    assert {"embed", "bigram", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.left.q.b", "l0.mix.left.o.b", "l0.mix.left.q.norm",
            "l0.mix.right.A_log", "l0.mix.right.a", "l0.mix.right.g", "l0.mix.right.q.conv", "l1.mix.a1", "l1.mix.g2", "l1.mix.dt_bias",
            "l0.mlp.e5.gate", "l0.mlp.router"} <= names
    assert not {"l0.mix.left.g", "l0.mix.right.a1", "l1.mix.a", "l3.norm2", "l0.mlp.correction", "l0.mlp.shared.up"} & names


def test_middles_that_only_the_checkpoint_gives(tmp_path):
    """Without the optional keys the narrow middles are as wide as the file's tensors."""
    from glassbox_amd.config import config_from_dir
    from glassbox_amd.weights.loader import build_model
    folder = folder_of(str(tmp_path), "A")
    raw = json.load(open(folder + "/config.json"))
    for layer in raw["layers"]:
        layer["mixer"].pop("decay_rank", None), layer["mixer"].pop("gate_rank", None)
    json.dump(raw, open(folder + "/config.json", "w"))
    specs = dict(build_model(config_from_dir(folder)).named_specs())
    assert specs["l1.mix.a1"].shape == (-1, 64) and specs["l1.mix.g2"].shape == (32, -1)


def test_parts_refuse_what_they_do_not_serve():
    from glassbox_amd.parts.attention import GatedAttention
    from glassbox_amd.parts.delta_rule import GatedDeltaRule
    from glassbox_amd.parts.moe import RoutedExperts
    from glassbox_amd.parts.side_by_side import SideBySide
    with pytest.raises(ValueError):
        GatedDeltaRule(64, 3, 2, 16, 16, 4, 1e-5)
    with pytest.raises(ValueError):
        GatedDeltaRule(64, 2, 2, 16, 16, 4, 1e-5, decay="channel", gate="full")
    with pytest.raises(ValueError):
        SideBySide(GatedDeltaRule(64, 2, 2, 16, 16, 4, 1e-5), GatedDeltaRule(64, 2, 2, 16, 16, 4, 1e-5))
    with pytest.raises(ValueError):
        RoutedExperts(64, 4, 2, 16, shared_ff=8, weigh_in=True)
    with pytest.raises(ValueError):
        GatedAttention(64, 2, 2, 16, 16, 0.25, 1e-5, gate="row")
    wide = GatedDeltaRule(64, 2, 2, 300, 16, 9, 1e-5)
    assert {a for a, _ in wide.problems(torch.bfloat16, 16)} == {"dim", "taps"}
