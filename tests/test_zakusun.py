"""Zakusun without a device: the plain implementation pinned by what fixes it beside its own text, the configuration's
checks, and the tensors, cache layers and state the model declares."""
from __future__ import annotations

import copy
import math

import pytest
import torch

from plain import zakusun as pz
from zakusun_cases import CASES, folder_of

F64 = torch.float64


# ------------------------------------------------------------------------------------------ the plain implementation
def test_the_position_vector_by_hand():
    out = pz.sinusoid(torch.tensor([0, 1, 7]), 6)
    assert out[0].tolist() == [0.0, 1.0, 0.0, 1.0, 0.0, 1.0]
    for t, p in ((1, 1), (2, 7)):
        for i in range(3):
            ang = p / 10000.0 ** (2 * i / 6)
            assert out[t, 2 * i] == pytest.approx(math.sin(ang)) and out[t, 2 * i + 1] == pytest.approx(math.cos(ang))
    # a shift of the position turns every pair by a fixed angle
    a, b = pz.sinusoid(torch.tensor([5, 9]), 4), pz.sinusoid(torch.tensor([105, 109]), 4)
    assert (a[0] * a[1]).sum() == pytest.approx(float((b[0] * b[1]).sum()))
    assert pz.sinusoid(torch.tensor([3]), 5)[0, 4] == pytest.approx(math.sin(3 * 10000.0 ** (-4 / 5)))   # an odd width ends on a sine


def test_the_norm_divides_every_group_by_its_own_root_mean_square():
    x = torch.tensor([[3.0, 4.0, 0.0, 0.0, 1.0, -1.0]], dtype=F64)
    w = torch.tensor([1.0, 2.0, 5.0, 5.0, -1.0, 3.0], dtype=F64)
    out = pz.group_norm(x, w, 3, 0.0 + 1e-12)
    r = math.sqrt(12.5)
    assert out[0].tolist() == pytest.approx([3 / r, 8 / r, 0.0, 0.0, -1.0, -3.0])
    assert torch.allclose(pz.group_norm(x, torch.ones(6, dtype=F64), 1, 0.5), x / math.sqrt(27 / 6 + 0.5))   # eps inside the root
    big = x.clone()
    big[0, 0] *= 100.0      # another group's size changes nothing
    assert torch.allclose(pz.group_norm(big, w, 3, 1e-12)[0, 2:], out[0, 2:])


def test_what_a_sublayer_reads_is_the_row_plus_a_causal_correlation():
    torch.manual_seed(0)
    x, taps = torch.randn(11, 5, dtype=F64), torch.randn(5, 4, dtype=F64)
    want = x + torch.nn.functional.conv1d(torch.nn.functional.pad(x.t()[None], (3, 0)), taps[:, None, :], groups=5)[0].t()
    assert torch.allclose(pz.with_conv(x, taps), want, atol=1e-12)
    one = torch.zeros(6, 1, dtype=F64)
    one[2] = 1.0     # the last tap weighs the token itself, the first the oldest
    assert pz.with_conv(one, torch.tensor([[1.0, 10.0, 100.0]], dtype=F64))[:, 0].tolist() == [0.0, 0.0, 101.0, 10.0, 1.0, 0.0]


def test_the_sum_over_depth_weighs_the_results_before_any_sum():
    hist = [torch.full((2, 3), float(v), dtype=F64) for v in (1.0, 10.0, 100.0)]
    assert torch.equal(pz.depth_average(torch.tensor([2.0, -1.0, 0.5], dtype=F64), hist), torch.full((2, 3), 42.0, dtype=F64))


def test_the_sink_takes_its_share_and_gives_nothing():
    torch.manual_seed(2)
    T, H = 7, 3
    s = torch.randn(H, T, T, dtype=F64)
    sink = torch.tensor([0.0, 2.0, -30.0], dtype=F64)
    p = pz.softmax_with_sink(s, sink)
    for h in range(H):
        for i in range(T):
            e = torch.exp(s[h, i, :i + 1])
            assert p[h, i, :i + 1].tolist() == pytest.approx((e / (e.sum() + math.exp(float(sink[h])))).tolist())
            assert float(p[h, i, i + 1:].abs().sum()) == 0.0
    assert float(p[2].sum(-1).min()) == pytest.approx(1.0) and float(p[1].sum(-1).max()) < 0.95


def test_queries_taken_into_the_latents_space_give_the_same_attention():
    torch.manual_seed(4)
    d, T = 20, 9
    m = {"heads": 3, "dim": 5, "vdim": 7, "kv_rank": 11, "scale": 0.7}
    r = lambda *s: torch.randn(*s, dtype=F64)
    w = {"x.q": r(15, d), "x.dkv": r(11, d), "x.dkv.norm": r(11), "x.uk": r(15, 11), "x.uv": r(21, 11), "x.sink": r(3), "x.g": r(21, d),
         "x.o": r(d, 21)}
    h = r(T, d)
    a, b = pz.latent_attention(w, "x.", m, 1e-5, h), pz.latent_attention_absorbed(w, "x.", m, 1e-5, h)
    assert torch.allclose(a, b, atol=1e-10)
    # one token: the softmax over its own key and the sink, written out
    c = h[:1] @ w["x.dkv"].T
    c = c / torch.sqrt((c ** 2).mean() + 1e-5) * w["x.dkv.norm"]
    o = torch.zeros(21, dtype=F64)
    for k in range(3):
        s = float((h[0] @ w["x.q"][5 * k:5 * k + 5].T) @ (w["x.uk"][5 * k:5 * k + 5] @ c[0])) * 0.7
        share = math.exp(s) / (math.exp(s) + math.exp(float(w["x.sink"][k])))
        o[7 * k:7 * k + 7] = share * (w["x.uv"][7 * k:7 * k + 7] @ c[0])
    o = o * torch.sigmoid(w["x.g"] @ h[0])
    assert torch.allclose(a[0], w["x.o"] @ o, atol=1e-10)


def test_the_router_chooses_by_logits_and_weighs_by_their_softmax():
    z = torch.tensor([[2.0, -1.0, 1.0, 3.0, 0.0]], dtype=F64)
    ids, wts = pz.route(z, 2)
    assert ids[0].tolist() == [3, 0] and float(wts.sum()) == pytest.approx(1.0)
    assert wts[0].tolist() == pytest.approx([math.e / (1 + math.e), 1 / (1 + math.e)])
    assert float(pz.route_margin(z, 2)) == pytest.approx(1.0) and math.isinf(float(pz.route_margin(z, 5)))
    assert torch.allclose(pz.route(z, 5)[1].sort().values, torch.softmax(z, -1).sort().values)


def test_clamped_units_by_hand_and_the_experts_weighted_sum():
    torch.manual_seed(3)
    d, E, ff, limit = 6, 4, 5, 0.6
    w = {f"m.e{e}.{n}": torch.randn(*s, dtype=F64) for e in range(E) for n, s in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff)))}
    w.update({"m.router": torch.randn(E, d, dtype=F64), "m.router.b": torch.randn(E, dtype=F64) * 3})
    mlp = {"expert": {"ff": ff, "limit": limit}, "router": {"experts": E, "top": 2}}
    x = torch.randn(9, d, dtype=F64)

    def unit(e, v):
        out = torch.zeros(d, dtype=F64)
        for j in range(ff):
            g, u = float(w[f"m.e{e}.gate"][j] @ v), float(w[f"m.e{e}.up"][j] @ v)
            g, u = min(g, limit), max(-limit, min(u, limit))          # the gate is not bounded from below
            out += w[f"m.e{e}.down"][:, j] * (g / (1 + math.exp(-1.702 * g)) * (u + 1))
        return out
    got = pz.experts(w, "m.", mlp, x)
    ids, wts = pz.route(x @ w["m.router"].T + w["m.router.b"], 2)
    for t in range(9):
        want = sum(float(a) * unit(e, x[t]) for e, a in zip(ids[t].tolist(), wts[t]))
        assert torch.allclose(got[t], want, atol=1e-12)
    plain, _ = pz.route(x @ w["m.router"].T, 2)
    assert not torch.equal(ids.sort(-1).values, plain.sort(-1).values)     # the bias takes part in the choice


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = str(tmp_path_factory.mktemp("zakusun"))
    return {name: folder_of(base, name) for name in CASES}


@pytest.mark.parametrize("name", list(CASES))
def test_every_layer_is_causal_and_reaches_everything_before(folders, name):
    cfg, w = pz.load_folder(folders[name])
    torch.manual_seed(5)
    toks = torch.randint(0, cfg["vocab"], (40,)).tolist()
    base = pz.forward(cfg, w, toks)
    other = list(toks)
    other[11] = (toks[11] + 1) % cfg["vocab"]
    moved = pz.forward(cfg, w, other)
    assert torch.allclose(moved[:11], base[:11], atol=1e-12) and not torch.allclose(moved[11], base[11], atol=1e-6)
    assert not torch.allclose(moved[-1], base[-1], atol=1e-9)
    # every tensor matters
    for key in ("l0.dwa", "l0.mix.sink", "l0.norm1", "l1.mix.dkv.norm"):
        ww = dict(w)
        ww[key] = w[key] + 0.1
        assert not torch.allclose(pz.forward(cfg, ww, toks), base, atol=1e-6), key


# ------------------------------------------------------------------------------------------ configuration and model
def test_the_configuration_keeps_the_nested_keys_and_refuses_what_the_design_has_not():
    from glassbox_amd.config import ConfigError, config_from_dict
    for raw in CASES.values():
        cfg = config_from_dict(raw)
        assert cfg.architecture == "Zakusun" and config_from_dict(cfg.to_dict()) == cfg
    cfg = config_from_dict(CASES["A"])
    assert (cfg.norm_groups, cfg.canon_taps, cfg.logit_scale, cfg.norm_eps) == (3, 3, 0.5, 1e-5)
    assert config_from_dict(CASES["E"]).canon_taps == 0

    def broken(change):
        raw = copy.deepcopy(CASES["A"])
        change(raw)
        with pytest.raises(ConfigError):
            config_from_dict(raw)
    broken(lambda r: r["norm"].update(groups=5))                        # 96 channels in five groups
    broken(lambda r: r["norm"].update(eps=0.0))
    broken(lambda r: r.pop("norm"))
    broken(lambda r: r["layers"][0]["mixer"].pop("kv_rank"))
    broken(lambda r: r["layers"][0]["mixer"].update(heads=0))
    broken(lambda r: r["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda r: r["layers"][0]["mlp"]["expert"].update(limit=-1.0))
    broken(lambda r: r["layers"][0]["mlp"]["expert"].pop("limit"))
    broken(lambda r: r["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda r: r["layers"][0].update(type="attention"))
    broken(lambda r: r.update(layers=[]))


def test_the_model_declares_the_checkpoints_tensors_one_latent_a_position_and_the_convolutions_rows(folders):
    from glassbox_amd.config import config_from_dict
    from glassbox_amd.engine.engine import check_supported, sharing_obstacles
    from glassbox_amd.weights import SafetensorsFile
    from glassbox_amd.weights.loader import build_model, checkpoint_layout
    for name, raw in CASES.items():
        model = build_model(config_from_dict(raw))
        _, shapes = checkpoint_layout(model)
        f = SafetensorsFile(folders[name] + "/model.safetensors")
        assert set(shapes) == set(f.names())
        f.close()
        taps = (raw.get("canon") or {"taps": 0})["taps"]
        assert model.num_cache_layers == len(raw["layers"])
        for i, layer in enumerate(raw["layers"]):
            spec, state = model.cache_specs()[i], model.state_specs()[i]
            assert (spec.num_kv_heads, spec.head_dim, spec.values) == (1, layer["mixer"]["kv_rank"], False)
            if taps > 1:
                assert tuple(state.shape) == (1 if layer["mlp"] is None else 2, taps - 1, raw["width"]) and state.dtype == torch.float32
            else:
                assert state is None
            assert tuple(shapes[f"l{i}.dwa"]) == (i + 2,)
        check_supported(model, torch.float32, 16)
        check_supported(model, torch.bfloat16, 16)
        assert bool(sharing_obstacles(model)) == (taps > 1)
    names = set(checkpoint_layout(build_model(config_from_dict(CASES["A"])))[1])
    assert {"embed", "l0.norm1", "l0.norm2", "l0.canon1", "l0.canon2", "l0.mix.q", "l0.mix.dkv", "l0.mix.dkv.norm", "l0.mix.uk", "l0.mix.uv",
            "l0.mix.sink", "l0.mix.g", "l0.mix.o", "l0.mlp.e5.gate", "l0.mlp.router", "l0.mlp.router.b", "l2.dwa", "final.norm"} <= names
    assert not {"l2.norm2", "l2.canon2", "head", "l0.mlp.e6.up", "l3.dwa"} & names


def test_sizes_beyond_the_kernels_are_refused_when_the_engine_is_built():
    from glassbox_amd.config import config_from_dict
    from glassbox_amd.engine.engine import EngineError, check_supported
    from glassbox_amd.weights.loader import build_model

    def refused(change, key):
        raw = copy.deepcopy(CASES["A"])
        change(raw)
        with pytest.raises(EngineError, match=key):
            check_supported(build_model(config_from_dict(raw)), torch.bfloat16, 16)
    refused(lambda r: r["canon"].update(taps=9), "canon.taps")
    refused(lambda r: r["layers"][0]["mixer"].update(kv_rank=4096), "kv_rank")
    refused(lambda r: r["layers"][0]["mlp"]["router"].update(experts=600), "router.experts")
    refused(lambda r: r["layers"][0]["mlp"]["router"].update(experts=40, top=17), "router.top")
    refused(lambda r: (r.update(width=960), r["norm"].update(groups=96)), "norm.groups")


def test_recorded_launches_take_a_tensor_that_moves_with_the_layer():
    """A layer's residual buffer is one of the ranges that recorded launches are moved by, set anew in every step."""
    from glassbox_amd import ops
    a, b = torch.zeros(4, 3), torch.zeros(8)
    fixed = ops.TapeOperands([b], places=1)
    other = ops.TapeOperands([torch.zeros(8)], places=1)
    fixed.place(0, a)
    other.place(0, torch.zeros(4, 3))
    assert fixed.count == 2 and fixed.ptrs[1] == a.data_ptr() and fixed.bytes[1] == 48 and fixed.sizes == other.sizes
    assert fixed.maps_onto(other)
    with pytest.raises(ops.KernelError):
        fixed.place(0, torch.zeros(3, 4).t())
