"""The Zozezen decoder without a GPU: its configuration, the tensors its parts declare, what its
layers ask of the cache manager, the plain implementation's own pieces on cases worked out by hand,
and the engine's own logic (row tables, cache manager, keys read from another layer, step function,
replay) against the plain implementation with the kernels replaced by torch stand-ins."""
import copy
import math
import shutil

import pytest
import torch

import emulated_ops
import schedules
from plain import zozezen as P
from replay_common import collect, make_requests
from tiny_zozezen import TINY, assert_matches_plain, read_model_dir, write_tiny

from kappai_amd.cache import CacheBundle, FixedState, PagedKV
from kappai_amd.config import ConfigError, config_from_dict
from kappai_amd.config.zozezen import ZozezenConfig
from kappai_amd.engine.replay import TraceReplayer, make_replay_cache
from kappai_amd.models import build_model, load_model

F64 = torch.float64
LENGTHS = {"A": [70, 45, 100, 37], "B": [66, 35, 90], "C": [50, 181, 36], "D": [40, 75],
           "E": [61, 30, 45]}
MIXED_LENGTHS = {"A": [70, 45, 100, 37, 83, 64, 29, 58], "B": [66, 35, 90, 41, 23, 77, 50, 62, 88],
                 "C": [50, 181, 36, 67, 44, 72, 90, 33, 58], "D": [40, 75, 52, 33, 61, 28],
                 "E": [61, 30, 45, 38, 52, 27, 66]}


@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    base = tmp_path_factory.mktemp("zozezen")
    return {name: write_tiny(name, base / name) for name in TINY}


# ---------------------------------------------------------------------------------------------
# configuration and weights
# ---------------------------------------------------------------------------------------------
def test_config_reads_every_size_from_the_file():
    raw = copy.deepcopy(TINY["A"][0])
    cfg = config_from_dict(raw)
    assert isinstance(cfg, ZozezenConfig)
    assert (cfg.vocab_size, cfg.width, cfg.norm_eps) == (211, 72, 1e-5)
    assert cfg.layers[0].mixer == {"heads": 6, "kv_heads": 2, "dim": 16, "vdim": 24, "scale": 0.3,
                                   "rot": {"base": 10000.0, "dims": 8}, "kv_from": None}
    assert cfg.layers[0].mlp == {"ff": 24, "limit": 1.5, "experts": 7, "top": 2, "identity": 2,
                                 "groups": 3, "keep_groups": 2, "shared_ff": 40,
                                 "shared_limit": 0.9}
    assert cfg.layers[1].mixer == {"heads": 6, "vdim": 12, "state": 20, "groups": 3, "conv": 3,
                                   "norm_groups": 2}
    assert cfg.layers[2].mixer["kv_from"] == 0 and cfg.layers[2].mlp is None
    assert cfg.layers[3].mlp["shared_ff"] is None and cfg.layers[3].mlp["groups"] == 1
    b = config_from_dict(copy.deepcopy(TINY["B"][0]))
    assert b.layers[0].mixer["rot"] is None and b.layers[2].mlp["identity"] == 0
    assert cfg.to_dict() == raw
    raw["layers"][1]["mlp"]["shared"] = raw["layers"][1]["mlp"]["router"]["groups"] = None
    raw["layers"][1]["mlp"]["router"]["identity"] = None
    m = config_from_dict(raw).layers[1].mlp
    assert (m["shared_ff"], m["groups"], m["identity"]) == (None, 1, 0)


@pytest.mark.parametrize("change,match", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0].update(type="mingru"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv heads"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "rot.dims"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "no keys and values"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=8), "vdim differs"),
    (lambda c: c["layers"][2]["mixer"].pop("rot"), "rot differs"),
    (lambda c: c["layers"][1]["mixer"].update(groups=4), "groups"),
    (lambda c: c["layers"][1]["mixer"].update(norm_groups=5), "norm_groups"),
    (lambda c: c["layers"][1]["mixer"].pop("state"), "state"),
    (lambda c: c["layers"][1]["mixer"].update(conv=0), "conv"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "identity"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "keep"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "chosen"),
])
def test_config_errors_name_the_key(change, match):
    raw = copy.deepcopy(TINY["A"][0])
    change(raw)
    with pytest.raises(ConfigError, match=match):
        config_from_dict(raw)


def test_tensor_names_and_shapes():
    model = build_model(config_from_dict(copy.deepcopy(TINY["A"][0])), "float32")
    shapes = {s.name: tuple(s.shape) for s in model.tensor_specs()}
    assert shapes["embed"] == shapes["head"] == (211, 72) and shapes["final.norm"] == (72,)
    for n in ("l0.norm1", "l0.norm1b", "l0.norm2", "l1.norm2b", "l2.norm1b"):
        assert shapes[n] == (72,)
    assert shapes["l0.mix.q"] == (96, 72) and shapes["l0.mix.k"] == (32, 72)
    assert shapes["l0.mix.v"] == (48, 72) and shapes["l0.mix.g"] == (6, 72)
    assert shapes["l0.mix.o"] == (72, 144) and shapes["l0.mix.k.norm"] == (16,)
    assert shapes["l2.mix.q.norm"] == (16,) and shapes["l2.mix.g"] == (6, 72)
    assert not any(n in shapes for n in ("l2.mix.k", "l2.mix.v", "l2.mix.k.norm", "l2.norm2",
                                         "l2.norm2b", "l2.mlp.router", "l0.mix.sink"))
    assert shapes["l1.mix.in"] == (2 * 72 + 2 * 60 + 6, 72)
    assert shapes["l1.mix.conv"] == (192, 3) and shapes["l1.mix.conv.b"] == (192,)
    assert shapes["l1.mix.dt_bias"] == shapes["l1.mix.A_log"] == shapes["l1.mix.D"] == (6,)
    assert shapes["l1.mix.norm"] == (72,) and shapes["l1.mix.o"] == (72, 72)
    assert shapes["l0.mlp.router"] == (9, 72) and shapes["l0.mlp.correction"] == (9,)
    assert shapes["l0.mlp.e6.gate"] == (24, 72) and "l0.mlp.e7.gate" not in shapes
    assert shapes["l0.mlp.shared.down"] == (72, 40) and shapes["l0.mlp.shared.sg"] == (1, 72)
    assert "l3.mlp.shared.gate" not in shapes and "l3.mlp.shared.sg" not in shapes


def test_a_file_may_hold_what_a_layer_without_feed_forward_leaves_unused(tmp_path, model_dirs):
    from kappai_amd.weights import WeightsError
    from kappai_amd.weights.safetensors_io import write_safetensors
    _, tensors = read_model_dir(model_dirs["A"])
    tensors["l2.norm2"] = tensors["l2.norm2b"] = torch.zeros(72, dtype=torch.bfloat16)
    folder = tmp_path / "more"
    folder.mkdir()
    shutil.copy(model_dirs["A"] / "config.json", folder / "config.json")
    write_safetensors(folder / "model.safetensors", tensors)
    assert load_model(folder, "float32", device="cpu").bound
    tensors["l2.mix.k"] = torch.zeros(32, 72, dtype=torch.bfloat16)
    write_safetensors(folder / "model.safetensors", tensors)
    with pytest.raises(WeightsError, match="unexpected tensors .1.: l2.mix.k"):
        load_model(folder, "float32", device="cpu")


def test_parts_refuse_what_they_do_not_do():
    from kappai_amd.kernels import ops
    from kappai_amd.parts import MixtureOfExperts, ScoredAttention, StateSpaceDual, SwiGLU
    clamp = ops.ClampedGate(1.0)
    with pytest.raises(ValueError, match="constants"):
        MixtureOfExperts("f.", 8, 8, 4, 2, torch.float32, activation="clamped")
    with pytest.raises(ValueError, match="constants"):
        SwiGLU("f.", 8, 8, torch.float32, clamp=clamp)
    with pytest.raises(ValueError, match="shared expert"):
        MixtureOfExperts("f.", 8, 8, 4, 2, torch.float32, scoring="softmax_all", shared_gate=True)
    with pytest.raises(ValueError, match="groups of 5"):
        MixtureOfExperts("f.", 8, 8, 4, 2, torch.float32, scoring="softmax_all", identity=1,
                         groups=2)
    with pytest.raises(ValueError, match="another layer"):
        ScoredAttention("a.", 8, 1, 1, 8, 8, 1.0, torch.float32, own_keys=False)
    with pytest.raises(ValueError, match="groups"):
        StateSpaceDual("m.", 8, 3, 8, 8, 2, 4, 1, 1e-5, torch.float32)
    with pytest.raises(ValueError, match="equal parts"):
        StateSpaceDual("m.", 8, 3, 8, 8, 1, 4, 5, 1e-5, torch.float32)
    with pytest.raises(ValueError, match="taps"):
        StateSpaceDual("m.", 8, 3, 8, 8, 1, 99, 1, 1e-5, torch.float32)
    own = ScoredAttention("a.", 8, 1, 1, 8, 8, 1.0, torch.float32, head_qk_norm=True)
    other = ScoredAttention("a.", 8, 1, 1, 8, 8, 1.0, torch.float32, head_qk_norm=True,
                            own_keys=False)
    for part, shared in ((own, True), (other, False)):
        with pytest.raises(ValueError, match="keys"):
            part.forward(torch.zeros(1, 8), None, None, shared_cache=shared)


def test_what_the_layers_ask_of_the_cache_manager():
    model = build_model(config_from_dict(copy.deepcopy(TINY["A"][0])), "float32")
    specs = model.cache_specs()
    assert specs[0] == PagedKV(2, 32) and specs[2] is None
    assert specs[1] == CacheBundle((("state", FixedState((6, 12, 20), "float32")),
                                    ("conv", FixedState((2, 192), "float32"))))
    assert [model.cache_id(i) for i in range(4)] == [0, 1, 0, 3]
    b = build_model(config_from_dict(copy.deepcopy(TINY["B"][0])), "float32")
    assert b.cache_specs()[1] == FixedState((2, 24, 16), "float32")      # one tap: no history
    assert [b.cache_id(i) for i in range(6)] == [0, 1, 2, 0, 4, 0]


# ---------------------------------------------------------------------------------------------
# pieces worked out by hand
# ---------------------------------------------------------------------------------------------
def test_plain_softmax_with_a_one_in_the_denominator():
    w = P.plus_one_softmax(torch.tensor([[0.0, -math.inf], [0.0, math.log(2.0)]], dtype=F64))
    assert torch.allclose(w, torch.tensor([[0.5, 0.0], [0.25, 0.5]], dtype=F64))
    far = P.plus_one_softmax(torch.tensor([[800.0, 800.0]], dtype=F64))
    assert torch.allclose(far, torch.tensor([[0.5, 0.5]], dtype=F64))
    assert float(P.plus_one_softmax(torch.tensor([[-800.0]], dtype=F64))) == 0.0


def test_plain_rotation_turns_pairs_half_apart():
    x = torch.tensor([1.0, 2.0, 3.0, 4.0, 9.0], dtype=F64).repeat(3, 1, 1)
    y = P.rotate(x, 100.0, 4)
    assert torch.equal(y[0], x[0]) and float(y[2, 0, 4]) == 9.0
    c, s = math.cos(0.2), math.sin(0.2)                    # pair 1 turns by p * 100^(-2 / 4)
    assert float(y[2, 0, 1]) == pytest.approx(2 * c - 4 * s)
    assert float(y[2, 0, 3]) == pytest.approx(4 * c + 2 * s)
    assert float(y[1, 0, 0]) == pytest.approx(math.cos(1) - 3 * math.sin(1))


def test_plain_state_space_two_tokens():
    x = torch.tensor([2.0, 5.0], dtype=F64).reshape(2, 1, 1)
    B = torch.tensor([[1.0, 0.5], [0.0, 2.0]], dtype=F64).reshape(2, 1, 2)
    C = torch.tensor([[1.0, 1.0], [3.0, 1.0]], dtype=F64).reshape(2, 1, 2)
    dt = torch.tensor([[0.5], [0.25]], dtype=F64)
    y = P.state_space(x, B, C, dt, torch.tensor([2.0], dtype=F64), torch.tensor([0.1], dtype=F64))
    assert float(y[0]) == pytest.approx(1.0 + 0.5 + 0.2)
    a = math.exp(-0.5)
    assert float(y[1]) == pytest.approx(3 * a + (0.5 * a + 2.5) + 0.5)


def test_plain_convolution_and_group_norm():
    x = torch.tensor([[1.0], [2.0], [3.0]], dtype=F64)
    y = P.short_conv(x, torch.tensor([[0.5, 10.0]]), torch.tensor([1.0]))
    want = torch.tensor([11.0, 21.5, 32.0], dtype=F64)
    assert torch.allclose(y[:, 0], want * torch.sigmoid(want))
    g = P.gated_group_norm(torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=F64),
                           torch.full((1, 4), 50.0, dtype=F64), torch.tensor([1.0, 1.0, 1.0, 3.0]),
                           2, 0.0)
    assert torch.allclose(g, torch.tensor([[3 / 12.5 ** .5, 4 / 12.5 ** .5, 0.0, 3 * 2 ** .5]],
                                          dtype=F64))


def test_plain_choice_by_groups_with_negative_scores():
    """All choice scores are negative: experts of a group that is not kept are out, not at zero; the
    group with the single best expert wins against the better pair.  The router's stand-in chooses
    alike."""
    s = torch.tensor([0.4, 0.1, 0.25, 0.25], dtype=F64)
    corr = torch.tensor([-1.0, -2.0, -0.95, -0.95], dtype=F64)
    router = {"experts": 3, "identity": 1, "top": 2, "groups": {"count": 2, "keep": 1}}
    order, gap = P.choose(s, corr, router)
    assert order == [0, 1] and gap == pytest.approx(0.1)
    chosen, wts, gate = emulated_ops.moe_route_scored(
        torch.cat([torch.log(s).float(), torch.tensor([math.log(3.0)])])[None], torch.eye(5), 2, 2.0,
        correction=corr.float(), groups=2, keep_groups=1, score="softmax", group_best=1, gate=True)
    assert chosen[0].tolist() == [0, 1] and torch.allclose(wts, torch.tensor([[0.8, 0.2]]))
    assert gate.tolist() == pytest.approx([0.75])


def test_plain_clamped_expert():
    t = {"gate": torch.tensor([[4.0], [-3.0]]), "up": torch.tensor([[5.0], [-0.25]]),
         "down": torch.eye(2)}
    y = P.expert(torch.ones(1, 1, dtype=F64), t, "", 2.0)
    sig = lambda z: 1 / (1 + math.exp(-z))
    assert y[0].tolist() == pytest.approx([2 * sig(3.404) * 3, -3 * sig(-5.106) * 0.75])


def test_plain_experts_that_hand_their_input_on():
    """One expert of tensors against two that hand their input on: the output is the input times the
    weights of the latter where only they are chosen."""
    W = 4
    x = torch.eye(W, dtype=F64)[:2] * 3
    t = {"router": torch.zeros(3, W), "correction": torch.tensor([-5.0, 0.0, 0.0])}
    out = P.moe_ff(x, t, "", {"expert": {"limit": 1.0}, "router": {"experts": 1, "identity": 2,
                                                                   "top": 2}})
    assert torch.allclose(out, x * 2 / 3)


# ---------------------------------------------------------------------------------------------
# norms on both sides of a sublayer
# ---------------------------------------------------------------------------------------------
def test_rms_norms_between_sublayers_in_one_pass_and_apart(monkeypatch):
    """A norm that applies the pending update itself gives what ``norm_output`` and a plain norm give
    one after the other; for a mixture's terms, partial sums and rows; for some rows only."""
    from kappai_amd.kernels import ops
    from kappai_amd.parts import RMSNorm
    from kappai_amd.parts.base import NormedUpdate, summed_delta
    emulated_ops.install(monkeypatch)
    W, T, eps = 12, 5, 1e-5
    g = torch.Generator().manual_seed(3)
    norms = []
    for name in ("a", "b"):
        n = RMSNorm(name, W, eps, torch.float32, suffix="", weight_offset=1.0)
        n.bind({name: 0.3 * torch.randn(W, generator=g)})
        norms.append(n)
    experts = torch.tensor([[0, 2], [1, 0], [2, 1], [2, 0], [1, 2]])       # 2: hands its input on
    plan = emulated_ops.moe_plan(experts, 2)
    y = torch.randn(T, 2, W, generator=g)
    y[experts == 2] = float("nan")
    terms = ops.ExpertTerms(y, torch.rand(T, 2, generator=g), plan,
                            also=torch.randn(3, T, W, generator=g),
                            also_gate=torch.rand(T, generator=g), rows=torch.randn(T, W, generator=g))
    for upd in (torch.randn(T, W, generator=g), torch.randn(4, T, W, generator=g), terms):
        x = torch.randn(T, W, generator=g)
        one, two = x.clone(), x.clone()
        rows = norms[1].add_norm(one, summed_delta(norms[1], NormedUpdate(upd, norms[0])))
        norms[0].norm_output(two, upd)
        want = norms[1].add_norm(two, None)
        assert torch.allclose(one, two, atol=1e-6) and torch.allclose(rows, want, atol=1e-6)
        pick = torch.tensor([3, 1], dtype=torch.int32)
        kept = x.clone()
        some = norms[1].add_norm(kept, NormedUpdate(upd, norms[0]), rows=pick)
        assert torch.equal(kept, x) and torch.allclose(some, want[pick.long()], atol=1e-6)


# ---------------------------------------------------------------------------------------------
# the engine's own logic, with stand-ins for the kernels
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", ["A", "B", "C", "D", "E"])
@pytest.mark.parametrize("family", ["prefill_then_decode", "changing_portions", "mixed"])
def test_schedules_with_stand_ins(tmp_path, monkeypatch, model_dirs, name, family):
    """Every logit of every request, pages and slots taken again (the mixed family's pool is smaller
    than its requests together) and poisoned before their first use."""
    emulated_ops.install(monkeypatch)
    requests = make_requests(TINY[name][0]["vocab"],
                             MIXED_LENGTHS[name] if family == "mixed" else LENGTHS[name], seed=21)
    steps, index, peak = getattr(schedules, family)(requests)
    model = load_model(model_dirs[name], "float32", device="cpu")
    cache = make_replay_cache(model, peak, 16, num_slots=4)
    cache.allocate_storage(model.dtype, "cpu", poison=True)
    replayer = TraceReplayer(emulated_ops.make_cpu_runner(model, cache), tmp_path / "out")
    outputs = {}
    for obj in steps:
        res = replayer.run_step(obj)
        if res is not None:
            outputs[obj["step"]] = res
        cache.check()
    got = collect(index, outputs, model.vocab_size)
    assert len(got) == sum(len(t) for t in requests.values())
    assert_matches_plain(got, model_dirs[name], requests, "float32", (name, family))


def test_the_named_shapes_are_configurations():
    from kappai_amd.config import named_shape
    for name in ("zozezen-w1024", "zozezen-w2048", "zozezen-tiny"):
        conf = config_from_dict(named_shape(name))
        model = build_model(conf, "float32")
        assert isinstance(conf, ZozezenConfig) and len(model.tensor_specs()) > 20
        assert any(c.reads_cache_of is not None for c in model.schedule)
