"""The Nuzivik decoder without a GPU: its configuration, the tensors its parts declare, what its
layers ask of the cache manager (windows that keep the first tokens), the plain implementation's
own pieces on cases worked out by hand, and the engine's own logic (row tables, cache manager,
step function, replay) against the plain implementation with the kernels replaced by torch
stand-ins."""
import copy
import json
import math
import shutil

import pytest
import torch

import emulated_ops
import schedules
from plain import nuzivik as P
from replay_common import collect, make_requests
from tiny_nuzivik import TINY, assert_matches_plain, read_model_dir, write_tiny

from kappai_amd.cache import CacheManager, PagedKV
from kappai_amd.config import ConfigError, config_from_dict
from kappai_amd.config.nuzivik import NuzivikConfig
from kappai_amd.engine.replay import TraceReplayer, make_replay_cache
from kappai_amd.models import build_model, load_model

LENGTHS = {"A": [70, 45, 100, 37], "B": [66, 35, 90], "C": [50, 81, 36], "D": [40, 75],
           "E": [61, 30, 45]}
MIXED_LENGTHS = {"A": [70, 45, 100, 37, 83, 64, 29, 58], "B": [66, 35, 90, 41, 23, 77, 50, 62, 88],
                 "C": [50, 81, 36, 67, 44, 72, 90, 33, 58], "D": [40, 75, 52, 33, 61, 28],
                 "E": [61, 30, 45, 38, 52, 27, 66]}


@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    base = tmp_path_factory.mktemp("nuzivik")
    return {name: write_tiny(name, base / name) for name in TINY}


# ---------------------------------------------------------------------------------------------
# configuration and weights
# ---------------------------------------------------------------------------------------------
def test_config_reads_every_size_from_the_file():
    raw = copy.deepcopy(TINY["A"][0])
    cfg = config_from_dict(raw)
    assert isinstance(cfg, NuzivikConfig)
    assert (cfg.vocab_size, cfg.width, cfg.norm_eps, cfg.embedding_scale) == (211, 72, 1e-5, 8.5)
    m = cfg.layers[0].mixer
    assert (m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], m["bias_max"],
            m["buckets"], m["window"], m["keep_first"]) == (6, 2, 16, 16, 0.3, 50.0, 10, 24, 3)
    assert cfg.layers[0].mlp == {"ff": 24, "experts": 6, "top": 2, "scale": 1.7, "groups": 3,
                                 "keep_groups": 2}
    assert cfg.layers[1].mixer["keep_first"] == 0 and cfg.layers[1].mlp is None
    assert cfg.layers[2].mlp["groups"] == cfg.layers[2].mlp["keep_groups"] == 1
    b = config_from_dict(copy.deepcopy(TINY["B"][0]))
    assert b.embedding_scale == 1.0 and b.layers[0].mixer["window"] is None
    assert b.layers[0].mlp["scale"] == 1.0
    assert cfg.to_dict() == raw


@pytest.mark.parametrize("change,match", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0].update(type="mingru"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv heads"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=24), "vdim"),
    (lambda c: c["layers"][0]["mixer"].update(bias_max=0.5), "bias_max"),
    (lambda c: c["layers"][0]["mixer"]["mask"].pop("size"), "size"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "expert"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "keep"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "chosen"),
])
def test_config_errors_name_the_key(change, match):
    raw = copy.deepcopy(TINY["A"][0])
    change(raw)
    with pytest.raises(ConfigError, match=match):
        config_from_dict(raw)


def test_tensor_names_and_shapes():
    model = build_model(config_from_dict(copy.deepcopy(TINY["A"][0])), "float32")
    shapes = {s.name: tuple(s.shape) for s in model.tensor_specs()}
    assert shapes["embed"] == (211, 72) and "head" not in shapes
    for n in ("l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l1.norm1b", "final.norm"):
        assert shapes[n] == shapes[n + ".b"] == (72,) and shapes[n + ".alpha"] == ()
    assert shapes["l0.mix.q"] == (96, 72) and shapes["l0.mix.k"] == (32, 72)
    assert shapes["l0.mix.o"] == (72, 96) and shapes["l0.mix.rel"] == (10, 6)
    assert shapes["l0.mix.sink"] == (6,) and "l0.mix.v" not in shapes
    assert not any("q.norm" in n or "k.norm" in n for n in shapes)
    assert shapes["l0.mlp.router"] == (6, 72) and shapes["l0.mlp.correction"] == (6,)
    assert shapes["l0.mlp.e5.gate"] == (24, 72) and shapes["l0.mlp.e0.down"] == (72, 24)
    assert not any(n.startswith(("l1.norm2", "l1.mlp")) for n in shapes)


def test_a_file_without_the_tables_rows_takes_them_from_the_tensor(tmp_path, model_dirs):
    raw = copy.deepcopy(TINY["A"][0])
    for layer in raw["layers"]:
        layer["mixer"].pop("buckets")
    with pytest.raises(ValueError, match="buckets"):
        build_model(config_from_dict(copy.deepcopy(raw)), "float32")
    folder = tmp_path / "bare"
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(raw))
    shutil.copy(model_dirs["A"] / "model.safetensors", folder / "model.safetensors")
    model = load_model(folder, "float32", device="cpu")
    assert [l.mixer["buckets"] for l in model.config.layers] == [10, 7, 16]


def test_a_file_may_hold_what_a_layer_without_feed_forward_leaves_unused(tmp_path, model_dirs):
    from kappai_amd.weights import WeightsError
    from kappai_amd.weights.safetensors_io import write_safetensors
    _, tensors = read_model_dir(model_dirs["A"])
    tensors["l1.norm2"] = tensors["l1.norm2b.b"] = torch.zeros(72, dtype=torch.bfloat16)
    tensors["l1.norm2b.alpha"] = torch.zeros((), dtype=torch.bfloat16)
    folder = tmp_path / "more"
    folder.mkdir()
    shutil.copy(model_dirs["A"] / "config.json", folder / "config.json")
    write_safetensors(folder / "model.safetensors", tensors)
    assert load_model(folder, "float32", device="cpu").bound
    tensors["l1.mix.v"] = torch.zeros(4, 72, dtype=torch.bfloat16)
    write_safetensors(folder / "model.safetensors", tensors)
    with pytest.raises(WeightsError, match="unexpected tensors .1.: l1.mix.v"):
        load_model(folder, "float32", device="cpu")


def test_parts_refuse_what_they_do_not_do():
    from kappai_amd.parts import MixtureOfExperts, SandwichNormBlock, ScoredAttention, TanhNorm
    from kappai_amd.parts import LayerNorm
    with pytest.raises(ValueError, match="sigmoid"):
        MixtureOfExperts("f.", 8, 8, 4, 2, torch.float32, groups=2, keep_groups=1)
    with pytest.raises(ValueError, match="groups"):
        MixtureOfExperts("f.", 8, 8, 4, 3, torch.float32, scoring="sigmoid", groups=2,
                         keep_groups=1)
    with pytest.raises(ValueError, match="keep_first"):
        ScoredAttention("a.", 8, 1, 1, 8, 8, 1.0, torch.float32, window=4, keep_first=-1)
    norm = TanhNorm("n", 8, torch.float32)
    with pytest.raises(ValueError, match="norm_output"):
        SandwichNormBlock(norm, None, LayerNorm("m", 8, 1e-5, torch.float32))
    with pytest.raises(ValueError, match="come together"):
        SandwichNormBlock(norm, None, norm, ffn_norm=norm)


# ---------------------------------------------------------------------------------------------
# the cache manager: windows that keep the first tokens
# ---------------------------------------------------------------------------------------------
def test_what_the_layers_ask_of_the_cache_manager():
    model = build_model(config_from_dict(copy.deepcopy(TINY["A"][0])), "float32")
    assert model.cache_specs() == [PagedKV(2, 16, 24, 3), PagedKV(3, 32, 40, 0),
                                   PagedKV(1, 48, 17, 20)]
    b = build_model(config_from_dict(copy.deepcopy(TINY["B"][0])), "float32")
    assert b.cache_specs()[0] == PagedKV(1, 16, None, 0)


@pytest.mark.parametrize("keep,pages_kept", [(0, 0), (1, 1), (16, 1), (17, 2), (40, 3), (100, 7)])
def test_a_window_gives_back_all_pages_but_those_of_the_first_tokens(keep, pages_kept):
    """Token by token and in portions: at every length the request holds the pages of its first
    ``keep`` tokens and those its window still reaches, and nothing else."""
    window, ps = 20, 16
    for portions in ([1] * 180, [50, 1, 1, 60, 3, 65], [180]):
        cm = CacheManager([PagedKV(1, 16, window, keep), PagedKV(1, 16, None)], ps, 14, 1)
        rc = cm.open("a")
        for n in portions:
            cm.extend(rc, n)
            cm.commit(rc, n)
            cm.check()
            first_needed = rc.length - window + 1
            for b, page in enumerate(rc.blocks[0]):
                want = b < pages_kept or (b + 1) * ps > first_needed
                assert (page >= 0) == want, (rc.length, b)
        assert rc.length == 180
        cm.close(rc)
        cm.check()
        assert cm.num_free_pages(0) == 14


def test_dump_shows_the_window_and_the_kept_tokens():
    cm = CacheManager([PagedKV(1, 16, 20, 18)], 16, 14, 1)
    cm.allocate_storage(torch.float32, "cpu")
    rc = cm.open("a")
    for _ in range(100):
        cm.extend_one(rc)
        page = rc.blocks[0][rc.length // 16]
        cm.paged_groups[0].pools[0]["k"][page, 0, rc.length % 16] = float(rc.length)
        cm.commit_one(rc)
    d = cm.dump(rc)["caches"][0]
    assert d["first_position"] == 80 and d["k"][0, 0, 0] == 80.0
    assert d["kept"]["k"].shape[0] == 18
    assert d["kept"]["k"][:, 0, 0].tolist() == [float(i) for i in range(18)]


# ---------------------------------------------------------------------------------------------
# pieces worked out by hand
# ---------------------------------------------------------------------------------------------
def test_plain_masks_and_buckets_and_sink():
    ok = P.seen(7, 2, 1)
    assert ok[5].tolist() == [True, False, False, False, True, True, False]
    assert P.seen(7, 2, 0)[5].tolist() == [False] * 4 + [True, True, False]
    assert P.seen(4, None, 0).tolist() == torch.ones(4, 4).tril().bool().tolist()
    assert [P.bucket_of(n, 8, 64) for n in (0, 3, 4, 7, 8, 15, 16, 31, 32, 64, 999)] == [
        0, 3, 4, 4, 5, 5, 6, 6, 7, 7, 7]
    w = P.sink_softmax(torch.zeros(1, 2, 2, dtype=torch.float64), P.seen(2, None, 0),
                       torch.tensor([math.log(3.0)], dtype=torch.float64))
    assert torch.allclose(w[0], torch.tensor([[0.25, 0.0], [0.2, 0.2]], dtype=torch.float64))


@pytest.mark.parametrize("rows,far", [(8, 64), (10, 50.0), (7, 300.0), (16, 33), (2, 30), (32, 1000),
                                      (9, 25), (64, 4096)])
def test_the_bias_table_by_distance(rows, far):
    from kappai_amd.parts.scored_attention import distance_bias_columns
    table = torch.randn(rows, 3)
    cols = distance_bias_columns(table, far)
    for n in list(range(cols.shape[1])) + [cols.shape[1] + 5, 10 ** 6]:
        want = table[P.bucket_of(n, rows, far)]
        assert torch.equal(cols[:, min(n, cols.shape[1] - 1)], want), n


def test_plain_choice_by_groups_with_negative_scores():
    """All choice scores are negative: experts of a group that is not kept are out, not at zero;
    the group with the single best expert loses against the better pair."""
    s = torch.tensor([0.9, 0.1, 0.5, 0.5], dtype=torch.float64)
    corr = torch.tensor([-1.0, -2.0, -1.0, -1.0], dtype=torch.float64)
    router = {"experts": 4, "top": 2, "groups": {"count": 2, "keep": 1}}
    order, gap = P.choose(s, corr, router)
    assert order == [2, 3] and gap == pytest.approx(min(-1.0 - (-2.0), math.inf))
    chosen, wts = emulated_ops.moe_route_scored(
        torch.log(s / (1 - s)).float()[None], torch.eye(4), 2, 1.5, correction=corr.float(),
        groups=2, keep_groups=1)
    assert sorted(chosen[0].tolist()) == [2, 3] and torch.allclose(wts, torch.tensor([[0.75, 0.75]]))


def test_norms_of_another_kind_between_the_same_sublayers(monkeypatch):
    """The block with a norm before and behind every sublayer is not tied to one kind of norm: RMS
    norms, and each kind reading what the other left pending."""
    from kappai_amd.parts import RMSNorm, SandwichNormBlock, TanhNorm
    from kappai_amd.parts.base import Hidden, summed_delta
    emulated_ops.install(monkeypatch)
    W, eps = 12, 1e-5
    g = torch.Generator().manual_seed(3)

    class Map:
        capturable, step_tables = True, None

        def __init__(self):
            self.w = torch.randn(W, W, generator=g)

        def forward(self, x, *rest, **more):
            return x @ self.w.T

    def make(kind, name):
        n = TanhNorm(name, W, torch.float32) if kind == "t" else RMSNorm(
            name, W, eps, torch.float32, suffix="")
        t = {s.name: (0.7 + 0.3 * torch.rand(s.shape, generator=g)) for s in n.tensor_specs()}
        n.bind(t)
        if kind == "t":
            return n, lambda x: torch.tanh(t[name + ".alpha"] * x) * t[name] + t[name + ".b"]
        return n, lambda x: x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * t[name]

    for kinds in ("tttt", "rrrr", "trtr", "rtrt", "ttrr"):
        norms, fns = zip(*(make(k, f"n{i}") for i, k in enumerate(kinds)))
        a, b = Map(), Map()
        block = SandwichNormBlock(norms[0], a, norms[1], norms[2], b, norms[3])
        last, last_fn = make("t" if kinds[3] == "r" else "r", "last")
        x = torch.randn(5, W, generator=g)
        want = x + fns[1](fns[0](x) @ a.w.T)
        want = want + fns[3](fns[2](want) @ b.w.T)
        h = block.forward(Hidden(x.clone()), None, None)
        got = last.add_norm(h.resid, summed_delta(last, h.delta, h.resid))
        assert torch.allclose(got, last_fn(want), atol=1e-5), kinds


# ---------------------------------------------------------------------------------------------
# the engine with emulated kernels
# ---------------------------------------------------------------------------------------------
def run_emulated(monkeypatch, model_dir, steps, index, max_tokens, tmp_path):
    emulated_ops.install(monkeypatch)
    model = load_model(model_dir, "float32", device="cpu")
    cache = make_replay_cache(model, max_tokens, 16, num_slots=4)
    cache.allocate_storage(model.dtype, "cpu", poison=True)
    rep = TraceReplayer(emulated_ops.make_cpu_runner(model, cache), tmp_path / "out")
    outputs = {}
    for obj in steps:
        res = rep.run_step(obj)
        if res is not None:
            outputs[obj["step"]] = res
        cache.check()
    assert not cache.live_requests()
    assert all(g.allocator.num_used == 0 for g in cache.paged_groups)
    return collect(index, outputs, model.vocab_size)


@pytest.mark.parametrize("name,family", [("A", f) for f in
                                         ("whole", "prefill_then_decode", "changing_portions",
                                          "mixed")] + [("B", "mixed"), ("C", "mixed"),
                                                       ("D", "changing_portions"),
                                                       ("E", "mixed")])
def test_schedules_float32(monkeypatch, tmp_path, model_dirs, name, family):
    cfg = TINY[name][0]
    lengths = MIXED_LENGTHS[name] if family == "mixed" else LENGTHS[name]
    requests = make_requests(cfg["vocab"], lengths, seed=21)
    steps, index, peak = getattr(schedules, family)(requests)
    if family == "mixed":
        assert sum(len(t) for t in requests.values()) > peak, "the pool must be reused"
    got = run_emulated(monkeypatch, model_dirs[name], steps, index, peak, tmp_path)
    assert len(got) == sum(len(t) for t in requests.values())
    assert_matches_plain(got, model_dirs[name], requests, "float32", (name, family))
