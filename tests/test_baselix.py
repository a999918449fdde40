"""Baselix on the host: the configuration, whose latent a layer reads and how long it is kept, what is refused, the stream
in units of the sublayers' factor, and the plain implementation's own mechanisms (tests/plain_baselix.py)."""
import copy
import math

import pytest
import torch

import baselix_models
import plain_baselix as plain
from bare_cuda_4gib_amd.config import BaselixConfig
from bare_cuda_4gib_amd.config.registry import architecture_for
from bare_cuda_4gib_amd.errors import ConfigError, EngineError


def described(config):
    arch = architecture_for(config)
    assert arch.name == "Baselix"
    cfg = arch.config_class.from_dict(config)
    from bare_cuda_4gib_amd.engine.model import Model
    return cfg, Model(arch.describe(cfg))


@pytest.mark.parametrize("name", sorted(baselix_models.CONFIGS))
def test_the_model_wants_exactly_the_tensors_of_the_design(name):
    config = baselix_models.CONFIGS[name]
    _, model = described(config)
    want = {k: tuple(v.shape) for k, v in baselix_models.tensors_for(config, 1).items()}
    specs = model.expected_weights()
    assert {k: tuple(v.shape) for k, v in specs.items() if not v.optional} == want
    assert [k for k, v in specs.items() if v.optional] == ["head.weight"]         # (the head is the embedding table)


def test_the_configuration_reads_back():
    for config in baselix_models.CONFIGS.values():
        cfg = BaselixConfig.from_dict(config)
        again = BaselixConfig.from_dict(cfg.to_dict())
        assert again == cfg and architecture_for(cfg.to_dict()).name == "Baselix"


def test_whose_latent_a_layer_reads_and_how_long_it_is_kept():
    from bare_cuda_4gib_amd.cache.specs import PagedLatent
    _, model = described(baselix_models.CONFIGS["A"])
    assert [(e.layer, e.cache, e.writes) for e in model.schedule] == [(0, 0, True), (1, 0, False), (2, 0, False), (3, 3, True)]
    # layer 0's stream is kept as far back as the widest of its readers looks (9, 23 and 4 keys); each layer keeps its own window
    assert model.cache_streams() == {0: PagedLatent(20, 0, 23), 3: PagedLatent(13, 0, 17)}
    assert [layer.mixer.window for layer in model.layers] == [9, 23, 4, 17]
    assert [layer.mixer.borrows for layer in model.layers] == [False, True, True, False]
    _, model = described(baselix_models.CONFIGS["D"])           # a reader of every key
    assert model.cache_streams() == {0: PagedLatent(68, 0, 0), 2: PagedLatent(40, 0, 16)}
    a, b = PagedLatent(8, 0, 5), PagedLatent(8, 0, 7)
    assert a.covering(b) == b.covering(a) == b and a.covering(PagedLatent(8, 0, 0)).window == 0
    assert a.covering(PagedLatent(9, 0, 5)) is None and a.covering(PagedLatent(8, 2, 5)) is None and a.covering("other") is None


def test_layers_whose_rows_differ_cannot_share_a_stream():
    from bare_cuda_4gib_amd.engine.model import Model
    cfg = BaselixConfig.from_dict(baselix_models.CONFIGS["A"])
    spec = architecture_for(baselix_models.CONFIGS["A"]).describe(cfg)
    spec.layers[1].mixer.params["kv_rank"] = 21
    with pytest.raises(ConfigError, match="another spec"):
        Model(spec).cache_streams()


def test_pages_go_back_once_the_widest_reader_has_passed_them():
    from bare_cuda_4gib_amd.cache.manager import CacheManager
    from bare_cuda_4gib_amd.cache.specs import PagedLatent
    cache = CacheManager({"s": PagedLatent(6, 0, 4).covering(PagedLatent(6, 0, 10))}, page_tokens=4, num_pages=6, max_requests=2, max_tokens=64,
                         dtype=torch.float32, device="cpu")
    cache.admit("r")
    held = []
    for n in (3, 6, 4, 1, 9):               # lengths 3, 9, 13, 14, 23: the next row reads from length - 9 on
        cache.reserve([("r", n)])
        cache.advance("r", n)
        held.append((cache.length("r"), [i for i, p in enumerate(cache.table(("window", 10), "r")) if p >= 0]))
    assert held == [(3, [0]), (9, [0, 1, 2]), (13, [1, 2, 3]), (14, [1, 2, 3]), (23, [3, 4, 5])]
    cache.release("r")
    assert cache.pages_in_use() == 0


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].__setitem__("type", "attention"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "lacks scale"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_from", 1), "itself"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_from", 3), "earlier"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_from", -1), "earlier"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 1), "of its own"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_rank", 21), "kv_rank"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "gelu"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 7), "7 of 6"),
    (lambda c: c.__setitem__("residual_mult", 0.0), "residual_mult"),
    (lambda c: c.__setitem__("logit_softcap", -2.0), "softcap"),
    (lambda c: c.pop("max_positions"), "max_positions"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("kv_rank", 0), "kv_rank"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("kv_rank", 5000), "beyond"),
])
def test_what_is_refused(change, message):
    config = copy.deepcopy(baselix_models.CONFIGS["A"])
    change(config)
    with pytest.raises(ConfigError, match=message):
        described(config)


def test_absent_keys_have_the_design_s_defaults():
    config = copy.deepcopy(baselix_models.CONFIGS["C"])
    del config["residual_mult"]
    cfg, model = described(config)
    assert cfg.residual_mult == 1.0 and cfg.softcap == 0.0 and model.head.part.softcap == 0.0
    assert model.layers[1].mixer.window == 0 and model.layers[0].ffn is None and model.layers[0].ffn_norm is None
    routed = model.layers[1].ffn
    assert routed.over_chosen and routed.router_bias and not routed.correction and not routed.shared_gate and not routed.normalize
    assert (routed.limit, routed.shared_limit, routed.shared_ff, routed.slope) == (0.9, 4.0, 30, 1.702)


def test_the_stream_is_kept_in_units_of_the_factor(tmp_path):
    """x += m f(N(x)) with eps is u += f(N(u)) with eps / m^2 for x = m u: the plain model once more with its tables over m,
    a factor of one and that eps gives the same logits; the parts are built with these numbers."""
    for name in ("A", "D"):
        config = baselix_models.CONFIGS[name]
        m = config["residual_mult"]
        cfg, model = described(config)
        assert model.embedding.part.scale == 1.0 / m and model.embedding.part.position_limit == config["max_positions"]
        norms = [layer.mixer_norm for layer in model.layers] + [layer.ffn_norm for layer in model.layers if layer.ffn] + [model.final_norm.part]
        assert all(abs(n.eps - config["norm"]["eps"] / m ** 2) < 1e-18 and n.offset == 1.0 for n in norms)
        assert all(layer.mixer.eps == config["norm"]["eps"] for layer in model.layers)             # (the latent is not the stream)
        theirs = plain.PlainBaselix(baselix_models.write_folder(tmp_path, name, "float32"))
        ids = [(5 * i + 2) % config["vocab"] for i in range(30)]
        want, layers = theirs.forward(ids, return_layers=True)
        latent_eps, stream_eps = theirs.eps, theirs.eps / m ** 2
        theirs.w["embed.in"], theirs.w["pos"] = theirs.w["embed"] / m, theirs.w["pos"] / m
        u, latents = plain.placed_embedding(theirs.w["embed.in"], theirs.w["pos"], ids), {}
        for i, entry in enumerate(config["layers"]):
            theirs.eps = latent_eps
            u = u + theirs.mixer(i, entry["mixer"], plain.norm_about_one(u, theirs.w[f"l{i}.norm1"], stream_eps), latents)
            if entry["mlp"] is not None:
                u = u + theirs.feed_forward(f"l{i}.mlp.", entry["mlp"], plain.norm_about_one(u, theirs.w[f"l{i}.norm2"], stream_eps))
            assert torch.allclose(u * m, layers[i], atol=1e-9, rtol=1e-9)
        got = plain.capped(plain.norm_about_one(u, theirs.w["final.norm"], stream_eps) @ theirs.w["embed"].T, config["logit_softcap"])
        assert torch.allclose(got.float(), want, atol=1e-5, rtol=1e-5)


def test_into_how_many_parts_a_window_s_keys_are_cut():
    """Few rows over a long context cut the keys into parts; with a window there are no more parts than it has tiles."""
    from bare_cuda_4gib_amd.csrc import ops
    assert ops.latent_splits([0, 1], 16, 4096) == 64
    assert ops.latent_splits([0, 1], 16, 4096, 100) == -(-(100 + 4 + 31) // 32)
    assert ops.latent_splits([0, 1], 16, 40, 100) == 2                     # (a context shorter than the window)
    assert ops.latent_splits([0, 4096], 16, 4096, 100) == 1


def test_a_part_without_a_latent_does_not_write():
    from bare_cuda_4gib_amd.parts.latent_attention import LatentAttention
    part = LatentAttention(hidden_size=8, heads=2, dim=4, vdim=4, kv_rank=6, scale=0.5, eps=1e-5, borrows=True)
    assert set(part.weight_specs()) == {"q", "uk", "uv", "o", "sink"}
    with pytest.raises(ConfigError, match="cannot write"):
        part.forward(torch.zeros(1, 8), None, None, None, writes=True)


def test_requests_end_where_the_table_of_positions_does():
    """An executor takes no more tokens a request than the table has rows, also for a caller who wants positions beyond the
    configuration's."""
    from bare_cuda_4gib_amd.engine import Executor, Runtime, StepEntry
    config = dict(copy.deepcopy(baselix_models.CONFIGS["F"]), max_positions=20)
    _, model = described(config)
    model.rt = Runtime(torch.device("cpu"), torch.float32)                 # (nothing runs: the step is refused before)
    with pytest.raises(EngineError, match="positions"):
        Executor(model, num_pages=8, max_requests=1, max_tokens=64, page_tokens=8)
    ex = Executor(model, num_pages=8, max_requests=1, max_tokens=64, page_tokens=8, beyond_positions=True)
    ex.admit("r")
    with pytest.raises(EngineError, match="21 tokens"):
        ex.step([StepEntry("r", [1] * 21)])
    assert ex.cache.max_tokens == 20 and ex.length("r") == 0 and ex.cache.pages_in_use() == 0


def test_the_plain_mechanisms():
    torch.manual_seed(0)
    f64 = torch.float64
    v, w = torch.randn(5, 12, dtype=f64), torch.randn(12, dtype=f64) * 0.3
    normed = plain.norm_about_one(v, w, 0.0) / (1.0 + w)
    assert torch.allclose((normed ** 2).mean(-1), torch.ones(5, dtype=f64)) and torch.equal(plain.norm_about_one(v, w * 0, 0.5), plain.unit_rms(v, 0.5))
    table, places = torch.randn(7, 4, dtype=f64), torch.randn(9, 4, dtype=f64)
    assert torch.equal(plain.placed_embedding(table, places, [3, 3, 0], first=5), table[[3, 3, 0]] + places[[5, 6, 7]])
    assert plain.window_mask(4, 2).int().tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]
    assert plain.window_mask(3, 0).int().tolist() == [[1, 0, 0], [1, 1, 0], [1, 1, 1]]
    s, mask, sink = torch.randn(2, 6, 6, dtype=f64), plain.window_mask(6, 3), torch.tensor([0.5, -2.0], dtype=f64)
    p = plain.sink_softmax(s, mask, sink)
    e = torch.exp(s) * mask
    assert torch.allclose(p, e / (torch.exp(sink)[:, None, None] + e.sum(-1, keepdim=True))) and bool((p.sum(-1) < 1.0).all())
    big = plain.sink_softmax(s + 800.0, mask, sink)
    assert bool(torch.isfinite(big).all()) and torch.allclose(big.sum(-1), torch.ones(2, 6, dtype=f64))
    assert float(plain.sink_softmax(s, mask, sink + 800.0).max()) < 1e-300
    assert plain.squared_relu(torch.tensor([-2.0, 0.0, 3.0])).tolist() == [0.0, 0.0, 9.0]
    unit = plain.clamped_unit(torch.tensor([5.0, -5.0, 0.5]), torch.tensor([9.0, -9.0, 0.25]), 2.0)
    want = [2.0 / (1 + math.exp(-1.702 * 2.0)) * 3.0, -5.0 / (1 + math.exp(1.702 * 5.0)) * -1.0, 0.5 / (1 + math.exp(-1.702 * 0.5)) * 1.25]
    assert torch.allclose(unit, torch.tensor(want))
    chosen, weights, margin = plain.route(torch.tensor([[0.0, 2.0, -1.0, 1.5]], dtype=f64), 2)
    assert chosen.tolist() == [[1, 3]] and abs(float(weights[0, 0]) - 1.0 / (1.0 + math.exp(-0.5))) < 1e-12 and abs(float(margin) - 1.5) < 1e-12
    assert torch.allclose(plain.capped(torch.tensor([0.01, 100.0, -100.0]), 2.0), torch.tensor([0.01, 2.0, -2.0]), atol=1e-6)
    assert torch.equal(plain.capped(v, None), v)


@pytest.mark.parametrize("name", sorted(baselix_models.CONFIGS))
def test_the_plain_model_does_not_look_ahead_and_every_piece_counts(name, tmp_path):
    folder = baselix_models.write_folder(tmp_path, name, "float32")
    model = plain.PlainBaselix(folder)
    ids = [(7 * i + 3) % model.cfg["vocab"] for i in range(40)]
    whole, after = model.forward(ids, return_layers=True)
    assert len(after) == len(model.cfg["layers"]) and bool(torch.isfinite(whole).all())
    assert torch.allclose(model.forward(ids[:23]), whole[:23], atol=1e-5, rtol=1e-5)
    keys = ["pos", "l0.mix.sink", "final.norm", "l0.mix.dkv.norm"] + [k for k in model.w if k.endswith("router.b")]
    for key in keys:
        kept = model.w[key].clone()
        model.w[key] = kept * 1.1 if not key.endswith("router.b") else kept + torch.arange(len(kept)) * 0.1
        moved = float((model.forward(ids) - whole).abs().max())
        assert moved > 1e-4 or (key.endswith("router.b") and len(kept) == 1), key
        model.w[key] = kept


def test_the_random_weights_mode_writes_a_folder_that_loads(tmp_path):
    """The framework's own random-weights mode over a Baselix configuration: every tensor the design names, norm weights
    around zero, a folder whose configuration reads back."""
    from bare_cuda_4gib_amd.config.registry import load_config
    from bare_cuda_4gib_amd.weights import write_random_model
    from safetensors.torch import load_file
    folder = write_random_model(baselix_models.CONFIGS["A"], 5, str(tmp_path / "random"), "bfloat16")
    arch, cfg = load_config(folder)
    assert arch.name == "Baselix" and cfg.residual_mult == 0.4 and cfg.softcap == 9.0
    tensors = load_file(folder + "/model.safetensors")
    assert set(tensors) == set(baselix_models.tensors_for(baselix_models.CONFIGS["A"], 1))
    assert float(tensors["l0.norm1"].float().abs().max()) < 0.2 and tuple(tensors["pos"].shape) == (310, 48)
    assert bool((tensors["l0.mix.dkv.norm"] == 1.0).all())
