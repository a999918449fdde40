"""Varolix on the host: the configuration, the order of the layer runs and the cache each asks for, what is refused, which
mixers can stand beside each other, and the plain implementation's own mechanisms (tests/plain_varolix.py)."""
import copy
import math

import pytest
import torch

import plain_varolix as plain
import varolix_models
from bare_cuda_4gib_amd.config import VarolixConfig
from bare_cuda_4gib_amd.config.registry import architecture_for
from bare_cuda_4gib_amd.errors import ConfigError


def described(config):
    arch = architecture_for(config)
    assert arch.name == "Varolix"
    cfg = arch.config_class.from_dict(config)
    from bare_cuda_4gib_amd.engine.model import Model
    return cfg, Model(arch.describe(cfg))


@pytest.mark.parametrize("name", sorted(varolix_models.CONFIGS))
def test_the_model_wants_exactly_the_tensors_of_the_design(name):
    config = varolix_models.CONFIGS[name]
    _, model = described(config)
    want = {k: tuple(v.shape) for k, v in varolix_models.tensors_for(config, 1).items()}
    assert {k: tuple(v.shape) for k, v in model.expected_weights().items()} == want


def test_the_configuration_reads_back():
    for config in varolix_models.CONFIGS.values():
        cfg = VarolixConfig.from_dict(config)
        again = VarolixConfig.from_dict(cfg.to_dict())
        assert again == cfg and architecture_for(cfg.to_dict()).name == "Varolix"


def test_the_order_of_the_runs_and_a_cache_for_each():
    from bare_cuda_4gib_amd.cache.specs import Bundle, PagedHeads, PagedLatent, States
    _, model = described(varolix_models.CONFIGS["A"])
    assert [(e.layer, e.cache, e.writes) for e in model.schedule] == [
        (0, (0, 0), True), (1, (1, 0), True), (0, (0, 1), True), (1, (1, 1), True), (2, (2, 0), True)]
    both = Bundle((("left", PagedHeads(2, 12, 2, 10)), ("right", States((("S", (3, 8, 14), "float32"), ("n", (3, 8), "float32"), ("m", (3,), "float32"))))))
    heads = PagedHeads(3, 10, 3, 14)
    assert model.cache_streams() == {(0, 0): both, (1, 0): heads, (0, 1): both, (1, 1): heads, (2, 0): PagedLatent(20, 6)}
    for name in sorted(varolix_models.CONFIGS):
        config = varolix_models.CONFIGS[name]
        cfg, _ = described(config)
        class Order:                      # noqa: E306
            cfg = config
        assert [i for i, _ in VarolixConfig.from_dict(config).runs()] == plain.PlainVarolix.order(Order)
    config = copy.deepcopy(varolix_models.CONFIGS["A"])
    config["loop"] = dict(start=1, stop=1, times=4)              # (an empty run of layers)
    assert VarolixConfig.from_dict(config).runs() == [(0, 0), (1, 0), (2, 0)]


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].__setitem__("type", "attention_2"), "type"),
    (lambda c: c["layers"].__setitem__(1, 7), "type"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].pop("kv_heads"), "lacks kv_heads"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_heads", 4), "cannot share"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 12), "12 rotated"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][0]["mixer"].pop("left"), "left"),
    (lambda c: c["layers"][0]["mixer"].pop("right_scale"), "right_scale"),
    (lambda c: c["layers"][0]["mixer"]["right"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][0]["mixer"]["right"].__setitem__("gate_cap", 0.0), "cap"),
    (lambda c: c["layers"][0]["mixer"]["right"].__setitem__("dim", 300), "256"),
    (lambda c: c["layers"][0]["mixer"]["left"]["q_temp"].__setitem__("every", 0), "every"),
    (lambda c: c["layers"][2]["mixer"].pop("q_rank"), "lacks q_rank"),
    (lambda c: c["layers"][2]["mixer"]["rot"].__setitem__("dims", 8), "rotated"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_rank", 5000), "beyond"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "moe"), "kind"),
    (lambda c: c["loop"].__setitem__("stop", 4), "does not fit"),
    (lambda c: c["loop"].__setitem__("times", 0), "does not fit"),
    (lambda c: c["norm"].__setitem__("eps", -1.0), "eps"),
    (lambda c: c.__setitem__("layers", []), "layers"),
])
def test_what_is_refused(change, message):
    config = copy.deepcopy(varolix_models.CONFIGS["A"])
    change(config)
    with pytest.raises(ConfigError, match=message):
        described(config)


def test_absent_keys_have_the_design_s_defaults():
    cfg, model = described(varolix_models.CONFIGS["C"])
    assert model.layers[0].mixer.position is None and model.layers[1].ffn is None and model.layers[1].ffn_norm is None
    left = model.layers[1].mixer.sides["left"]
    assert left.temperature is None and left.head_norm and left.out_bias and left.bias and not left.sink and not left.unit_sink
    assert model.layers[2].mixer.position.scaling is None
    assert [e.cache for e in model.schedule] == [(0, 0), (1, 0), (2, 0), (3, 0)] and cfg.max_seq_len == 1 << 20


def test_which_mixers_can_stand_beside_each_other():
    """Any two that say so, whichever side they stand on; those with a convolution or heads that mix their weights do not."""
    from bare_cuda_4gib_amd.engine.spec import PartSpec
    from bare_cuda_4gib_amd.parts import build_part
    memory = PartSpec("matrix_memory", dict(hidden_size=16, heads=2, dim=4, vdim=6, gate_cap=5.0, eps=1e-5))
    heads = dict(hidden_size=16, heads=2, kv_heads=1, dim=4, vdim=8, scale=0.5, sink=False)
    part = build_part("mixer", PartSpec("parallel", dict(left=memory, right=PartSpec("sink_attention", heads))))
    assert set(part.weight_specs()) == {"left." + n for n in ("q", "k", "v", "g", "i", "i.b", "f", "f.b", "norm", "o")} | {
        "right." + n for n in ("q", "k", "v", "o")}
    assert [n for n, _ in part.cache_spec().members] == ["left", "right"]
    for other, message in ((PartSpec("sink_attention", dict(heads, conv_taps=3)), "cannot stand"),
                           (PartSpec("sink_attention", dict(heads, talking=True)), "cannot stand"),
                           (PartSpec("retention", dict(hidden_size=16, heads=1, dim=4, vdim=4, decay=[0.9], eps=1e-5)), "cannot stand"),
                           (PartSpec("sink_attention", dict(heads, hidden_size=24)), "widths")):
        with pytest.raises(ConfigError, match=message):
            build_part("mixer", PartSpec("parallel", dict(left=memory, right=other)))
    # the work of a step is the two sides' own, counted once
    from bare_cuda_4gib_amd.engine.batch import HostBatch
    batch = HostBatch(n_tokens=3, n_seqs=1, seq_start=[0, 3], seq_ctx=[5], seq_slots=[0], max_q_len=3, max_kv_len=8)
    alone = [side.step_work(batch, 3, 2) for side in part.sides.values()]
    assert part.step_work(batch, 3, 2) == (alone[0][0] + alone[1][0], alone[0][1] + alone[1][1])


def test_parts_that_do_not_fit_together_are_refused():
    from bare_cuda_4gib_amd.parts.feedforward import SwiGLU
    from bare_cuda_4gib_amd.parts.latent_attention import LatentAttention
    from bare_cuda_4gib_amd.parts.linear_attention import MatrixMemory
    from bare_cuda_4gib_amd.parts.sink_attention import SinkAttention
    base = dict(hidden_size=8, heads=2, kv_heads=2, dim=4, vdim=4, scale=1.0)
    for make, message in ((lambda: SinkAttention(**base, head_norm=True, row_norm=True), "not both"),
                          (lambda: SinkAttention(**base, temperature=(0.1, 0)), "temperature"),
                          (lambda: SwiGLU(8, 8, act="relu"), "activation"),
                          (lambda: LatentAttention(hidden_size=8, heads=2, dim=4, vdim=4, kv_rank=6, scale=0.5, eps=1e-5, pairing="other"), "pairing"),
                          (lambda: MatrixMemory(hidden_size=8, heads=0, dim=4, vdim=4, gate_cap=1.0, eps=1e-5), "heads")):
        with pytest.raises(ConfigError, match=message):
            make()
    with pytest.raises(ConfigError, match="moved"):
        MatrixMemory(hidden_size=8, heads=1, dim=4, vdim=4, gate_cap=1.0, eps=1e-5).run_heads(torch.zeros(1, 18), None, None, writes=False)


def test_a_latent_s_tensors_with_and_without_a_latent_of_the_queries():
    from bare_cuda_4gib_amd.parts.latent_attention import LatentAttention
    base = dict(hidden_size=8, heads=2, dim=4, rot_dim=2, rot_dims=2, vdim=4, kv_rank=6, scale=0.5, eps=1e-5, sink=False)
    assert set(LatentAttention(**base).weight_specs()) == {"q", "dkv", "dkv.norm", "uk", "uv", "o"}
    low = LatentAttention(**base, q_rank=3, head_gate=True).weight_specs()
    assert set(low) == {"dq", "dq.norm", "uq", "g", "dkv", "dkv.norm", "uk", "uv", "o"} and low["uq"].shape == (12, 3) and low["g"].shape == (2, 8)


def test_the_rotary_part_s_frequencies_are_the_plain_ones():
    from bare_cuda_4gib_amd.parts.position import Rotary
    for dims, base, scaling in ((6, 10000.0, (8.0, 64, 8.0, 1.0)), (32, 100.0, (4.0, 100, 20.0, 2.0)), (16, 50.0, (2.0, 7, 1.0, 1.0)), (8, 1e6, None), (2, 3.0, (5.0, 40, 3.0, 1.0))):
        s = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
        mine, amp = Rotary(base, dims, scaling=s).frequencies()
        theirs, amplitude = plain.turning_speeds(dims, base, s)
        assert torch.allclose(torch.tensor(mine, dtype=torch.float64), theirs, rtol=1e-12) and abs(amp - amplitude) < 1e-12


def test_the_plain_mechanisms():
    torch.manual_seed(0)
    f64 = torch.float64
    z = torch.linspace(-6, 6, 50, dtype=f64)
    assert torch.allclose(plain.gelu_by_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert plain.query_temperature(torch.tensor([0, 2, 3, 6, 7, 70]), 0.5, 4).tolist() == [
        1.0, 1.0, 1.0 + 0.5 * math.log(2.0), 1.0 + 0.5 * math.log(2.0), 1.0 + 0.5 * math.log(3.0), 1.0 + 0.5 * math.log(18.0)]
    v, pos = torch.randn(4, 2, 7, dtype=f64), torch.tensor([0, 1, 9, 50])
    speeds, amp = plain.turning_speeds(4, 100.0)
    turned = plain.turn_halves(v, pos, speeds, amp)
    assert torch.equal(turned[0], v[0]) and torch.equal(turned[..., 4:], v[..., 4:])
    assert torch.allclose((turned[..., :4] ** 2).sum(-1), (v[..., :4] ** 2).sum(-1))
    c, s = math.cos(9 * 0.1), math.sin(9 * 0.1)                  # (the second pair: elements 1 and 3, speed 100^(-1/2))
    assert torch.allclose(turned[2, :, 1], v[2, :, 1] * c - v[2, :, 3] * s) and torch.allclose(turned[2, :, 3], v[2, :, 3] * c + v[2, :, 1] * s)
    scores, sink = torch.randn(2, 5, 5, dtype=f64), torch.tensor([0.3, -1.0], dtype=f64)
    w = plain.causal_weights(scores, sink)
    e = torch.tril(torch.exp(scores))
    assert torch.allclose(w, e / (torch.exp(sink)[:, None, None] + e.sum(-1, keepdim=True))) and torch.allclose(
        plain.causal_weights(scores).sum(-1), torch.ones(2, 5, dtype=f64))
    # the memory without its maximum: sums of exponentials of the gates, divided by their own size or one
    T, d, n = 9, 4, 3
    q, k, vv = torch.randn(T, d, dtype=f64), torch.randn(T, d, dtype=f64), torch.randn(T, n, dtype=f64)
    i, f = torch.randn(T, dtype=f64) * 3, plain.log_forget_gate(torch.randn(T, dtype=f64) * 4, 5.0)
    out, (S, nn, m) = plain.matrix_memory(q, k, vv, i, f)
    F = torch.cumsum(f, 0)
    for t in range(T):
        wt = torch.exp(F[t] - F[:t + 1] + i[:t + 1]) * (k[:t + 1] @ q[t])
        top = max([float(F[t])] + [float(F[t] - F[j] + i[j]) for j in range(t + 1)])
        want = (wt @ vv[:t + 1]) * math.exp(-top) / (max(abs(float(wt.sum())) * math.exp(-top), math.exp(-top)) + 1e-6)
        assert torch.allclose(out[t], want, atol=1e-12)
    assert abs(float(m) - top) < 1e-12
    head, state = plain.matrix_memory(q[:4], k[:4], vv[:4], i[:4], f[:4])
    rest, end = plain.matrix_memory(q[4:], k[4:], vv[4:], i[4:], f[4:], state)
    assert torch.allclose(torch.cat([head, rest]), out) and torch.allclose(end[0], S) and torch.allclose(end[1], nn)


@pytest.mark.parametrize("name", sorted(varolix_models.CONFIGS))
def test_the_plain_model_does_not_look_ahead_and_every_piece_counts(name, tmp_path):
    folder = varolix_models.write_folder(tmp_path, name, "float32")
    model = plain.PlainVarolix(folder)
    ids = [(7 * i + 3) % model.cfg["vocab"] for i in range(40)]
    whole, after = model.forward(ids, return_layers=True)
    assert len(after) == len(model.order()) and bool(torch.isfinite(whole).all())
    assert torch.allclose(model.forward(ids[:23]), whole[:23], atol=1e-5, rtol=1e-5)
    for key in sorted(model.w):
        kept = model.w[key].clone()
        # (another draw of the same size rather than a multiple: a norm behind a tensor would take a multiple back out)
        model.w[key] = kept + torch.randn(kept.shape, generator=torch.Generator().manual_seed(1), dtype=kept.dtype) * float(kept.abs().mean()) * 0.5
        moved = float((model.forward(ids) - whole).abs().max())
        unused = key.endswith(".k.b") and ".left." not in key and "rot" not in model.cfg["layers"][int(key[1])]["mixer"]    # (the same for every key: the softmax takes it out)
        assert moved > 1e-5 or unused, key
        model.w[key] = kept


def test_the_random_weights_mode_writes_a_folder_that_loads(tmp_path):
    from bare_cuda_4gib_amd.config.registry import load_config
    from bare_cuda_4gib_amd.weights import write_random_model
    from safetensors.torch import load_file
    folder = write_random_model(varolix_models.CONFIGS["A"], 5, str(tmp_path / "random"), "bfloat16")
    arch, cfg = load_config(folder)
    assert arch.name == "Varolix" and cfg.norm_eps == 1e-5
    tensors = load_file(folder + "/model.safetensors")
    assert set(tensors) == set(varolix_models.tensors_for(varolix_models.CONFIGS["A"], 1))
    assert bool((tensors["l0.norm1"] == 1.0).all()) and bool((tensors["l2.mix.dq.norm"] == 1.0).all())
