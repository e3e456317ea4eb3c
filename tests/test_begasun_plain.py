"""The plain implementation of Begasun pinned by cases worked out by hand, and the package's side of the design that needs
no GPU: configuration, tensors' names, run order, caches."""
import copy
import math

import pytest
import torch

import plain_begasun as P
from begasun_configs import CONFIGS, model_dir, tensors_of

F = torch.float64
t64 = lambda *v: torch.tensor(v, dtype=F)


# ---- the plain implementation ----------------------------------------------------------------------------------------------
def test_norms():
    x = t64([3.0, 4.0])
    r = 1 / math.sqrt(12.5 + 0.5)
    assert torch.allclose(P.rms(x, 0.5), x * r)
    assert torch.allclose(P.norm_zero(x, t64(0.0, -1.0), 0.5), t64([3.0 * r, 0.0]))


def test_gelu():
    z = t64(-3.0, -0.5, 0.0, 1.0, 4.0)
    assert torch.allclose(P.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))


def test_frequencies():
    f, mag = P.frequencies(4, 100.0)
    assert f == [1.0, 0.1] and mag == 1.0
    # every pair faster than "fast" stays, every pair slower than "slow" is divided by the factor
    sc = {"factor": 10.0, "original": 1000, "fast": 1e9, "slow": 1e8}
    f, mag = P.frequencies(8, 100.0, sc)
    assert all(abs(a - b / 10.0) < 1e-15 for a, b in zip(f[1:], P.frequencies(8, 100.0)[0][1:])) and abs(mag - (0.1 * math.log(10) + 1)) < 1e-15
    f, _ = P.frequencies(8, 100.0, dict(sc, fast=1e-6, slow=1e-7))
    assert f == P.frequencies(8, 100.0)[0]
    # between them a ramp over the pairs' indices: dim(t) = 8 ln(1000 / (2 pi t)) / (2 ln 100)
    sc = {"factor": 4.0, "original": 1000, "fast": 100.0, "slow": 2.0}
    dim = lambda t: 8 * math.log(1000 / (2 * math.pi * t)) / (2 * math.log(100.0))
    lo, hi = math.floor(dim(100.0)), math.ceil(dim(2.0))
    assert (lo, hi) == (0, 4)
    f, _ = P.frequencies(8, 100.0, sc)
    plain = P.frequencies(8, 100.0)[0]
    assert all(abs(f[i] - plain[i] * (1 - i / 4 + i / 16)) < 1e-15 for i in range(4))


def test_rotations():
    x = torch.arange(1.0, 7.0, dtype=F).view(1, 1, 6)
    p = torch.tensor([3])
    c, s = math.cos(3.0), math.sin(3.0)
    c2, s2 = math.cos(0.3), math.sin(0.3)
    assert torch.allclose(P.rotate_pairs(x, p, 4, 100.0)[0, 0], t64(c - 2 * s, 2 * c + s, 3 * c2 - 4 * s2, 4 * c2 + 3 * s2, 5.0, 6.0))
    assert torch.allclose(P.rotate_half(x, p, 4, 100.0)[0, 0], t64(c - 3 * s, 2 * c2 - 4 * s2, 3 * c + s, 4 * c2 + 2 * s2, 5.0, 6.0))
    assert torch.equal(P.rotate_half(x, p, 0, 100.0), x)


def test_one_token_of_each_attention():
    """One key: the softmax is one, the output the value (times the head's gate)."""
    g = torch.Generator().manual_seed(0)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=F)
    m = {"heads": 2, "dim": 3, "rot_dim": 2, "vdim": 4, "kv_rank": 5, "scale": 0.7, "rot": {"base": 10.0}}
    w = {"q": rnd(10, 6), "dkv": rnd(7, 6), "dkv.norm": rnd(5), "uk": rnd(6, 5), "uv": rnd(8, 5), "g": rnd(2, 6), "o": torch.eye(8, dtype=F)}
    h = rnd(1, 6)
    c = P.rms((h @ w["dkv"].T)[:, :5], 1e-5) * w["dkv.norm"]
    want = (c @ w["uv"].T).view(2, 4) * torch.sigmoid(h @ w["g"].T).view(2, 1)
    assert torch.allclose(P.latent_attention(h, w, m, 1e-5).view(2, 4), want)
    m = {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 2, "scale": 0.7}
    w = {"q": rnd(12, 6), "k": rnd(6, 6), "v": rnd(4, 6), "q.norm": rnd(3), "k.norm": rnd(3), "o": torch.eye(8, dtype=F)}
    v = (h @ w["v"].T).view(2, 2)
    assert torch.allclose(P.attention(h, w, m, 1e-5).view(4, 2), v[[0, 0, 1, 1]])


def test_convolution_through_a_history():
    x, w, b = t64([1.0], [10.0], [100.0]), t64([0.5, 2.0]), t64(7.0)
    assert P.causal_conv(x, w, b).tolist() == [[9.0], [27.5], [212.0]]
    assert P.causal_conv(x[1:], w, b, history=x[:1]).tolist() == [[27.5], [212.0]]


def test_gates_and_walk_by_hand():
    """Two blocks of one channel: r and i from a channel's own number; the square root of 1 - a^2; a state handed on."""
    w = {"ra": t64([[2.0]], [[-1.0]]), "ra.b": t64([0.5], [0.0]), "ri": t64([[1.0]], [[3.0]]), "ri.b": t64([0.0], [-1.0]), "lam": t64(0.3, -2.0)}
    u = t64([1.5, -0.5])
    la, add = P.lru_gates(u, w, 2)
    sg = lambda z: 1 / (1 + math.exp(-z))
    sp = lambda z: math.log1p(math.exp(z))
    for c, (r, i) in enumerate(((sg(3.5), sg(1.5)), (sg(0.5), sg(-2.5)))):
        a = math.exp(-8 * r * sp(float(w["lam"][c])))
        assert abs(float(la[0, c]) - math.log(a)) < 1e-12
        assert abs(float(add[0, c]) - math.sqrt(1 - a * a) * i * float(u[0, c])) < 1e-12
    la, add = torch.log(t64([0.5], [0.25], [1.0])), t64([1.0], [2.0], [3.0])
    out, S = P.lru_scan(la, add)
    assert torch.allclose(out, t64([1.0], [2.25], [5.25])) and torch.allclose(S, t64(5.25))
    again, _ = P.lru_scan(la[1:], add[1:], out[0])
    assert torch.allclose(again, out[1:])


def test_clipped_feed_forward():
    eye = torch.eye(1, dtype=F)
    w = {"gate": eye, "up": -3 * eye, "down": eye}
    f = lambda z: float(P.clipped_mlp(t64([z]), w, 2.0))
    sg = lambda z: 1 / (1 + math.exp(-1.702 * z))
    assert abs(f(0.5) - 0.5 * sg(0.5) * (1 - 1.5)) < 1e-12
    assert abs(f(5.0) - 2.0 * sg(2.0) * (1 - 2.0)) < 1e-12            # gate and up at their limits
    assert abs(f(-5.0) + 5.0 * sg(-5.0) * (1 + 2.0)) < 1e-12          # the gate has no lower limit


def test_token_side():
    w = {"gate": t64([1.0, 0.0]), "proj": t64([2.0], [1.0]), "norm": t64(1.0, 3.0)}
    w["gate"] = w["gate"].view(1, 2)
    y = P.token_side(t64([0.8, 9.0]), t64([-1.5]), w, 1e-12)
    r = math.sqrt((4 + 1) / 2)
    assert torch.allclose(y, t64([-2.0 / r, -3.0 / r]))                # the norm leaves the sign


def test_run_order():
    assert P.run_order(4, None) == [(i, False) for i in range(4)]
    assert P.run_order(4, {"start": 1, "stop": 3, "times": 2}) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert P.run_order(2, {"start": 0, "stop": 1, "times": 1}) == [(0, True), (1, False)]
    assert P.run_order(2, {"start": 1, "stop": 1, "times": 5}) == [(0, False), (1, False)]


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_prefix_does_not_depend_on_what_follows(name):
    toks = [(7 * i + 3) % CONFIGS[name]["vocab"] for i in range(40)]
    full = P.forward(CONFIGS[name], tensors_of(name), toks)
    part = P.forward(CONFIGS[name], tensors_of(name), toks[:23])
    assert torch.allclose(full[:23], part, atol=1e-9)
    trace = []
    P.forward(CONFIGS[name], tensors_of(name), toks, trace=trace)
    assert len(trace) == len(P.run_order(len(CONFIGS[name]["layers"]), CONFIGS[name].get("loop")))


# ---- the package's side, without a GPU -----------------------------------------------------------------------------------
def _description(name):
    from pico_vllm_amd.config.registry import load_model_description
    return load_model_description(model_dir(name))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_model_description_names_exactly_the_checkpoints_tensors(name):
    from pico_vllm_amd.parts.model import model_param_specs
    _, cfg, spec = _description(name)
    want = {p.name: tuple(p.shape) for p in model_param_specs(spec)}
    assert want == {n: tuple(v.shape) for n, v in tensors_of(name).items()} == P.tensor_shapes(CONFIGS[name])
    assert [(e.layer, e.mix_input) for e in spec.run_order] == P.run_order(len(CONFIGS[name]["layers"]), CONFIGS[name].get("loop"))
    assert all(e.cache_of is None and not e.add_input for e in spec.run_order)       # every pass has a cache of its own


def test_what_the_configuration_says_and_does_not_say():
    from pico_vllm_amd.config.begasun import BegasunConfig
    a, c = BegasunConfig.from_dict(CONFIGS["a"]), BegasunConfig.from_dict(CONFIGS["c"])
    assert (a.embed_scale, a.logit_scale, a.loop, a.side_dim) == (3.0, 0.3, (1, 3, 3), 10)
    assert a.layers[1].mixer.scaling == (4.0, 24.0, 8.0, 1.0) and a.layers[1].mlp is None and a.layers[0].mlp.limit == 0.7
    assert (c.embed_scale, c.logit_scale, c.loop, c.side_dim) == (1.0, 1.0, None, 0)
    assert c.layers[1].mixer.rot is None and c.layers[2].mixer.rot_dim == 0
    empty = dict(CONFIGS["a"], loop={"start": 1, "stop": 1, "times": 4})
    assert BegasunConfig.from_dict(empty).loop is None


def test_what_the_configuration_refuses():
    from pico_vllm_amd.config.begasun import BegasunConfig
    from pico_vllm_amd.config.model_config import ConfigError

    def broken(change):
        raw = copy.deepcopy(CONFIGS["a"])
        change(raw)
        with pytest.raises(ConfigError):
            BegasunConfig.from_dict(raw)
    broken(lambda r: r["layers"][0].update(type="other"))
    broken(lambda r: r["layers"][0]["mixer"].pop("scale"))
    broken(lambda r: r["layers"][0]["mixer"].update(heads=4, kv_heads=3))
    broken(lambda r: r["layers"][0]["mixer"]["rot"].update(dims=7))
    broken(lambda r: r["layers"][1]["mixer"].pop("rot"))
    broken(lambda r: r["layers"][2]["mixer"].update(blocks=5))               # 36 channels
    broken(lambda r: r["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda r: r["layers"][0]["mlp"].pop("limit"))
    broken(lambda r: r["loop"].update(stop=9))
    broken(lambda r: r.pop("norm"))
    broken(lambda r: r.update(layers=[]))


def test_every_pass_of_the_loop_asks_for_a_cache_or_state_of_its_own():
    from pico_vllm_amd.cache.manager import CacheManager
    from pico_vllm_amd.parts.model import DecoderModel
    _, _, spec = _description("a")
    model = DecoderModel(spec, torch.float32, "cpu")
    specs = model.cache_specs()
    # runs: attention; latent, recurrence three times over
    assert [specs[i].kind for i in range(7)] == ["paged_kv"] + ["paged_kv", "state"] * 3 and len(specs) == 7
    assert specs[2].state_shape == (36, 4) and specs[2].state_dtype == "float32"
    m = CacheManager(specs, 8, 64, 3)
    assert sorted(len(g.layers) for g in m.groups) == [1, 3]
    assert model.is_graph_safe() and model.is_graph_safe(prompts=True)


def test_the_weights_stored_around_zero_and_the_logits_constant():
    from pico_vllm_amd.parts.norm import RMSNorm
    n = RMSNorm(3, 1e-5, weight_name="", offset=1.0, gain=0.5)
    n.load({"": torch.tensor([-1.0, 0.0, 0.25])}, torch.device("cpu"), torch.float32)
    assert n.weight.tolist() == [0.0, 0.5, 0.625]


def test_a_checkpoint_with_tensors_that_a_layer_does_not_use():
    """The second norms and vector of a layer without feed-forward may be there; anything else unknown is an error."""
    from pico_vllm_amd.weights.loader import WeightsError, load_checkpoint
    from pico_vllm_amd.parts.model import model_param_specs
    from begasun_configs import write_model
    cfg, t = CONFIGS["a"], dict(tensors_of("a"))
    t.update({"l1.norm2": torch.zeros(72), "l1.norm2b": torch.zeros(72), "l1.ls2": torch.ones(72)})
    from pico_vllm_amd.config.registry import load_model_description
    d = write_model(cfg, t)
    _, _, spec = load_model_description(d)
    load_checkpoint(d, model_param_specs(spec), torch.float32, optional=spec.ignored_tensors)
    d = write_model(cfg, dict(t, **{"l1.mix.q.b": torch.zeros(60)}))
    with pytest.raises(WeightsError):
        load_checkpoint(d, model_param_specs(spec), torch.float32, optional=spec.ignored_tensors)


def test_a_layer_names_a_whole_feed_forward_or_none():
    from pico_vllm_amd.parts.block import SandwichBlock
    from pico_vllm_amd.parts.mlp import ClippedGLUMLP
    from pico_vllm_amd.parts.norm import RMSNorm
    n = lambda: RMSNorm(8, 1e-5, weight_name="")
    with pytest.raises(ValueError):
        SandwichBlock({"norm1": n(), "mixer": None, "post1": n(), "ff": ClippedGLUMLP(8, 4, 1.0)}, size=8)
    assert [p.name for p in SandwichBlock({"norm1": n(), "mixer": None, "post1": n()}, size=8).own_param_specs()] == ["ls1"]
