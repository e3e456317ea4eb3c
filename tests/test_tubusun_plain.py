"""The plain implementation of Tubusun pinned by cases worked out by hand, and the package's side of the design that needs no
GPU: configuration, tensors' names, run order, caches."""
import copy
import math

import pytest
import torch

import plain_tubusun as P
from begasun_configs import write_model
from tubusun_configs import CONFIGS, model_dir, tensors_of

F = torch.float64
t64 = lambda *v: torch.tensor(v, dtype=F)
sigmoid = lambda z: 1 / (1 + math.exp(-z))


# ---- the plain implementation ----------------------------------------------------------------------------------------------
def test_norm_and_activations():
    assert torch.allclose(P.rms(t64([3.0, 4.0]), 0.5), t64([3.0, 4.0]) / math.sqrt(13.0))
    z = t64(-3.0, -0.5, 0.0, 1.0, 4.0)
    assert torch.allclose(P.gelu_erf(z), torch.nn.functional.gelu(z))
    assert torch.allclose(P.silu(z), torch.nn.functional.silu(z))


def test_rotation_of_neighbours():
    x = torch.arange(1.0, 7.0, dtype=F).view(1, 1, 6)
    c, s, c2, s2 = math.cos(3.0), math.sin(3.0), math.cos(0.3), math.sin(0.3)
    got = P.rotate_pairs(x, torch.tensor([3]), 4, 100.0)[0, 0]
    assert torch.allclose(got, t64(c - 2 * s, 2 * c + s, 3 * c2 - 4 * s2, 4 * c2 + 3 * s2, 5.0, 6.0))
    assert torch.equal(P.rotate_pairs(x, torch.tensor([3]), 0, 100.0), x)


def test_a_window_of_three_sees_itself_and_two_in_front():
    assert P.seen(5, 3).int().tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [1, 1, 1, 0, 0], [0, 1, 1, 1, 0], [0, 0, 1, 1, 1]]
    assert P.seen(3, 0).int().tolist() == [[1, 0, 0], [1, 1, 0], [1, 1, 1]]


def test_a_sink_counts_once_unscaled_and_never_overflows():
    s = torch.log(t64([2.0, 7.0], [3.0, 5.0]))
    p = P.sink_softmax(s, P.seen(2, 0), torch.tensor(math.log(4.0), dtype=F))
    assert torch.allclose(p, t64([2 / 6, 0.0], [3 / 12, 5 / 12]))
    p = P.sink_softmax(t64([1.0]), P.seen(1, 0), torch.tensor(2000.0, dtype=F))
    assert p.tolist() == [[0.0]]


def test_one_token_of_attention():
    """One key: its score is scale times dk (unit lengths: a root mean square of one) whatever its size, if it is the query."""
    g = torch.Generator().manual_seed(0)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=F)
    m = {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 2, "scale": 0.7, "mask": {"size": 4}, "rot": {"dims": 2, "base": 10.0}}
    k = rnd(2, 3, 6)
    w = {"q": 5 * k.repeat_interleave(2, dim=0).reshape(12, 6), "k": k.reshape(6, 6), "v": rnd(4, 6), "g": rnd(4, 6), "sink": t64(0.5, -1.0, 2.0, 3.0)}
    h = rnd(1, 6)
    v = (h @ w["v"].T).view(2, 2)[[0, 0, 1, 1]]
    e = math.exp(0.7 * 3)
    want = v * torch.sigmoid(h @ w["g"].T).view(4, 1) * (e / (e + torch.exp(w["sink"]))).view(4, 1)
    assert torch.allclose(P.attention(h, w, m, 1e-15, first_pos=9).view(4, 2), want)


def test_decayed_sums_by_hand_and_from_a_state():
    q, k, v = t64([[1.0]], [[2.0]], [[1.0]]), t64([[3.0]], [[1.0]], [[0.0]]), t64([[2.0]], [[5.0]], [[7.0]])
    o, S = P.decayed_sums(q, k, v, [0.5])
    assert o.flatten().tolist() == [6.0, 16.0, 4.0] and S.flatten().tolist() == [4.0]
    again, _ = P.decayed_sums(q[1:], k[1:], v[1:], [0.5], S0=t64([[6.0]]))
    assert again.flatten().tolist() == [16.0, 4.0]
    # two heads, keys and values of two entries: the sums written out
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(4, 2, 2, generator=g, dtype=F) for _ in range(3))
    o, _ = P.decayed_sums(q, k, v, [0.3, 0.9])
    for h, d in enumerate((0.3, 0.9)):
        want = sum(d ** (3 - j) * (q[3, h] @ k[j, h]) * v[j, h] for j in range(4))
        assert torch.allclose(o[3, h], want)


def test_one_token_of_lightning_attention():
    """All heads are normed as one row."""
    w = {"q": t64([1.0], [2.0]), "k": t64([-1.0], [0.5]), "v": t64([3.0], [1.0]), "g": t64([0.0], [2.0]), "norm": t64(1.0, 4.0)}
    x = 0.8
    si = lambda z: z * sigmoid(z)
    o = [si(1 * x) * si(-1 * x) * si(3 * x), si(2 * x) * si(0.5 * x) * si(1 * x)]
    r = math.sqrt((o[0] ** 2 + o[1] ** 2) / 2 + 1e-3)
    got = P.lightning(t64([x]), w, {"heads": 2, "dim": 1, "vdim": 1, "decay": [0.5, 0.9]}, 1e-3)
    assert torch.allclose(got, t64([o[0] / r * 0.5, o[1] / r * 4 * sigmoid(2 * x)]))


def test_two_mixers_side_by_side():
    cfg, t = CONFIGS["a"], {k: v.to(F) for k, v in tensors_of("a").items()}
    m, w = cfg["layers"][0]["mixer"], P.under("l0.mix", t)
    h = torch.randn(5, 72, generator=torch.Generator().manual_seed(0), dtype=F)
    both = P.parallel(h, w, m, 1e-5)
    only = lambda ls, rs: P.parallel(h, w, dict(m, left_scale=ls, right_scale=rs), 1e-5)
    assert torch.allclose(both, 0.6 * only(1.0, 0.0) + 1.5 * only(0.0, 1.0))
    assert torch.allclose(P.parallel(h, w, {k: m[k] for k in ("left", "right")}, 1e-5), only(1.0, 1.0))


def test_dense_feed_forward():
    w = {"up": t64([2.0]), "up.b": t64(-1.0), "down": t64([3.0]), "down.b": t64(0.25)}
    z = 2 * 0.7 - 1
    assert torch.allclose(P.dense_mlp(t64([0.7]), w), t64([3 * 0.5 * z * (1 + math.erf(z / math.sqrt(2))) + 0.25]))


def test_the_choice_of_experts_by_groups():
    """The expert with the largest score may stand in a group that is not kept; with one expert a group its score is the
    group's; the weights are the scores as they are."""
    eye = torch.eye(6, dtype=F)
    z = t64([3.0, -5.0, 1.0, 1.2, 2.0, -1.0])
    s = lambda *i: torch.sigmoid(z[0, list(i)])
    c, w = P.route(z, eye, {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}})
    assert c.tolist() == [[3, 2]] and torch.allclose(w[0], s(3, 2))
    c, w = P.route(z, eye, {"experts": 6, "top": 3, "groups": {"count": 3, "keep": 2}})        # sums 0.96, 1.50, 1.15
    assert c.tolist() == [[4, 3, 2]] and torch.allclose(w[0], s(4, 3, 2))
    for r in ({"experts": 6, "top": 2}, {"experts": 6, "top": 2, "groups": {"count": 1, "keep": 1}},
              {"experts": 6, "top": 2, "groups": {"count": 6, "keep": 2}}):
        assert P.route(z, eye, r)[0].tolist() == [[0, 4]]
    m = P.route_margin(z, eye, {"experts": 6, "top": 1, "groups": {"count": 3, "keep": 1}})
    assert torch.allclose(m, torch.minimum((s(2) + s(3) - s(4) - s(5)) / 2, s(3) - s(2)))


def test_an_expert_at_and_beyond_its_limits_and_the_weight_on_its_output():
    one = t64([1.0])
    f = lambda z: float(P.expert(t64([z]), one, -3 * one, one, 2.0))
    sg = lambda z: 1 / (1 + math.exp(-1.702 * z))
    assert abs(f(0.5) - 0.5 * sg(0.5) * (1 - 1.5)) < 1e-12
    assert abs(f(5.0) - 2.0 * sg(2.0) * (1 - 2.0)) < 1e-12
    assert abs(f(-5.0) + 5.0 * sg(-5.0) * (1 + 2.0)) < 1e-12                # the gate has no lower limit
    w = {"router": t64([0.4]), "e0.gate": one, "e0.up": -3 * one, "e0.down": one}
    got = P.routed_mlp(t64([5.0]), w, {"expert": {"limit": 2.0}, "router": {"experts": 1, "top": 1}})
    assert abs(float(got) - sigmoid(2.0) * f(5.0)) < 1e-12


def test_run_order():
    assert P.run_order(3, None) == [(0, None), (1, None), (2, None)]
    assert P.run_order(4, {"start": 1, "stop": 3, "times": 2}) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert P.run_order(2, {"start": 0, "stop": 1, "times": 1}) == [(0, 0), (1, None)]
    assert P.run_order(2, {"start": 1, "stop": 1, "times": 5}) == [(0, None), (1, None)]


def test_a_pass_adds_its_own_vector_once():
    """Layers whose outputs' norms have weights of zero leave the stream alone: what is left are the vectors."""
    cfg, t = CONFIGS["b"], {k: v.clone() for k, v in tensors_of("b").items()}
    for k in t:
        if k.endswith(("norm1b", "norm2b")):
            t[k].zero_()
    trace = []
    P.forward(cfg, t, [5, 9], trace=trace)
    x, st = t["embed"][[5, 9]].to(F) * 0.5, t["loop.step"].to(F)
    want = [x, x + st[0], x + st[0], x + st[0] + st[1], x + st[0] + st[1], x + st[0] + st[1]]
    assert len(trace) == 6 and all(torch.allclose(a, b) for a, b in zip(trace, want))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_prefix_does_not_depend_on_what_follows(name):
    toks = [(7 * i + 3) % CONFIGS[name]["vocab"] for i in range(40)]
    full = P.forward(CONFIGS[name], tensors_of(name), toks)
    part = P.forward(CONFIGS[name], tensors_of(name), toks[:23])
    assert torch.allclose(full[:23], part, atol=1e-9)
    cap = CONFIGS[name].get("logit_softcap")
    assert not cap or float(full.abs().max()) < cap


# ---- the package's side, without a GPU -----------------------------------------------------------------------------------
def _description(name):
    from pico_vllm_amd.config.registry import load_model_description
    return load_model_description(model_dir(name))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_model_description_names_exactly_the_checkpoints_tensors(name):
    from pico_vllm_amd.parts.model import model_param_specs
    _, cfg, spec = _description(name)
    want = {p.name: tuple(p.shape) for p in model_param_specs(spec)}
    have = {n: tuple(v.shape) for n, v in tensors_of(name).items()}
    unused = {n for n in have if n in spec.ignored_tensors}                # the second norms of a layer without feed-forward
    assert want == {n: s for n, s in have.items() if n not in unused} and have == P.tensor_shapes(CONFIGS[name])
    assert all(n.endswith(("norm2", "norm2b")) for n in unused)
    assert [(e.layer, e.add_vector) for e in spec.run_order] == P.run_order(len(CONFIGS[name]["layers"]), CONFIGS[name].get("loop"))
    assert all(e.cache_of is None and not e.add_input and not e.mix_input for e in spec.run_order)     # every pass: a cache of its own


def test_what_the_configuration_says_and_does_not_say():
    from pico_vllm_amd.config.tubusun import TubusunConfig
    a, c = TubusunConfig.from_dict(CONFIGS["a"]), TubusunConfig.from_dict(CONFIGS["c"])
    assert (a.embed_scale, a.logit_softcap, a.loop) == (3.0, 8.0, (1, 3, 3))
    m = a.layers[0].mixer
    assert (m.left.window, m.left.rot_dims, m.left.rot_base, m.left_scale, m.right_scale) == (21, 10, 300.0, 0.6, 1.5)
    assert a.layers[1].mlp is None and (a.layers[2].mlp.groups, a.layers[2].mlp.keep, a.layers[2].mlp.limit) == (3, 2, 0.7)
    assert (c.embed_scale, c.logit_softcap, c.loop) == (1.0, 0.0, None)
    assert (c.layers[0].mixer.left.window, c.layers[0].mixer.left.rot_dims, c.layers[0].mixer.left_scale) == (0, 0, 1.0)
    assert (c.layers[0].mlp.groups, c.layers[0].mlp.keep) == (1, 1)
    assert TubusunConfig.from_dict(dict(CONFIGS["a"], loop={"start": 1, "stop": 1, "times": 4})).loop is None


def test_what_the_configuration_refuses():
    from pico_vllm_amd.config.tubusun import TubusunConfig
    from pico_vllm_amd.config.model_config import ConfigError

    def broken(change):
        raw = copy.deepcopy(CONFIGS["a"])
        change(raw)
        with pytest.raises(ConfigError):
            TubusunConfig.from_dict(raw)
    mixer = lambda r: r["layers"][0]["mixer"]
    broken(lambda r: r["layers"][0].update(type="other"))
    broken(lambda r: mixer(r).pop("right"))
    broken(lambda r: mixer(r)["left"].pop("scale"))
    broken(lambda r: mixer(r)["left"].update(heads=4, kv_heads=3))
    broken(lambda r: mixer(r)["left"]["rot"].update(dims=7))
    broken(lambda r: mixer(r)["left"]["mask"].update(size=0))
    broken(lambda r: mixer(r)["right"].update(decay=[0.5]))
    broken(lambda r: mixer(r)["right"].update(decay=[0.5, 1.5]))
    broken(lambda r: r["layers"][0]["mlp"].update(kind="other"))
    broken(lambda r: r["layers"][2]["mlp"]["router"]["groups"].update(count=4))          # nine experts
    broken(lambda r: r["layers"][2]["mlp"]["router"].update(top=7))                      # two groups of three
    broken(lambda r: r["layers"][2]["mlp"]["expert"].pop("limit"))
    broken(lambda r: r["loop"].update(stop=9))
    broken(lambda r: r.pop("norm"))
    broken(lambda r: r.update(layers=[]))


def test_every_pass_of_the_loop_asks_for_a_cache_and_a_state_of_its_own():
    from pico_vllm_amd.cache.manager import CacheManager
    from pico_vllm_amd.parts.model import DecoderModel
    _, _, spec = _description("a")
    model = DecoderModel(spec, torch.float32, "cpu")
    specs = model.cache_specs()
    assert sorted(specs) == [(i, s) for i in range(7) for s in (0, 1)]
    assert all(specs[(i, 0)].kind == "paged_kv" and specs[(i, 1)].kind == "state" for i in range(7))
    assert [specs[(i, 0)].window for i in range(7)] == [21, 5, 33, 5, 33, 5, 33]
    assert specs[(1, 1)].state_shape == (3, 12, 8) and specs[(1, 1)].state_dtype == "float32"
    m = CacheManager(specs, 8, 64, 3)
    assert sorted(len(g.layers) for g in m.groups) == [1, 3, 3]
    assert model.is_graph_safe() and model.is_graph_safe(prompts=True)


def test_the_joined_products_of_two_mixers():
    """Columns and rows of both sides in one matrix each, padded with zeros to whole eights between them."""
    from pico_vllm_amd.parts.model import DecoderModel
    _, _, spec = _description("a")
    model = DecoderModel(spec, torch.float32, "cpu")
    part = model.layers[0].mixer
    t = {n[len("l0.mix."):]: v.float() for n, v in tensors_of("a").items() if n.startswith("l0.mix.")}
    part.load(t, torch.device("cpu"), torch.float32)
    n = 3 * 24 + 24 + 40 + 3
    assert part.in_rows == [n, 2 * (9 + 9 + 11 + 11)] and part.in_at == (0, 144) and part.out_at == (0, 120) and part.out_total == 144
    w = part.proj.weight
    assert torch.equal(w[:72], t["left.q"]) and torch.equal(w[136:139], t["left.g"]) and float(w[139:144].abs().max()) == 0
    assert torch.equal(w[144:162], t["right.q"]) and torch.equal(w[202:224], t["right.g"])
    assert torch.equal(part.o.weight[:, :120], t["left.o"]) and torch.equal(part.o.weight[:, 120:142], t["right.o"])
    assert float(part.o.weight[:, 142:].abs().max()) == 0
    assert part.left.out_scale == 0.6 and torch.allclose(part.right.norm_weight, 1.5 * t["right.norm"])


def test_a_sum_of_mixers_wants_mixers_that_open_their_products():
    from pico_vllm_amd.parts.registry import build_part
    from pico_vllm_amd.parts.spec import PartSpec
    r = PartSpec("lightning_attention", {"hidden_size": 8, "num_heads": 1, "key_dim": 4, "value_dim": 4, "decay": (0.5,), "norm_eps": 1e-5})
    g = PartSpec("retention", dict(r.params))
    build_part("mixer", PartSpec("mixer_sum", {"hidden_size": 8, "left": r, "right": r}))
    with pytest.raises(TypeError):
        build_part("mixer", PartSpec("mixer_sum", {"hidden_size": 8, "left": r, "right": g}))


def test_a_run_order_that_adds_a_vector_the_model_does_not_have():
    import dataclasses
    from pico_vllm_amd.parts.model import DecoderModel
    _, _, spec = _description("a")
    with pytest.raises(ValueError):
        DecoderModel(dataclasses.replace(spec, run_vectors=("loop.step", 2)), torch.float32, "cpu")


def test_a_checkpoint_with_tensors_that_a_layer_does_not_use():
    """The second norms of a layer without feed-forward may be there or not; anything else unknown is an error."""
    from pico_vllm_amd.config.registry import load_model_description
    from pico_vllm_amd.parts.model import model_param_specs
    from pico_vllm_amd.weights.loader import WeightsError, load_checkpoint
    cfg, t = CONFIGS["a"], dict(tensors_of("a"))
    less = {k: v for k, v in t.items() if k not in ("l1.norm2", "l1.norm2b")}
    for tensors in (t, less):
        d = write_model(cfg, tensors)
        _, _, spec = load_model_description(d)
        load_checkpoint(d, model_param_specs(spec), torch.float32, optional=spec.ignored_tensors)
    d = write_model(cfg, dict(t, **{"l1.mix.left.q.b": torch.zeros(20)}))
    with pytest.raises(WeightsError):
        load_checkpoint(d, model_param_specs(spec), torch.float32, optional=spec.ignored_tensors)
