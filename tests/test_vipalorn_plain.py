"""The plain Vipalorn pinned by cases worked out by hand, and the design's reader, spec and cache needs (CPU)."""

import copy
import math

import pytest
import torch

import plain_vipalorn as plain
from vipalorn_fixtures import CONFIGS

F64 = torch.float64


def test_layer_norm_by_hand():
    x = torch.tensor([[1.0, 3.0, 5.0, 7.0]], dtype=F64)                 # mean 4, deviations -3 -1 1 3, variance 5
    out = plain.layer_norm(x, torch.tensor([1.0, 2.0, 1.0, 0.0], dtype=F64), 4.0)
    assert torch.allclose(out, torch.tensor([[-1.0, -2 / 3, 1 / 3, 0.0]], dtype=F64))


def test_the_rotation_pairs_the_halves():
    x = torch.arange(1, 7, dtype=F64).view(1, 1, 6)
    rot = {"dims": 4, "base": 100.0}
    assert plain.rotate(x, rot).flatten().tolist() == [1, 2, 3, 4, 5, 6]        # position 0 turns nothing
    a0, a1 = 3.0, 3.0 * 100.0 ** -0.5
    want = [1 * math.cos(a0) - 3 * math.sin(a0), 2 * math.cos(a1) - 4 * math.sin(a1),
            3 * math.cos(a0) + 1 * math.sin(a0), 4 * math.cos(a1) + 2 * math.sin(a1), 5, 6]
    assert torch.allclose(plain.rotate(x, rot, first_position=3).flatten(), torch.tensor(want, dtype=F64))


def test_a_query_sees_itself_and_what_came_before():
    p = plain.causal_softmax(torch.zeros(1, 3, 3, dtype=F64))[0]
    assert torch.allclose(p, torch.tensor([[1, 0, 0], [0.5, 0.5, 0], [1 / 3, 1 / 3, 1 / 3]], dtype=F64))


def test_a_convolution_starts_from_zeros_and_ends_with_the_current_token():
    u = torch.tensor([[1.0], [10.0], [100.0]], dtype=F64)
    w = torch.tensor([[2.0, 3.0, 5.0]], dtype=F64)
    assert plain.short_convolution(u, w).flatten().tolist() == [5.0, 53.0, 532.0]


def test_the_delta_rule_by_hand():
    # one key row, one value column: S <- g S; u = beta (v - S k); S <- S + k u; o = S q, the write seen by the read
    q, k = torch.tensor([[2.0], [1.0]], dtype=F64), torch.tensor([[1.0], [0.5]], dtype=F64)
    v, beta, decay = torch.tensor([[4.0], [6.0]], dtype=F64), torch.tensor([0.5, 1.0], dtype=F64), torch.tensor([0.9, 0.25], dtype=F64)
    out, S = plain.delta_rule_scan(q, k, v, beta, decay, torch.tensor([[2.0]], dtype=F64))
    s1 = 1.8 + 0.5 * (4.0 - 1.8)
    s2 = 0.25 * s1 + 0.5 * (6.0 - 0.5 * 0.25 * s1)
    assert torch.allclose(out, torch.tensor([[2 * s1], [s2]], dtype=F64)) and torch.allclose(S, torch.tensor([[s2]], dtype=F64))


def test_an_expert_cuts_its_sums_off():
    s = lambda g: g / (1 + math.exp(-1.702 * g))                       # noqa: E731
    gate = torch.tensor([5.0, -5.0, 0.5], dtype=F64)                   # above the limit; far below: not cut; inside
    up = torch.tensor([3.0, -3.0, 0.25], dtype=F64)                    # cut at both ends; inside
    want = [s(1.0) * 2.0, s(-5.0) * 0.0, s(0.5) * 1.25]
    assert torch.allclose(plain.clipped_gate(gate, up, 1.0), torch.tensor(want, dtype=F64))


def test_a_routing_choice_by_hand():
    z = torch.tensor([[0.0, 2.0, 1.0, 2.0]], dtype=F64)
    chosen, weights = plain.route(z, 3)
    assert chosen.tolist() == [[1, 3, 2]]                               # a tie goes to the lower index
    total = 2 * math.e ** 2 + math.e                                    # only the chosen share the softmax
    assert torch.allclose(weights, torch.tensor([[math.e ** 2, math.e ** 2, math.e]], dtype=F64) / total)


# ----------------------------------------------------------------------------------- reader, registry, spec
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_reader_and_the_spec(name):
    import tie_amd  # noqa: F401
    from tie_amd.cache.spec import FixedState, PagedKV
    from tie_amd.models.builder import model_from_config

    config = CONFIGS[name]
    model = model_from_config(config)
    assert model.spec.architecture == "Vipalorn"
    shapes = {s.name: tuple(s.shape) for s in model.expected_tensors()}
    assert {"embed", "embed.norm", "final.norm"} <= set(shapes) and "head" not in shapes
    needs = [g.need for g in model.cache_plan.groups]
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        assert f"l{i}.norm1" in shapes and f"l{i}.norm2" not in shapes
        if layer["type"] == "latent_attention":
            assert shapes[p + "g"] == (m["heads"], config["width"])                  # one gate a head
            size = -(-(m["kv_rank"] + m["rot_dim"]) // 16) * 16
            assert PagedKV(1, size, None) in needs                                   # one head: nothing per head
        else:
            assert shapes[p + "a"] == (m["heads"], config["width"]) and shapes[p + "dt_bias"] == (m["heads"],)
            assert shapes[p + "g"] == (m["heads"] * m["vdim"], config["width"])
            assert FixedState((m["heads"], m["dim"], m["vdim"])) in needs
            channels = 2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"]
            assert m["conv"] == 1 or FixedState((m["conv"] - 1, channels)) in needs
        mlp = layer["mlp"]
        assert (f"l{i}.mlp.router.b" in shapes) == (mlp is not None)
        if mlp is not None:
            experts = mlp["router"]["experts"]
            assert {f"l{i}.mlp.e{e}.{k}" for e in range(experts) for k in ("gate", "up", "down")} <= set(shapes)
            assert f"l{i}.mlp.e{experts}.up" not in shapes
    assert model.capturable()


def test_what_does_not_fit_is_refused():
    import tie_amd  # noqa: F401
    from tie_amd.errors import InvalidArgument, LoadError, UnsupportedError
    from tie_amd.models.builder import model_from_config

    def changed(path, value):
        config = copy.deepcopy(CONFIGS["A"])
        node = config
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = value
        return config

    for path, value, error in [
        (("layers", 1, "mixer", "kv_heads"), 3, LoadError),
        (("layers", 0, "mixer", "rot", "dims"), 10, LoadError),               # more than the rotated part holds
        (("layers", 0, "mixer", "rot", "dims"), 3, LoadError),
        (("layers", 0, "mixer", "rot"), None, LoadError),
        (("layers", 0, "mixer", "kv_rank"), 0, LoadError),
        (("layers", 0, "mlp", "router", "top"), 7, LoadError),
        (("layers", 0, "mlp", "expert", "limit"), 0.0, LoadError),
        (("layers", 0, "mlp", "kind"), "dense", UnsupportedError),
        (("layers", 1, "mixer", "conv"), 0, LoadError),
        (("layers", 1, "mixer", "conv"), 9, InvalidArgument),                 # more taps than the kernels take
        (("layers", 2, "type"), "attention", UnsupportedError),
        (("norm", "eps"), 0.0, LoadError),
        (("width",), 0, LoadError),
        (("layers",), [], LoadError),
    ]:
        with pytest.raises(error):
            model_from_config(changed(path, value))


def test_keys_that_may_be_absent():
    import tie_amd  # noqa: F401
    from tie_amd.config.vipalorn import VipalornConfig

    config = copy.deepcopy(CONFIGS["A"])
    config.pop("residual_mult")
    config.pop("logit_scale")
    for key in ("kv_heads", "vdim", "conv"):
        config["layers"][1]["mixer"].pop(key)
    config["layers"][0]["mixer"].pop("vdim")
    config["layers"][0]["mixer"]["rot"].pop("dims")
    read = VipalornConfig.from_json(config)
    assert read.residual_mult == 1.0 and read.logit_scale == 1.0
    delta, latent = read.layers[1].mixer, read.layers[0].mixer
    assert (delta.kv_heads, delta.vdim, delta.conv) == (delta.heads, delta.dim, 1)
    assert latent.vdim == latent.dim and latent.rotation.dims == latent.rot_dim


def test_layers_of_one_shape_may_run_from_one_launch_list():
    import tie_amd  # noqa: F401
    from tie_amd.models.builder import model_from_config

    config = copy.deepcopy(CONFIGS["D"])
    model = model_from_config(config)
    model._find_layers_alike()
    assert model._alike == {0: 5}
    config["layers"][2]["mlp"]["expert"]["limit"] = 2.0
    model = model_from_config(config)
    model._find_layers_alike()
    assert model._alike == {}                       # no four alike in a row
