"""The plain Vosurax pinned by cases worked out by hand, and the design's reader, spec and cache needs (CPU)."""

import copy
import math

import pytest
import torch

import plain_vosurax as plain
from vosurax_fixtures import CONFIGS

F64 = torch.float64


def t64(values):
    return torch.tensor(values, dtype=F64)


def test_norms_by_hand():
    x = t64([[3.0, -4.0]])                                             # mean square 12.5
    assert torch.allclose(plain.over_rms(x, 0.0), x / math.sqrt(12.5))
    assert torch.allclose(plain.over_rms(x, 3.5), x / 4.0)             # the eps is inside the root
    assert torch.allclose(plain.stream_norm(x, t64([0.5, -1.0]), 3.5), t64([[1.125, 0.0]]))


def test_the_rotation_pairs_the_halves_and_leaves_the_rest():
    x = torch.arange(1, 7, dtype=F64).view(1, 1, 6)
    rot = {"dims": 4, "base": 100.0}
    assert plain.rotate(x, rot).flatten().tolist() == [1, 2, 3, 4, 5, 6]        # position 0 turns nothing
    a0, a1 = 3.0, 3.0 * 100.0 ** -0.5
    want = [1 * math.cos(a0) - 3 * math.sin(a0), 2 * math.cos(a1) - 4 * math.sin(a1),
            3 * math.cos(a0) + 1 * math.sin(a0), 4 * math.cos(a1) + 2 * math.sin(a1), 5, 6]
    assert torch.allclose(plain.rotate(x, rot, first_position=3).flatten(), t64(want))


def test_a_query_sees_its_own_chunk_up_to_itself():
    seen = plain.seen_in_chunks(5, 2).tolist()
    assert [[j for j in range(5) if row[j]] for row in seen] == [[0], [0, 1], [2], [2, 3], [4]]
    assert [sum(row) for row in plain.seen_in_chunks(3, None).tolist()] == [1, 2, 3]


def test_attention_by_hand():
    # one token: the softmax is 1, so the output is the value (with its bias) times the gate
    m = {"heads": 2, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 1.0, "mask": {"size": 4}}
    w = {"q": t64([[1.0], [1.0]]), "q.b": t64([0.0, 0.0]), "k": t64([[1.0]]), "k.b": t64([0.0]), "v": t64([[3.0]]),
         "v.b": t64([0.5]), "q.norm": t64([1.0]), "k.norm": t64([1.0]), "g": t64([[0.0], [math.log(3.0)]]),
         "o": t64([[1.0, 10.0]])}
    got = plain.chunked_attention(w, "", m, t64([[1.0]]), 1e-12)
    assert torch.allclose(got, t64([[3.5 * 0.5 + 10.0 * 3.5 * 0.75]]))
    # two tokens whose normed keys are both 1 (the norm takes the size away): half of each value
    w["g"] = t64([[100.0], [100.0]])
    got = plain.chunked_attention(w, "", m, t64([[1.0], [2.0]]), 1e-12)
    assert torch.allclose(got[1], t64([11.0 * (3.5 + 6.5) / 2]))
    # ... unless the second begins a chunk of its own
    got = plain.chunked_attention(w, "", {**m, "mask": {"size": 1}}, t64([[1.0], [2.0]]), 1e-12)
    assert torch.allclose(got[1], t64([11.0 * 6.5]))


def test_the_matrix_memory_by_hand():
    q, k, v = t64([[1.0], [2.0]]), t64([[2.0], [1.0]]), t64([[3.0], [5.0]])
    li, lf = t64([-1.0, 0.5]), t64([-0.25, -2.0])
    out, (S, n, m) = plain.matrix_memory_scan(q, k, v, li, lf)
    # the running maximum starts at 0 and not at minus infinity: m_1 = max(-0.25 + 0, -1)
    m1 = -0.25
    s1, n1 = 6.0 * math.exp(-1.0 - m1), 2.0 * math.exp(-1.0 - m1)
    assert torch.allclose(out[0], t64([s1 / (max(n1, math.exp(-m1)) + 1e-6)]))      # here the floor counts
    assert n1 < math.exp(-m1)
    m2 = max(-2.0 + m1, 0.5)
    s2 = math.exp(-2.0 + m1 - m2) * s1 + math.exp(0.5 - m2) * 5.0
    n2 = math.exp(-2.0 + m1 - m2) * n1 + math.exp(0.5 - m2) * 1.0
    assert 2 * n2 > math.exp(-m2)                                                   # here the normaliser
    assert torch.allclose(out[1], t64([2 * s2 / (2 * n2 + 1e-6)]))
    assert torch.allclose(S, t64([[s2]])) and torch.allclose(n, t64([n2])) and m == m2
    # cut after the first token
    first, state = plain.matrix_memory_scan(q[:1], k[:1], v[:1], li[:1], lf[:1])
    second, _ = plain.matrix_memory_scan(q[1:], k[1:], v[1:], li[1:], lf[1:], state)
    assert torch.allclose(torch.cat([first, second]), out)


def test_gates_are_capped():
    assert torch.allclose(plain.capped(t64([1e9, -1e9, 0.0]), 4.0), t64([4.0, -4.0, 0.0]))
    assert torch.allclose(plain.capped(t64([2.0]), 4.0), t64([4.0 * math.tanh(0.5)]))


def test_retention_by_hand():
    out, S = plain.retention_scan(t64([[1.0], [3.0]]), t64([[2.0], [0.5]]), t64([[4.0], [6.0]]), 0.5, t64([[10.0]]))
    s1 = 5.0 + 8.0
    s2 = s1 / 2 + 3.0
    assert torch.allclose(out, t64([[s1], [3 * s2]])) and torch.allclose(S, t64([[s2]]))


def test_both_branches_are_normed_before_they_are_halved():
    eps, h = 1e-5, torch.randn(3, 6, dtype=F64, generator=torch.Generator().manual_seed(1))
    m = {"left": {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0},
         "right": {"heads": 1, "dim": 2, "vdim": 2, "gate_cap": 5.0}}
    g = torch.Generator().manual_seed(2)
    shapes = {"left.q": (2, 6), "left.q.b": (2,), "left.k": (2, 6), "left.k.b": (2,), "left.v": (2, 6), "left.v.b": (2,),
              "left.q.norm": (2,), "left.k.norm": (2,), "left.g": (2, 6), "left.o": (6, 2), "right.q": (2, 6),
              "right.k": (2, 6), "right.v": (2, 6), "right.g": (2, 6), "right.o": (6, 2), "right.norm": (2,),
              "right.i": (1, 6), "right.i.b": (1,), "right.f": (1, 6), "right.f.b": (1,), "left.out": (6,),
              "right.out": (6,)}
    w = {n: torch.randn(*s, dtype=F64, generator=g) for n, s in shapes.items()}
    base = plain.parallel_mixer(w, "", m, h, eps)
    big = plain.parallel_mixer({**w, "left.o": w["left.o"] * 1000.0}, "", m, h, 0.0)
    assert torch.allclose(base, big, atol=1e-2)                    # a branch's size does not count, its direction does
    alone = plain.parallel_mixer({**w, "left.out": w["left.out"] * 0.0, "right.out": t64([1.0] * 6)}, "", m, h, 0.0)
    assert torch.allclose((alone * alone).mean(-1), t64([0.25] * 3))


def test_gelu_tanh_by_its_limits():
    z = t64([-20.0, 0.0, 20.0, 1.0])
    inner = math.sqrt(2 / math.pi) * 1.044715
    assert torch.allclose(plain.gelu_tanh(z), t64([0.0, 0.0, 20.0, 0.5 * (1 + math.tanh(inner))]))


def test_a_routing_choice_by_hand():
    chosen, weights = plain.route(t64([[0.0, 2.0, 1.0, 2.0]]), 3)
    assert chosen.tolist() == [[1, 3, 2]]                               # a tie goes to the lower index
    s = lambda z: 1 / (1 + math.exp(-z))                                # noqa: E731
    assert torch.allclose(weights, t64([[s(2), s(2), s(1)]]))           # as they are, not made to sum to 1


def test_a_weight_multiplies_the_experts_input():
    w = {"router": t64([[0.0]]), "e0.gate": t64([[2.0]]), "e0.up": t64([[3.0]]), "e0.down": t64([[1.0]])}
    got = plain.routed_experts(w, "", {"expert": {"ff": 1}, "router": {"experts": 1, "top": 1}}, t64([[4.0]]))
    x = 0.5 * 4.0                                                       # sigmoid(0) times the row
    assert torch.allclose(got, t64([[2 * x / (1 + math.exp(-2 * x)) * 3 * x]]))
    w.update({"shared.gate": w["e0.gate"], "shared.up": w["e0.up"], "shared.down": w["e0.down"]})
    both = plain.routed_experts(w, "", {"expert": {"ff": 1}, "router": {"experts": 1, "top": 1}, "shared": {"ff": 1}},
                                t64([[4.0]]))
    assert torch.allclose(both - got, t64([[8 / (1 + math.exp(-8.0)) * 12]]))       # the shared one sees the row itself


def test_the_run_order_of_a_loop():
    layers = [None] * 4
    assert plain.run_order({"layers": layers}) == [(0, None), (1, None), (2, None), (3, None)]
    assert plain.run_order({"layers": layers, "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert plain.run_order({"layers": layers, "loop": {"start": 3, "stop": 4, "times": 3}})[3:] == [(3, 0), (3, 1), (3, 2)]


# ----------------------------------------------------------------------------------- reader, registry, spec
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_reader_and_the_spec(name):
    import tie_amd  # noqa: F401
    from tie_amd.cache.spec import FixedState, PagedKV
    from tie_amd.models.builder import model_from_config

    config = CONFIGS[name]
    model = model_from_config(config)
    assert model.spec.architecture == "Vosurax"
    shapes = {s.name: tuple(s.shape) for s in model.expected_tensors()}
    assert {"embed", "head", "final.norm"} <= set(shapes)
    order = plain.run_order(config)
    assert [c.layer for c in model.spec.order] == [i for i, _ in order]
    assert {i: s.row for i, s in model.stages.items()} == {i: t for i, (_, t) in enumerate(order) if t is not None}
    loop = config.get("loop")
    assert shapes.get("loop.step") == ((loop["times"], config["width"]) if loop else None)
    groups = {g.need: g.num_planes for g in model.cache_plan.groups}
    expected = {}
    for i, _ in order:                                          # every run of a layer has a cache of its own
        m = config["layers"][i]["mixer"]
        if config["layers"][i]["type"] == "retention":
            needs = [FixedState((m["heads"], m["dim"], m["vdim"]))]
        else:
            left, right = m["left"], m["right"]
            size = max(left["dim"], left["vdim"])
            size = -(-size // 16) * 16
            needs = [PagedKV(left["kv_heads"], size, None, (left.get("mask") or {}).get("size")),
                     FixedState((right["heads"], right["dim"], right["vdim"])),
                     FixedState((right["heads"], -(-right["vdim"] // 32), right["dim"] + 1))]
        for need in needs:
            expected[need] = expected.get(need, 0) + 1
    assert groups == expected
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        if layer["type"] == "parallel":
            left, right = m["left"], m["right"]
            assert shapes[p + "left.g"] == (left["heads"] * left["vdim"], config["width"])
            assert shapes[p + "left.q.norm"] == (left["dim"],) and shapes[p + "left.v.b"] == (left["kv_heads"] * left["vdim"],)
            assert shapes[p + "right.norm"] == (right["heads"] * right["vdim"],) and shapes[p + "right.f.b"] == (right["heads"],)
            assert shapes[p + "left.out"] == shapes[p + "right.out"] == (config["width"],)
        else:
            assert shapes[p + "g"] == (m["heads"] * m["vdim"], config["width"]) and p + "norm" not in shapes
        mlp = layer["mlp"]
        assert (f"l{i}.norm2" in shapes) == (mlp is not None)
        assert (f"l{i}.mlp.router" in shapes) == (mlp is not None and mlp["kind"] == "moe")
        assert (f"l{i}.mlp.shared.up" in shapes) == (mlp is not None and "shared" in mlp)
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

    left, right = ("layers", 0, "mixer", "left"), ("layers", 0, "mixer", "right")
    for path, value, error in [
        ((*left, "kv_heads"), 4, LoadError),
        ((*left, "scale"), 0.0, LoadError),
        ((*left, "mask", "size"), 0, LoadError),
        ((*right, "gate_cap"), 0.0, LoadError),
        ((*right, "heads"), 0, LoadError),
        ((*right, "dim"), 513, InvalidArgument),                               # more than the kernels keep
        (("layers", 0, "mixer", "right"), None, LoadError),
        (("layers", 1, "mixer", "decay"), [0.9, 0.99, 1.0], LoadError),        # one head's is missing
        (("layers", 1, "mixer", "decay"), [0.9, 0.99, 1.0, -0.5], LoadError),
        (("layers", 1, "mixer", "rot", "dims"), 18, LoadError),
        (("layers", 1, "mixer", "rot", "dims"), 5, LoadError),
        (("layers", 1, "mlp", "router", "top"), 7, LoadError),
        (("layers", 1, "mlp", "shared", "ff"), 0, LoadError),
        (("layers", 1, "mlp", "kind"), "gated", UnsupportedError),
        (("layers", 2, "type"), "attention", UnsupportedError),
        (("loop", "stop"), 6, LoadError),
        (("loop", "stop"), 1, LoadError),
        (("loop", "times"), 0, LoadError),
        (("norm", "eps"), 0.0, LoadError),
        (("width",), 0, LoadError),
        (("layers",), [], LoadError),
    ]:
        with pytest.raises(error):
            model_from_config(changed(path, value))


def test_keys_that_may_be_absent():
    import tie_amd  # noqa: F401
    from tie_amd.config.vosurax import VosuraxConfig

    config = copy.deepcopy(CONFIGS["A"])
    config["loop"] = None
    for node, keys in ((config["layers"][0]["mixer"]["left"], ("kv_heads", "vdim", "mask")),
                       (config["layers"][0]["mixer"]["right"], ("vdim",)), (config["layers"][1]["mixer"], ("vdim",)),
                       (config["layers"][1]["mixer"]["rot"], ("dims",)), (config["layers"][1]["mlp"], ("shared",))):
        for key in keys:
            node.pop(key)
    read = VosuraxConfig.from_json(config)
    assert read.loop is None
    left, right = read.layers[0].mixer.left, read.layers[0].mixer.right
    assert (left.kv_heads, left.vdim, left.chunk) == (left.heads, left.dim, None) and right.vdim == right.dim
    assert read.layers[1].mixer.vdim == read.layers[1].mixer.dim == read.layers[1].mixer.rotation.dims
    assert read.layers[1].mlp.shared_ff is None


def test_layers_of_one_shape_may_run_from_one_launch_list():
    import tie_amd  # noqa: F401
    from tie_amd.models.builder import model_from_config

    def alike(config):
        model = model_from_config(config)
        model._find_layers_alike()
        return model._alike

    assert alike(CONFIGS["D"]) == {0: 5}
    assert alike(CONFIGS["F"]) == {4: 9}
    assert alike({**CONFIGS["D"], "loop": {"start": 0, "stop": 1, "times": 1}}) == {1: 5}      # a vector comes before it
    config = copy.deepcopy(CONFIGS["D"])
    config["layers"][2]["mixer"]["right"]["gate_cap"] = 5.5
    assert alike(config) == {}                      # no four alike in a row
    config = copy.deepcopy(CONFIGS["F"])
    config["layers"][3]["mixer"]["decay"][1] = 0.98
    assert alike(config) == {}
