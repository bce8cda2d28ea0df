"""Kokuvik without a GPU: the configuration reader, where checkpoint tensors land in the fused input / output projections and
the stacked experts, what the cache manager sets up for the design, and the oracle's own mechanisms on hand-made inputs."""

import copy
import math

import pytest
import torch

from tests import _kokuvik as T
from tests import _layered as L


def _geometry(cfg):
    from lite_llama_amd.model_layers import LayeredGeometry

    return LayeredGeometry.from_config(cfg, name="kokuvik")


def test_reader_takes_every_size_and_constant_from_the_configuration():
    geo = _geometry(T.CONFIGS["mix"])
    assert geo.parallel and not (geo.sandwich or geo.token_shift or geo.tied_head or geo.post_norm) and (geo.width, geo.vocab_size) == (96, 83)
    a, r, b, r2 = (layer.mixer for layer in geo.layers)
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.kv_from) == ("window_attention", 4, 2, 16, 8, 9, 3, None)
    assert a.scale == pytest.approx(1.5 / 4.0)
    assert (a.rotary.dims, a.rotary.base, a.rotary.factor, a.rotary.low, a.rotary.high, a.rotary.original) == (8, 100.0, 4.0, 0.5, 4.0, 64.0)
    assert (b.kv_from, b.window, b.keep_first) == (0, 14, 0)
    assert (r.kind, r.heads, r.dim, r.vdim, r.rotary.dims, r.decay) == ("retention", 3, 16, 24, 16, (0.75, 0.9375, 0.984375))
    assert r2.rotary.dims == 16 and r2.rotary.factor == 0.0
    dense, moe, plain = geo.layers[0].mlp, geo.layers[1].mlp, geo.layers[2].mlp
    assert (dense.kind, dense.ff, dense.act, dense.bias) == ("dense", 72, "relu_square", True) and geo.layers[3].mlp is None
    assert (moe.kind, moe.experts, moe.top, moe.ff, moe.scoring, moe.group_count, moe.group_keep, moe.shared_ff) == \
        ("moe", 6, 2, 24, "softmax_groups", 3, 2, 40)
    assert (plain.group_count, plain.group_keep, plain.shared_ff) == (1, 1, 0)
    assert _geometry(T.CONFIGS["odd"]).eps == 1e-6


def test_reader_takes_what_a_layer_leaves_out():
    cfg = copy.deepcopy(T.CONFIGS["mix"])
    for key in ("mask", "rot", "kv_heads"):
        del cfg["layers"][0]["mixer"][key]
    del cfg["layers"][1]["mixer"]["rot"], cfg["layers"][0]["mlp"]["kind"]
    cfg["layers"][2] = dict(cfg["layers"][0], mlp=None)
    geo = _geometry(cfg)
    a = geo.layers[0].mixer
    assert (a.window, a.keep_first, a.rotary, a.kv_heads) == (0, 0, None, 4) and geo.layers[1].mixer.rotary is None


@pytest.mark.parametrize("bad", ["type", "heads", "rot", "odd_rot", "top", "groups", "keep", "kind", "decay", "later", "chain", "recurrent",
                                 "shape", "turn", "bands"])
def test_reader_refuses_what_it_cannot_build(bad):
    cfg = copy.deepcopy(T.CONFIGS["mix"])
    first, second, third = (entry["mixer"] for entry in cfg["layers"][:3])
    router = cfg["layers"][1]["mlp"]["router"]
    if bad == "type":
        cfg["layers"][1]["type"] = "lstm"
    elif bad == "heads":
        first["kv_heads"] = 3
    elif bad == "rot":
        second["rot"]["dims"] = 18
    elif bad == "odd_rot":
        second["rot"]["dims"] = 7
    elif bad == "top":
        router["top"] = 5                       # two of three groups of two hold four experts
    elif bad == "groups":
        router["groups"]["count"] = 4
    elif bad == "keep":
        router["groups"]["keep"] = 4
    elif bad == "kind":
        cfg["layers"][0]["mlp"]["kind"] = "conv"
    elif bad == "decay":
        second["decay"] = [0.5]
    elif bad == "later":
        first["kv_from"] = 2
    elif bad == "chain":
        cfg["layers"].append(copy.deepcopy(cfg["layers"][2]))
        cfg["layers"][4]["mixer"]["kv_from"] = 2
    elif bad == "recurrent":
        third["kv_from"] = 1
    elif bad == "shape":
        third["vdim"] = 16
    elif bad == "turn":
        third["rot"]["base"] = 50.0
    else:
        first["rot"]["scaling"]["low"] = 4.0
        third["rot"]["scaling"]["low"] = 4.0
    with pytest.raises(ValueError):
        _geometry(cfg)


@pytest.mark.parametrize("name", sorted(T.CONFIGS))
def test_checkpoint_lands_in_the_fused_projections(tmp_path, name):
    from lite_llama_amd.weights import load_pretrained

    cfg = T.CONFIGS[name]
    tens = T.tensors(cfg, seed=3)
    model = load_pretrained(L.write(tmp_path / name, cfg, tens), device="cpu", dtype=torch.float32)
    assert torch.equal(model.embed_tokens.weight, tens["embed"]) and torch.equal(model.lm_head.weight, tens["head"])
    for i, entry in enumerate(cfg["layers"]):
        layer, m, p = model.layers[i], entry["mixer"], f"l{i}."
        w, x, H = layer.mixer.in_proj.weight, layer.mixer, entry["mixer"]["heads"]
        seen = torch.zeros(w.shape[0], dtype=torch.bool)

        def lies(at, key):
            rows = tens[key].shape[0]
            assert torch.equal(w[at:at + rows], tens[key]), key
            assert not seen[at:at + rows].any()
            seen[at:at + rows] = True

        if entry["type"] == "retention":
            for at, leaf in ((0, "q"), (x.k_off, "k"), (x.v_off, "v"), (x.g_off, "g")):
                assert at % 8 == 0
                lies(at, p + "mix." + leaf)
        else:
            own = m.get("kv_from") is None
            lies(0, p + "mix.q")
            if own:
                lies(H * m["dim"], p + "mix.k")
                lies((H + m["kv_heads"]) * m["dim"], p + "mix.v")
            lies(x.gate_off, p + "mix.g")
            assert x.gate_off % 8 == 0 and torch.equal(x.sink, tens[p + "mix.sink"]) and x.kv_heads == (m["kv_heads"] if own else 0)
        hw = H * m["vdim"]
        out = layer.out_proj.weight
        assert torch.equal(out[:, :hw], tens[p + "mix.o"])
        mlp = entry["mlp"]
        if mlp is None:
            assert out.shape[1] == hw and layer.experts is None and layer.out_proj.bias is None
        elif mlp["kind"] == "dense":
            lies(x.extra_off, p + "mlp.up")
            ff = mlp["ff"]
            bias = layer.mixer.in_proj.bias
            assert torch.equal(bias[x.extra_off:x.extra_off + ff], tens[p + "mlp.up.b"])
            assert torch.count_nonzero(bias) == torch.count_nonzero(tens[p + "mlp.up.b"])      # nobody else has one
            assert torch.equal(out[:, hw:], tens[p + "mlp.down"]) and torch.equal(layer.out_proj.bias, tens[p + "mlp.down.b"])
        else:
            ff = mlp["expert"]["ff"]
            assert layer.out_proj.bias is None and torch.equal(layer.experts.router_weight, tens[p + "mlp.router"])
            if mlp.get("shared"):
                lies(x.extra_off, p + "mlp.shared.gate")
                lies(x.extra_off + mlp["shared"]["ff"], p + "mlp.shared.up")
                assert torch.equal(out[:, hw:], tens[p + "mlp.shared.down"])
            else:
                assert out.shape[1] == hw
            for e in range(mlp["router"]["experts"]):
                assert torch.equal(layer.experts.gate_up_weight[e, :ff], tens[f"{p}mlp.e{e}.gate"])
                assert torch.equal(layer.experts.gate_up_weight[e, ff:], tens[f"{p}mlp.e{e}.up"])
                assert torch.equal(layer.experts.down_weight[e], tens[f"{p}mlp.e{e}.down"])
        assert torch.count_nonzero(w[~seen]) == 0        # padding between the members


def test_loader_names_missing_and_unknown_tensors(tmp_path):
    from lite_llama_amd.weights import load_pretrained

    cfg = T.CONFIGS["odd"]
    tens = T.tensors(cfg)
    for key, param in (("l0.mlp.up.b", "layers.0.mixer.in_proj.bias"), ("l1.mix.sink", "layers.1.mixer.sink"),
                       ("l1.mlp.shared.down", "layers.1.out_proj.weight"), ("l3.mlp.e7.up", "layers.3.experts.gate_up_weight")):
        with pytest.raises(ValueError, match=param):
            load_pretrained(L.write(tmp_path / key, cfg, {k: v for k, v in tens.items() if k != key}), device="cpu", dtype=torch.float32)
    with pytest.raises(ValueError, match="l2.mix.k"):        # a layer that borrows its keys has no projection of them
        load_pretrained(L.write(tmp_path / "b", cfg, dict(tens, **{"l2.mix.k": torch.zeros(12, 58)})), device="cpu", dtype=torch.float32)


def test_family_is_registered_and_borrowing_layers_list_the_cache_of_their_source():
    from lite_llama_amd.executor.paged_kv import PagedStateCache
    from lite_llama_amd.model_layers import LayeredLM
    from lite_llama_amd.weights import MODEL_FAMILIES, model_family

    cfg = T.CONFIGS["odd"]
    assert model_family(cfg) == "kokuvik" and "kokuvik" in MODEL_FAMILIES
    runs = LayeredLM(_geometry(cfg), dtype=torch.float32).cache_runs()
    assert [r["kind"] for r in runs] == ["recurrent", "attention", "shared", "shared"] and runs[2]["source"] == runs[3]["source"] == 1
    cache = PagedStateCache.__new__(PagedStateCache)
    cache.runs, cache.device, cache.max_requests, cache.max_tokens, cache.prev_token = runs, "cpu", 2, 32, None
    cache.kv_buffer = cache._make_buffers(len(runs), 1, 1, torch.float32)
    assert cache.kv_buffer[0] is None and cache.kv_buffer[2] is cache.kv_buffer[1] and cache.kv_buffer[3] is cache.kv_buffer[1]
    assert tuple(cache.recurrent[0].shape) == (2, 5, 10, 6) and cache.recurrent[2] is None
    assert cache.state_bytes() == 4 * (2 * 5 * 10 * 6 + 32 * (12 + 10))        # borrowed buffers are counted once
    cache.runs = [runs[0], dict(runs[2], source=0)]
    with pytest.raises(ValueError):
        cache._make_buffers(2, 1, 1, torch.float32)


def test_frequency_bands_of_product_and_oracle_agree_and_hold_their_three_ranges():
    from lite_llama_amd.model_layers import RotarySpec
    from oracle import kokuvik as O

    for kw in (dict(), dict(base=10000.0, original=1000, factor=8.0, low=1.0, high=4.0), dict(base=500000.0, original=256, low=0.25, high=32.0),
               dict(scaled=False)):
        r = T.rot(40, **kw)
        got, amp = RotarySpec.from_config(r).table()
        want = O.banded_frequencies(r)
        assert amp == 1.0 and torch.allclose(torch.tensor(got, dtype=torch.float64), want, rtol=1e-14, atol=0)
    plain = [100.0 ** (-2 * i / 40) for i in range(20)]
    f = O.banded_frequencies(T.rot(40)).tolist()        # wavelengths from 6.3 to 500; kept below 16, divided above 128
    for fi, pi in zip(f, plain):
        wave = 2 * math.pi / pi
        if wave < 16:
            assert fi == pi
        elif wave > 128:
            assert fi == pi / 4
        else:
            assert pi / 4 <= fi <= pi
    assert f[0] == plain[0] and f[-1] == plain[-1] / 4 and any(p / 4 < x < p for x, p in zip(f, plain))


def test_oracle_rotations_mask_and_sink_on_hand_made_inputs():
    from oracle import kokuvik as O

    v = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 9.0]], [[1.0, 2.0, 3.0, 4.0, 9.0]]], dtype=torch.float64)
    pos = torch.tensor([0, 2])
    a, b = 2.0, 2.0 * 100.0 ** -0.5
    pairs = O.rotate_interleaved(v, pos, {"dims": 4, "base": 100.0})
    halves = O.rotate_halves(v, pos, {"dims": 4, "base": 100.0})
    turn = lambda x, y, t: [x * math.cos(t) - y * math.sin(t), y * math.cos(t) + x * math.sin(t)]   # noqa: E731
    (p0, p1), (p2, p3) = turn(1, 2, a), turn(3, 4, b)
    (h0, h2), (h1, h3) = turn(1, 3, a), turn(2, 4, b)
    assert torch.equal(pairs[0], v[0]) and torch.allclose(pairs[1, 0], torch.tensor([p0, p1, p2, p3, 9.0], dtype=torch.float64))
    assert torch.equal(halves[0], v[0]) and torch.allclose(halves[1, 0], torch.tensor([h0, h1, h2, h3, 9.0], dtype=torch.float64))
    seen = O.visible(7, 2, 3)
    assert seen[6].tolist() == [True, True, True, False, False, True, True] and seen[1].tolist() == [True, True] + [False] * 5
    s = torch.tensor([[0.0, math.log(3.0), 5.0]], dtype=torch.float64)
    mask = torch.tensor([[True, True, False]])
    w = O.sink_softmax(s, mask, torch.tensor(math.log(4.0)))
    assert torch.allclose(w, torch.tensor([[1 / 8, 3 / 8, 0.0]], dtype=torch.float64))
    assert torch.allclose(O.sink_softmax(s, mask, torch.tensor(-900.0)), torch.tensor([[0.25, 0.75, 0.0]], dtype=torch.float64))
    assert torch.equal(O.sink_softmax(s, mask, torch.tensor(900.0)), torch.zeros(1, 3, dtype=torch.float64))


def test_oracle_retention_is_the_sum_over_decayed_keys_and_continues_from_a_state():
    from oracle import kokuvik as O

    torch.manual_seed(0)
    T_, H, dk, dv = 9, 2, 3, 4
    q, k, v = (torch.randn(T_, H, n, dtype=torch.float64) for n in (dk, dk, dv))
    decay = [0.5, 1.0]
    o, S = O.retention_scan(q, k, v, decay)
    for t in range(T_):
        for h in range(H):
            want = sum(decay[h] ** (t - u) * (q[t, h] @ k[u, h]) * v[u, h] for u in range(t + 1))
            assert torch.allclose(o[t, h], want)
    first, mid = O.retention_scan(q[:4], k[:4], v[:4], decay)
    second, end = O.retention_scan(q[4:], k[4:], v[4:], decay, mid)
    assert torch.allclose(torch.cat([first, second]), o) and torch.allclose(end, S)


def test_oracle_feed_forwards_and_routing_on_hand_made_inputs():
    from oracle import kokuvik as O

    eye = torch.eye(2, dtype=torch.float64)
    t = {"up": eye, "up.b": torch.tensor([1.0, -1.0]), "down": 2 * eye, "down.b": torch.tensor([0.5, 0.0])}
    y = O.square_mlp(torch.tensor([[2.0, 3.0], [-4.0, 0.5]], dtype=torch.float64), t, "")
    assert torch.allclose(y, torch.tensor([[18.5, 8.0], [0.5, 0.0]], dtype=torch.float64))
    # group scores are the LARGEST member: the group {3, -9} beats {2, 1.9} although its sum (and second best) is smaller
    logits = torch.tensor([[3.0, -9.0, 2.0, 1.9, 0.0, 0.5]], dtype=torch.float64)
    h = torch.ones(1, 1, dtype=torch.float64)
    p = torch.softmax(logits, -1)[0]
    ids, w = O.route(h, logits.T, 2, {"count": 3, "keep": 1})
    assert ids.tolist() == [[0, 1]] and torch.allclose(w[0], p[[0, 1]] / (p[0] + p[1]))
    ids, w = O.route(h, logits.T, 3, {"count": 3, "keep": 2})
    assert ids.tolist() == [[0, 2, 3]] and torch.allclose(w[0], p[[0, 2, 3]] / p[[0, 2, 3]].sum())
    ids, _ = O.route(h, logits.T, 4)
    assert ids.tolist() == [[0, 2, 3, 5]]


def test_oracle_borrowing_layer_reads_its_sources_keys_and_values_and_nothing_else():
    from oracle import kokuvik as O

    cfg = T.CONFIGS["odd"]
    tens = T.tensors(cfg, seed=1)
    toks = L.prompt(cfg, 14)
    layers, changed = [], []
    O.forward(toks, tens, cfg, layers_out=layers)
    # with the source layer's own result switched off the borrowing layers still move when its keys do
    quiet = dict(tens, **{"l1.mix.o": torch.zeros_like(tens["l1.mix.o"])})
    base, moved = [], []
    O.forward(toks, quiet, cfg, layers_out=base)
    O.forward(toks, dict(quiet, **{"l1.mix.k": -tens["l1.mix.k"]}), cfg, layers_out=moved)
    assert torch.equal(base[1], moved[1]) and not torch.allclose(base[2], moved[2]) and not torch.allclose(base[1], layers[1])
