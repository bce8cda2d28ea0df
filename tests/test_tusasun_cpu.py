"""Tusasun without a GPU: the configuration reader (with the sizes that only a tensor's shape gives), where checkpoint tensors
land in the fused, padded, block-diagonal and transposed parameters, what the cache manager is asked to set up for the design,
the distance buckets, and the oracle's own mechanisms on hand-made inputs."""

import copy
import math

import pytest
import torch

from tests import _layered as L
from tests import _tusasun as T

F64 = torch.float64


def _folder(tmp_path, name, seed=0):
    cfg = T.CONFIGS[name]
    tens = T.tensors(cfg, seed=seed)
    return L.write(tmp_path / name, T.on_disk(cfg), tens), T.on_disk(cfg), tens


def _geometry(cfg, shapes=None):
    from lite_llama_amd.model_layers import LayeredGeometry

    return LayeredGeometry.from_config(cfg, name="tusasun", shapes=shapes)


def test_reader_takes_sizes_and_constants_from_the_configuration_and_the_rest_from_shapes(tmp_path):
    from lite_llama_amd.weights import tensor_shapes

    folder, cfg, _ = _folder(tmp_path, "mix")
    geo = _geometry(cfg, tensor_shapes(folder))
    assert (geo.width, geo.vocab_size, geo.streams, geo.norm_base) == (96, 83, 4, 1.0) and not (geo.tied_head or geo.token_shift or geo.loop_mix)
    assert geo.run_order() == [(0, 0, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False), (3, 0, False)]
    a, b, c, e = (layer.mixer for layer in geo.layers)
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.conv_taps, a.decay_rank, a.gate_rank) == ("channel_delta", 4, 2, 16, 24, 4, 8, 16)
    assert (b.kind, b.heads, b.kv_heads, b.dim, b.vdim, b.bias_rows, b.bias_max, b.softcap) == ("distance_attention", 4, 2, 16, 8, 16, 40.0, 15.0)
    assert b.scale == pytest.approx(1.5 / 4) and (c.kind, c.width, c.blocks, c.conv_taps) == ("rglru", 48, 3, 3)
    assert e.bias_rows == 8 and geo.layers[3].mlp is None
    m = geo.layers[0].mlp
    assert (m.kind, m.experts, m.top, m.ff, m.shared_ff, m.scoring, m.act) == ("moe", 6, 3, 24, 40, "sigmoid_plain", "relu_square")
    with pytest.raises(ValueError):
        _geometry(cfg)                     # (without the shapes the ranks and the number of buckets are unknown)


@pytest.mark.parametrize("bad", ["type", "heads", "blocks", "top", "kind", "reach", "streams", "loop", "taps"])
def test_reader_refuses_what_it_cannot_build(bad):
    cfg = copy.deepcopy(T.on_disk(T.CONFIGS["mix"]))
    shapes = {"l0.mix.a1": (8, 96), "l0.mix.g1": (16, 96), "l1.mix.rel": (16, 4), "l3.mix.rel": (8, 2)}
    _geometry(cfg, shapes)
    if bad == "type":
        cfg["layers"][0]["type"] = "lstm"
    elif bad == "heads":
        cfg["layers"][0]["mixer"]["kv_heads"] = 3
    elif bad == "blocks":
        cfg["layers"][2]["mixer"]["blocks"] = 5
    elif bad == "top":
        cfg["layers"][1]["mlp"]["router"]["top"] = 5
    elif bad == "kind":
        cfg["layers"][0]["mlp"]["kind"] = "dense"
    elif bad == "reach":
        cfg["layers"][1]["mixer"]["bias_max"] = 8
    elif bad == "streams":
        cfg["streams"] = 0
    elif bad == "loop":
        cfg["loop"]["stop"] = 9
    else:
        cfg["layers"][2]["mixer"]["conv"] = 0
    with pytest.raises(ValueError):
        _geometry(cfg, shapes)


@pytest.mark.parametrize("name", sorted(T.CONFIGS))
def test_checkpoint_lands_in_the_fused_parameters(tmp_path, name):
    from lite_llama_amd.weights import load_pretrained

    folder, cfg, tens = _folder(tmp_path, name, seed=3)
    model = load_pretrained(folder, device="cpu", dtype=torch.float32)
    assert torch.equal(model.embed_tokens.weight, tens["embed"]) and torch.equal(model.lm_head.weight, tens["head"])
    assert not hasattr(model, "loop_in")
    for i, entry in enumerate(cfg["layers"]):
        layer, p, m = model.layers[i], f"l{i}.", entry["mixer"]
        x = layer.mixer
        w, run = x.in_proj.weight, x.cache_run()
        for n in (1, 2) if entry["mlp"] else (1,):
            mix = getattr(layer, f"mix{n}")
            for leaf, got in (("hc%d.in", mix.gather), ("hc%d.out", mix.out), ("hc%d.mix", mix.mix), ("ls%d", mix.scale)):
                assert torch.equal(got, tens[p + leaf % n])
        if entry["type"] == "attention":
            q, k, v = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
            for leaf, first, count in (("q", 0, q), ("k", q, k), ("v", q + k, v)):
                assert torch.equal(w[first:first + count], tens[p + "mix." + leaf])
                assert torch.equal(x.in_proj.bias[first:first + count], tens[p + f"mix.{leaf}.b"])
            assert torch.equal(x.o_proj.bias, tens[p + "mix.o.b"]) and torch.equal(x.bias_table, tens[p + "mix.rel"])
            assert run == {"kind": "attention", "kv_heads": m["kv_heads"], "dk": m["dim"], "dv": m["vdim"]}
        elif entry["type"] == "channel_delta":
            qk, v, gk = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"], m["heads"] * m["dim"]
            at = 0
            for leaf, count in (("q", qk), ("k", qk), ("v", v)):
                assert torch.equal(w[at:at + count], tens[p + "mix." + leaf])
                assert torch.equal(x.conv_weight[at:at + count], tens[p + f"mix.{leaf}.conv"])
                at += count
            ra, rg = tens[p + "mix.a1"].shape[0], tens[p + "mix.g1"].shape[0]
            assert torch.equal(w[x.low_off:x.low_off + ra], tens[p + "mix.a1"]) and torch.equal(w[x.low_off + ra:x.low_off + ra + rg], tens[p + "mix.g1"])
            assert torch.equal(w[x.beta_off:x.beta_off + m["heads"]], tens[p + "mix.b"])
            assert x.low_off % 8 == 0 and x.beta_off % 8 == 0 and w.shape[0] % 8 == 0
            used = torch.zeros(w.shape[0], dtype=torch.bool)
            for lo, count in ((0, 2 * qk + v), (x.low_off, ra + rg), (x.beta_off, m["heads"])):
                used[lo:lo + count] = True
            assert not w[~used].any()                             # (padding between the members stays zero)
            low = x.low_proj.weight
            assert torch.equal(low[:gk, :ra], tens[p + "mix.a2"]) and torch.equal(low[x.gate_off:x.gate_off + v, ra:], tens[p + "mix.g2"])
            assert not low[:gk, ra:].any() and not low[x.gate_off:, :ra].any()
            assert run == {"kind": "recurrent", "heads": m["heads"], "dk": m["dim"], "dv": m["vdim"], "conv_taps": m["conv"],
                           "conv_channels": 2 * qk + v}
        else:
            C, bs = m["width"], m["width"] // m["blocks"]
            assert torch.equal(w[:C], tens[p + "mix.x"]) and torch.equal(w[x.y_off:x.y_off + C], tens[p + "mix.y"])
            assert torch.equal(x.in_proj.bias[x.y_off:x.y_off + C], tens[p + "mix.y.b"])
            for b in range(m["blocks"]):
                assert torch.equal(x.gate_weight[b, :, :bs], tens[p + "mix.ra"][b].T) and torch.equal(x.gate_weight[b, :, bs:], tens[p + "mix.ri"][b].T)
            assert torch.equal(x.r_bias, tens[p + "mix.ra.b"].flatten()) and torch.equal(x.i_bias, tens[p + "mix.ri.b"].flatten())
            assert run == {"kind": "recurrent", "heads": 1, "dk": 1, "dv": C, "conv_taps": m["conv"], "conv_channels": C}
        mlp = entry["mlp"]
        if mlp is None:
            assert layer.mlp is None
            continue
        for e in range(mlp["router"]["experts"]):
            assert torch.equal(layer.mlp.up_weight[e], tens[f"{p}mlp.e{e}.up"]) and torch.equal(layer.mlp.down_weight[e], tens[f"{p}mlp.e{e}.down"])
        assert torch.equal(layer.mlp.shared_scale_weight, tens[p + "mlp.shared.sg"])


def test_loader_names_missing_partial_and_unknown_tensors(tmp_path):
    from lite_llama_amd.weights import load_pretrained

    cfg = T.CONFIGS["mix"]
    tens = T.tensors(cfg)
    for k, leaf in enumerate(("l0.mix.dt_bias", "l0.mix.b", "l0.mix.g2", "l2.mix.ri", "l1.hc2.mix")):   # (whole parameters, and parts of fused ones)
        missing = dict(tens)
        del missing[leaf]
        with pytest.raises(ValueError, match="never written|partially written"):
            load_pretrained(L.write(tmp_path / f"a{k}", T.on_disk(cfg), missing), device="cpu", dtype=torch.float32)
    extra = dict(tens, **{"l1.mix.sink": torch.zeros(2)})
    with pytest.raises(ValueError, match="sink"):
        load_pretrained(L.write(tmp_path / "b", T.on_disk(cfg), extra), device="cpu", dtype=torch.float32)


def test_cache_keeps_one_set_per_layer_run(tmp_path):
    """A layer that runs several times keeps its rows or its state, and its carried convolution rows, once per pass."""
    from lite_llama_amd.weights import load_pretrained

    folder, _, _ = _folder(tmp_path, "odd")
    runs = load_pretrained(folder, device="cpu", dtype=torch.float32).cache_runs()
    assert [r["kind"] for r in runs] == ["recurrent"] * 6 + ["attention", "recurrent"]
    assert [r.get("conv_taps") for r in runs] == [6, 1, 6, 1, 6, 1, None, 6]


def test_the_trace_replay_and_the_engine_know_the_family():
    from lite_llama_amd.weights import MODEL_FAMILIES, model_family

    assert model_family({"architecture": "Tusasun"}) == "tusasun" and "tusasun" in MODEL_FAMILIES


@pytest.mark.parametrize("rows,far", [(16, 40.0), (8, 20.0), (6, 9.0), (32, 300.0), (2, 2.0), (64, 2048.0), (10, 5.5), (32, 64.0)])
def test_distance_buckets_of_the_product_and_of_the_oracle(rows, far):
    from lite_llama_amd.model_layers import distance_buckets
    from oracle import tusasun as O

    table = distance_buckets(rows, far)
    assert table[-1] == rows - 1 and table.count(rows - 1) == 1 and table == sorted(table)
    for n in range(int(far) + 40):
        assert table[min(n, len(table) - 1)] == O.distance_bucket(n, rows, far)


# ------------------------------------------------------------------------------------------------------------------- #
# the oracle's mechanisms on inputs small enough to do by hand
# ------------------------------------------------------------------------------------------------------------------- #
def test_oracle_buckets_by_hand():
    from oracle import tusasun as O

    # eight buckets up to 64: 0 .. 3 one distance each, then 4, 8, 16 and 32 open the others
    got = [O.distance_bucket(n, 8, 64.0) for n in (0, 3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 1000)]
    assert got == [0, 3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]


def test_oracle_scores_cap_first_then_add_the_unscaled_bias():
    from oracle import tusasun as O

    q, k = torch.tensor([[0.0], [4.0]], dtype=F64), torch.tensor([[3.0], [1.0]], dtype=F64)
    s = O.attention_scores(q, k, 0.5, 2.0, torch.tensor([10.0, 20.0], dtype=F64), 2.0)
    assert s[0, 0] == 10.0 and s[0, 1] == -math.inf
    assert s[1, 0].item() == pytest.approx(2.0 * math.tanh(6.0 / 2.0) + 20.0) and s[1, 1].item() == pytest.approx(2.0 * math.tanh(1.0) + 10.0)


def test_oracle_delta_rule_decays_corrects_and_reads_its_own_write():
    from oracle import tusasun as O

    k = torch.tensor([[1.0, 0.0], [1.0, 0.0]], dtype=F64)
    q = torch.tensor([[1.0, 0.0], [2.0, 0.0]], dtype=F64)
    v, beta = torch.tensor([[8.0], [4.0]], dtype=F64), torch.tensor([0.5, 0.25], dtype=F64)
    g = torch.tensor([[0.9, 0.1], [0.5, 0.1]], dtype=F64)
    o, S = O.delta_scan(q, k, v, g, beta)
    # token 0: u = 0.5 * 8 = 4; token 1: S = 2, u = 0.25 * (4 - 2) = 0.5, S = 2.5
    assert o[:, 0].tolist() == [4.0, 5.0] and S[:, 0].tolist() == [2.5, 0.0]


def test_oracle_real_gated_recurrence_has_no_special_first_token():
    from oracle import tusasun as O

    lam = torch.tensor([0.3], dtype=F64)
    r, i, u = torch.tensor([[0.5], [1.0]], dtype=F64), torch.tensor([[0.5], [1.0]], dtype=F64), torch.tensor([[4.0], [2.0]], dtype=F64)
    S, last = O.real_gated_scan(u, r, i, lam)
    sp = math.log1p(math.exp(0.3))
    a0, a1 = math.exp(-4.0 * sp), math.exp(-8.0 * sp)
    s0 = math.sqrt(1 - a0 * a0) * 2.0
    assert S[0, 0].item() == pytest.approx(s0) and last[0].item() == pytest.approx(a1 * s0 + math.sqrt(1 - a1 * a1) * 2.0)


def test_oracle_gates_use_one_matrix_per_part():
    from oracle import tusasun as O

    w = torch.tensor([[[1.0, 2.0], [0.0, 0.0]], [[0.0, 0.0], [3.0, 4.0]]], dtype=F64)   # [part, out, in]
    b = torch.tensor([[0.0, 5.0], [6.0, 0.0]], dtype=F64)
    got = torch.logit(O.block_gates(torch.tensor([[1.0, 10.0, -1.0, 1.0]], dtype=F64) * 0.1, w, b))
    assert torch.allclose(got, torch.tensor([[2.1, 5.0, 6.0, 0.1]], dtype=F64))


def test_oracle_streams_mix_from_row_to_column_all_at_once():
    from oracle import tusasun as O

    xs = torch.tensor([[[1.0]], [[10.0]]], dtype=F64)
    mix = torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=F64)
    got = O.stream_update(xs, torch.tensor([[100.0]], dtype=F64), mix, torch.tensor([1.0, 0.5], dtype=F64))
    assert got.flatten().tolist() == [1.0 + 30.0 + 100.0, 2.0 + 40.0 + 50.0]
    assert O.stream_input(xs, torch.tensor([2.0, 0.5], dtype=F64)).item() == 7.0


def test_oracle_weight_multiplies_the_expert_input_and_is_not_renormalised():
    from oracle import tusasun as O

    one = torch.ones(1, 1, dtype=F64)
    t = {"router": torch.tensor([[0.0], [1.0]], dtype=F64), "e0.up": one, "e0.down": one, "e1.up": 2 * one, "e1.down": one,
         "shared.up": -one, "shared.down": one, "shared.sg": one}
    ids, w = O.route(one, t, "", 2)
    s = 1 / (1 + math.exp(-1.0))
    assert ids[0].tolist() == [1, 0] and w[0].tolist() == pytest.approx([s, 0.5])
    y = O.moe(one * 1.0, t, "", {"router": {"experts": 2, "top": 2}, "shared": {"ff": 1}})
    assert y.item() == pytest.approx((2 * s) ** 2 + 0.25)          # (squares of the WEIGHTED input; the shared relu is shut)


def test_oracle_norm_weight_is_stored_around_zero():
    from oracle import tusasun as O

    x = torch.tensor([[3.0, 4.0]], dtype=F64)
    assert torch.allclose(O.shifted_norm(x, torch.tensor([0.0, 1.0], dtype=F64), 0.0), torch.tensor([[3.0, 8.0]], dtype=F64) / math.sqrt(12.5))
