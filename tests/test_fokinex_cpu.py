"""Host-side parts of the Fokinex decoder: its configuration and its errors, the model as data, what its parts ask of the cache
manager (a layer's rows kept for as long as any layer reads them), weights loaded into fused layouts, stretched wavelengths, and
the plain implementation's own properties."""
import json
import math

import pytest
import torch

import plain_fokinex as P
from test_gpu_fokinex import F1, F2, F3, _drawn_config, _latent, _parallel, _write_model

from infinicore_infer_amd.config import ConfigError, ExecEntry, PartSpec, config_from_dict
from infinicore_infer_amd.parts import Runtime, build_model
from infinicore_infer_amd.parts.base import build_part


def _cpu_model(cfg, dtype=torch.float32):
    return build_model(config_from_dict(cfg).model_spec(), Runtime(dtype, "cpu"))


def test_config_to_model_spec():
    cfg = config_from_dict(F1)
    spec = cfg.model_spec()
    assert spec.architecture == "Fokinex" and spec.vocab_size == 211 and spec.hidden_size == 96 and spec.residual_streams == 1
    assert [(e.layer, e.cache, e.writes_cache) for e in spec.schedule] == [(0, 0, True), (1, 1, True), (2, 0, False), (3, 0, False)]
    assert [l.mixer.kind for l in spec.layers] == ["latent_attention", "parallel", "latent_attention", "latent_attention"]
    assert all(l.block.kind == "shared_norm_residual" and l.feed_forward_norm is None for l in spec.layers)
    assert spec.embedding.params["scale"] == 7.0 and spec.embedding.params["tensor"] == "embed" and spec.head.params["tensor"] == "head"
    a = spec.layers[0].mixer.params
    assert (a["num_heads"], a["head_dim"], a["rot_dim"], a["value_dim"], a["q_rank"], a["kv_rank"]) == (4, 24, 16, 40, 40, 64)
    assert (a["softmax_scale"], a["window"], a["sink"], a["gate"], a["own_rows"], a["norm_eps"]) == (0.2, 37, True, False, True, 1e-5)
    assert (a["rot_base"], a["rot_dims"]) == (10000.0, 16)
    assert a["rot_scaling"] == {"factor": 4.0, "original": 64.0, "fast": 8.0, "slow": 1.0}
    assert not spec.layers[2].mixer.params["own_rows"] and spec.layers[2].mixer.params["window"] == 70
    (left, ls), (right, rs) = spec.layers[1].mixer.params["branches"]
    assert (ls, rs, left.kind, right.kind) == (0.8, 1.3, "span_attention", "gated_delta")
    p = left.params
    assert (p["num_heads"], p["num_kv_heads"], p["key_dim"], p["value_dim"], p["softmax_scale"], p["softcap"], p["window"]) == (4, 2, 40, 40, 0.3, 3.0, 29)
    assert p["values_from_keys"] and p["gate"] and p["qk_norm"] == "row" and p["distance_slopes"] == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    r = right.params
    assert (r["heads"], r["kv_heads"], r["key_dim"], r["value_dim"], r["conv_taps"], r["decay"]) == (4, 2, 24, 40, 4, "head")
    assert spec.layers[0].feed_forward.params["intermediate_size"] == 112 and spec.layers[3].feed_forward is None
    assert config_from_dict(cfg.to_dict()).model_spec().layers[1].mixer == spec.layers[1].mixer
    assert config_from_dict(F1, max_tokens=300).max_positions == 300 and cfg.context_is_open
    # what may be absent: windows, stretching, the cap, kv_heads, the embedding's scale
    bare = json.loads(json.dumps(F2))
    bare.pop("embedding")
    for k in ("softcap", "kv_heads", "vdim"):
        bare["layers"][0]["mixer"]["left"].pop(k)
    spec = config_from_dict(bare).model_spec()
    p = spec.layers[0].mixer.params["branches"][0][0].params
    assert (p["softcap"], p["num_kv_heads"], p["value_dim"], p["window"]) == (None, 3, 10, None) and spec.embedding.params["scale"] == 1.0
    assert spec.layers[1].mixer.params["rot_scaling"] is None and spec.layers[1].mixer.params["window"] is None
    for seed in range(14):                                    # every drawn configuration is one the reader takes
        assert len(config_from_dict(_drawn_config(seed)).model_spec().layers) >= 2


@pytest.mark.parametrize("change,what", [
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), "base"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("original"), "original"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=32), "kv_rank"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(base=77.0), "rot"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(vdim=24), "vdim"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("conv"), "conv"),
    (lambda c: c["layers"][1]["mixer"].pop("right_scale"), "right_scale"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "dense"),
    (lambda c: c["layers"][0]["mlp"].update(ff=0), "ff"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_config_errors(change, what):
    cfg = json.loads(json.dumps(F1))
    change(cfg)
    with pytest.raises(ConfigError) as e:
        config_from_dict(cfg)
    assert what in str(e.value)


def test_part_errors():
    rt = Runtime(torch.float32, "cpu")
    latent = {"hidden_size": 16, "num_heads": 2, "head_dim": 8, "rot_dim": 4, "value_dim": 8, "q_rank": 8, "kv_rank": 16, "softmax_scale": 0.3,
              "rot_base": 100.0}
    for bad in ({"window": 0}, {"window": -3}, {"kv_rank": 513}, {"rot_dims": 6}, {"rot_dims": 3}):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("latent_attention", "a.", dict(latent, **bad)), rt)
    span = {"hidden_size": 16, "num_heads": 2, "num_kv_heads": 1, "key_dim": 8, "value_dim": 8, "softmax_scale": 0.3}
    for bad in ({"values_from_keys": True, "value_dim": 4}, {"values_from_keys": True, "conv_taps": 2}, {"distance_slopes": [1.0]},
                {"values_from_keys": True, "rot_dims": 4, "rot_base": 10.0}, {"values_from_keys": True, "value_mix": "keep"}):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("span_attention", "a.", dict(span, **bad)), rt)
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("gated_delta", "a.", {"hidden_size": 16, "heads": 2, "kv_heads": 1, "key_dim": 8, "value_dim": 8, "conv_taps": 3,
                                                           "norm_eps": 1e-5, "decay": "token"}), rt)
    norm = build_part("norm", PartSpec("rmsnorm", "", {"size": 16, "eps": 1e-5, "tensor": "n"}), rt)
    mixer = build_part("mixer", PartSpec("latent_attention", "a.", latent), rt)
    from infinicore_infer_amd.parts.block import SharedNormResidualBlock
    for bad in ({"mixer": None, "mixer_norm": norm}, {"mixer": mixer, "mixer_norm": None},
                {"mixer": mixer, "mixer_norm": norm, "feed_forward_norm": norm}):
        with pytest.raises(ValueError):
            SharedNormResidualBlock("b.", rt, **bad)


def test_cache_needs_follow_the_widest_reader():
    """A slot's pages are given back once the widest window of all layers that read it has passed; one reader without a window
    keeps every page."""
    model = _cpu_model(F1)
    rows, par = model.cache_needs()                         # the reading layers have no slot of their own
    assert (rows.kind, rows.planes, rows.n_kv_heads, rows.head_dim, rows.window) == ("kv", 1, 1, 80, 70)
    state = (4 * 40 * 24 + 3 * (2 * 2 * 24 + 4 * 40) + 3) // 4 * 4
    assert (par.kind, par.n_kv_heads, par.plane_dims, par.window, par.state_shape) == ("kv+state", 2, (40, 40), 29, (state,))
    assert model.cache_needs()[0] == rows and model.layers[0].mixer.cache_need().window == 37
    keeps = _cpu_model(F3).cache_needs()
    assert keeps[0].window is None and keeps[0].head_dim == 160 and keeps[1].kind == "none" and keeps[2].window == 48 and keeps[3].window == 130
    # a reader that wants another row is refused
    spec = config_from_dict(F1).model_spec()
    spec.schedule[1] = ExecEntry(layer=1, cache=0, writes_cache=False)
    with pytest.raises(ValueError):
        build_model(spec, Runtime(torch.float32, "cpu"))


def test_window_pages_live_as_long_as_a_reader_needs_them():
    from infinicore_infer_amd.cache import CacheManager, GroupSpec
    need = _cpu_model(F1).cache_needs()[0]
    cm = CacheManager([GroupSpec("window", need.n_kv_heads, need.head_dim, need.window, (0,), need.planes)], [64], 16, 2)
    cm.admit("a")
    for length in range(1, 300):
        cm.append("a", 1)
        # the next token sits at position `length` and reads keys above length - 70
        cm.trim("a")
        oldest = max(0, length - need.window + 1)
        assert all(p >= 0 for p in cm.block_table("a", 0)[oldest // 16:]) and all(p < 0 for p in cm.block_table("a", 0)[:oldest // 16])
    cm.check_invariants()


def test_weights_and_fused_layouts(tmp_path):
    folder = str(tmp_path / "m")
    W = _write_model(folder, F1, 5)
    model = _cpu_model(F1)
    model.load_from_dir(folder)
    m = model.layers[0].mixer
    assert torch.equal(m.w_down, torch.cat([W["l0.mix.dq"], W["l0.mix.dkv"]])) and torch.equal(m.w_ukv, torch.cat([W["l0.mix.uk"], W["l0.mix.uv"]]))
    assert torch.equal(m.w_uk_t, W["l0.mix.uk"].view(4, 24, 64).transpose(1, 2)) and torch.equal(m.w_uv, W["l0.mix.uv"].view(4, 40, 64))
    assert torch.equal(m.sinks, W["l0.mix.sink"])
    reader = model.layers[2].mixer
    assert torch.equal(reader.w_down, W["l2.mix.dq"]) and reader.kvn_w is None and not any(k.startswith("l2.mix.dkv") for k in model.weight_specs())
    left, right = model.layers[1].mixer.children
    assert torch.equal(left.w_rows, torch.cat([W["l1.mix.left." + n] for n in "qkg"])) and "l1.mix.left.v" not in model.weight_specs()
    assert torch.equal(right.w_rows, torch.cat([W["l1.mix.right." + n] for n in ("q", "k", "v", "g", "b", "a")]))
    assert torch.allclose(right.rate, torch.exp(W["l1.mix.right.A_log"]))
    assert left.state_base == 0 and right.state_base == 0 and (left.out_buffer, right.out_buffer) == ("mixer_out_0", "mixer_out_1")
    assert set(model.weight_specs()) == set(W)
    # the query latent's size may stand in the tensors alone
    open_cfg = json.loads(json.dumps(F1))
    for i in (0, 2, 3):
        open_cfg["layers"][i]["mixer"].pop("q_rank")
    other = _cpu_model(open_cfg)
    other.load_from_dir(folder)
    assert [other.layers[i].mixer.Rq for i in (0, 2, 3)] == [40, 24, 40] and torch.equal(other.layers[0].mixer.w_down, m.w_down)
    # an unexpected tensor is named
    from infinicore_infer_amd.weights.loader import WeightError
    from safetensors.torch import save_file
    save_file({k: v.to(torch.bfloat16) for k, v in dict(W, **{"l2.mix.dkv": W["l0.mix.dkv"]}).items()}, folder + "/model.safetensors")
    with pytest.raises(WeightError) as e:
        _cpu_model(F1).load_from_dir(folder)
    assert "l2.mix.dkv" in str(e.value)


def test_who_hands_rows_on():
    """Which blocks take half-normed rows, and what the parallel mixers pass on to their children."""
    model = _cpu_model(F1)
    assert all(l.entry_norm() is l.mixer_norm and l.fuses_successor for l in model.layers)
    assert model.layers[1].mixer.accepts_deferred and model.layers[1].mixer.adds_into_stream and model.layers[1].mixer.yields_branches
    other = build_part("mixer", PartSpec("rglru", "r.", {"hidden_size": 96, "width": 32, "blocks": 2, "conv_taps": 2}), Runtime(torch.float32, "cpu"))
    from infinicore_infer_amd.parts.block import SharedNormResidualBlock
    assert SharedNormResidualBlock("b.", other.runtime, mixer=other, mixer_norm=model.layers[0].mixer_norm).entry_norm() is None


@pytest.mark.parametrize("dims,base,scaling", [(48, 10000.0, (10.0, 300, 24.0, 1.0)), (64, 5e5, (40.0, 4096, 32.0, 1.0)), (6, 10.0, (2.0, 4, 3.0, 3.0)),
                                               (16, 100.0, (1.0, 64, 8.0, 1.0)), (8, 1000.0, (4.0, 1, 32.0, 16.0))])
def test_stretched_wavelengths(dims, base, scaling):
    from infinicore_infer_amd.parts.rotary import pair_frequencies, stretched_magnitude
    s = dict(zip(("factor", "original", "fast", "slow"), scaling))
    plain, f = pair_frequencies(dims, base).double().sum(0), pair_frequencies(dims, base, s).double().sum(0)
    want, mult = P.stretched_frequencies(dims, base, s)
    assert torch.allclose(f, torch.tensor(want, dtype=torch.float64), rtol=1e-13)
    assert stretched_magnitude(s) == mult == 0.1 * math.log(scaling[0]) + 1.0 and stretched_magnitude(None) == 1.0
    # between the two ends, slower pairs stretched at least as much as faster ones
    ratio = plain / f
    assert bool((ratio >= 1.0 - 1e-12).all()) and bool((ratio <= scaling[0] + 1e-9).all()) and bool((ratio[1:] - ratio[:-1] > -1e-9).all())


def test_plain_implementation_is_causal_and_forgets_what_it_should():
    """The oracle's own properties: a later token changes nothing before it; latent layers alone forget a token once every window
    has passed; a tail's logits do not depend on what follows."""
    g = torch.Generator().manual_seed(1)
    toks = torch.randint(0, 211, (120,), generator=g).tolist()
    changed = list(toks)
    changed[10] = (changed[10] + 1) % 211
    first, second = json.loads(json.dumps([F1["layers"][0], F1["layers"][3]]))       # windows of 37 and of 18 keys
    for shared in (True, False):
        # a layer with rows of its own sees what the layer before it has mixed in; one that reads that layer's rows does not
        reach = 36 if shared else 36 + 17
        second["mixer"].pop("kv_from", None)
        if shared:
            second["mixer"]["kv_from"] = 0
        cfg = dict(F1, layers=[first, second])
        W = P.random_weights(cfg, 3)
        full, other = P.forward(cfg, W, toks), P.forward(cfg, W, changed)
        assert torch.allclose(P.forward(cfg, W, toks[:70]), full[:70], atol=1e-9)
        moved = (other - full).abs().amax(1)
        assert float(moved[:10].max()) < 1e-12 and float(moved[10]) > 1e-3
        assert float(moved[10 + reach]) > 1e-9 and float(moved[10 + reach + 1:].max()) < 1e-12
    # the recurrence beside the attention does not forget
    W = P.random_weights(F1, 3)
    moved = (P.forward(F1, W, changed) - P.forward(F1, W, toks)).abs().amax(1)
    assert float(moved[100:].max()) > 1e-9


def test_plain_sink_and_softmax():
    s = torch.tensor([[1.0, 2.0, -math.inf]], dtype=torch.float64)
    z = torch.tensor(0.5, dtype=torch.float64)
    e = [math.exp(v) for v in (1.0, 2.0)]
    want = torch.tensor([[e[0], e[1], 0.0]], dtype=torch.float64) / (sum(e) + math.exp(0.5))
    assert torch.allclose(P.softmax_with_sink(s, z), want) and torch.allclose(P.softmax_with_sink(s), torch.softmax(s, -1))
    assert P.seen_keys(5, 2).int().tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 1, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 1, 1]]
    assert bool(torch.equal(P.seen_keys(4, None), torch.tril(torch.ones(4, 4, dtype=torch.bool))))
