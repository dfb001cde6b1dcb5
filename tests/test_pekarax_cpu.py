"""Host-side parts of the Pekarax decoder: its configuration and its errors, the model as data, what its parts ask of the
cache manager, weights loaded into fused layouts with inner sizes that only the file knows, and the plain
implementation's own properties."""
import json
import math

import pytest
import torch

import plain_pekarax as P
from test_gpu_pekarax import K1, K2, _delta, _drawn_config, _gla, _moe, _parallel, _write_model

from infinicore_infer_amd.config import ConfigError, PartSpec, config_from_dict
from infinicore_infer_amd.parts import Runtime, build_model
from infinicore_infer_amd.parts.base import build_part


def test_config_to_model_spec():
    cfg = config_from_dict(K1)
    spec = cfg.model_spec()
    assert spec.architecture == "Pekarax" and spec.vocab_size == 211 and spec.hidden_size == 96 and spec.residual_streams == 1
    assert [(e.layer, e.cache) for e in spec.schedule] == [(0, 0), (1, 1), (2, 2)]
    assert [l.mixer.kind for l in spec.layers] == ["gated_delta", "parallel", "gated_linear_attention"]
    assert all(l.block.kind == "sum_norm_residual" and l.block.params["alpha"] == 1.7 for l in spec.layers)
    a = spec.layers[0].mixer.params
    assert (a["heads"], a["kv_heads"], a["key_dim"], a["value_dim"], a["conv_taps"], a["norm_eps"]) == (4, 2, 24, 40, 4, 1e-5)
    (left, ls), (right, rs) = spec.layers[1].mixer.params["branches"]
    assert (ls, rs, left.kind, right.kind) == (0.8, 1.3, "span_attention", "exponential_memory")
    assert (left.name, right.name) == ("l1.mix.left.", "l1.mix.right.")
    p = left.params
    assert (p["num_heads"], p["num_kv_heads"], p["key_dim"], p["value_dim"], p["conv_taps"], p["softmax_scale"]) == (4, 2, 32, 64, 3, 0.3)
    assert (p["rot_dims"], p["rot_base"], p["qk_norm"], p["qk_norm_weight"], p["qk_norm_eps"]) == (16, 10000.0, "head", False, 1e-5)
    assert (right.params["heads"], right.params["key_dim"], right.params["value_dim"], right.params["gate_cap"]) == (3, 20, 28, 4.0)
    g = spec.layers[2].mixer.params
    assert (g["heads"], g["key_dim"], g["value_dim"], g["tau"]) == (3, 20, 36, 4.0)
    f = spec.layers[0].feed_forward.params
    assert (f["experts"], f["top"], f["expert_size"], f["groups"], f["group_keep"], f["identity"], f["scale"]) == (9, 3, 48, 3, 2, 3, 1.5)
    assert (f["scores"], f["renormalize"], f["weight_on"], f["correction"], f["unit"], f["limit"], f["slope"]) == (
        "softmax", True, "output", True, "clamped", 2.0, 1.702)
    assert spec.layers[0].mixer_norm.params["tensor"] == "l0.norm1" and spec.layers[0].feed_forward_norm.params["tensor"] == "l0.norm2"
    assert spec.final_norm.params["weight_offset"] == 1.0 and spec.layers[2].mixer_norm.params["weight_offset"] == 1.0
    assert config_from_dict(cfg.to_dict()).model_spec().layers[1].mixer == spec.layers[1].mixer
    assert config_from_dict(K1, max_tokens=300).max_positions == 300 and cfg.context_is_open
    # no feed-forward, no groups, no identity experts
    plain = config_from_dict(K2).model_spec()
    assert plain.layers[0].feed_forward is None and plain.layers[0].feed_forward_norm is None and plain.layers[2].feed_forward is None
    f = plain.layers[1].feed_forward.params
    assert (f["groups"], f["group_keep"], f["identity"]) == (1, 1, 0)
    bare = json.loads(json.dumps(K2))
    left = bare["layers"][0]["mixer"]["left"]
    for k in ("rot", "conv", "kv_heads", "vdim"):
        left.pop(k)
    p = config_from_dict(bare).model_spec().layers[0].mixer.params["branches"][0][0].params
    assert (p["rot_dims"], p["conv_taps"], p["num_kv_heads"], p["value_dim"]) == (0, 0, 3, 10)
    for seed in range(12):                                    # every drawn configuration is one the reader takes
        assert len(config_from_dict(_drawn_config(seed)).model_spec().layers) >= 2


@pytest.mark.parametrize("change,what", [
    (lambda c: c["layers"][0].update(type="lightning"), "type"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("postln_alpha"), "postln_alpha"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("right_scale"), "right_scale"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].pop("base"), "base"),
    (lambda c: c["layers"][2]["mixer"].pop("tau"), "tau"),
    (lambda c: c["layers"][2]["mixer"].update(dim=0), "dim"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "moe"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=13), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=5), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=9), "groups"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_config_errors(change, what):
    cfg = json.loads(json.dumps(K1))
    change(cfg)
    with pytest.raises(ConfigError) as e:
        config_from_dict(cfg)
    assert what in str(e.value)


def test_part_errors():
    rt = Runtime(torch.float32, "cpu")
    delta = {"hidden_size": 16, "heads": 2, "kv_heads": 1, "key_dim": 8, "value_dim": 8, "conv_taps": 3, "norm_eps": 1e-5}
    for bad in ({"kv_heads": 3}, {"conv_taps": 9}, {"key_dim": 2000}, {"value_dim": 0}):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("gated_delta", "a.", dict(delta, **bad)), rt)
    gla = {"hidden_size": 16, "heads": 2, "key_dim": 8, "value_dim": 8, "tau": 0.0, "norm_eps": 1e-5}
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("gated_linear_attention", "a.", gla), rt)
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("exponential_memory", "a.", dict({k: v for k, v in gla.items() if k != "tau"}, gate_cap=-1.0)), rt)
    span = {"hidden_size": 16, "num_heads": 2, "num_kv_heads": 1, "key_dim": 8, "value_dim": 8, "softmax_scale": 0.3}
    for bad in ({"conv_taps": 9}, {"rot_dims": 6, "rot_base": None}, {"rot_dims": 5, "rot_base": 10.0}, {"rot_dims": 10, "rot_base": 10.0},
                {"rot_dims": 4, "rot_base": 10.0, "qkv_bias": True}, {"conv_taps": 2, "qk_norm": "row"}):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("span_attention", "a.", dict(span, **bad)), rt)
    s = PartSpec("span_attention", "a.", span)
    for branches in ([], [(s, 1.0)] * 3, [(s, 1.0), (s, 1.0)], [(PartSpec("mamba2", "m.", {
            "hidden_size": 16, "heads": 2, "head_dim": 8, "state_dim": 4, "groups": 1, "norm_groups": 1, "conv_taps": 2, "norm_eps": 1e-5}), 1.0)]):
        with pytest.raises((ValueError, TypeError)):           # none, too many, two paged caches, a mixer with a fixed place
            build_part("mixer", PartSpec("parallel", "p.", {"branches": branches}), rt)
    moe = {"hidden_size": 16, "experts": 6, "top": 2, "expert_size": 8, "weight_on": "output"}
    for bad in ({"groups": 4}, {"groups": 3, "group_keep": 4}, {"groups": 6, "group_keep": 1}, {"unit": "clamped"}, {"unit": "relu"},
                {"identity": 1, "weight_on": "input"}, {"unit": "clamped", "limit": 1.0, "shared_size": 8}):
        with pytest.raises(ValueError):
            build_part("feed_forward", PartSpec("routed_experts", "f.", dict(moe, **bad)), rt)


def test_cache_needs_of_the_mixers():
    model = build_model(config_from_dict(K1).model_spec(), Runtime(torch.float32, "cpu"))
    delta, par, gla = model.cache_needs()
    # state rows: S and the convolution's inputs, rounded up to whole 16-byte pieces
    assert delta.kind == "state" and delta.state_shape == (4 * 40 * 24 + 3 * (2 * 2 * 24 + 4 * 40),)
    assert gla.kind == "state" and gla.state_shape == (3 * 36 * 20,)
    conv = 2 * (4 * 32 + 2 * 32 + 2 * 64)
    assert (par.kind, par.n_kv_heads, par.plane_dims, par.window) == ("kv+state", 2, (32, 64), None)
    mlstm = 3 * 29 * 20 + 3
    assert par.state_shape == (conv + (mlstm + 3) // 4 * 4,) and par.state_dtype == torch.float32
    left, right = model.layers[1].mixer.children
    assert (left.state_base, right.state_base) == (0, conv) and left.out_buffer != right.out_buffer
    # one tap keeps no inputs: the left branch has no state, the right one starts at zero
    model2 = build_model(config_from_dict(K2).model_spec(), Runtime(torch.float32, "cpu"))
    left, right = model2.layers[0].mixer.children
    assert left.state_size == 0 and right.state_base == 0 and model2.cache_needs()[0].kind == "kv+state"
    assert model2.cache_needs()[3].state_shape == ((3 * 6 * 9 + 3) // 4 * 4,)


def test_weights_load_into_fused_layouts(tmp_path):
    from safetensors.torch import save_file
    from infinicore_infer_amd.weights.loader import WeightError
    W = _write_model(str(tmp_path), K1, seed=3)                # inner sizes 8 and 15: only the file knows them
    f = lambda name: W[name].to(torch.float32)
    for dtype in (torch.float32, torch.bfloat16):
        model = build_model(config_from_dict(K1).model_spec(), Runtime(dtype, "cpu"))
        assert set(model.weight_specs()) == set(W)
        model.load_from_dir(str(tmp_path))
        delta, par, gla = (l.mixer for l in model.layers)
        assert (delta.ra, delta.rg) == (8, 15) and gla.w_a2.shape == (60, 8)
        assert torch.equal(delta.w_rows.float(), torch.cat([f("l0.mix." + s) for s in ("q", "k", "v", "a1", "g1", "b")]))
        assert delta.conv_w.dtype == torch.float32 and torch.equal(delta.conv_w, torch.cat([f("l0.mix.%s.conv" % s) for s in "qkv"]))
        assert torch.allclose(delta.rate.double(), torch.exp(W["l0.mix.A_log"].double()), rtol=1e-6) and delta.dt_bias.dtype == torch.float32
        left, right = par.children
        assert torch.equal(left.w_rows.float(), torch.cat([f("l1.mix.left." + s) for s in "qkv"])) and left.norm_weight is False
        want = torch.tensor([10000.0 ** (-2.0 * i / 16) for i in range(8)], dtype=torch.float64)
        assert torch.allclose(left.freq[0].double() + left.freq[1].double(), want, atol=1e-15, rtol=1e-13)
        assert torch.equal(right.w_gates.float(), torch.cat([f("l1.mix.right.i"), f("l1.mix.right.f")])) and right.b_f.dtype == torch.float32
        assert torch.equal(gla.w_rows.float(), torch.cat([f("l2.mix." + s) for s in ("q", "k", "v", "g", "a1")]))
        moe = model.layers[0].feed_forward
        assert tuple(moe.w_gate_up.shape) == (9, 96, 96) and tuple(moe.w_router.shape) == (12, 96) and moe.correction.dtype == torch.float32
        assert torch.equal(moe.w_gate_up[8].float(), torch.cat([f("l0.mlp.e8.gate"), f("l0.mlp.e8.up")]))
        # a norm's weight is stored around zero
        assert torch.allclose(model.layers[1].mixer_norm.weight.double(), 1.0 + f("l1.norm1").double(), atol=1e-6)
        assert torch.allclose(model.final_norm.weight.double(), 1.0 + f("final.norm").double(), atol=1e-6)
    for name, tensor in (("l0.mlp.correction", None), ("l0.mix.a2", W["l0.mix.a2"][:, :5]), ("l2.mix.a1", W["l2.mix.a1"][:3])):
        broken = {k: v.to(torch.bfloat16).contiguous() for k, v in W.items() if k != name}
        if tensor is not None:
            broken[name] = tensor.to(torch.bfloat16).contiguous()
        save_file(broken, str(tmp_path / "model.safetensors"))
        with pytest.raises(WeightError) as e:                  # a missing tensor; two halves of a product that do not fit
            build_model(config_from_dict(K1).model_spec(), Runtime(torch.float32, "cpu")).load_from_dir(str(tmp_path))
        assert name.rsplit(".", 1)[0] in str(e.value)


def test_the_plain_implementation_is_causal():
    for cfg in (K1, K2):
        W = P.random_weights(cfg, 1)
        toks = list(range(5, 45))
        full = P.forward(cfg, W, toks)
        assert torch.allclose(P.forward(cfg, W, toks[:17]), full[:17], atol=1e-9)      # what follows changes nothing
        other = P.forward(cfg, W, toks[:16] + [61] + toks[17:])
        assert torch.allclose(other[:16], full[:16], atol=1e-9) and not torch.allclose(other[16:], full[16:], atol=1e-3)


def test_the_plain_pieces_do_what_they_say():
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    # the convolution's last column is the current token's
    x, w = r(9, 3), r(3, 4)
    pad = torch.cat([torch.zeros(3, 3, dtype=torch.float64), x])
    assert torch.allclose(P.short_conv(x, w), sum(w[:, k] * pad[k:k + 9] for k in range(4)))
    # halves turn by position * base^(-2i/dims); what lies behind dims stays
    x = torch.arange(12, dtype=torch.float64).reshape(1, 2, 6) + 1
    y = P.rotate_halves(x, [5], 4, 100.0)
    a = 5 * 100.0 ** (-2 / 4)
    assert torch.allclose(y[0, 0, [1, 3]], torch.tensor([2 * math.cos(a) - 4 * math.sin(a), 4 * math.cos(a) + 2 * math.sin(a)], dtype=torch.float64))
    assert torch.equal(y[..., 4:], x[..., 4:]) and torch.equal(P.rotate_halves(x, [0], 6, 10.0), x)
    # linear attention with a decay per channel is a sum over earlier tokens with products of the decays between
    q, k, v, d = r(6, 2, 3), r(6, 2, 3), r(6, 2, 4), torch.rand(6, 2, 3, generator=g, dtype=torch.float64)
    want = torch.zeros(6, 2, 4, dtype=torch.float64)
    for t in range(6):
        for j in range(t + 1):
            want[t] += (q[t] * k[j] * d[j + 1:t + 1].prod(0)).sum(-1, keepdim=True) * v[j]
    assert torch.allclose(P.channel_decay_memory(q, k, v, d), want)
    # the delta rule without decay and with full steps stores a value that its (unit) key reads back, whatever was there
    k = P.unit_rms(r(6, 2, 3), 0) / math.sqrt(3)
    out = P.delta_memory(k, k, v, torch.ones(6, 2, 3, dtype=torch.float64), torch.ones(6, 2, dtype=torch.float64))
    assert torch.allclose(out, v)
    # the running maximum changes nothing but the floor: the memory equals the plain sums of exp(gates), divided by
    # max(|n q|, 1) up to the small constant
    li, lf = r(6, 2), -P.softplus(r(6, 2))
    q = r(6, 2, 3)
    got = P.matrix_memory(q, k, v, li, lf)
    for t in range(6):
        wgt = [torch.exp(li[j] + lf[j + 1:t + 1].sum(0)) for j in range(t + 1)]
        num = sum(wgt[j][:, None] * (q[t] * k[j]).sum(-1, keepdim=True) * v[j] for j in range(t + 1))
        n = sum(wgt[j] * (q[t] * k[j]).sum(-1) for j in range(t + 1))
        assert torch.allclose(got[t], num / torch.clamp(n.abs(), min=1.0)[:, None], atol=1e-4)
    # the choice: a group is as good as its best member, members of other groups are out even when all scores are negative
    s, c = torch.tensor([0.3, 0.1, 0.2, 0.05, 0.25, 0.1]), torch.full((6,), -1.0)
    assert P.choose(s, torch.zeros(6), 3, 3, 2) == [0, 4, 1] and P.choose(s, c, 3, 3, 2) == [0, 4, 1]
    assert P.choose(s, torch.tensor([0.0, 0, 0, 1, 0, 0]), 2, 2, 1) == [3, 4] and P.choose(torch.zeros(6), torch.zeros(6), 2, 3, 1) == [0, 1]
    # bounded branches: the gate from above only, the up branch on both sides
    W = {"m.gate": torch.eye(1, dtype=torch.float64), "m.up": torch.eye(1, dtype=torch.float64), "m.down": torch.eye(1, dtype=torch.float64)}
    unit = lambda z: float(P.bounded_unit(torch.tensor([[z]], dtype=torch.float64), W, "m.", 2.0))
    sig = lambda z: 1 / (1 + math.exp(-z))
    assert abs(unit(5.0) - 2 * sig(3.404) * 3) < 1e-12 and abs(unit(-5.0) - (-5 * sig(-8.51) * -1)) < 1e-12
    # identity experts return their input, times the weight
    W = {"m.router": torch.zeros(3, 2, dtype=torch.float64), "m.correction": torch.tensor([0.0, 5.0, 4.0], dtype=torch.float64)}
    h = r(4, 2)
    assert torch.allclose(P.routed_experts(h, W, "m.", _moe(1, 2, 4, 1.0, None, 2, 1.7)), 1.7 * h)


def test_layers_of_each_kind_stand_alone():
    """Layers of each kind alone make a model (no layer rests on another's presence)."""
    for layer in (_delta(2, 1, 8, 8, 3, None), _gla(2, 8, 8, 2.0, _moe(3, 1, 8, 1.0)),
                  _parallel((2, 1, 8, 8, 3, 0.3, 8, 100.0), (1, 8, 8, 5.0), (1.0, 0.5), None)):
        cfg = {"architecture": "Pekarax", "vocab": 30, "width": 16, "norm": {"eps": 1e-5}, "postln_alpha": 2.0, "layers": [layer]}
        model = build_model(config_from_dict(cfg).model_spec(), Runtime(torch.float32, "cpu"))
        assert len(model.layers) == 1 and set(model.weight_specs()) == set(P.random_weights(cfg, 0))
