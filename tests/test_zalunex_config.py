"""The Zalunex design without a GPU: its configuration and the errors it names, the parts, cache groups and tensors a
configuration becomes, the learned positions as a limit that no option lifts, random model folders, and pins of the plain
implementation (tests/plain_zalunex.py) on inputs with known answers."""
import copy
import json

import numpy as np
import pytest
import torch

import plain_zalunex as plain
import zalunex_cases as cases


def test_configurations_round_trip_and_name_every_bad_key():
    from kvcm_amd.config.model_config import ConfigError
    from kvcm_amd.config.zalunex_config import ZalunexConfig
    for raw in cases.CONFIGS.values():
        cfg = ZalunexConfig.from_dict(raw)
        assert ZalunexConfig.from_dict(cfg.to_dict()) == cfg
        assert ZalunexConfig.from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    r = ZalunexConfig.from_dict(cases.CONFIGS["R"])
    assert r.loop is None and r.logit_softcap == 0.0 and r.layers[1].mixer.left.window == 0 and r.layers[0].mixer.right.decay == (0.0, 0.9, 0.3)
    assert ZalunexConfig.from_dict(cases.CONFIGS["P"]).layers[2].mlp is None
    bad = copy.deepcopy(cases.CONFIGS["Q"])
    bad["layers"][0]["mixer"]["left"]["kv_heads"] = 3
    bad["layers"][0]["mixer"]["left"]["mask"] = {}
    bad["layers"][0]["mixer"]["left_scale"] = "big"
    bad["layers"][0]["mixer"]["right"]["decay"] = [0.5]
    bad["layers"][0]["mlp"]["router"]["top"] = 9
    bad["layers"][1]["mixer"]["right"]["decay"] = [0.5, 1.5]
    del bad["layers"][1]["mlp"]["limit"]
    bad["layers"][2]["mixer"]["right"]["decay"] = 0.5
    bad["layers"][2]["mlp"]["kind"] = "sparse"
    bad["logit_softcap"] = -1.0
    del bad["width"], bad["max_positions"]
    bad["loop"] = {"start": 2, "stop": 9, "times": 2}
    with pytest.raises(ConfigError) as e:
        ZalunexConfig.from_dict(bad)
    text = str(e.value)
    for piece in ("config.width", "config.max_positions", "left: heads 4 is not a multiple of kv_heads 3", "left.mask.size", "left_scale must be a number",
                  "right.decay has 1 numbers for 4 heads", "top 9 exceeds", "decay must lie between 0 and 1", "mlp.limit", "decay must be a list",
                  "'sparse' is not supported", "logit_softcap", "layers 2 .. 8 are not a stretch"):
        assert piece in text, (piece, text)
    with pytest.raises(ConfigError, match="'mamba2' is not supported"):
        ZalunexConfig.from_dict(dict(cases.CONFIGS["R"], layers=[{"type": "mamba2", "mixer": {}, "mlp": None}]))
    with pytest.raises(ConfigError, match="needs 'left' and 'right'"):
        ZalunexConfig.from_dict(dict(cases.CONFIGS["R"], layers=[{"type": "parallel", "mixer": {"left": {}}, "mlp": None}]))
    # what a file may leave out
    lean = copy.deepcopy(cases.CONFIGS["Q"])
    m = lean["layers"][1]["mixer"]
    del m["left"]["kv_heads"], m["left"]["vdim"], m["left"]["mask"], m["right"]["vdim"], m["left_scale"], m["right_scale"]
    del lean["residual_mult"], lean["logit_softcap"], lean["loop"], lean["layers"][2]["mlp"]
    cfg = ZalunexConfig.from_dict(lean)
    p = cfg.layers[1].mixer
    assert (p.left.kv_heads, p.left.vdim, p.left.window, p.right.vdim, p.left_scale, p.right_scale) == (2, 32, 0, 64, 1.0, 1.0)
    assert (cfg.residual_mult, cfg.logit_softcap, cfg.loop, cfg.layers[2].mlp) == (1.0, 0.0, None, None)
    assert ZalunexConfig.from_dict(cfg.to_dict()) == cfg


def test_parts_cache_groups_and_tensors_of_a_configuration():
    from kvcm_amd.architectures.zalunex import zalunex_spec
    from kvcm_amd.config.zalunex_config import ZalunexConfig
    from kvcm_amd.engine.runner import plan_groups
    from kvcm_amd.parts.base import BuildContext, KVCacheNeed, StateNeed
    from kvcm_amd.parts.model import Model
    from kvcm_amd.weights.random_init import expected_tensors
    cfg = ZalunexConfig.from_dict(cases.CONFIGS["P"])
    spec = zalunex_spec(cfg)
    assert [l.name for l in spec.layers] == ["l0", "l1", "l2", "l3", "l1.pass1", "l2.pass1", "l3.pass1"]
    assert [("ffn" in l.parts) for l in spec.layers] == [True, True, False, True, True, False, True]
    assert (spec.max_position, spec.max_position_fixed, spec.keep_embedding) == (333, True, False)
    model = Model(spec, BuildContext(torch.bfloat16, torch.device("cpu"), spec.hidden_size, 16, None))
    assert model.capturable, model.not_capturable()
    plans = {g.need: [name for name, _ in g.layers] for g in model.groups}
    # every pass has places of its own
    assert plans[KVCacheNeed(3, 8, 33, value_dim=24)] == ["l1", "l1.pass1"]
    assert plans[StateNeed((2, 20, 8), torch.float32)] == ["l1", "l1.pass1"] and plans[StateNeed((3, 12, 20), torch.float32)] == ["l0"]
    windows = sorted((g.kind, g.window) for g in plan_groups(model, 50, 4) if g.kind != "state")
    assert windows == [("window", 7), ("window", 20), ("window", 33), ("window", 50)]
    names = expected_tensors("Zalunex", cfg)
    for n in ("embed", "pos", "final.norm", "head", "l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l0.mix.left.q", "l0.mix.left.k", "l0.mix.left.v",
              "l0.mix.left.g", "l0.mix.left.o", "l0.mix.left.q.norm", "l0.mix.left.k.norm", "l0.mix.left.sink", "l0.mix.right.q", "l0.mix.right.k",
              "l0.mix.right.v", "l0.mix.right.g", "l0.mix.right.o", "l0.mix.right.norm", "l0.mlp.gate", "l0.mlp.up", "l0.mlp.down", "l1.mlp.router",
              "l1.mlp.e4.up", "l1.mlp.e4.down"):
        assert n in names, n
    assert "l2.norm2" not in names and "l2.mlp.up" not in names and "l1.mlp.e0.gate" not in names and "l0.mlp.router" not in names
    assert names["pos"] == ((333, 48), "table") and names["l0.mix.left.g"][0] == (4, 48) and names["l0.mix.left.sink"] == ((4,), "bias")
    assert names["l0.mix.left.q.norm"] == ((16,), "vector") and names["l0.norm1b"][1] == "bias" and names["l0.mix.right.norm"] == ((60,), "vector")


def test_what_the_parts_make_of_their_weights():
    """Norm weights around one with the residual's factor in the outer ones; the two halves as one product at each end, their factors
    in what stands before it; passes share all of it."""
    from kvcm_amd.architectures.zalunex import zalunex_spec
    from kvcm_amd.config.zalunex_config import ZalunexConfig
    from kvcm_amd.parts.base import BuildContext
    from kvcm_amd.parts.model import Model
    from kvcm_amd.weights.loader import DictSource, load_weights
    cfg, tensors = cases.tensors_for(cases.CONFIGS["P"], seed=3)
    spec = zalunex_spec(cfg)
    model = Model(spec, BuildContext(torch.float32, torch.device("cpu"), spec.hidden_size, 16, None))
    load_weights(model, DictSource(tensors), torch.float32, torch.device("cpu"))
    first, second = (next(p for l, p in zip(spec.layers, model.layer_parts) if l.name == n) for n in ("l1", "l1.pass1"))
    np.testing.assert_allclose(first["norm_mixer"].w["weight"].numpy(), 1.0 + tensors["l1.norm1"].numpy(), rtol=1e-6)
    np.testing.assert_allclose(first["norm_ffn_out"].w["weight"].numpy(), 0.6 * (1.0 + tensors["l1.norm2b"].numpy()), rtol=1e-6)
    np.testing.assert_allclose(model.final_norm.w["weight"].numpy(), 1.0 + tensors["final.norm"].numpy(), rtol=1e-6)
    a, b = first["mixer"], second["mixer"]
    for key in ("w_in", "w_out"):
        assert a.w[key].data_ptr() == b.w[key].data_ptr()
    at = 0
    for m in a.members:
        for name, shape in m.in_sources():
            assert torch.equal(a.w["w_in"][at:at + shape[0]], tensors[name]), name
            at += shape[0]
    assert torch.equal(a.w["w_out"], torch.cat([tensors["l1.mix.left.o"], tensors["l1.mix.right.o"]], 1))
    np.testing.assert_allclose(a.members[1].w["norm"].numpy(), tensors["l1.mix.right.norm"].numpy() * np.float32(0.5), rtol=1e-6)
    np.testing.assert_allclose(a.members[1].w["decay"].numpy(), [0.97, 0.7], rtol=1e-6)


def test_parts_refuse_what_they_cannot_be():
    from kvcm_amd.parts.base import BuildContext
    from kvcm_amd.parts.chunk_attention_parts import ChunkAttention
    from kvcm_amd.parts.recurrent_parts import LightningAttention
    from kvcm_amd.parts.routed_parts import RoutedExperts
    ctx = BuildContext(torch.float32, torch.device("cpu"), 16, 16, None)
    sizes = {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 1.0, "eps": 1e-5}
    with pytest.raises(ValueError, match="beside a window"):
        ChunkAttention({**sizes, "chunk": 4, "window": 4}, "a.", ctx)
    with pytest.raises(ValueError, match="sink 'some'"):
        ChunkAttention({**sizes, "sink": "some"}, "a.", ctx)
    with pytest.raises(ValueError, match="1 decays for 2 heads"):
        LightningAttention({"heads": 2, "dim": 8, "vdim": 8, "decay": (0.5,), "eps": 1e-5}, "r.", ctx)
    with pytest.raises(ValueError, match="weigh 'both'"):
        RoutedExperts({"experts": 2, "top": 1, "ff": 8, "weigh": "both"}, "e.", ctx)
    with pytest.raises(ValueError, match="routing 'tanh'"):
        RoutedExperts({"experts": 2, "top": 1, "ff": 8, "routing": "tanh"}, "e.", ctx)
    with pytest.raises(ValueError, match="activation 'swish'"):
        RoutedExperts({"experts": 2, "top": 1, "ff": 8, "activation": "swish"}, "e.", ctx)


def test_learned_positions_are_a_limit_that_no_option_lifts(capsys):
    from kvcm_amd.config.engine_config import EngineConfig
    from kvcm_amd.engine.build import within_max_position
    ec = EngineConfig(max_seq_len=512)
    assert within_max_position(ec, 333, fixed=True).max_seq_len == 333
    assert "333 learned positions" in capsys.readouterr().err
    far = EngineConfig(max_seq_len=512, beyond_max_position=True)
    assert within_max_position(far, 333, fixed=True).max_seq_len == 333
    assert within_max_position(far, 333).max_seq_len == 512      # rotated positions: the option lifts it
    assert within_max_position(ec, 600, fixed=True).max_seq_len == 512


def test_random_model_folders_of_the_design(tmp_path):
    from kvcm_amd.config.zalunex_config import ZalunexConfig
    from kvcm_amd.engine.build import read_model_config
    from kvcm_amd.weights.random_init import write_model_dir
    cfg = ZalunexConfig.from_dict(cases.CONFIGS["P"])
    d = write_model_dir(str(tmp_path / "m"), "Zalunex", cfg, seed=4, dtype=torch.bfloat16, std=0.1, norm_jitter=0.1, device="cpu")
    arch, again = read_model_config(d)
    assert arch.name == "Zalunex" and again == cfg
    t = plain.read_tensors(str(tmp_path / "m" / "model.safetensors"))
    assert abs(t["l1.norm1b"].mean()) < 0.1 and abs(t["l1.mix.right.norm"].mean() - 1.0) < 0.1 and t["pos"].shape == (333, 48)
    logits = plain.forward(cases.CONFIGS["P"], t, [5, 17, 3, 90])
    assert logits.shape == (4, 97) and np.isfinite(logits).all() and np.abs(logits).max() < 12.0


# ---------------------------------------------------------------- pins of the plain implementation
def test_plain_norms_gates_and_caps_on_known_inputs():
    np.testing.assert_allclose(plain.offset_norm(np.array([3.0, 4.0]), np.array([0.0, 0.5]), 0.0), [3 / 12.5 ** 0.5, 6 / 12.5 ** 0.5])
    np.testing.assert_allclose(plain.gelu(np.array([0.0, 1.0, -1.0])), [0.0, 0.8413447460685429, -0.15865525393145707])
    np.testing.assert_allclose(plain.clamped_gate(np.array([0.0, 9.0, -9.0]), np.array([5.0, 9.0, -9.0]), 2.0),
                               [0.0, 2.0 / (1 + np.exp(-3.404)) * 3.0, -9.0 / (1 + np.exp(1.702 * 9)) * -1.0])
    np.testing.assert_allclose(plain.softcap(np.array([0.0, 1e9, -5.0]), 10.0), [0.0, 10.0, -10 * np.tanh(0.5)])
    assert plain.softcap(7.0, None) == 7.0
    np.testing.assert_allclose(plain.embedding({"embed": np.array([[1.0], [2.0]]), "pos": np.array([[10.0], [20.0], [30.0]])}, [1, 0], first=1)[:, 0], [22, 31])


def test_plain_window_and_sink_on_known_inputs():
    np.testing.assert_allclose(plain.sink_softmax(np.array([0.0, np.log(2.0), -np.inf]), 0.0), [0.25, 0.5, 0.0])
    np.testing.assert_allclose(plain.sink_softmax(np.array([0.0, 0.0]), np.log(2.0)), [0.25, 0.25])
    np.testing.assert_allclose(plain.sink_softmax(np.array([-800.0, -800.0]), 3.0), [0.0, 0.0])
    # a window of 3: position 5 sees 3, 4, 5; a sink of exp(0) shares with equal scores of 0; two heads with sinks of their own
    q, k, v = np.zeros((6, 2, 2)), np.zeros((6, 1, 2)), np.arange(6.0).reshape(6, 1, 1)
    out = plain.window_attention(q, k, v, 1.0, np.array([0.0, np.log(3.0)]), np.arange(6), np.arange(6), 3)
    np.testing.assert_allclose(out[[0, 1, 5], 0, 0], [0.0, 1 / 3, 12 / 4])
    np.testing.assert_allclose(out[[0, 1, 5], 1, 0], [0.0, 1 / 5, 12 / 6])
    np.testing.assert_allclose(plain.window_attention(q, k, v, 1.0, np.zeros(2), np.arange(6), np.arange(6))[5, 0, 0], 15 / 7)


def test_plain_recurrence_routing_and_layer_order_on_known_inputs():
    one = np.ones((3, 2, 1))
    np.testing.assert_allclose(plain.decayed_state(one, one, one, [0.5, 0.0])[:, :, 0], [[1, 1], [1.5, 1], [1.75, 1]])
    np.testing.assert_allclose(plain.decayed_state(2 * one, one, 3 * one, [1.0, 1.0])[:, 0, 0], [6, 12, 18])
    chosen, weight = plain.choose_experts(np.array([[0.0, np.log(3.0), -1.0, np.log(9.0)]]), 2)
    assert chosen.tolist() == [[3, 1]]
    np.testing.assert_allclose(weight, [[0.9, 0.75]])
    # the weight acts before the activation: gelu(0.75 * 2), not 0.75 * gelu(2)
    w = {"router": np.array([[np.log(3.0)]]), "e0.up": np.array([[2.0]]), "e0.down": np.array([[1.0]])}
    np.testing.assert_allclose(plain.mixture(np.array([[1.0]]), w, "", {"router": {"top": 1}}), plain.gelu(np.array([[1.5]])))
    assert plain.layer_runs(cases.CONFIGS["P"]) == [0, 1, 2, 3, 1, 2, 3] and plain.layer_runs(cases.CONFIGS["S"]) == [0, 0, 0, 1, 2]
    assert plain.layer_runs(cases.CONFIGS["U"]) == [0, 1, 0, 1] and plain.layer_runs(cases.CONFIGS["V"]) == [0] and plain.layer_runs(cases.CONFIGS["R"]) == [0, 1, 2]
