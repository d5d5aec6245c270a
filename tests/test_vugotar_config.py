"""The Vugotar design without a GPU: its configuration and the errors it names, the parts, cache groups and tensors a
configuration becomes, pages given back chunk by chunk, random model folders, and pins of the plain implementation
(tests/plain_vugotar.py) on inputs with known answers."""
import copy
import json

import numpy as np
import pytest
import torch

import plain_vugotar as plain
import vugotar_cases as cases


def test_configurations_round_trip_and_name_every_bad_key():
    from kvcm_amd.config.model_config import ConfigError
    from kvcm_amd.config.vugotar_config import VugotarConfig
    for raw in cases.CONFIGS.values():
        cfg = VugotarConfig.from_dict(raw)
        assert VugotarConfig.from_dict(cfg.to_dict()) == cfg
        assert VugotarConfig.from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    r = VugotarConfig.from_dict(cases.CONFIGS["R"])
    assert r.loop is None and r.layers[2].mlp is None and r.layers[1].mlp.shared_ff == 0
    bad = copy.deepcopy(cases.CONFIGS["Q"])
    bad["layers"][0]["mixer"]["left"]["kv_heads"] = 3
    bad["layers"][0]["mixer"]["left"]["rot"]["dims"] = 7
    bad["layers"][0]["mixer"]["left"]["mask"] = {}
    bad["layers"][0]["mixer"]["right"]["kv_heads"] = 3
    bad["layers"][0]["mixer"]["left_scale"] = "big"
    bad["layers"][0]["mlp"]["router"]["top"] = 9
    bad["layers"][1]["mixer"]["groups"] = 3
    bad["layers"][1]["mixer"]["norm_groups"] = 3
    bad["layers"][2]["mlp"]["kind"] = "sparse"
    del bad["layers"][2]["mixer"]["right"]["conv"]
    del bad["layers"][3]["mixer"]["state"]
    del bad["width"]
    bad["loop"] = {"start": 3, "stop": 9, "times": 2}
    with pytest.raises(ConfigError) as e:
        VugotarConfig.from_dict(bad)
    text = str(e.value)
    for piece in ("config.width", "left: heads 4 is not a multiple of kv_heads 3", "right: heads 4 is not a multiple of kv_heads 3", "rot.dims 7",
                  "left.mask.size", "left_scale must be a number", "top 9 exceeds", "heads 4 is not a multiple of groups 3",
                  "heads x vdim 128 is not a multiple of norm_groups 3", "'sparse' is not supported", "right.conv", "mixer.state", "layers 3 .. 8 are not a stretch"):
        assert piece in text, (piece, text)
    with pytest.raises(ConfigError, match="'mlstm' is not supported"):
        VugotarConfig.from_dict(dict(cases.CONFIGS["R"], layers=[{"type": "mlstm", "mixer": {}, "mlp": None}]))
    with pytest.raises(ConfigError, match="needs 'left' and 'right'"):
        VugotarConfig.from_dict(dict(cases.CONFIGS["R"], layers=[{"type": "parallel", "mixer": {"left": {}}, "mlp": None}]))
    # what a file may leave out
    lean = copy.deepcopy(cases.CONFIGS["Q"])
    m = lean["layers"][2]["mixer"]
    del m["left"]["kv_heads"], m["left"]["vdim"], m["left"]["rot"]["base"], m["left"]["mask"], m["right"]["kv_heads"], m["right"]["vdim"]
    del m["left_scale"], m["right_scale"], lean["layers"][1]["mixer"]["groups"], lean["layers"][1]["mixer"]["norm_groups"]
    del lean["layers"][0]["mlp"]["router"]["scale"]
    cfg = VugotarConfig.from_dict(lean)
    p, s = cfg.layers[2].mixer, cfg.layers[1].mixer
    assert (p.left.kv_heads, p.left.vdim, p.left.rot_base, p.left.chunk) == (2, 32, 10000.0, 0)
    assert (p.right.kv_heads, p.right.vdim, p.left_scale, p.right_scale, s.groups, s.norm_groups) == (2, 64, 1.0, 1.0, 1, 1)
    assert cfg.layers[0].mlp.scale == 1.0 and VugotarConfig.from_dict(cfg.to_dict()) == cfg


def test_parts_cache_groups_and_tensors_of_a_configuration():
    from kvcm_amd.architectures.vugotar import vugotar_spec
    from kvcm_amd.config.vugotar_config import VugotarConfig
    from kvcm_amd.engine.runner import plan_groups
    from kvcm_amd.parts.base import BuildContext, KVCacheNeed, StateNeed
    from kvcm_amd.parts.model import Model
    from kvcm_amd.weights.random_init import expected_tensors
    cfg = VugotarConfig.from_dict(cases.CONFIGS["P"])
    spec = vugotar_spec(cfg)
    assert [l.name for l in spec.layers] == ["l0", "l1", "l2", "l3", "l1.pass1", "l2.pass1", "l3.pass1", "l4"]
    assert [("again" in l.parts) for l in spec.layers] == [False, False, False, False, True, False, False, False]
    assert spec.keep_embedding and not vugotar_spec(VugotarConfig.from_dict(cases.CONFIGS["U"])).keep_embedding
    model = Model(spec, BuildContext(torch.bfloat16, torch.device("cpu"), spec.hidden_size, 16, None))
    assert model.capturable, model.not_capturable()
    plans = {g.need: [name for name, _ in g.layers] for g in model.groups}
    # every pass has places of its own
    assert plans[KVCacheNeed(2, 16, value_dim=12, chunk=20)] == ["l1", "l1.pass1"]
    assert plans[StateNeed((6, 12, 20), torch.float32)] == ["l1", "l1.pass1"] and plans[StateNeed((3, 2 * 3 * 12 + 6 * 20), torch.float32)] == ["l1", "l1.pass1"]
    assert plans[StateNeed((3, 24, 16), torch.float32)] == ["l2", "l2.pass1"] and plans[StateNeed((2, 4 * 12 + 2 * 2 * 10), torch.float32)] == ["l0"]
    chunks = sorted((g.kind, g.window, g.chunk) for g in plan_groups(model, 50, 4) if g.kind != "state")
    assert chunks == [("window", 7, 7), ("window", 20, 20), ("window", 33, 33)]
    names = expected_tensors("Vugotar", cfg)
    for n in ("embed", "final.norm", "head", "l0.norm1", "l0.mix.in", "l0.mix.conv", "l0.mix.conv.b", "l0.mix.D", "l0.mix.o", "l0.mlp.gate.b", "l0.mlp.down.b",
              "l1.mix.left.q", "l1.mix.left.o", "l1.mix.right.q.conv", "l1.mix.right.v.conv", "l1.mix.right.b", "l1.mix.right.a", "l1.mix.right.A_log",
              "l1.mix.right.dt_bias", "l1.mix.right.norm", "l1.mix.right.g", "l1.mlp.e4.down", "l1.mlp.router", "l1.mlp.shared.gate", "l1.mlp.shared.sg"):
        assert n in names, n
    assert "l2.mlp.router" not in names and "l1.mlp.gate" not in names and "l1.norm2" not in names and "l1.mlp.shared.gate.b" not in names
    assert names["l1.mlp.shared.sg"][0] == (1, 48) and names["l0.mix.in"][0] == (4 * 12 + (4 * 12 + 2 * 2 * 10) + 4, 48)
    assert names["l1.mix.right.norm"] == ((20,), "vector") and names["l0.norm1"][1] == "bias"
    # no shared expert, no gate of one
    q = expected_tensors("Vugotar", VugotarConfig.from_dict(cases.CONFIGS["Q"]))
    assert "l1.mlp.shared.sg" not in q and "l1.mlp.shared.up" not in q and "l0.mlp.shared.sg" in q
    # one tap: nothing of the convolution is kept
    r = Model(vugotar_spec(VugotarConfig.from_dict(cases.CONFIGS["R"])), BuildContext(torch.float32, torch.device("cpu"), 32, 8, None))
    assert sum(isinstance(g.need, StateNeed) and len(g.need.shape) == 2 for g in r.groups) == 1


def test_passes_share_what_is_made_of_their_weights():
    """Layers that run again name the same tensors, and the fused, padded and interleaved matrices made of them exist once."""
    from kvcm_amd.architectures.vugotar import vugotar_spec
    from kvcm_amd.parts.base import BuildContext
    from kvcm_amd.parts.model import Model
    from kvcm_amd.weights.loader import DictSource, load_weights
    cfg, tensors = cases.tensors_for(cases.CONFIGS["P"], seed=3)
    spec = vugotar_spec(cfg)
    model = Model(spec, BuildContext(torch.float32, torch.device("cpu"), spec.hidden_size, 16, None))
    load_weights(model, DictSource(tensors), torch.float32, torch.device("cpu"))
    first, second = (next(p for l, p in zip(spec.layers, model.layer_parts) if l.name == n)["mixer"] for n in ("l1", "l1.pass1"))
    for key in ("w_in", "w_out"):
        assert first.w[key].data_ptr() == second.w[key].data_ptr()
    assert first.members[2].w["w_up"].data_ptr() == second.members[2].w["w_up"].data_ptr()
    assert first.members[2].w["w_up"].shape == (5, 64, 48)      # 20 columns padded to 32, gate and up interleaved
    # the joined matrices: the members' sources under one another, their last matrices side by side
    at = 0
    for m in first.members:
        for name, shape in m.in_sources():
            assert torch.equal(first.w["w_in"][at:at + shape[0]], tensors[name]), name
            at += shape[0]
    assert first.w["w_in"].shape[0] == -(-at // 16) * 16 and not first.w["w_in"][at:].any()
    assert torch.equal(first.w["w_out"], torch.cat([tensors["l1.mix.left.o"], tensors["l1.mix.right.o"], tensors["l1.mlp.shared.down"]], 1))
    np.testing.assert_allclose(first.members[1].w["norm"].numpy(), np.tile(tensors["l1.mix.right.norm"].numpy(), 6) * np.float32(1.3), rtol=1e-6)


def test_pages_are_given_back_chunk_by_chunk():
    """A chunked group keeps the pages of the chunk that the next token belongs to (its first one may be shared with the chunk
    before) and gives back everything earlier, whatever the portions."""
    from kvcm_amd.cache.manager import CacheGroupSpec, HostCore
    B = 8
    sizes = (20, 5, 8, 32, 1)
    core = HostCore([CacheGroupSpec("window", c, 64, chunk=c) for c in sizes], block_size=B, max_seq_len=256, max_num_seqs=2, watermark_blocks=0)
    core.seq_new(1, list(range(30)))
    core.admit(1)
    done = 0
    for n in (30, 7, 1, 1, 1, 50, 1, 5, 40):
        if done:
            core.seq_push_tokens(1, list(range(n)))
            assert core.append_slot(1)
        done += n
        core.set_computed(1, done)
        core.commit(1)
        for g, c in enumerate(sizes):
            first = done // c * c // B
            assert all((p >= 0) == (i >= first) for i, p in enumerate(core.seq_table(1, g))), (done, c)
    core.release(1)
    assert [core.blocks_in_use(g) for g in range(len(sizes))] == [0] * len(sizes)
    with pytest.raises(Exception, match="only a windowed group"):
        HostCore([CacheGroupSpec("full", 0, 8, chunk=3)], block_size=B, max_seq_len=64, max_num_seqs=1)
    with pytest.raises(ValueError, match="no window"):
        from kvcm_amd.parts.base import KVCacheNeed
        KVCacheNeed(1, 8, window=4, chunk=4)


def test_members_that_do_not_offer_their_ends_are_refused():
    from kvcm_amd.parts.base import BuildContext, PartSpec
    from kvcm_amd.parts.joined_parts import JoinedSublayers
    from kvcm_amd.parts.routed_parts import RoutedExperts
    ctx = BuildContext(torch.float32, torch.device("cpu"), 16, 16, None)
    with pytest.raises(ValueError, match="does not offer its ends"):
        JoinedSublayers({"members": (("ffn", "ffn", PartSpec("plain_mlp", {"intermediate_size": 8}, "a.")),)}, "l0.", ctx)
    with pytest.raises(ValueError, match="no members"):
        JoinedSublayers({"members": ()}, "l0.", ctx)
    with pytest.raises(ValueError, match="no product to join"):
        RoutedExperts({"experts": 2, "top": 1, "ff": 8, "routing": "table", "joined": True}, "e.", ctx)
    with pytest.raises(ValueError, match="needs one"):
        RoutedExperts({"experts": 2, "top": 1, "ff": 8, "shared_gate": "sg"}, "e.", ctx)


def test_random_model_folders_of_the_design(tmp_path):
    from kvcm_amd.config.vugotar_config import VugotarConfig
    from kvcm_amd.engine.build import read_model_config
    from kvcm_amd.weights.random_init import write_model_dir
    cfg = VugotarConfig.from_dict(cases.CONFIGS["P"])
    d = write_model_dir(str(tmp_path / "m"), "Vugotar", cfg, seed=4, dtype=torch.bfloat16, std=0.1, norm_jitter=0.1, device="cpu")
    arch, again = read_model_config(d)
    assert arch.name == "Vugotar" and again == cfg
    t = plain.read_tensors(str(tmp_path / "m" / "model.safetensors"))
    assert abs(t["l1.norm1"].mean()) < 0.1 and abs(t["l1.mix.right.norm"].mean() - 1.0) < 0.1 and t["l0.mlp.down.b"].shape == (48,)
    logits = plain.forward(cases.CONFIGS["P"], t, [5, 17, 3, 90])
    assert logits.shape == (4, 97) and np.isfinite(logits).all()


# ---------------------------------------------------------------- pins of the plain implementation
def test_plain_norms_rotation_and_sink_on_known_inputs():
    np.testing.assert_allclose(plain.offset_norm(np.array([3.0, 4.0]), np.array([0.0, 0.5]), 0.0), [3 / 12.5 ** 0.5, 6 / 12.5 ** 0.5])
    np.testing.assert_allclose(plain.rotate_pairs(np.array([[[1.0, 0.0, 2.0, 0.0, 7.0]]]), [1], 4, 100.0),
                               [[[np.cos(1), np.sin(1), 2 * np.cos(0.1), 2 * np.sin(0.1), 7.0]]], atol=1e-12)
    np.testing.assert_allclose(plain.sink_softmax(np.array([0.0, np.log(2.0), -np.inf])), [0.25, 0.5, 0.0])
    np.testing.assert_allclose(plain.sink_softmax(np.array([-800.0, -800.0])), [0.0, 0.0])
    # chunks of 3: position 5 sees 3, 4, 5; position 6 itself alone; equal scores of 0 share with the sink
    q, k, v = np.zeros((7, 1, 2)), np.zeros((7, 1, 2)), np.arange(7.0).reshape(7, 1, 1)
    out = plain.chunk_attention(q, k, v, 1.0, np.arange(7), np.arange(7), 3)
    np.testing.assert_allclose(out[[2, 3, 5, 6], 0, 0], [3 / 4, 3 / 2, 12 / 4, 6 / 2])
    np.testing.assert_allclose(plain.chunk_attention(q, k, v, 1.0, np.arange(7), np.arange(7))[6, 0, 0], 21 / 8)


def test_plain_recurrences_on_known_inputs():
    x = np.arange(1.0, 6.0).reshape(5, 1)
    np.testing.assert_allclose(plain.causal_conv(x, np.array([[100.0, 10.0, 1.0]]))[:, 0], [1, 12, 123, 234, 345])
    np.testing.assert_allclose(plain.causal_conv(x, np.array([[2.0]]), np.array([1.0]))[:, 0], [3, 5, 7, 9, 11])
    np.testing.assert_allclose(plain.softplus(np.array([0.0, 800.0, -800.0])), [np.log(2), 800.0, 0.0])
    # a full rate replaces what the key held; a rate of a half goes half way; the read-out sees the write
    k = np.array([[[1.0, 0.0]], [[0.0, 1.0]], [[1.0, 0.0]], [[1.0, 0.0]]])
    v = np.array([[[4.0]], [[6.0]], [[8.0]], [[0.0]]])
    o = plain.gated_delta(k, k, v, np.ones((4, 1)), np.array([[1.0], [1.0], [0.5], [1.0]]))
    np.testing.assert_allclose(o[:, 0, 0], [4, 6, 6, 0])
    # the decay acts before the removal: 4 decays to 2, a rate of a half towards 8 gives 5
    o = plain.gated_delta(k[[0, 0]], k[[0, 0]], v[[0, 2]], np.array([[1.0], [0.5]]), np.array([[1.0], [0.5]]))
    np.testing.assert_allclose(o[:, 0, 0], [4, 5])
    y = plain.state_space(np.ones((3, 1, 1)), np.ones((3, 1, 1)), np.ones((3, 1, 1)), np.full((3, 1), np.log(2.0)), np.zeros(1), np.array([10.0]))
    np.testing.assert_allclose(y[:, 0, 0], 10 + np.log(2.0) * np.array([1, 1.5, 1.75]))


def test_plain_routing_and_layer_order_on_known_inputs():
    chosen, weight = plain.choose_experts(np.array([[0.0, 2.0, 1.0, 2.0 + np.log(3.0)]]), 2, 2.5)
    assert chosen.tolist() == [[3, 1]]
    np.testing.assert_allclose(weight, [[0.75 * 2.5, 0.25 * 2.5]])
    assert plain.layer_runs(cases.CONFIGS["P"]) == [(0, False), (1, False), (2, False), (3, False), (1, True), (2, False), (3, False), (4, False)]
    assert plain.layer_runs(cases.CONFIGS["S"]) == [(0, False), (0, True), (0, True), (1, False), (2, False)]
    assert plain.layer_runs(cases.CONFIGS["U"]) == [(0, False), (1, False)] and plain.layer_runs(cases.CONFIGS["R"]) == [(i, False) for i in range(3)]
