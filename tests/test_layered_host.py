"""CPU-side checks of the layered models' plumbing: configuration, layer order, slots, step tables, the checkpoint
reader, the library's exported surface, and the plain implementation's own consistency."""

import json
import re
import struct
import subprocess
from pathlib import Path

import pytest
import torch

REPO = Path(__file__).resolve().parent.parent


def _cfg():
    return {
        "architecture": "Bavesun", "vocab": 19, "width": 12, "norm": {"eps": 1e-6}, "embedding": {"scale": 2.5},
        "token_side": {"dim": 2}, "loop": {"start": 1, "stop": 3, "times": 3},
        "layers": [
            {"type": "retention", "mlp": {"kind": "dense", "ff": 10},
             "mixer": {"heads": 2, "dim": 4, "vdim": 6, "decay": [0.5, 0.75], "rot": {"dims": 2, "base": 100.0}}},
            {"type": "latent_attention", "mlp": {"kind": "moe", "expert": {"ff": 5}, "router": {"experts": 3, "top": 2}},
             "mixer": {"heads": 3, "dim": 2, "rot_dim": 4, "vdim": 2, "kv_rank": 6, "scale": 0.4,
                       "rot": {"dims": 4, "base": 50.0}}},
            {"type": "retention", "mlp": None,
             "mixer": {"heads": 1, "dim": 2, "vdim": 2, "decay": [1.0], "rot": {"dims": 2, "base": 7.0}}},
            {"type": "latent_attention", "mlp": None,
             "mixer": {"heads": 1, "dim": 2, "rot_dim": 2, "vdim": 4, "kv_rank": 4, "scale": 0.5,
                       "rot": {"dims": 2, "base": 50.0}}},
        ]}


def test_config_reads_every_size_and_the_layer_order():
    from lit_gpt.config import LayeredConfig

    c = LayeredConfig.from_dict(_cfg())
    assert (c.vocab, c.width, c.norm_eps, c.embedding_scale, c.side_dim) == (19, 12, 1e-6, 2.5, 2)
    assert c.layer_runs == [0, 1, 2, 1, 2, 1, 2, 3]
    m = c.layers[1].mixer
    assert (m.kind, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale) == ("latent_attention", 3, 2, 4, 2, 6, 0.4)
    assert c.layers[1].mlp.experts == 3 and c.layers[1].mlp.top == 2 and c.layers[1].mlp.ff == 5
    assert c.layers[0].mixer.decay == [0.5, 0.75] and c.layers[2].mlp is None
    f = c.layers[3].mixer.rot.inv_freq()
    assert f == [1.0]
    assert c.layers[1].mixer.rot.inv_freq() == pytest.approx([1.0, 50.0 ** -0.5])
    d = _cfg()
    del d["loop"], d["token_side"]
    c2 = LayeredConfig.from_dict(d)
    assert c2.layer_runs == [0, 1, 2, 3] and c2.side_dim == 0


def test_config_rejects_what_does_not_fit():
    from lit_gpt.config import LayeredConfig

    for change in (lambda d: d["loop"].update(stop=9), lambda d: d["layers"][0]["mixer"].update(decay=[0.5]),
                   lambda d: d["layers"][1]["mlp"]["router"].update(top=4),
                   lambda d: d["layers"][0].update(type="convolution"),
                   lambda d: d["layers"][0]["mixer"]["rot"].update(dims=6)):
        d = _cfg()
        change(d)
        with pytest.raises(ValueError):
            LayeredConfig.from_dict(d)


def test_registry_picks_the_class_by_config_json(tmp_path):
    from lit_gpt.config import LayeredConfig, load_config, model_class

    (tmp_path / "config.json").write_text(json.dumps(_cfg()))
    c = load_config(tmp_path)
    assert isinstance(c, LayeredConfig)
    assert model_class(c).__name__ == "LayeredGPT"
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nonesuch"}))
    with pytest.raises(ValueError, match="not registered"):
        load_config(tmp_path)


def test_tensor_shapes_name_every_checkpoint_tensor():
    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT

    shapes = LayeredGPT.tensor_shapes(LayeredConfig.from_dict(_cfg()))
    assert shapes["embed"] == (19, 12) and shapes["side.embed"] == (19, 8) and shapes["final.norm"] == (12,)
    assert shapes["l0.mix.q"] == (8, 12) and shapes["l0.mix.v"] == (12, 12) and shapes["l0.mix.o"] == (12, 12)
    assert shapes["l1.mix.q"] == (18, 12) and shapes["l1.mix.dkv"] == (10, 12) and shapes["l1.mix.uk"] == (6, 6)
    assert shapes["l1.mix.uv"] == (6, 6) and shapes["l1.mix.sink"] == (3,) and shapes["l1.mix.dkv.norm"] == (6,)
    assert shapes["l1.mlp.router"] == (3, 12) and shapes["l1.mlp.e2.down"] == (12, 5)
    assert shapes["l0.mlp.gate"] == (10, 12) and shapes["l3.side.proj"] == (12, 2)
    assert not any(k.startswith("l2.mlp") for k in shapes)


def test_slot_pool_hands_out_the_lowest_free_slot():
    from generate.batch import SlotPool

    p = SlotPool()
    assert [p.take() for _ in range(4)] == [0, 1, 2, 3]
    p.give(2)
    p.give(0)
    assert p.take() == 0 and p.take() == 2 and p.take() == 4
    with pytest.raises(ValueError):
        p.give(9)
    p.give(1)
    with pytest.raises(ValueError):
        p.give(1)


def test_step_table():
    from lit_gpt.mixers import StepBatch

    s = StepBatch.build([(3, 0, [5, 6, 7]), (0, 10, [1])], torch.device("cpu"))
    assert (s.T, s.B) == (4, 2)
    assert s.tokens.tolist() == [5, 6, 7, 1] and s.slot.tolist() == [3, 3, 3, 0] and s.pos.tolist() == [0, 1, 2, 10]
    assert s.seq_start.tolist() == [0, 3, 4] and s.seq_slot.tolist() == [3, 0] and s.seq_pos0.tolist() == [0, 10]
    assert s.tokens.dtype == torch.int32
    with pytest.raises(ValueError):
        StepBatch.build([(0, 0, [])], torch.device("cpu"))


def test_safetensors_reader(tmp_path):
    from lit_gpt.utils import read_safetensors

    a = torch.randn(3, 5).to(torch.bfloat16)
    b = torch.arange(7, dtype=torch.int32)
    blob = a.view(torch.uint8).numpy().tobytes() + b.view(torch.uint8).numpy().tobytes()
    header = {"a": {"dtype": "BF16", "shape": [3, 5], "data_offsets": [0, 30]},
              "b": {"dtype": "I32", "shape": [7], "data_offsets": [30, 58]}, "__metadata__": {"x": "y"}}
    hj = json.dumps(header).encode()
    path = tmp_path / "m.safetensors"
    path.write_bytes(struct.pack("<Q", len(hj)) + hj + blob)
    out = read_safetensors(path)
    assert set(out) == {"a", "b"} and torch.equal(out["a"], a) and torch.equal(out["b"], b)
    header["a"]["data_offsets"] = [0, 28]
    hj = json.dumps(header).encode()
    path.write_bytes(struct.pack("<Q", len(hj)) + hj + blob)
    with pytest.raises(ValueError):
        read_safetensors(path)


def test_library_exports_every_header_symbol():
    from lit_gpt import seq_ops

    text = re.sub(r"/\*.*?\*/", "", (REPO / "include" / "litgpt_seq.h").read_text(), flags=re.S)
    declared = sorted(set(re.findall(r"\b(lgs_[a-z0-9_]+)\s*\(", text)))
    assert declared == sorted(seq_ops.SIGNATURES)
    if not seq_ops.LIB_PATH.is_file():
        subprocess.run(["make", "-C", str(REPO / "lit-gpt_amd" / "csrc"), "-j8", "seq"], check=True)
    lib = seq_ops.load_library()
    assert lib.lgs_version() >= 1
    rc = lib.lgs_linear(None, 1, 0, None, 0, 0, None, 1, 0, 1, 1, 1, 1, 0, 0, None, None, 0, 0, None, None, 1, None)
    assert rc != 0 and b"null" in lib.lgs_last_error_string()
    with pytest.raises(RuntimeError, match="GPU tensor"):
        seq_ops.rmsnorm(torch.zeros(2, 8), torch.ones(8), offset=0.0, eps=1e-5)


def test_oracle_is_causal_and_loops_share_weights():
    """The plain implementation itself: a later token never changes earlier logits, rotations keep lengths, and the
    routing weights of the chosen experts sum to one."""
    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT
    from oracle import bavesun as ob

    cfg = _cfg()
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=1)
    toks = [3, 1, 4, 1, 5, 9, 2, 6]
    full = ob.forward(cfg, w, toks)
    assert torch.allclose(ob.forward(cfg, w, toks[:5]), full[:5], atol=1e-12)
    assert ob.layer_order(cfg) == [0, 1, 2, 1, 2, 1, 2, 3]
    x = torch.randn(8, dtype=torch.float64)
    for f in (ob.rope_half, ob.rope_interleaved):
        y = f(x, 17, 6, 100.0)
        assert torch.allclose(y.norm(), x.norm()) and torch.equal(y[6:], x[6:])
        assert torch.allclose(f(x, 0, 6, 100.0), x)
    assert ob.rope_half(torch.tensor([1.0, 0, 0, 0], dtype=torch.float64), 1, 4, 100.0)[2] == pytest.approx(
        torch.sin(torch.tensor(1.0, dtype=torch.float64)).item())
    assert ob.rope_interleaved(torch.tensor([1.0, 0, 0, 0], dtype=torch.float64), 1, 4, 100.0)[1] == pytest.approx(
        torch.sin(torch.tensor(1.0, dtype=torch.float64)).item())


# ------------------------------------------------------------------------------------------------ Rigulorn
def _rig_cfg():
    att = {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 10, "diff": 0.3, "softcap": 9.0, "scale": 0.35,
           "mask": {"size": 5}, "rot": {"dims": 4, "base": 300.0}}
    return {
        "architecture": "Rigulorn", "vocab": 23, "width": 16, "norm": {"eps": 1e-5}, "embedding": {"scale": 4.0},
        "streams": 2,
        "layers": [
            {"type": "mamba2", "mlp": None,
             "mixer": {"heads": 4, "vdim": 3, "state": 5, "groups": 2, "norm_groups": 3, "conv": 4}},
            {"type": "attention", "mlp": {"kind": "dense", "ff": 14, "limit": 1.25}, "mixer": dict(att)},
            {"type": "attention", "mlp": None, "mixer": dict(att, kv_from=1, mask={"size": 3})},
        ]}


def test_rigulorn_config_and_tensor_names():
    from lit_gpt.config import LayeredConfig, model_class
    from lit_gpt.layered import LayeredGPT

    c = LayeredConfig.from_dict(_rig_cfg())
    assert model_class(c) is LayeredGPT
    assert (c.streams, c.stream_weights, c.design.block, c.design.tied_head) == (2, True, "sequential", False)
    s, a, b = (l.mixer for l in c.layers)
    assert (s.kind, s.heads, s.vdim, s.state, s.groups, s.norm_groups, s.conv) == ("mamba2", 4, 3, 5, 2, 3, 4)
    assert (a.kv_heads, a.diff, a.softcap, a.mask_size, a.scale, a.rot.dims, a.kv_from) == (2, 0.3, 9.0, 5, 0.35, 4, None)
    assert (b.kv_from, b.mask_size) == (1, 3) and c.layers[1].mlp.limit == 1.25
    shapes = LayeredGPT.tensor_shapes(c)
    assert shapes["head"] == (23, 16) and shapes["l0.mix.in"] == (2 * 12 + 2 * 2 * 5 + 4, 16)
    assert shapes["l0.mix.conv"] == (12 + 20, 4) and shapes["l0.hc1.mix"] == (2, 2) and "l0.hc2.in" not in shapes
    assert shapes["l1.mix.q"] == (48, 16) and shapes["l1.mix.k"] == (24, 16) and shapes["l1.mix.v"] == (20, 16)
    assert "l2.mix.k" not in shapes and "l2.mix.v" not in shapes and "l2.norm2" not in shapes
    assert shapes["l1.norm2"] == (16,) and shapes["l1.mix.lq2"] == (6,)
    w = LayeredGPT.random_weights(c)
    assert set(w) == set(shapes) and all(tuple(w[k].shape) == shapes[k] for k in shapes)
    plain = dict(_rig_cfg())
    del plain["streams"]
    p = LayeredConfig.from_dict(plain)
    assert p.streams == 1 and not p.stream_weights and "l0.hc1.in" not in LayeredGPT.tensor_shapes(p)


@pytest.mark.parametrize("edit", [
    lambda c: c["layers"][2]["mixer"].update(kv_from=0),  # not an attention layer
    lambda c: c["layers"][2]["mixer"].update(kv_from=2),  # itself
    lambda c: c["layers"][2]["mixer"].update(kv_heads=4),  # other key heads than its source
    lambda c: c["layers"][1]["mixer"].update(kv_heads=3),
    lambda c: c["layers"][0]["mixer"].update(groups=3),
    lambda c: c["layers"][0]["mixer"].update(norm_groups=5),
    lambda c: c["layers"][1]["mixer"]["rot"].update(dims=8),
    lambda c: c.update(streams=9),
])
def test_rigulorn_config_rejects_what_does_not_fit(edit):
    from lit_gpt.config import LayeredConfig

    c = _rig_cfg()
    edit(c)
    with pytest.raises(ValueError):
        LayeredConfig.from_dict(c)


def test_rigulorn_plain_implementation_is_causal_and_chunked():
    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT
    from oracle import rigulorn as orc

    cfg = _rig_cfg()
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=3)
    toks = [3, 7, 1, 0, 22, 5, 9, 9, 4, 13, 2, 8]
    full = orc.forward(cfg, w, toks)
    assert torch.allclose(orc.forward(cfg, w, toks[:7]), full[:7], atol=1e-10)
    # attention alone: a token before the query's chunk cannot reach it (values are per-token maps of the embedding)
    only = dict(cfg, layers=[dict(cfg["layers"][1], mlp=None)])
    w1 = {k: v for k, v in LayeredGPT.random_weights(LayeredConfig.from_dict(only), seed=4).items()}
    a = orc.forward(only, w1, toks)
    other = list(toks)
    other[4] = 11  # the last position of the first chunk of 5
    b = orc.forward(only, w1, other)
    assert torch.allclose(a[5:], b[5:], atol=1e-12) and not torch.allclose(a[4], b[4], atol=1e-6)
    assert orc.visible(9, 5, {"size": 5}) and not orc.visible(9, 4, {"size": 5}) and not orc.visible(4, 5, None)
    # a kernel that is 1 in column taps - 1 and 0 elsewhere copies its input
    u = torch.arange(6.0, dtype=torch.float64).view(6, 1)
    got = orc.causal_conv(u, torch.tensor([[0.0, 0.0, 1.0]], dtype=torch.float64), torch.zeros(1, dtype=torch.float64))
    assert torch.equal(got, u)


# ------------------------------------------------------------------------------------------------ Ravelorn
def _rav_cfg():
    return {
        "architecture": "Ravelorn", "vocab": 23, "width": 16, "norm": {"eps": 1e-5}, "residual_mult": 0.4,
        "logit_softcap": 7.0, "max_positions": 30,
        "layers": [
            {"type": "channel_delta", "mlp": {"kind": "moe", "expert": {"ff": 6}, "router": {"experts": 3, "identity": 2, "top": 2}},
             "mixer": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 5, "conv": 3, "decay_rank": 3, "gate_rank": 4}},
            {"type": "parallel", "mlp": None,
             "mixer": {"left": {"heads": 6, "kv_heads": 2, "dim": 4, "vdim": 3, "scale": 0.3, "q_temp": {"coef": 0.5, "every": 4}},
                       "right": {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 6, "conv": 2},
                       "left_scale": 1.5, "right_scale": 0.25}},
        ]}


def test_ravelorn_config_and_tensor_names():
    from lit_gpt.config import LayeredConfig, model_class
    from lit_gpt.layered import LayeredGPT

    c = LayeredConfig.from_dict(_rav_cfg())
    assert model_class(c) is LayeredGPT
    d = c.design
    assert (d.block, d.norm, d.positions, d.moe, d.tied_head) == ("post", "layer", "learned", "scores", False)
    assert (c.residual_mult, c.logit_softcap, c.max_positions) == (0.4, 7.0, 30)
    a, p = (l.mixer for l in c.layers)
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.conv) == ("channel_delta", 4, 2, 6, 5, 3)
    assert (p.left.kind, p.left.heads, p.left.kv_heads, p.left.scale, p.left.q_temp_coef, p.left.q_temp_every) == \
        ("sink_attention", 6, 2, 0.3, 0.5, 4)
    assert (p.right.kind, p.right.heads, p.right.kv_heads, p.right.conv, p.left_scale, p.right_scale) == \
        ("gated_delta", 2, 1, 2, 1.5, 0.25)
    f = c.layers[0].mlp
    assert (f.experts, f.identity, f.top, f.ff) == (3, 2, 2, 6) and c.layers[1].mlp is None
    shapes = LayeredGPT.tensor_shapes(c)
    assert shapes["pos"] == (30, 16) and shapes["head"] == (23, 16) and shapes["final.norm.b"] == (16,)
    assert shapes["l0.norm1.b"] == (16,) and shapes["l0.norm2.b"] == (16,) and "l1.norm2" not in shapes
    assert shapes["l0.mix.q"] == (12, 16) and shapes["l0.mix.v"] == (20, 16) and shapes["l0.mix.k.conv"] == (12, 3)
    assert shapes["l0.mix.a1"] == (3, 16) and shapes["l0.mix.a2"] == (24, 3) and shapes["l0.mix.dt_bias"] == (24,)
    assert shapes["l0.mix.g2"] == (20, 4) and shapes["l0.mix.norm"] == (5,) and shapes["l0.mix.b"] == (4, 16)
    assert shapes["l0.mlp.router"] == (5, 16) and shapes["l0.mlp.correction"] == (5,) and "l0.mlp.e3.up" not in shapes
    assert shapes["l0.mlp.e2.gate"] == (6, 16) and shapes["l0.mlp.e2.down"] == (16, 6)
    assert shapes["l1.mix.left.q"] == (24, 16) and shapes["l1.mix.left.k"] == (8, 16) and shapes["l1.mix.left.v"] == (6, 16)
    assert shapes["l1.mix.left.sink"] == (6,) and shapes["l1.mix.left.o"] == (16, 18)
    assert shapes["l1.mix.right.a"] == (2, 16) and shapes["l1.mix.right.dt_bias"] == (2,) and shapes["l1.mix.right.g"] == (12, 16)
    w = LayeredGPT.random_weights(c)
    assert set(w) == set(shapes) and all(tuple(w[k].shape) == shapes[k] for k in shapes)
    bare = _rav_cfg()
    del bare["layers"][1]["mixer"]["left"]["q_temp"]
    assert LayeredConfig.from_dict(bare).layers[1].mixer.left.q_temp_every == 0


@pytest.mark.parametrize("edit", [
    lambda c: c["layers"][0]["mixer"].update(kv_heads=3),  # heads no multiple of the key heads
    lambda c: c["layers"][0]["mixer"].update(conv=0),
    lambda c: c["layers"][0]["mixer"].update(dim=600),
    lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4),
    lambda c: c["layers"][1]["mixer"]["right"].update(kv_heads=0),
    lambda c: c["layers"][0]["mlp"]["router"].update(top=6),  # more than experts + identity experts
    lambda c: c.update(max_positions=0),
])
def test_ravelorn_config_rejects_what_does_not_fit(edit):
    from lit_gpt.config import LayeredConfig

    c = _rav_cfg()
    edit(c)
    with pytest.raises(ValueError):
        LayeredConfig.from_dict(c)


def test_ravelorn_plain_implementation():
    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT
    from oracle import ravelorn as orc

    cfg = _rav_cfg()
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=3)
    toks = [3, 7, 1, 0, 22, 5, 9, 9, 4, 13, 2, 8]
    full = orc.forward(cfg, w, toks)
    assert torch.allclose(orc.forward(cfg, w, toks[:7]), full[:7], atol=1e-10)  # causal
    assert float(full.abs().max()) < cfg["logit_softcap"]
    # a convolution kernel that is 1 in column taps - 1 and 0 elsewhere passes its input to the activation
    u = torch.linspace(-2, 2, 6, dtype=torch.float64).view(6, 1)
    assert torch.allclose(orc.causal_conv_silu(u, torch.tensor([[0.0, 0.0, 1.0]], dtype=torch.float64)), orc.silu(u))
    # the delta rule stores a value under a key and returns it to a query along that key; a second write under the
    # same key replaces it (beta 1, no decay)
    k = torch.tensor([[1.0, 0.0], [1.0, 0.0], [0.0, 1.0]], dtype=torch.float64)
    v = torch.tensor([[2.0, 3.0], [5.0, 7.0], [1.0, 1.0]], dtype=torch.float64)
    o = orc.delta_rule(k, k, v, torch.ones(3, dtype=torch.float64), torch.ones(3, 2, dtype=torch.float64))
    assert torch.allclose(o, v)
    # a sink as large as the only score halves the output; identity experts return the input
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0}
    eye = torch.eye(2, dtype=torch.float64)
    h = torch.tensor([[1.0, 1.0]], dtype=torch.float64)
    aw = {"q": eye, "k": eye, "v": eye, "o": eye}
    plain = orc.sink_attention(h, aw, m, 0.0)
    score = 2.0  # unit-RMS q . k
    halved = orc.sink_attention(h, dict(aw, sink=torch.tensor([score], dtype=torch.float64)), m, 0.0)
    assert torch.allclose(plain, h) and torch.allclose(halved, 0.5 * h)
    rw = {"router": torch.tensor([[0.0, 0.0], [9.0, 9.0]], dtype=torch.float64)}
    out = orc.moe_ff(h, rw, {"router": {"experts": 0, "identity": 2, "top": 1}})
    assert torch.allclose(out, torch.softmax(torch.tensor([0.0, 18.0], dtype=torch.float64), 0)[1] * h)


# ------------------------------------------------------------------------------------------------ the Gatutar design
def _gat_cfg():
    return {
        "architecture": "Gatutar", "vocab": 23, "width": 16, "norm": {"eps": 1e-5},
        "layers": [
            {"type": "parallel_2", "mlp": {"kind": "dense", "ff": 10},
             "mixer": {"left": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 6, "scale": 0.3, "q_temp": {"coef": 0.5, "every": 4}},
                       "right": {"heads": 2, "dim": 5, "vdim": 3, "decay": [0.5, 0.9]}}},
            {"type": "parallel", "mlp": {"kind": "moe", "expert": {"ff": 6}, "router": {"experts": 3, "top": 2},
                                         "shared": {"ff": 4}},
             "mixer": {"left": {"heads": 6, "kv_heads": 3, "dim": 4, "vdim": 2, "scale": 0.5,
                                "rot": {"dims": 2, "base": 100.0,
                                        "scaling": {"factor": 2.0, "low": 1.0, "high": 4.0, "original": 16}}},
                       "right": {"heads": 2, "dim": 3, "vdim": 5, "tau": 3.0}}},
            {"type": "parallel", "mlp": None,
             "mixer": {"left": {"heads": 1, "kv_heads": 1, "dim": 4, "vdim": 4, "scale": 0.5},
                       "right": {"heads": 1, "dim": 2, "vdim": 2, "tau": 1.0}}},
        ],
    }


def test_gatutar_config_and_tensor_names():
    from lit_gpt.config import LayeredConfig, model_class
    from lit_gpt.layered import LayeredGPT

    c = LayeredConfig.from_dict(_gat_cfg())
    assert model_class(c) is LayeredGPT
    d = c.design
    assert (d.block, d.norm, d.dense_ff, d.moe, d.tied_head, d.norm_offset) == ("sandwich", "rms", "relu2", "sigmoid", False, 0.0)
    a, b, e = (l.mixer for l in c.layers)
    assert (a.kind, a.branch_norm, a.left_scale, a.right_scale) == ("parallel", True, 0.5, 0.5)
    assert (a.left.kind, a.left.heads, a.left.kv_heads, a.left.qk_norm, a.left.sink_kind, a.left.values, a.left.head_gate,
            a.left.q_temp_coef, a.left.q_temp_every, a.left.rot.dims) == \
        ("key_value_attention", 4, 2, "weight", "none", "keys", True, 0.5, 4, 0)
    assert (a.right.kind, a.right.decay, a.right.dim, a.right.vdim) == ("lightning", [0.5, 0.9], 5, 3)
    assert (b.left.kind, b.left.qk_norm, b.left.sink_kind, b.left.values, b.left.head_gate, b.left.rot.dims) == \
        ("rotary_attention", "none", "one", "own", False, 2)
    assert b.left.rot.scaling == {"factor": 2.0, "low": 1.0, "high": 4.0, "original": 16.0}
    assert (b.right.kind, b.right.tau) == ("gated_linear", 3.0) and e.left.rot.dims == 0
    f = c.layers[1].mlp
    assert (f.experts, f.top, f.ff, f.shared_ff) == (3, 2, 6, 4) and c.layers[2].mlp is None
    assert c.layers[0].mlp.kind == "dense" and c.layers[0].mlp.ff == 10
    shapes = LayeredGPT.tensor_shapes(c)
    assert shapes["head"] == (23, 16) and shapes["final.norm"] == (16,) and "pos" not in shapes
    for n in ("norm1", "norm1b", "norm2", "norm2b", "ls1", "ls2"):
        assert shapes[f"l0.{n}"] == (16,)
    assert "l2.norm2" not in shapes and "l2.ls2" not in shapes and shapes["l2.ls1"] == (16,)
    assert shapes["l0.mix.left.q"] == (24, 16) and shapes["l0.mix.left.k"] == (12, 16) and "l0.mix.left.v" not in shapes
    assert shapes["l0.mix.left.q.norm"] == (6,) and shapes["l0.mix.left.g"] == (4, 16) and shapes["l0.mix.left.o"] == (16, 24)
    assert shapes["l0.mix.right.q"] == (10, 16) and shapes["l0.mix.right.v"] == (6, 16) and shapes["l0.mix.right.norm"] == (6,)
    assert shapes["l0.mix.left.out"] == (16,) and shapes["l0.mix.right.out"] == (16,)
    assert shapes["l0.mlp.up"] == (10, 16) and "l0.mlp.gate" not in shapes
    assert shapes["l1.mix.left.v"] == (6, 16) and shapes["l1.mix.left.o"] == (16, 12) and "l1.mix.left.sink" not in shapes
    assert shapes["l1.mix.right.a2"] == (6, 16) and shapes["l1.mix.right.a2.b"] == (6,) and shapes["l1.mix.right.norm"] == (5,)
    assert shapes["l1.mlp.router"] == (3, 16) and shapes["l1.mlp.e2.up"] == (6, 16) and "l1.mlp.e2.gate" not in shapes
    assert shapes["l1.mlp.shared.up"] == (4, 16) and shapes["l1.mlp.shared.sg"] == (1, 16)
    w = LayeredGPT.random_weights(c)
    assert set(w) == set(shapes) and all(tuple(w[k].shape) == shapes[k] for k in shapes)


@pytest.mark.parametrize("edit", [
    lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3),  # heads no multiple of the key heads
    lambda c: c["layers"][0]["mixer"]["left"].update(vdim=5),  # values that are the keys have the keys' size
    lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5]),  # one decay per head
    lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=6),  # more rotary dims than the head has
    lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=3),
    lambda c: c["layers"][1]["mixer"]["right"].update(tau=0.0),
    lambda c: c["layers"][1]["mixer"]["right"].update(dim=600),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=4),
])
def test_gatutar_config_rejects_what_does_not_fit(edit):
    from lit_gpt.config import LayeredConfig

    c = _gat_cfg()
    edit(c)
    with pytest.raises(ValueError):
        LayeredConfig.from_dict(c)


def test_gatutar_plain_implementation():
    import math

    from lit_gpt.config import LayeredConfig, RotarySpec
    from lit_gpt.layered import LayeredGPT
    from oracle import gatutar as orc

    cfg = _gat_cfg()
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=3)
    toks = [3, 7, 1, 0, 22, 5, 9, 9, 4, 13, 2, 8]
    full = orc.forward(cfg, w, toks)
    assert torch.allclose(orc.forward(cfg, w, toks[:7]), full[:7], atol=1e-10)  # causal
    D = torch.float64
    eye = torch.eye(2, dtype=D)
    h = torch.tensor([[1.0, 1.0]], dtype=D)
    # one key whose score is 0: with the extra one in the denominator the weight is a half
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 0.0}
    out = orc.rope_attention(h, m, {"q": eye, "k": eye, "v": eye, "o": eye})
    assert torch.allclose(out, 0.5 * h)
    # a rotation by position p turns the pair (1, 0) by the angle p * f; dims beyond the rotated ones pass
    r = orc.rotate_half(torch.tensor([1.0, 5.0, 0.0, 7.0], dtype=D)[[0, 2, 1, 3]], 3, [0.25])  # pairs (0, 1) of a 2-dim rotation
    assert torch.allclose(r, torch.tensor([math.cos(0.75), math.sin(0.75), 5.0, 7.0], dtype=D))
    # frequency bands: short waves kept, long ones divided by the factor, the same numbers as the product's table
    rot = {"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 40}}
    f = orc.scaled_frequencies(rot)
    assert f[0] == 1.0 and f[-1] == pytest.approx(100.0 ** -0.75 / 4.0)
    assert f == pytest.approx(RotarySpec(8, 100.0, rot["scaling"]).inv_freq(), rel=1e-12)
    # the linear rule: without decay the state is the sum of the outer products
    q = torch.tensor([[[1.0, 0.0]], [[0.0, 1.0]]], dtype=D)
    k = torch.tensor([[[1.0, 0.0]], [[1.0, 1.0]]], dtype=D)
    v = torch.tensor([[[2.0]], [[3.0]]], dtype=D)
    o = orc.linear_recurrence(q, k, v, torch.ones(2, 1, 2, dtype=D))
    assert o.view(-1).tolist() == [2.0, 3.0]
    o = orc.linear_recurrence(q.flip(0), k, v, torch.full((2, 1, 2), 0.5, dtype=D))
    assert o.view(-1).tolist() == [0.0, 0.5 * 2.0 + 3.0]
    # the router's score scales the expert's input: with relu^2 experts the output goes with its square
    fw = {"router": torch.tensor([[0.0, 0.0], [1.0, 1.0]], dtype=D), "e0.up": eye, "e0.down": eye, "e1.up": eye, "e1.down": eye}
    out = orc.feed_forward(h, {"kind": "moe", "router": {"experts": 2, "top": 1}}, fw)
    assert torch.allclose(out, torch.sigmoid(torch.tensor(2.0, dtype=D)) ** 2 * h)
    # a shut shared gate leaves the routed experts alone; an open one adds the shared expert
    fs = dict(fw, **{"shared.up": eye, "shared.down": eye, "shared.sg": torch.tensor([[-50.0, 0.0]], dtype=D)})
    shut = orc.feed_forward(h, {"kind": "moe", "router": {"experts": 2, "top": 1}, "shared": {"ff": 2}}, fs)
    assert torch.allclose(shut, out)
    fs["shared.sg"] = torch.tensor([[50.0, 0.0]], dtype=D)
    opened = orc.feed_forward(h, {"kind": "moe", "router": {"experts": 2, "top": 1}, "shared": {"ff": 2}}, fs)
    assert torch.allclose(opened, out + h)


# ------------------------------------------------------------------------------------------------ the Zaronex design
def _zar_cfg():
    return {
        "architecture": "Zaronex", "vocab": 23, "width": 16, "norm": {"eps": 1e-5},
        "layers": [
            {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 10},
             "mixer": {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 5, "kv_rank": 6, "q_rank": 7, "scale": 0.4,
                       "rot": {"dims": 4, "base": 100.0}, "mask": {"size": 5}}},
            {"type": "parallel", "mlp": None,
             "mixer": {"left": {"heads": 6, "kv_heads": 3, "dim": 4, "vdim": 2, "scale": 0.5, "mask": {"size": 3, "pool": 2},
                                "rot": {"dims": 2, "base": 100.0}},
                       "right": {"heads": 2, "dim": 3, "vdim": 5, "tau": 3.0}}},
            {"type": "parallel_2", "mlp": {"kind": "dense", "ff": 9},
             "mixer": {"left": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 4, "scale": 0.3, "mask": {"size": 4},
                                "rot": {"dims": 4, "base": 50.0, "scaling": {"factor": 2.0}}},
                       "right": {"inner": 10, "state": 3, "dt_rank": 2, "conv": 4}}},
        ],
    }


def test_zaronex_config_and_tensor_names():
    from lit_gpt.config import LayeredConfig, model_class
    from lit_gpt.layered import LayeredGPT

    c = LayeredConfig.from_dict(_zar_cfg())
    assert model_class(c) is LayeredGPT
    d = c.design
    assert (d.block, d.norm, d.dense_ff, d.tied_head, d.norm_offset, d.mask, d.depth_average) == \
        ("prenorm", "rms", "gelu_tanh", False, 0.0, "window", True)
    a, b, e = (l.mixer for l in c.layers)
    assert (a.kind, a.q_rank, a.kv_rank, a.rot_dim, a.window, a.mask_size, a.sink_kind) == ("latent_attention", 7, 6, 4, 5, 0, "none")
    assert (b.kind, b.branch_norm, b.left_scale, b.right_scale) == ("parallel", True, 0.5, 0.5)
    assert (b.left.kind, b.left.window, b.left.pool, b.left.bias, b.left.out_gate, b.left.sink_kind, b.left.qk_norm,
            b.left.rot_layout, b.left.rot_values) == ("pooled_attention", 3, 2, True, True, "learned", "none", "half", False)
    assert (b.right.kind, b.right.tau) == ("gated_linear", 3.0)
    assert (e.left.kind, e.left.window, e.left.pool, e.left.bias, e.left.out_gate, e.left.sink_kind, e.left.qk_norm,
            e.left.rot_layout, e.left.rot_values) == \
        ("rotated_value_attention", 4, 0, False, False, "none", "joint", "interleaved", True)
    assert e.left.rot.inv_freq() == pytest.approx([0.5, 50.0 ** -0.5 / 2.0])
    assert (e.right.kind, e.right.inner, e.right.state, e.right.dt_rank, e.right.conv) == ("mamba", 10, 3, 2, 4)
    assert c.layers[1].mlp is None and c.layers[2].mlp.ff == 9
    s = LayeredGPT.tensor_shapes(c)
    assert [s[f"l{i}.dwa"] for i in range(3)] == [(2,), (3,), (4,)]
    assert s["head"] == (23, 16) and s["final.norm"] == (16,) and "l1.norm2" not in s and s["l2.norm2"] == (16,)
    assert s["l0.mix.dq"] == (7, 16) and s["l0.mix.dq.norm"] == (7,) and s["l0.mix.uq"] == (14, 7) and "l0.mix.q" not in s
    assert s["l0.mix.dkv"] == (10, 16) and s["l0.mix.uk"] == (6, 6) and s["l0.mix.uv"] == (10, 6) and "l0.mix.sink" not in s
    assert s["l0.mix.g"] == (10, 16) and s["l0.mix.o"] == (16, 10)
    assert s["l1.mix.left.q.b"] == (24,) and s["l1.mix.left.k.b"] == (12,) and s["l1.mix.left.v.b"] == (6,)
    assert s["l1.mix.left.sink"] == (6,) and s["l1.mix.left.g"] == (12, 16) and s["l1.mix.left.o"] == (16, 12)
    assert s["l1.mix.right.a2.b"] == (6,) and s["l1.mix.right.out"] == (16,) and s["l1.mix.left.out"] == (16,)
    assert s["l2.mix.left.q.norm"] == (24,) and s["l2.mix.left.k.norm"] == (12,) and "l2.mix.left.g" not in s
    assert s["l2.mix.right.in"] == (20, 16) and s["l2.mix.right.conv"] == (10, 4) and s["l2.mix.right.x"] == (8, 10)
    assert s["l2.mix.right.dt"] == (10, 2) and s["l2.mix.right.A_log"] == (10, 3) and s["l2.mix.right.o"] == (16, 10)
    w = LayeredGPT.random_weights(c)
    assert set(w) == set(s) and all(tuple(w[k].shape) == s[k] for k in s)
    # a mask's size keeps its older meaning in the designs with aligned chunks
    assert LayeredConfig._mixer_spec("attention", {"heads": 1, "dim": 2, "vdim": 2, "mask": {"size": 9}}).mask_size == 9


@pytest.mark.parametrize("edit", [
    lambda c: c["layers"][0]["mixer"].update(kv_rank=2000),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6),  # more rotary dims than the rotated part has
    lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4),  # heads no multiple of the key heads
    lambda c: c["layers"][1]["mixer"]["left"].update(mask={"pool": 4}),  # pooled blocks need a window
    lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=3),
    lambda c: c["layers"][1]["mixer"]["right"].update(tau=0.0),
    lambda c: c["layers"][2]["mixer"]["left"].update(vdim=3),  # rotated values have an even size
    lambda c: c["layers"][2]["mixer"]["right"].update(state=300),
    lambda c: c["layers"][2]["mixer"]["right"].update(conv=20),
    lambda c: c.update(loop={"start": 0, "stop": 2, "times": 2}),  # one weight vector per layer, not per pass
])
def test_zaronex_config_rejects_what_does_not_fit(edit):
    from lit_gpt.config import LayeredConfig

    c = _zar_cfg()
    edit(c)
    with pytest.raises(ValueError):
        LayeredConfig.from_dict(c)


def test_input_projection_gathers_biases():
    from lit_gpt.layered import _fuse_rows
    from lit_gpt.mixers import InputReader

    class Part(InputReader):
        def __init__(self, parts, bias):
            super().__init__()
            self.parts, self.bias = parts, bias

        def in_parts(self):
            return self.parts

        def in_bias(self):
            return self.bias

    a = Part([("q", torch.ones(3, 4)), ("k", 2 * torch.ones(8, 4))], {"k": torch.arange(8.0)})
    b = Part([("g", 3 * torch.ones(2, 4))], {})
    w, bias = _fuse_rows([a, b], 4, torch.device("cpu"), torch.float32)
    assert a.off == {"q": 0, "k": 8} and b.off == {"g": 16} and w.shape == (24, 4) and bias.shape == (24,)
    assert torch.equal(bias[8:16], torch.arange(8.0)) and bias[:8].abs().sum() == 0 and bias[16:].abs().sum() == 0
    assert w[3:8].abs().sum() == 0 and (w[16:18] == 3).all()
    assert _fuse_rows([b], 4, torch.device("cpu"), torch.float32)[1] is None
    with pytest.raises(ValueError):
        _fuse_rows([Part([("q", torch.ones(3, 4))], {"q": torch.ones(2)})], 4, torch.device("cpu"), torch.float32)


def test_zaronex_plain_implementation():
    import math

    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT
    from oracle import zaronex as orc

    cfg = _zar_cfg()
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=3)
    toks = [3, 7, 1, 0, 22, 5, 9, 9, 4, 13, 2, 8]
    full = orc.forward(cfg, w, toks)
    assert torch.allclose(orc.forward(cfg, w, toks[:7]), full[:7], atol=1e-10)  # causal
    D = torch.float64
    # a window of 2 with blocks of 2, all scores equal: position 5 sees tokens 4, 5 and blocks (0, 1), (2, 3); position 4
    # sees tokens 3, 4 and block (0, 1) - token 2 has left the window and its block is not complete before it
    q, k = torch.zeros(6, 1, 1, dtype=D), torch.zeros(6, 1, 1, dtype=D)
    v = torch.tensor([1.0, 3.0, 10.0, 20.0, 100.0, 200.0], dtype=D).view(6, 1, 1)
    out = orc.window_attention(q, k, v, 1.0, size=2, pool=2).view(-1)
    assert out.tolist() == pytest.approx([1.0, 2.0, 6.5, (10 + 20 + 2) / 3, (20 + 100 + 2) / 3, (100 + 200 + 2 + 15) / 4])
    assert orc.window_attention(q, k, v, 1.0, size=2).view(-1).tolist() == pytest.approx([1.0, 2.0, 6.5, 15.0, 60.0, 150.0])
    # a sink of score 0 beside one key of score 0 takes half
    assert orc.window_attention(q[:1], k[:1], v[:1], 1.0, 1, 0, torch.zeros(1, dtype=D)).item() == pytest.approx(0.5)
    # rotations: layouts, and turning back undoes turning
    x = torch.tensor([[[1.0, 0.0, 0.0, 5.0]]], dtype=D)
    half = orc.rotate(x, [3], [0.25], "half")[0, 0]
    assert torch.allclose(half, torch.tensor([math.cos(0.75), math.sin(0.75), 0.0, 5.0], dtype=D))
    inter = orc.rotate(x, [3], [0.25, 0.5], "interleaved")[0, 0]
    assert torch.allclose(inter, torch.tensor([math.cos(0.75), math.sin(0.75), -5 * math.sin(1.5), 5 * math.cos(1.5)], dtype=D))
    assert torch.allclose(orc.rotate(orc.rotate(x, [3], [0.25, 0.5], "half"), [3], [0.25, 0.5], "half", -1.0), x)
    # the scan: one channel, one state, A = -ln 2 and dt = 1 halve the state per token
    one = torch.ones(3, 1, dtype=D)
    y, S = orc.channel_scan(one, one, torch.full((1, 1), -math.log(2.0), dtype=D), one, one, torch.zeros(1, dtype=D))
    assert y.view(-1).tolist() == pytest.approx([1.0, 1.5, 1.75]) and S.item() == pytest.approx(1.75)
    c = orc.causal_conv(torch.tensor([[1.0], [2.0], [3.0]], dtype=D), torch.tensor([[10.0, 1.0]], dtype=D), torch.zeros(1, dtype=D))
    assert c.view(-1).tolist() == [1.0, 12.0, 23.0]
    assert orc.depth_average([one, 2 * one], torch.tensor([3.0, 0.5], dtype=D))[0].item() == 4.0


# ------------------------------------------------------------------------------------------------ the Fazolorn design
def _faz_cfg():
    moe = {"kind": "moe", "expert": {"ff": 5}, "router": {"experts": 8, "top": 3, "groups": {"count": 4, "keep": 2}, "scale": 1.5}}
    return {
        "architecture": "Fazolorn", "vocab": 23, "width": 16, "norm": {"eps": 1e-5}, "logit_scale": 0.3,
        "loop": {"start": 1, "stop": 3, "times": 3},
        "layers": [
            {"type": "attention", "mlp": {"kind": "dense", "ff": 10, "limit": 1.25},
             "mixer": {"heads": 6, "kv_heads": 3, "dim": 4, "vdim": 4, "scale": 0.5, "mask": {"size": 3},
                       "rot": {"dims": 2, "base": 100.0}}},
            {"type": "mingru", "mlp": moe, "mixer": {"width": 11}},
            {"type": "latent_attention", "mlp": moe,
             "mixer": {"heads": 2, "dim": 3, "rot_dim": 8, "vdim": 5, "kv_rank": 6, "q_rank": 7, "scale": 0.4,
                       "rot": {"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "original": 100, "fast": 4.0, "slow": 0.5}}}},
            {"type": "mingru", "mlp": None, "mixer": {"width": 9}},
        ],
    }


def test_fazolorn_config_and_tensor_names():
    import math

    from lit_gpt.config import LayeredConfig, RotarySpec, model_class
    from lit_gpt.layered import LayeredGPT
    from oracle import fazolorn as orc

    c = LayeredConfig.from_dict(_faz_cfg())
    assert model_class(c) is LayeredGPT
    d = c.design
    assert (d.block, d.norm, d.dense_ff, d.tied_head, d.norm_offset, d.mask, d.depth_average, d.moe) == \
        ("prenorm", "rms", "clamped_swish", False, 0.0, "chunk", False, "group_scores")
    assert c.layer_runs == [0, 1, 2, 1, 2, 1, 2, 3] and c.loop_inputs and c.logit_scale == 0.3
    a, g, l, _ = (s.mixer for s in c.layers)
    assert (a.kind, a.weights, a.values, a.bias, a.qk_norm, a.sink_kind, a.mask_size, a.window, a.rot_layout) == \
        ("sigmoid_attention", "sigmoid", "keys", True, "none", "none", 3, 0, "half")
    assert (g.kind, g.inner) == ("mingru", 11)
    assert (l.kind, l.q_rank, l.out_gate, l.sink_kind, l.window) == ("latent_attention", 7, False, "none", 0)
    f = c.layers[1].mlp
    assert (f.experts, f.top, f.groups, f.keep, f.route_scale, f.identity) == (8, 3, 4, 2, 1.5, 0)
    assert c.layers[0].mlp.limit == 1.25 and c.layers[3].mlp is None
    s = LayeredGPT.tensor_shapes(c)
    assert s["loop.step"] == (3, 16) and s["head"] == (23, 16) and "l3.norm2" not in s
    assert s["l0.mix.q.b"] == (24,) and s["l0.mix.k.b"] == (12,) and s["l0.mix.pb"] == (6,) and "l0.mix.v" not in s
    assert "l0.mix.v.b" not in s and s["l0.mix.o"] == (16, 24)
    assert s["l1.mix.z"] == (11, 16) and s["l1.mix.z.b"] == (11,) and s["l1.mix.x.b"] == (11,) and "l1.mix.g.b" not in s
    assert s["l1.mlp.router"] == (8, 16) and s["l1.mlp.correction"] == (8,) and s["l1.mlp.e7.gate"] == (5, 16)
    assert "l2.mix.g" not in s and s["l2.mix.uq"] == (22, 7) and s["l2.mix.dkv"] == (14, 16)
    w = LayeredGPT.random_weights(c)
    assert set(w) == set(s) and all(tuple(w[k].shape) == s[k] for k in s)
    # the other designs' latent attention keeps its output gate, and their layer types keep their meaning
    assert LayeredConfig._mixer_spec("latent_attention", dict(_faz_cfg()["layers"][2]["mixer"])).out_gate
    assert LayeredConfig._mixer_spec("attention", {"heads": 1, "dim": 2, "vdim": 2}).kind == "attention"
    # without a loop nothing joins the residual
    plain = _faz_cfg()
    del plain["loop"]
    plain = LayeredConfig.from_dict(plain)
    assert not plain.loop_inputs and "loop.step" not in LayeredGPT.tensor_shapes(plain) and plain.layer_runs == [0, 1, 2, 3]
    # YaRN: the corner indices by hand (dims 8, base 100, original 100): 4 turns at 1.19 -> lo 1, half a turn at 3.01 -> hi 4
    r = l.rot
    assert r.mult == pytest.approx(1.0 + 0.1 * math.log(4.0))
    base = [100.0 ** (-i / 4.0) for i in range(4)]
    ramp = [0.0, 0.0, 1.0 / 3.0, 2.0 / 3.0]
    assert r.inv_freq() == pytest.approx([b / 4.0 * t + b * (1.0 - t) for b, t in zip(base, ramp)])
    for dims, b0, sc in ((8, 100.0, r.scaling), (32, 5e4, {"factor": 8.0, "original": 300, "fast": 32.0, "slow": 1.0}),
                         (6, 40.0, {"factor": 0.5, "original": 9000, "fast": 1.0, "slow": 1.0})):
        want, mult = orc.rot_frequencies({"dims": dims, "base": b0, "scaling": sc})
        got = RotarySpec(dims, b0, sc)
        assert got.inv_freq() == pytest.approx(want, rel=1e-12) and got.mult == pytest.approx(mult)
    assert RotarySpec(4, 10.0, {"factor": 2.0}).mult == 1.0 and RotarySpec(4, 10.0).mult == 1.0


@pytest.mark.parametrize("edit", [
    lambda c: c["layers"][0]["mixer"].update(vdim=5),  # values that are the keys have their size
    lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3),
    lambda c: c["layers"][1]["mixer"].update(width=0),
    lambda c: c["layers"][2]["mixer"].update(kv_rank=2000),
    lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].update(original=0),
    lambda c: c["layers"][2]["mixer"]["rot"].update(base=1.0),
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=3),  # no equal groups
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=5),
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=1),  # three experts out of a group of two
    lambda c: c["layers"][1]["mlp"]["router"].update(experts=512),
    lambda c: c["loop"].update(stop=9),
    lambda c: c["loop"].update(times=0),
])
def test_fazolorn_config_rejects_what_does_not_fit(edit):
    from lit_gpt.config import LayeredConfig

    c = _faz_cfg()
    edit(c)
    with pytest.raises(ValueError):
        LayeredConfig.from_dict(c)


def test_fazolorn_plain_implementation():
    import math

    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT
    from oracle import fazolorn as orc

    cfg = _faz_cfg()
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=3)
    toks = [3, 7, 1, 0, 22, 5, 9, 9, 4, 13, 2, 8]
    full = orc.forward(cfg, w, toks)
    assert torch.allclose(orc.forward(cfg, w, toks[:7]), full[:7], atol=1e-10)  # causal
    assert torch.allclose(orc.forward(dict(cfg, logit_scale=0.6), w, toks), 2.0 * full)
    D = torch.float64
    # the recurrence: z = 0 halves the distance to the candidate; u = 1.5 gives 2, u = -ln 3 gives 1 / 4
    z = torch.zeros(3, 1, dtype=D)
    S, last = orc.mingru_scan(z, torch.tensor([[1.5], [-math.log(3.0)], [0.0]], dtype=D))
    assert S.view(-1).tolist() == pytest.approx([1.0, 0.625, 0.5625]) and last.item() == pytest.approx(0.5625)
    assert orc.mingru_scan(z[:1] - 60.0, z[:1], torch.tensor([5.0], dtype=D))[1].item() == pytest.approx(5.0)
    # chunks of 2: position 3 sees 2 and 3; every weight is sigmoid(0 + bias) on its own
    q = torch.zeros(4, 2, 1, dtype=D)
    k = torch.tensor([1.0, 10.0, 100.0, 1000.0], dtype=D).view(4, 1, 1)
    out = orc.sigmoid_attention(q, k, k, 1.0, 2, torch.tensor([0.0, math.log(3.0)], dtype=D))
    assert out[..., 0].tolist() == [pytest.approx([0.5 * s, 0.75 * s]) for s in (1.0, 11.0, 100.0, 1100.0)]
    assert [orc.visible(i, 3) for i in (0, 2, 3, 5)] == [[0], [0, 1, 2], [3], [3, 4, 5]] and orc.visible(2, 0) == [0, 1, 2]
    # routing: the pair 0.5 + 0.4 beats 0.8 + 0.0, and a negative choice score can still be chosen
    s = torch.tensor([0.8, 0.01, 0.5, 0.4], dtype=D)
    picks = orc.route(torch.log(s / (1 - s)), torch.zeros(4, dtype=D), 2, 2, 1, 2.0)
    assert picks == pytest.approx({2: 1.0, 3: 0.8})
    picks = orc.route(torch.log(s / (1 - s)), torch.tensor([-9.0, -9.0, -1.0, -2.0], dtype=D), 1, 2, 1, 1.0)
    assert picks == pytest.approx({2: 0.5})
    # the clamped unit: gate 3 -> 1, up -7 -> -1: the unit vanishes; up 7 -> 1 doubles it
    one = torch.ones(1, 1, dtype=D)
    u = orc.clamped_feed_forward(one, {"gate": 3 * one, "up": -7 * one, "down": one}, 1.0)
    assert u.item() == pytest.approx(0.0)
    u = orc.clamped_feed_forward(one, {"gate": 3 * one, "up": 7 * one, "down": one}, 1.0)
    assert u.item() == pytest.approx(2.0 / (1.0 + math.exp(-1.702)))
