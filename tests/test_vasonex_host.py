"""Host side of the Vasonex integration on the CPU: registry and configuration, checkpoint names and merged layouts, layers
that share weights, the cache specifications the engine sizes its pools from, rotation frequencies, and the oracle's own
consistency (closed forms that do not go through its loops)."""

import copy
import json
import math

import pytest
import torch

from oracle import vasonex as O
from vasonex_cases import aligned_config, attention, config, dense, mixed_config, odd_config, plain_config, random_checkpoint

F64 = torch.float64


def _model(cfg, dtype=torch.bfloat16):
    from byox_vllm_amd.models.vasonex import VasonexForCausalLM, vasonex_config
    default = torch.get_default_dtype()
    torch.set_default_dtype(dtype)
    try:
        return VasonexForCausalLM(vasonex_config(cfg, dtype=dtype))
    finally:
        torch.set_default_dtype(default)


def test_registry_and_configuration():
    from byox_vllm_amd.models import registry
    assert registry.model_class({"architecture": "Vasonex"}).__name__ == "VasonexForCausalLM"
    cfg = mixed_config()
    hf = registry.read_config(cfg, None)
    assert (hf.vocab_size, hf.hidden_size, hf.num_hidden_layers, hf.norm_eps) == (150, 96, 6, 1e-4)
    assert not hf.tie_word_embeddings
    hf.layers[1]["mixer"]["heads"] = 99                     # the given dict is left as it was
    assert cfg["layers"][1]["mixer"]["heads"] == 3


def test_config_from_a_model_folder(tmp_path):
    from safetensors.torch import save_file

    from byox_vllm_amd.config import Config
    cfg = odd_config()
    with open(tmp_path / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in random_checkpoint(cfg, 1).items()}, str(tmp_path / "model.safetensors"))
    c = Config(str(tmp_path), dtype="float32", kvcache_block_size=32, max_num_seqs=3)
    assert c.portioned and c.num_state_slots == 3 and c.hf_config.dtype == torch.float32
    assert c.hf_config.layers[3]["weights_of"] == 1


def test_layers_that_share_weights():
    from byox_vllm_amd.models.vasonex import vasonex_config, weight_owner
    cfg = mixed_config()
    assert [weight_owner(cfg["layers"], i) for i in range(6)] == [0, 1, 0, 3, 1, 0] == [O.owner(cfg, i) for i in range(6)]
    model = _model(cfg)
    assert len(model.layers) == 3 and model.order == [(0, 0), (1, 0), (0, 1), (2, 0), (1, 1), (0, 2)]
    caches = model.page_layers()
    assert len({id(c) for c in caches}) == 6                 # every layer keeps keys and values of its own
    assert [c.page_spec()["width"] for c in caches] == [2 * (16 + 24), 3 * (24 + 8), 80, 32 + 16, 96, 80]
    assert model.state_layers() == []
    assert model.checkpoint_target("l2.norm1") is None and model.checkpoint_target("l3.norm1") == ("layers.2.norm1.pre", None)
    other = copy.deepcopy(cfg)
    other["layers"][4]["mixer"]["scale"] = 0.5
    with pytest.raises(AssertionError):
        vasonex_config(other)
    circle = copy.deepcopy(cfg)
    circle["layers"][0]["weights_of"] = 2
    with pytest.raises(AssertionError):
        vasonex_config(circle)
    # the owner may come later than the layer that uses its weights
    late = config(40, 32, [(attention(2, 1, 8, 8, 0.3), dense(24)), 0])
    late["layers"][0], late["layers"][1] = late["layers"][1], late["layers"][0]
    late["layers"][0]["weights_of"] = 1
    model = _model(late)
    assert model.order == [(0, 0), (0, 1)] and model.checkpoint_target("l1.mix.q") == ("layers.0.mix.inp.weight", "q")


def test_every_checkpoint_tensor_has_a_parameter_and_every_parameter_a_tensor():
    from byox_vllm_amd.utils.loader import load_state_dict_packed
    for make in (mixed_config, odd_config, aligned_config, plain_config):
        cfg = make()
        W = random_checkpoint(cfg, 3)
        model = _model(cfg)
        for p in model.parameters():
            p.data.fill_(float("nan"))
        load_state_dict_packed(model, W, model.cfg)
        unused = [n for n, p in model.named_parameters() if torch.isnan(p.float()).any()]
        assert not unused, unused
        for name in ("l0.mix.nothing", "l99.norm1", "l0.mlp.e99.up", "l0.norm3", "tail"):
            assert model.checkpoint_target(name) is None


def test_merged_layouts():
    from byox_vllm_amd.utils.loader import load_state_dict_packed
    cfg = mixed_config()
    W = random_checkpoint(cfg, 4)
    model = _model(cfg)
    load_state_dict_packed(model, W, model.cfg)
    att = model.layers[0].mix                                # 6 query heads on 2 key heads of 16, values of 24
    assert att.inp.weight.shape == (6 * 16 + 2 * 16 + 2 * 24 + 6, 96)
    assert torch.equal(att.inp.weight[96:128], W["l0.mix.k"]) and torch.equal(att.inp.weight[-6:], W["l0.mix.g"])
    assert torch.equal(att.inp.weight[128:176], W["l0.mix.v"]) and torch.equal(att.o.weight, W["l0.mix.o"])
    mix = model.layers[0].mlp
    assert torch.equal(mix.up[3], W["l0.mlp.e3.up"]) and torch.equal(mix.down[4], W["l0.mlp.e4.down"]) and mix.up.shape[0] == 5
    assert torch.equal(mix.router.weight[:5], W["l0.mlp.router"]) and torch.equal(mix.router.weight[5:], W["l0.mlp.shared.sg"])
    assert torch.equal(mix.shared_up.weight, W["l0.mlp.shared.up"])
    ff = model.layers[1].mlp
    assert torch.equal(ff.gate_up.weight[56:], W["l1.mlp.up"]) and torch.equal(ff.gate_up.bias[:56], W["l1.mlp.gate.b"])
    assert torch.equal(ff.gate_up.bias[56:], W["l1.mlp.up.b"]) and torch.equal(ff.down.bias, W["l1.mlp.down.b"])
    assert torch.equal(model.layers[1].norm2.post, W["l1.norm2b"]) and torch.equal(model.layers[1].norm1.post, W["l1.norm1b"])
    assert model.layers[2].mlp is None and model.checkpoint_target("l3.norm2b") == (None, None)
    assert torch.equal(model.head.weight, W["head"]) and torch.equal(model.final_norm.pre, W["final.norm"])
    # a shared expert of the experts' size is stored behind them
    aligned = _model(aligned_config())
    W = random_checkpoint(aligned_config(), 5)
    load_state_dict_packed(aligned, W, aligned.cfg)
    mix = aligned.layers[0].mlp
    assert mix.up.shape == (9, 64, 128) and torch.equal(mix.up[8], W["l0.mlp.shared.up"])
    assert torch.equal(mix.down[8], W["l0.mlp.shared.down"])


def test_rotation_frequencies_match_the_oracle():
    from byox_vllm_amd.layers.rotary_embedding import scaled_inv_freq

    def scaling(*v):
        return dict(zip(("factor", "low", "high", "original"), v))
    for rot in ({"base": 10000.0, "dims": 16}, {"base": 500.0, "dims": 8, "scaling": scaling(8.0, 1.0, 4.0, 64)},
                {"base": 1e6, "dims": 64, "scaling": scaling(4.0, 1.0, 4.0, 4096)},
                {"base": 50.0, "dims": 4, "scaling": scaling(2.0, 0.5, 8.0, 16)},
                {"base": 200.0, "dims": 12, "scaling": scaling(2.0, 2.0, 2.0, 100)}):      # no band between the two
        f, mag = scaled_inv_freq(rot["dims"], rot["base"], rot.get("scaling"))
        assert torch.allclose(f.double(), O.frequencies(rot), rtol=1e-6, atol=0) and mag == 1.0
    # by hand: wavelengths 2 pi, 2 pi 10, 2 pi 100 against original / high = 25 and original / low = 100
    f = O.frequencies({"base": 1000.0, "dims": 6, "scaling": scaling(4.0, 1.0, 4.0, 100)})
    s = (100 / (20 * math.pi) - 1.0) / 3.0
    want = [1.0, (1 - s) * 0.1 / 4 + s * 0.1, 0.01 / 4]
    assert torch.allclose(f, torch.tensor(want, dtype=F64), rtol=1e-12)


# ------------------------------------------------------------------------------------------------ the oracle itself
def test_oracle_is_causal():
    cfg = mixed_config()
    W = random_checkpoint(cfg, 5)
    torch.manual_seed(0)
    a = torch.randint(0, cfg["vocab"], (30,)).tolist()
    b = list(a)
    b[25] = (b[25] + 1) % cfg["vocab"]
    la, lb = O.forward(a, W, cfg), O.forward(b, W, cfg)
    # (a batched product may round a row differently as other rows' experts change)
    assert torch.allclose(la[:25], lb[:25], rtol=1e-12, atol=1e-12) and not torch.allclose(la[25:], lb[25:])


def test_window_with_kept_first_tokens():
    m = O.visible(10, {"size": 3, "keep_first": 2})
    assert m[9].nonzero()[:, 0].tolist() == [0, 1, 7, 8, 9] and m[3].nonzero()[:, 0].tolist() == [0, 1, 2, 3]
    assert m[1].nonzero()[:, 0].tolist() == [0, 1]
    assert torch.equal(O.visible(10, {"size": 3}), O.visible(10, {"size": 3, "keep_first": 0}))
    assert torch.equal(O.visible(10, None), O.visible(10, {"size": 10, "keep_first": 4}))


def test_rotation_turns_neighbours_and_depends_on_distance_only():
    g = torch.Generator().manual_seed(0)
    x, y = torch.randn(1, 1, 12, generator=g, dtype=F64), torch.randn(1, 1, 12, generator=g, dtype=F64)
    f = O.frequencies({"base": 100.0, "dims": 8})
    dots = []
    for p in (0, 7, 1000):
        a, b = O.rotate_pairs(x, torch.tensor([p + 5]), f), O.rotate_pairs(y, torch.tensor([p]), f)
        assert torch.allclose(a[..., 2:4].norm(), x[..., 2:4].norm()) and torch.equal(a[..., 8:], x[..., 8:])
        dots.append(float((a * b).sum()))
    assert max(dots) - min(dots) < 1e-9
    a = O.rotate_pairs(torch.tensor([[[1.0, 0.0, 0.0, 1.0]]], dtype=F64), torch.tensor([2]), torch.tensor([0.5, 0.25], dtype=F64))
    assert torch.allclose(a[0, 0], torch.tensor([math.cos(1), math.sin(1), -math.sin(0.5), math.cos(0.5)], dtype=F64))


def test_scores_are_not_renormalised_and_weigh_the_input():
    """With a linear stand-in for the activation both places of the weight agree; with the real one they do not."""
    z = torch.tensor([[2.0, -1.0, 0.0]], dtype=F64)
    idx, w = O.route(z, 2)
    assert idx.tolist() == [[0, 2]] and torch.allclose(w, torch.sigmoid(torch.tensor([[2.0, 0.0]], dtype=F64)))
    spec = {"router": {"experts": 1, "top": 1}, "expert": {"ff": 1}}
    one = torch.ones(1, 1, dtype=F64)
    W = {"router": 0.0 * one, "e0.up": one, "e0.down": one}
    h = torch.tensor([[1.5]], dtype=F64)
    assert torch.allclose(O.moe(h, W, "", spec), O.gelu_erf(0.5 * h))            # sigmoid(0) = 1/2 inside the unit
    assert abs(float(O.gelu_erf(torch.tensor(1.0, dtype=F64))) - 0.8413447460685429) < 1e-15
