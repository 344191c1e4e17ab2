"""Kakalorn on the CPU: configuration reading and refusals, tensor names, the parts a layer is made of, layers that share
rows, the rotation's frequencies, the cache's bookkeeping for kept first positions and for the convolutions' rows."""
import copy
import json
import random

import pytest
import torch

from rocml_amd.cache import Cache
from rocml_amd.cache.cache import planned_bytes
from rocml_amd.config import architecture_of
from rocml_amd.config.spec import RopeSpec, RopeStretch
from rocml_amd.engine.model import DecoderModel
from rocml_amd.errors import ConfigError
from rocml_amd.parts import BuildContext, build_position
from rocml_amd.parts.base import CompositeRequest, KVCacheRequest, LatentCacheRequest, StateRequest
from tests import kakalorn_models as km
from tests.plain import kakalorn_plain as plain


def _spec(cfg):
    arch = architecture_of(cfg)
    return arch, arch.to_spec(arch.read_config(cfg))


@pytest.mark.parametrize("name", sorted(km.CONFIGS))
def test_tensor_names_and_shapes(name):
    cfg, _ = km.CONFIGS[name]
    arch, spec = _spec(cfg)
    model = DecoderModel(spec, torch.float32, device="meta")
    names = arch.checkpoint_names(spec)
    mine = {names[k]: tuple(p.shape) for k, p in model.param_specs().items()}
    unused = set(arch.unused_tensors(spec))
    theirs = km.tensor_shapes(cfg)
    assert mine == {k: v for k, v in theirs.items() if k not in unused}
    assert unused == {f"l{i}.norm2{b}" for i, l in enumerate(cfg["layers"]) if l.get("mlp") is None for b in ("", "b")}
    assert model.kernel_families()[:3] == ("elementwise", "gemm", "attention") and "moe" not in model.kernel_families()
    assert model.graph_safe and model.prompt_graph_safe


def test_only_a_model_with_a_recurrence_needs_its_kernels():
    cfg = dict(km.CFG_D, layers=[l for l in km.CFG_D["layers"] if l["type"] == "attention"])
    _, spec = _spec(cfg)
    assert DecoderModel(spec, torch.float32, device="meta").kernel_families() == ("elementwise", "gemm", "attention")


def test_spec_carries_every_constant():
    _, spec = _spec(km.CFG_A)
    assert not spec.tie_lm_head and spec.final_norm.eps == 3e-6 and not spec.final_norm.unit_offset
    for b in spec.layers:
        assert b.arrangement == "sandwich_norm" and b.input_conv == 3
        for norm in (b.mixer_norm, b.mixer_out_norm) + ((b.ffn_norm, b.ffn_out_norm) if b.ffn is not None else ()):
            assert norm.kind == "rmsnorm" and not norm.unit_offset and norm.size == 72 and norm.eps == 3e-6
    lat, att, reader, rec = spec.layers[:4]
    m = lat.mixer
    assert (m.n_heads, m.head_dim, m.rot_dim, m.v_head_dim, m.q_rank, m.kv_rank, m.scale, m.window) == (3, 12, 8, 20, 28, 40, 0.35, None)
    assert m.gate and m.gate_per_head and m.own_rows and m.position.pairing == "neighbours"
    assert m.position.stretch == RopeStretch(4.0, 64.0, 8.0, 1.0) and (m.position.rot_dim, m.position.theta) == (8, 3000.0)
    a = att.mixer
    assert (a.n_heads, a.n_kv_heads, a.head_dim, a.scale, a.window, a.keep_first) == (6, 2, 24, 0.35, 7, 3)
    assert a.bias and a.o_bias is False and a.values_are_keys and a.sink and a.sink_learned and a.softcap is None
    assert a.qk_norm.size == 24 and a.qk_norm_span == "head" and (a.position.rot_dim, a.position.pairing) == (12, "halves")
    assert not reader.mixer.own_rows and reader.ffn is None and reader.ffn_norm is None
    assert (rec.mixer.kind, rec.mixer.n_heads, rec.mixer.head_dim, rec.mixer.v_head_dim, rec.mixer.eps) == ("hgrn2", 3, 20, 36, 3e-6)
    assert (lat.ffn.kind, lat.ffn.activation, lat.ffn.intermediate) == ("mlp", "relu2", 88)
    assert [(e.layer, e.reads_cache_of) for e in spec.schedule] == [(0, None), (1, None), (2, 0), (3, None), (4, None), (5, None), (6, None), (7, 5)]


def test_refusals():
    def broken(change):
        cfg = copy.deepcopy(km.CFG_A)
        change(cfg)
        with pytest.raises(ConfigError):
            _spec(cfg)
    broken(lambda c: c["layers"][0].update(type="retention"))
    broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=4))
    broken(lambda c: c["layers"][1]["mixer"].update(vdim=16))
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=13))
    broken(lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1))
    broken(lambda c: c["layers"][1]["mixer"]["mask"].pop("size"))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6))
    broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"))
    broken(lambda c: c["layers"][2]["mixer"].update(kv_from=1))             # no latent layer
    broken(lambda c: c["layers"][2]["mixer"].update(kv_from=5))             # a later one
    broken(lambda c: c["layers"][7]["mixer"].update(kv_from=2))             # one without rows of its own
    broken(lambda c: c["layers"][7]["mixer"].update(kv_from=0))             # rows of other sizes
    broken(lambda c: c["layers"][2]["mixer"]["rot"].update(base=100.0))     # another rotation
    broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda c: c.pop("canon"))
    broken(lambda c: c["canon"].update(taps=0))
    cfg = copy.deepcopy(km.CFG_A)
    cfg["canon"]["taps"] = 17                                                # more than the kernels slide over
    _, spec = _spec(cfg)
    with pytest.raises(ConfigError):
        DecoderModel(spec, torch.float32, device="meta")
    # a configuration survives the round trip through its typed form
    arch = architecture_of(km.CFG_A)
    assert arch.read_config(arch.read_config(km.CFG_A).to_dict()) == arch.read_config(km.CFG_A)


def test_an_input_convolution_needs_a_norm_before_the_mixer():
    import dataclasses
    from rocml_amd.parts import build_block
    _, spec = _spec(km.CFG_A)
    ctx = BuildContext(dtype=torch.float32, device=torch.device("meta"))
    block = spec.layers[3]
    assert build_block(dataclasses.replace(block, arrangement="pre_norm"), ctx).input_conv is not None
    for arrangement in ("post_norm", "sublayer_norm"):
        with pytest.raises(ConfigError):
            build_block(dataclasses.replace(block, arrangement=arrangement), ctx)


@pytest.mark.parametrize("dims,base,scaling", [(8, 3000.0, (4.0, 64, 8.0, 1.0)), (32, 1e5, (8.0, 128, 16.0, 2.0)), (64, 1e6, (2.5, 4096, 32.0, 1.0)),
                                               (2, 50.0, (1.0, 1000, 1.0, 1.0)), (12, 800.0, None), (16, 100.0, (3.0, 7, 50.0, 40.0))])
def test_frequencies(dims, base, scaling):
    rot = {"dims": dims, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    want, factor = plain.frequencies(rot)
    spec = RopeSpec(head_dim=dims, rot_dim=dims, theta=base, pairing="neighbours",
                    stretch=None if scaling is None else RopeStretch(*[float(v) for v in scaling]))
    part = build_position(spec, BuildContext(dtype=torch.float32, device=torch.device("cpu")))
    assert part.pairing == "neighbours" and part.magnitude == pytest.approx(factor, rel=1e-15)
    assert torch.allclose(part.inv_freq, torch.tensor(want, dtype=torch.float64), rtol=1e-15)


def test_cache_lines_of_layers_that_share_rows():
    _, spec = _spec(km.CFG_A)
    model = DecoderModel(spec, torch.float32, device="meta")
    requests = model.cache_requests()
    conv = StateRequest((2, 72), dtype=torch.float32)
    assert requests[0] == CompositeRequest((LatentCacheRequest(48, None), conv))
    assert requests[1] == CompositeRequest((KVCacheRequest(2, 24, 7, keep_first=3), conv))
    assert requests[2] == CompositeRequest((None, conv)), "a layer that reads another's rows keeps its convolution's rows itself"
    assert requests[3] == CompositeRequest((StateRequest((3, 36, 20)), conv))
    cache = Cache(requests, max_tokens=256, dtype=torch.float32, device="cpu", max_seqs=3)
    lines = [cache.line(i, 1) for i in range(8)]
    assert len({id(g) for g, _ in lines}) == 1 and sorted(line for _, line in lines) == list(range(8))
    assert sum(1 for g in cache.groups if type(g).__name__ == "LatentGroup") == 2

    class Step:
        block_tables = {g.name: None for g in cache.kv_groups}
        seq_slots = None
    own, reader = model.entry_view(0, cache, Step), model.entry_view(2, cache, Step)
    assert reader.parts[0].k.data_ptr() == own.parts[0].k.data_ptr(), "the rows are the first layer's"
    assert reader.parts[1].state.data_ptr() != own.parts[1].state.data_ptr()
    assert reader.parts[1].state.data_ptr() == cache.line(2, 1)[0].state[cache.line(2, 1)[1]].data_ptr()
    # a convolution of one tap keeps nothing
    _, spec_c = _spec(dict(km.CFG_D, canon={"taps": 1}))
    model_c = DecoderModel(spec_c, torch.float32, device="meta")
    assert model_c.cache_requests()[2] is None
    # states and kept rows start at zero when a slot is used again
    a = cache.new_sequence()
    for g, line in lines:
        g.state[line, a].fill_(2.0)
    cache.free_sequence(a)
    assert cache.new_sequence() == a and all(float(g.state[line, a].abs().max()) == 0.0 for g, line in lines)


def test_pages_of_kept_first_positions_stay():
    page = 64
    for window, keep in ((10, 1), (65, 64), (64, 65), (130, 200), (1, 0), (5, 20)):
        req = KVCacheRequest(1, 4, window, keep_first=keep)
        cache = Cache([req], max_tokens=64 * page, dtype=torch.float32, device="cpu", max_seqs=2)
        g = cache.kv_groups[0]
        s = cache.new_sequence()
        for n in list(range(1, 700, 37)) + [700, 701, 702]:
            cache.reserve([s], [n])
            cache.commit([s], [n])
            held = {i for i, p in enumerate(g.page_table(s)) if p >= 0}
            # what a query at position n (the next one) or later can see
            seen = {j // page for j in range(n) if n - j < window or j < keep}
            assert seen <= held, f"window {window}, kept {keep}, length {n}"
            allowed = seen | {i for i in held if i < -(-keep // page)} | {n // page, (n - 1) // page}
            assert held <= allowed | {max(0, n - window + 1) // page}, f"window {window}, kept {keep}, length {n}: pages nobody sees are held"
            cache.check()
        cache.free_sequence(s)
        assert g.n_free_pages == g.n_pages


def test_a_group_with_kept_positions_is_sized_for_them_and_plans_hold():
    """The bounded pool is large enough for any sequence, and what ``fits`` predicts is what happens."""
    page, rng = 64, random.Random(5)
    for window, keep in ((70, 3), (20, 130), (128, 64)):
        req = KVCacheRequest(1, 2, window, keep_first=keep)
        cache = Cache([req], max_tokens=4096, dtype=torch.float32, device="cpu", max_seqs=2, step_tokens=96)
        g = cache.kv_groups[0]
        assert g.n_pages == 2 * (-(-window // page) + 2 + -(-keep // page)) + 2
        assert planned_bytes([req], 4096, torch.float32, max_seqs=2, step_tokens=96) == g.k.numel() * 4 * 2
        for _ in range(20):
            a, b = cache.new_sequence(), cache.new_sequence()
            la = lb = 0
            for _ in range(12):
                pieces = []
                ta, tb = la, lb
                for _ in range(rng.randint(1, 3)):
                    na, nb = rng.randint(1, 60), rng.randint(1, 36)
                    ta, tb = ta + na, tb + nb
                    pieces.append([(a, ta), (b, tb)])
                assert cache.fits(pieces, final=[(a, ta + 300), (b, tb + 300)]) is None
                for piece in pieces:
                    cache.reserve([s for s, _ in piece], [n for _, n in piece])
                    cache.commit([s for s, _ in piece], [n for _, n in piece])
                la, lb = ta, tb
            cache.check()
            cache.free_sequence(a)
            cache.free_sequence(b)


def test_plain_mechanisms_on_cases_made_by_hand():
    """The oracle's own mask, sink and recurrence where the answer can be written down."""
    seen = plain.window_seen(6, 2, 1)
    assert seen.int().tolist() == [[1, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0], [1, 0, 1, 1, 0, 0], [1, 0, 0, 1, 1, 0],
                                   [1, 0, 0, 0, 1, 1]]
    w = plain.softmax_seen(torch.zeros(1, 3, dtype=torch.float64), torch.tensor([[True, True, False]]), torch.tensor(0.0, dtype=torch.float64))
    assert torch.allclose(w, torch.tensor([[1 / 3, 1 / 3, 0.0]], dtype=torch.float64))
    q = torch.ones(3, 1, 1, dtype=torch.float64)
    f = torch.tensor([0.5, 1.0, 0.0], dtype=torch.float64).view(3, 1, 1)
    v = torch.tensor([2.0, 7.0, 3.0], dtype=torch.float64).view(3, 1, 1)
    assert plain.gated_recurrence(q, f, v).flatten().tolist() == [1.0, 1.0, 3.0]
    h = torch.tensor([[1.0], [10.0], [100.0]])
    assert plain.added_conv(h, torch.tensor([[2.0, 3.0]])).flatten().tolist() == [4.0, 42.0, 420.0]


def test_random_model_folder_has_the_checkpoint_names(tmp_path):
    from safetensors import safe_open
    from rocml_amd.config.catalog import resolve
    from rocml_amd.weights import write_model_dir
    cfg = resolve("kakalorn-tiny").entry.config
    path = write_model_dir(str(tmp_path / "m"), cfg, 5, dtype=torch.bfloat16, norm_jitter=True)
    arch, spec = _spec(cfg)
    model = DecoderModel(spec, torch.float32, device="meta")
    names = arch.checkpoint_names(spec)
    with safe_open(f"{path}/model.safetensors", "pt") as f:
        found = {k: tuple(f.get_slice(k).get_shape()) for k in f.keys()}
    assert found == {names[k]: tuple(p.shape) for k, p in model.param_specs().items()}
    assert architecture_of(json.load(open(f"{path}/config.json"))).name == "Kakalorn"
