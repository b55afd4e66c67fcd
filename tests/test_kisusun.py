"""The Kisusun design against the plain implementation in ``tests/plain/kisusun_plain.py``: every mechanism alone, then
whole models of several small shapes replayed whole, token by token, in portions and in mixed batches (32-bit and bfloat16
through graphs), window edges and far tokens that stand out, and greedy generation through the engine's own entry point."""
import copy
import math

import numpy as np
import pytest
import torch
import torch.nn.functional as F

from tests import traces
from tests.plain import kisusun_plain as P
from tests.test_gidurax import BF16_NOISE, F32_ATOL, _Ctx, _replay, requests_for, write_model

gpu = pytest.mark.gpu


# ================================================================================================ configurations
def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, limit, experts, top, scale, groups=None, shared=None):
    d = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top, "scale": scale}}
    if groups is not None:
        d["router"]["groups"] = dict(zip(("count", "keep"), groups))
    if shared is not None:
        d["shared"] = dict(zip(("ff", "limit"), shared))
    return d


def attention(heads, kv_heads, dim, vdim, scale, mlp, rot=None, window=None, softcap=None, v_mix=False):
    """``rot``: (base, dims, factor or None)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix}
    if rot is not None:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
        if rot[2] is not None:
            m["rot"]["scaling"] = {"factor": rot[2]}
    if window is not None:
        m["mask"] = {"size": window}
    if softcap is not None:
        m["softcap"] = softcap
    return {"type": "attention", "mixer": m, "mlp": mlp}


def config(vocab, width, eps, embedding_scale, logit_scale, layers):
    return {"architecture": "Kisusun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embedding_scale},
            "logit_scale": logit_scale, "layers": layers}


# Shapes that differ in every size and in the order of their layers: values narrower and wider than keys and of their size;
# windows of one token, inside a page, across pages and none; caps from tight to none; rotation of some, all and no entries;
# blending that starts late, skips layers, and of a different number of heads than the layer before; a layer without a
# feed-forward; experts with and without groups, groups of one, two and more experts, with and without a shared one; pages of
# 4 to 16.
SHAPES = {
    "P": config(211, 96, 1e-5, 1.5, 0.3, [
        attention(6, 3, 20, 12, 0.3, moe(40, 1.2, 6, 2, 1.7, (3, 2), (24, 0.8)), (10000.0, 8, 3.0), 17, 4.0, True),
        attention(4, 1, 16, 36, 0.35, dense(72), (500.0, 16, None), 40, None, True),
        attention(5, 5, 12, 10, 0.4, None, None, None, 2.0, False)]),
    "Q": config(130, 72, 3e-6, 1.0, 0.4, [
        attention(2, 1, 24, 24, 0.25, dense(40), (100.0, 4, 2.0), 1, 10.0, False),
        attention(3, 1, 10, 14, 0.5, moe(28, 2.0, 5, 3, 0.6), (3000.0, 10, 8.0), 6, 7.0, True),
        attention(7, 7, 8, 2, 0.6, moe(20, 0.7, 4, 2, 1.0, (4, 2), (36, 1.1)), (50.0, 2, 1.5), None, 3.0, True)]),
    "R": config(97, 100, 1e-6, 2.5, 0.2, [
        attention(8, 2, 18, 26, 0.3, moe(36, 0.7, 8, 3, 2.0, (2, 1), (52, 3.0)), (3000.0, 14, 5.0), 9, 80.0, True),
        attention(3, 3, 6, 6, 0.5, dense(64), None, 33, 5.0, False),
        attention(4, 4, 14, 13, 0.35, moe(24, 1.5, 9, 4, 0.8, (3, 2), None), (20.0, 6, 2.0), None, 6.0, True)]),
}
# sizes that the matrix cores take in bfloat16: key sizes 32, 64 and 128, values of that size and narrower, widths of whole pieces
SHAPES["S"] = config(257, 160, 1e-5, 2.0, 0.25, [
    attention(10, 2, 32, 32, 0.25, dense(192), (10000.0, 16, 4.0), 48, 8.0, True),
    attention(6, 2, 64, 32, 0.18, moe(64, 1.5, 12, 4, 1.2, (4, 2), (96, 1.1)), (50000.0, 64, 2.0), 37, 30.0, True),
    attention(4, 1, 128, 64, 0.13, moe(64, 1.1, 4, 1, 0.9, (1, 1), None), (1000.0, 32, 1.0), None, 12.0, True)])
SHAPES["T"] = config(301, 128, 1e-5, 1.2, 0.3, [
    attention(9, 3, 64, 64, 0.2, moe(32, 0.9, 16, 5, 1.0, (4, 3), (64, 1.4)), (1000000.0, 48, 16.0), 64, 100.0, False),
    attention(3, 1, 128, 128, 0.12, dense(128), (5000.0, 128, 3.0), 80, None, True),
    attention(8, 4, 32, 16, 0.3, moe(48, 2.5, 6, 2, 1.4, (3, 1), (32, 0.6)), (700.0, 8, 2.5), 31, 20.0, False)])
PAGES = {"P": 16, "Q": 8, "R": 4, "S": 16, "T": 16}
SEEDS = {"P": 10, "Q": 7, "R": 9, "S": 2, "T": 1}      # (choices of experts that do not rest on rounding)


def tensor_shapes(cfg):
    """Names and shapes, stated here from the design (not asked of the product)."""
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "final.norm": (W,)}
    blending = [i for i, layer in enumerate(cfg["layers"]) if layer["mixer"]["v_mix"]]
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        a = p + "mix."
        out.update({p + "norm1": (W,), a + "q": (H * D, W), a + "k": (G * D, W), a + "v": (G * E, W), a + "q.norm": (H * D,),
                    a + "k.norm": (G * D,), a + "g": (H * E, W), a + "o": (W, H * E)})
        if i in blending[1:]:
            out[a + "vmix"] = ()
        if mlp is None:
            continue
        f = p + "mlp."
        out[p + "norm2"] = (W,)
        sizes = [(f, mlp["ff"])] if mlp["kind"] == "dense" else \
            [(f"{f}e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        if mlp["kind"] == "moe":
            out[f + "router"] = (mlp["router"]["experts"], W)
            if mlp.get("shared"):
                sizes.append((f + "shared.", mlp["shared"]["ff"]))
        for q, ff in sizes:
            out.update({q + "gate": (ff, W), q + "up": (ff, W), q + "down": (W, ff)})
    return out


def random_weights(cfg, seed, dtype=torch.bfloat16):
    """Weights large enough that every mechanism moves the logits: scores of order one and more, gates half open, clamps that
    are reached, blends far from 0 and 1.  Every token has a kind that its embedding leans towards and that the routers read,
    so that a choice of experts hardly ever rests on rounding."""
    g = torch.Generator().manual_seed(seed)
    W, V, scale = cfg["width"], cfg["vocab"], cfg["embedding"]["scale"]
    kinds = 6
    dirs = torch.linalg.qr(torch.randn(W, kinds, generator=g))[0].T              # [kinds, W], orthonormal
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g)
        if leaf in ("norm1", "norm2", "norm"):
            t = 1.0 + 0.2 * r
        elif name == "embed":
            t = 0.6 * r + math.sqrt(W) * dirs[torch.arange(V) % kinds]
        elif leaf == "vmix":
            t = 0.45 + 0.2 * r
        elif leaf == "router":
            n = shape[0]
            rank = torch.stack([torch.randperm(n, generator=g) for _ in range(kinds)], dim=1).float()   # [n, kinds]
            t = (rank / max(1, n - 1) * 4.0 - 2.0) @ dirs / (math.sqrt(W) * scale) + 0.02 * r / (math.sqrt(W) * scale)
        else:
            t = r * (1.3 / math.sqrt(shape[-1]))
        w[name] = t
    return {name: t.to(dtype).contiguous() for name, t in w.items()}


# ================================================================================================ the oracle's own pins
def test_plain_pieces_against_library_routines():
    torch.manual_seed(0)
    x = torch.randn(9, 6, dtype=torch.float64)
    w = torch.randn(6, dtype=torch.float64)
    assert torch.allclose(P.rms_norm(x, w, 1e-5), F.rms_norm(x, (6,), w, 1e-5), atol=1e-12)
    assert torch.allclose(P.silu(x), F.silu(x), atol=1e-12)
    # inside its limits the clamped form is a sigmoid-weighted product, outside the limit's own value
    g, u = torch.tensor([0.5, 9.0, -9.0]).double(), torch.tensor([0.25, 9.0, -9.0]).double()
    got = P.clamped_glu(g, u, 1.5)
    want = [0.5 * torch.sigmoid(torch.tensor(0.851, dtype=torch.float64)) * 1.25,
            1.5 * torch.sigmoid(torch.tensor(1.702 * 1.5, dtype=torch.float64)) * 2.5,
            -9.0 * torch.sigmoid(torch.tensor(-9.0 * 1.702, dtype=torch.float64)) * -0.5]
    assert all(abs(float(a) - float(b)) < 1e-12 for a, b in zip(got, want))
    # the rotation is a complex product with exp(i p f); the rest stays; the factor slows every pair alike
    f = P.frequencies(4, 100.0, 2.5)
    assert torch.allclose(f, torch.tensor([0.4, 0.04], dtype=torch.float64))
    v = torch.randn(5, 2, 7, dtype=torch.float64)
    pos = torch.tensor([0, 1, 2, 50, 1000])
    turn = torch.polar(torch.ones(5, 2, dtype=torch.float64), pos[:, None] * f[None, :])[:, None, :]
    got = P.rotate(v, pos, f)
    z = torch.complex(v[..., :2], v[..., 2:4]) * turn
    assert torch.allclose(got[..., :2], z.real, atol=1e-12) and torch.allclose(got[..., 2:4], z.imag, atol=1e-12)
    assert torch.equal(got[..., 4:], v[..., 4:])
    # one more score of zero in the softmax, dropped afterwards; scores so large that only the shift keeps them finite
    s = torch.tensor([[1.0, -2.0, 3.0], [800.0, 799.0, 0.0], [-900.0, -901.0, -950.0]], dtype=torch.float64)
    want = torch.softmax(torch.cat([s, torch.zeros(3, 1, dtype=torch.float64)], 1), 1)[:, :3]
    assert torch.allclose(P.one_plus_softmax(s), want, atol=1e-12)
    assert float(P.cap_scores(torch.tensor(1e6), 3.0)) == 3.0 and abs(float(P.cap_scores(torch.tensor(0.01), 3.0)) - 0.01) < 1e-6
    q, k, vv = torch.randn(7, 4, 5, dtype=torch.float64), torch.randn(7, 2, 5, dtype=torch.float64), torch.randn(7, 2, 3, dtype=torch.float64)
    got = P.windowed_attention(q, k, vv, 0.3, None, 3)
    i, j = torch.arange(7)[:, None], torch.arange(7)[None, :]
    seen = (j <= i) & (i - j < 3)
    for h in range(4):
        sc = (q[:, h] @ k[:, h // 2].T * 0.3).masked_fill(~seen, -math.inf)
        p = torch.exp(sc) / (1 + torch.exp(sc).sum(1, keepdim=True))
        assert torch.allclose(got[:, h], p @ vv[:, h // 2], atol=1e-12)


def test_plain_router_counts_a_group_as_its_two_best():
    logit = lambda p: torch.log(torch.tensor(p, dtype=torch.float64) / (1 - torch.tensor(p, dtype=torch.float64)))
    # the single best expert (0.9) sits in the group whose two best add up to less
    z = logit([[0.9, 0.1, 0.2, 0.6, 0.55, 0.05]])
    ids, w = P.route(z, 2, 1.5, (2, 1))
    assert ids == [[3, 4]] and abs(w[0][0] - 0.9) < 1e-12 and abs(w[0][1] - 0.825) < 1e-12
    ids, w = P.route(z, 2, 1.0, None)
    assert ids == [[0, 3]] and abs(sum(w[0]) - 1.5) < 1e-12
    ids, _ = P.route(z, 3, 1.0, (2, 2))
    assert ids == [[0, 3, 4]]
    ids, _ = P.route(z, 2, 1.0, (6, 2))         # groups of one expert count as that expert
    assert ids == [[0, 3]]


@pytest.mark.parametrize("dims,base,factor", [(32, 10000.0, None), (64, 500000.0, 8.0), (6, 50.0, 3.0), (2, 10.0, 1.0), (12, 2000.0, 0.5)])
def test_frequencies_of_the_product(dims, base, factor):
    from llm_infrence_engine_amd.parts.positions import scaled_frequencies

    f = scaled_frequencies(dims, base, {"factor": factor} if factor is not None else None)
    assert torch.allclose(f, P.frequencies(dims, base, factor or 1.0), rtol=1e-12, atol=0)


def test_config_reads_every_size_and_refuses_what_it_does_not_know():
    from llm_infrence_engine_amd.cache import CacheLayout
    from llm_infrence_engine_amd.config import ConfigError, config_from_dict, preset
    from llm_infrence_engine_amd.parts.model import Model

    for name, cfg in SHAPES.items():
        c = config_from_dict(copy.deepcopy(cfg))
        assert type(c).__name__ == "KisusunConfig" and c.to_dict() == cfg
        model = Model(c.to_spec())
        assert {s.name: tuple(s.shape) for s in model.tensor_specs()} == tensor_shapes(cfg)
        assert model.graph_safe() is True and hash(c.to_spec()) == hash(config_from_dict(copy.deepcopy(cfg)).to_spec())
        for layer, (kv, state, _) in zip(cfg["layers"], model.run_needs()):
            m = layer["mixer"]
            assert state is None and kv.window == (m["mask"]["size"] if "mask" in m else None)
            assert [(t.name, t.heads, t.width) for t in kv.tensors] == [("k", m["kv_heads"], m["dim"]), ("v", m["kv_heads"], m["vdim"])]
        # equal needs share a group
        needs = {(x["mixer"]["kv_heads"], x["mixer"]["dim"], x["mixer"]["vdim"], str(x["mixer"].get("mask"))) for x in cfg["layers"]}
        assert len(CacheLayout(model.run_needs()).group_keys) == len(needs)
    for change in (lambda c: c["layers"][0].__setitem__("type", "something_else"),
                   lambda c: c["layers"][0]["mixer"].pop("vdim"),
                   lambda c: c["layers"][0]["mixer"].pop("scale"),
                   lambda c: c["layers"][0]["mixer"].__setitem__("scale", 0),
                   lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 4),
                   lambda c: c["layers"][0]["mixer"].__setitem__("softcap", -1.0),
                   lambda c: c["layers"][0]["mixer"].__setitem__("mask", {"size": 0}),
                   lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 7),
                   lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 22),
                   lambda c: c["layers"][0]["mixer"]["rot"].pop("base"),
                   lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("factor"),
                   lambda c: c["layers"][2]["mixer"].__setitem__("v_mix", True),            # 50 values a token against 36
                   lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"),
                   lambda c: c["layers"][0]["mlp"]["router"].pop("scale"),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 7),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("groups", {"count": 4, "keep": 1}),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("groups", {"count": 6, "keep": 1}),
                   lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"),
                   lambda c: c["layers"][1]["mlp"].pop("ff"),
                   lambda c: c["layers"][1]["mlp"].__setitem__("kind", "sparse"),
                   lambda c: c["embedding"].pop("scale"),
                   lambda c: c.pop("logit_scale"),
                   lambda c: c.__setitem__("width", 0)):
        bad = copy.deepcopy(SHAPES["P"])
        change(bad)
        with pytest.raises(ConfigError):
            config_from_dict(bad)
    for size in ("0.5b", "7b"):
        c = config_from_dict(preset(f"kisusun-{size}"))
        assert len(Model(c.to_spec()).layers) == len(c.layers)


def test_tensors_a_layer_has_no_use_for_may_be_there():
    from llm_infrence_engine_amd.config import config_from_dict

    spec = lambda n: config_from_dict(copy.deepcopy(SHAPES[n])).to_spec()
    assert set(spec("P").ignorable) == {"l0.mix.vmix", "l2.mix.vmix", "l2.norm2"}
    assert set(spec("Q").ignorable) == {"l0.mix.vmix", "l1.mix.vmix"}


def test_parts_refuse_what_they_cannot_do():
    from llm_infrence_engine_amd.config import PartSpec
    from llm_infrence_engine_amd.parts.base import build_part

    heads = {"head_dim": 8, "eps": 1e-5, "dims": 4}
    build = lambda cat, kind, **p: build_part(cat, PartSpec(kind, "", p))
    with pytest.raises(ValueError):
        build("position", "qk_norm_rotary_half", **heads, over="projection")                    # how many heads?
    with pytest.raises(ValueError):
        build("position", "qk_norm_rotary_half", **heads, over="projection", heads=(2, 1), weighted=False)
    with pytest.raises(ValueError):
        build("position", "qk_norm_rotary_half", **heads, over="token")
    mixer = {"hidden_size": 32, "num_heads": 4, "num_kv_heads": 2, "head_dim": 8, "scale": 1.0, "qkv_bias": False}
    per_head = build("position", "qk_norm_rotary_half", **heads)
    for bad in ({"gate": "token"}, {"value_blend": "last"}, {"value_blend": "blend"}):          # (a norm per head stores no blend)
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("gqa_attention", "", dict(mixer, **bad)), position=per_head)
    with pytest.raises(ValueError):
        build("feed_forward", "routed_experts", hidden_size=32, expert_ff=16, experts=6, top=2, groups=(2, 1), group_top=3)


def test_values_lie_transposed_where_the_matrix_cores_read_them():
    from llm_infrence_engine_amd.config import PartSpec
    from llm_infrence_engine_amd.parts.base import build_part

    for d, dv, flipped in ((64, 64, True), (64, 32, True), (32, 16, True), (64, 40, False), (16, 32, False)):
        pos = build_part("position", PartSpec("qk_norm_rotary_half", "", {"head_dim": d, "eps": 1e-5}))
        m = build_part("mixer", PartSpec("gqa_attention", "", {"hidden_size": 32, "num_heads": 2, "num_kv_heads": 1, "head_dim": d,
                                                               "value_dim": dv, "scale": 1.0}), position=pos)
        assert (m.cache_need().tensors[1].transpose_at == 16) == flipped


def test_plain_model_prefix_property():
    """The plain model is causal: the logits of a prefix do not change when tokens follow."""
    cfg = SHAPES["R"]
    w = {k: v.double() for k, v in random_weights(cfg, 5).items()}
    toks = requests_for(cfg["vocab"], [23], 1)["r0"]
    full = P.forward(cfg, w, toks)
    assert torch.allclose(P.forward(cfg, w, toks[:9]), full[:9], atol=1e-9)


@pytest.mark.parametrize("name", list(SHAPES))
def test_every_mechanism_moves_the_logits_of_the_shapes(name):
    """What the shapes' tests can find: each mechanism, changed in the plain model alone, moves the logits by far more than the
    bounds below leave room for."""
    cfg = SHAPES[name]
    w = {k: v.double() for k, v in random_weights(cfg, SEEDS[name]).items()}
    toks = requests_for(cfg["vocab"], [110], 3)["r0"]
    base = P.forward(cfg, w, toks)

    def moved(edit_cfg=None, edit_w=None):
        c, ww = copy.deepcopy(cfg), dict(w)
        if edit_cfg:
            edit_cfg(c)
        if edit_w:
            edit_w(ww)
        return float((P.forward(c, ww, toks) - base).abs().max())

    for i, layer in enumerate(cfg["layers"]):
        m, mlp = layer["mixer"], layer["mlp"]
        keys = []
        if "mask" in m:
            keys.append(lambda c: c["layers"][i]["mixer"]["mask"].__setitem__("size", m["mask"]["size"] + 1))
        if "softcap" in m and m["softcap"] < 40:
            keys.append(lambda c: c["layers"][i]["mixer"].pop("softcap"))
        if "rot" in m and m["rot"].get("scaling", {}).get("factor", 1.0) != 1.0 and m.get("mask", {"size": 99})["size"] > 1:
            keys.append(lambda c: c["layers"][i]["mixer"]["rot"].pop("scaling"))
        if m["v_mix"] and f"l{i}.mix.vmix" in w:
            keys.append(lambda c: c["layers"][i]["mixer"].__setitem__("v_mix", False))
        if mlp and mlp["kind"] == "moe":
            keys.append(lambda c: c["layers"][i]["mlp"]["expert"].__setitem__("limit", mlp["expert"]["limit"] + 0.1))
            if mlp.get("shared"):       # (without one the norm behind the experts takes the scale out again)
                keys.append(lambda c: c["layers"][i]["mlp"]["router"].__setitem__("scale", mlp["router"]["scale"] * 1.1))
                keys.append(lambda c: c["layers"][i]["mlp"]["shared"].__setitem__("limit", mlp["shared"]["limit"] + 0.1))
        for k in keys:
            assert moved(k) > 5 * F32_ATOL, (name, i, keys.index(k))
        for t in ("mix.q.norm", "mix.k.norm", "mix.g"):
            if t != "mix.g" and m.get("mask", {"size": 99})["size"] == 1:
                continue
            assert moved(None, lambda ww: ww.__setitem__(f"l{i}.{t}", ww[f"l{i}.{t}"].flip(0))) > 5 * F32_ATOL, (name, i, t)


# ================================================================================================ kernels alone
@gpu
@pytest.mark.parametrize("N,H", [(1, 64), (3, 100), (9, 98), (130, 96), (17, 3584), (300, 260), (5, 2050), (2, 12400)])
def test_normed_sum_into_the_stream_and_the_stream_rounded(N, H):
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(N + H)
    top = 3
    x0, w1, w2 = torch.randn(N, H), 1 + 0.2 * torch.randn(H), 1 + 0.2 * torch.randn(H)
    part, weights = torch.randn(N * top, H), torch.rand(N, top)
    routed = (part.view(N, top, H).double() * weights.double()[:, :, None]).sum(1)
    for dtype in (torch.float32, torch.bfloat16):
        base = torch.randn(N, H + 4).to(dtype)[:, :H]
        dev = base.cuda()
        for y, yd in ((dev, base.double()), ((dev, part.cuda(), weights.cuda()), base.double() + routed),
                      ((None, part.cuda(), weights.cuda()), routed)):
            want = x0.double() + P.rms_norm(yd, w1.double(), 1e-5)
            for out_type in (torch.float32, torch.bfloat16):
                x = x0.cuda()
                out = ops.rms_norm_add(y, w1.cuda(), 1e-5, x, out=torch.full((N, H), 7.0, dtype=out_type, device="cuda"))
                assert (x.cpu().double() - want).abs().max() < 2e-5
                assert torch.equal(out, x.to(out_type))
                x = x0.cuda()
                out = ops.rms_norm_add(y, w1.cuda(), 1e-5, x, w2.cuda(), 3e-6, torch.empty(N, H, dtype=out_type, device="cuda"))
                ref = P.rms_norm(want, w2.double(), 3e-6)
                assert (out.cpu().double() - ref).abs().max() < (5e-5 if out_type == torch.float32 else 3e-2)
            x = x0.cuda()
            assert ops.rms_norm_add(y, w1.cuda(), 1e-5, x) is None
            assert (x.cpu().double() - want).abs().max() < 2e-5
    x = x0.cuda()
    assert torch.equal(ops.round_rows(x, torch.empty(N, H, dtype=torch.bfloat16, device="cuda")), x.bfloat16())
    with pytest.raises(ValueError):
        ops.rms_norm_add((None, part[:-1].contiguous().cuda(), weights.cuda()), w1.cuda(), 1e-5, x)


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,E,rot", [(6, 3, 20, 12, 8), (3, 1, 10, 14, 10), (8, 2, 64, 32, 32), (4, 4, 128, 128, 128), (7, 7, 8, 2, 0),
                                         (5, 1, 32, 16, 16), (28, 4, 128, 128, 64), (2, 1, 256, 256, 6)])
def test_norms_over_the_projection_rotation_blend_and_store(dtype, H, G, D, E, rot):
    """A token's q heads under one root mean square and its k heads under another, the rotation after it, values blended with
    another matrix's rows; every slot of the pages written where it should be and nowhere else."""
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(H * D)
    N, page, pages = 13, 16, 4
    width = (H + G) * D + G * E
    wide = (torch.randn(N, width + 24) * (1.0 + torch.arange(N)[:, None])).to(dtype)     # rows of very different sizes
    qw, kw = 1 + 0.3 * torch.randn(H * D), 1 + 0.3 * torch.randn(G * D)
    pos = torch.tensor([0, 1, 2, 3, 9, 17, 100, 101, 555, 1000, 4095, 20, 21], dtype=torch.int32)
    slots = torch.tensor([5, 0, 63, 16, -1, 31, 32, 17, -1, 40, 41, 2, 47], dtype=torch.int32)
    f = P.frequencies(rot, 500.0, 3.0) if rot else torch.empty(0, dtype=torch.float64)
    inv = f.float()
    first, lam = torch.randn(N, G * E + 8).to(dtype), torch.tensor(0.37)
    d = wide.double()
    q = P.rms_norm(d[:, :H * D], qw.double(), 1e-5).view(N, H, D)
    k = P.rms_norm(d[:, H * D:(H + G) * D], kw.double(), 1e-5).view(N, G, D)
    if rot:
        q, k = P.rotate(q, pos, f), P.rotate(k, pos, f)
    v = d[:, (H + G) * D:width]
    blended = P.blend_values(v, first[:, 8:].double(), 0.37)
    tol = 1e-3 if dtype == torch.float32 else 4e-2                 # (float angles of thousands of radians)
    for flipped in (False, True):
        for blend in (False, True):
            kp = torch.full((pages, G, page, D), 7.0, dtype=dtype, device="cuda")
            vp = torch.full((pages, G, E, page) if flipped else (pages, G, page, E), 7.0, dtype=dtype, device="cuda")
            x = wide.cuda()
            ops.qk_span_norm_store(x[:, :width], H, G, D, E, qw.cuda(), kw.cuda(), 1e-5, pos.cuda(), inv.cuda() if rot else None, rot,
                                   first.cuda()[:, 8:] if blend else None, lam.cuda() if blend else None, slots.cuda(), kp, vp, flipped)
            got = x.cpu().double()
            assert (got[:, :H * D].view(N, H, D) - q).abs().max() < tol * (1 + q.abs().max())
            assert torch.equal(x.cpu()[:, (H + G) * D:], wide[:, (H + G) * D:])      # v and what lies behind it stay
            want_v = blended if blend else v
            kd, vd = kp.cpu().double(), vp.cpu().double()
            if flipped:
                vd = vd.transpose(2, 3)
            used = set()
            for n, s in enumerate(slots.tolist()):
                if s < 0:
                    continue
                used.add(s)
                assert (kd[s // page, :, s % page] - k[n]).abs().max() < tol * (1 + k[n].abs().max()), n
                err = (vd[s // page, :, s % page].reshape(-1) - want_v[n]).abs() / (1 + want_v[n].abs())
                assert err.max() < (1e-6 if dtype == torch.float32 else 5e-3), n
            for s in range(pages * page):
                if s not in used:
                    assert (kd[s // page, :, s % page] == 7).all() and (vd[s // page, :, s % page] == 7).all()
    # nothing stored
    x = wide.cuda()
    ops.qk_span_norm_store(x[:, :width], H, G, D, E, qw.cuda(), kw.cuda(), 1e-5, pos.cuda(), inv.cuda() if rot else None, rot)
    assert (x.cpu().double()[:, :H * D].view(N, H, D) - q).abs().max() < tol * (1 + q.abs().max())


def _pages_of(lens, G, D, E, page, dtype, flipped, seed):
    """Pages in no order, full of what earlier users left, holding the keys and values of requests of these lengths."""
    from llm_infrence_engine_amd.parts.base import KVView

    g = torch.Generator().manual_seed(seed)
    need = sum(-(-n // page) for n in lens)
    order = [int(p) + 1 for p in torch.randperm(need + 3, generator=g)]
    kp, vp = (torch.full((need + 4, G, page, w), 9.0, dtype=dtype) for w in (D, E))
    table = torch.zeros(len(lens) + 1, max(-(-n // page) for n in lens) + 2, dtype=torch.int32)
    keys, values = [], []
    for r, n in enumerate(lens):
        keys.append(torch.randn(n, G, D, generator=g).to(dtype))
        values.append(torch.randn(n, G, E, generator=g).to(dtype))
        for p in range(-(-n // page)):
            table[r, p] = order.pop()

    def view():
        for r, n in enumerate(lens):
            for j in range(n):
                kp[table[r, j // page], :, j % page] = keys[r][j]
                vp[table[r, j // page], :, j % page] = values[r][j]
        v = vp.transpose(2, 3).contiguous() if flipped else vp
        return KVView({"k": kp.cuda(), "v": v.cuda()}, {"k": False, "v": flipped}, table.cuda(), None, True, None, None)

    return keys, values, view


def _plain_token(q, keys, values, t, scale, cap, window, slopes=None):
    """q [H, D] of the token at position t -> [H, E], from the request's keys and values."""
    lo = 0 if window is None else max(0, t - window + 1)
    rep = q.shape[0] // keys.shape[1]
    k, v = (a[lo:t + 1].double().repeat_interleave(rep, dim=1) for a in (keys, values))
    s = P.cap_scores(torch.einsum("hd,jhd->hj", q.double(), k) * scale, cap)
    if slopes is not None:
        s = s - slopes.double()[:, None] * (t - torch.arange(lo, t + 1).double())[None, :]
    return torch.einsum("hj,jhe->he", P.one_plus_softmax(s), v)


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,E", [(6, 2, 64, 64), (6, 2, 64, 32), (7, 1, 128, 128), (4, 4, 128, 80), (9, 3, 32, 32), (4, 2, 32, 16),
                                     (3, 1, 20, 36), (4, 2, 48, 24), (16, 1, 64, 48)])
@pytest.mark.parametrize("window,cap", [(None, 20.0), (33, 20.0), (50, None), (1, 5.0), (70, 75.0)])
def test_attention_with_cap_sink_window_and_a_gate_per_entry(dtype, H, G, D, E, window, cap):
    """Portions beside single tokens: every path (the vector kernel; on the matrix cores the bounded and the changed variant,
    values narrower than keys), with keys just inside and just outside every token's window that would take the whole weight."""
    from llm_infrence_engine_amd.kernels import ops

    page, scale = 16, 1.3 / math.sqrt(D)
    starts, q_lens = [0, 130, 63, 300, 15], [40, 1, 2, 77, 1]
    lens = [s + n for s, n in zip(starts, q_lens)]
    flipped = dtype == torch.bfloat16 and (E == D or (E < D and E % 16 == 0))
    keys, values, view = _pages_of(lens, G, D, E, page, dtype, flipped, seed=D + E)
    N = sum(q_lens)
    gen = torch.Generator().manual_seed(1)
    width = H * D + 24
    proj = torch.randn(N, width + H * E, generator=gen).to(dtype)
    n = 0
    for r, (s, m) in enumerate(zip(starts, q_lens)):
        for t in range(s, s + m):
            if window is not None and t % 3 == 0 and t - window >= 0:       # the token just outside would win everything
                keys[r][t - window] = proj[n, :H * D].view(G, H // G, D).float().mean(1).to(dtype) * 6
            n += 1
    kv = view()
    ctx = _Ctx(q_lens, list(range(len(lens))), starts)
    kv.table_rows = torch.arange(len(lens), dtype=torch.int32, device="cuda")
    pd = proj.cuda()
    for gate in ("entry", "head", None):
        g = {"entry": proj[:, width:], "head": proj[:, width:width + H], None: None}[gate]
        gd = {"entry": pd[:, width:], "head": pd[:, width:width + H], None: None}[gate]
        out = torch.full((N, H * E), 5.0, dtype=dtype, device="cuda")
        ops.paged_attention(pd[:, :width], kv, ctx, out, H, scale, window, torch.zeros(H, device="cuda"), cap or 0.0, None, gd)
        got, n = out.cpu().double(), 0
        for r, (s, m) in enumerate(zip(starts, q_lens)):
            for t in range(s, s + m):
                want = _plain_token(proj[n, :H * D].view(H, D), keys[r], values[r], t, scale, cap, window)
                if gate == "head":
                    want = want * torch.sigmoid(g[n].double())[:, None]
                want = want.reshape(-1)
                if gate == "entry":
                    want = want * torch.sigmoid(g[n].double())
                assert (got[n] - want).abs().max() < (2e-5 if dtype == torch.float32 else 2.5e-2), (gate, r, t)
                n += 1
    with pytest.raises(ValueError):
        ops.paged_attention(pd[:, :width], kv, ctx, out, H, scale, window, None, 0.0, None, pd[:, width:width + H + 1])


@gpu
@pytest.mark.parametrize("nt,waves,shares", [(1, 4, 1), (1, 8, 1), (1, 8, 2), (1, 8, 4), (2, 4, 1), (4, 4, 1), (0, 0, 0)])
@pytest.mark.parametrize("H,G,D,E", [(4, 2, 64, 64), (4, 2, 64, 16), (5, 1, 128, 128), (2, 2, 128, 96), (8, 2, 32, 32), (8, 2, 32, 16)])
def test_every_tile_of_the_matrix_core_attention_with_changed_scores(nt, waves, shares, H, G, D, E):
    """Every tile width, number of waves and share of the dims that has such a variant (others refuse), bounded scores and scores
    with slopes, with a learned sink."""
    from llm_infrence_engine_amd.kernels import build, ops

    page, scale, starts, q_lens = 16, 1.0 / math.sqrt(D), [90, 0, 201], [20, 35, 1]
    lens = [s + n for s, n in zip(starts, q_lens)]
    keys, values, view = _pages_of(lens, G, D, E, page, torch.bfloat16, True, seed=D)
    kv = view()
    N = sum(q_lens)
    proj = torch.randn(N, H * D + H * E, generator=torch.Generator().manual_seed(2)).bfloat16()
    sink = torch.linspace(-3.0, 3.0, H)
    slopes = torch.linspace(0.0, 0.1, H)
    ctx = _Ctx(q_lens, [0, 1, 2], starts)
    rows = torch.arange(3, dtype=torch.int32, device="cuda")
    pd, ran = proj.cuda(), 0
    lib = build.load()
    for sl in (None, slopes):
        for window in (None, 60):
            lib.ms_attention_mfma_force(nt, waves, shares)
            try:
                out = ops.paged_attention_mfma(pd, kv.k_pages, kv.v_pages, kv.block_table, ctx.q_start, ctx.context_lens,
                                               torch.empty(N, H * E, dtype=torch.bfloat16, device="cuda"), H, scale, ctx.max_q_len,
                                               ctx.max_context_len, window, rows, sink.cuda(), 9.0, sl.cuda() if sl is not None else None,
                                               pd[:, H * D:], 0.7)
            except ops.UnsupportedShape:
                continue
            finally:
                lib.ms_attention_mfma_force(0, 0, 0)
            ran += 1
            got, n = out.cpu().double(), 0
            for r, (s, m) in enumerate(zip(starts, q_lens)):
                for t in range(s, s + m):
                    lo = 0 if window is None else max(0, t - window + 1)
                    rep = H // G
                    k, v = (a[r][lo:t + 1].double().repeat_interleave(rep, dim=1) for a in (keys, values))
                    sc = P.cap_scores(torch.einsum("hd,jhd->hj", proj[n, :H * D].view(H, D).double(), k) * scale, 9.0)
                    if sl is not None:
                        sc = sc - sl.double()[:, None] * (t - torch.arange(lo, t + 1).double())[None, :]
                    p = torch.softmax(torch.cat([sc, sink.double()[:, None]], 1), 1)[:, :-1]
                    want = torch.einsum("hj,jhe->he", p, v).reshape(-1) * 0.7 * torch.sigmoid(proj[n, H * D:].double())
                    assert (got[n] - want).abs().max() < 2e-2, (sl is not None, window, r, t)
                    n += 1
    assert ran > 0 or nt == 4 or (E != D and shares > 1) or (D, nt) in ((128, 1), (32, 1))


@gpu
@pytest.mark.parametrize("H,G,D,E", [(4, 2, 64, 64), (7, 1, 128, 48), (2, 1, 32, 16), (5, 1, 128, 128)])
@pytest.mark.parametrize("window", [None, 1500])
def test_split_decode_with_a_gate_per_entry(H, G, D, E, window):
    """Single tokens behind long contexts: the keys spread over blocks and combined, bounded and unbounded scores."""
    from llm_infrence_engine_amd.kernels import ops

    page, scale, lens = 16, 1.2 / math.sqrt(D), [2500, 1100, 3001]
    keys, values, view = _pages_of(lens, G, D, E, page, torch.bfloat16, True, seed=D)
    proj = torch.randn(3, H * D + H * E, generator=torch.Generator().manual_seed(3)).bfloat16()
    for r in (0, 2):       # a far key that stands out, and one just outside the window that must not
        keys[r][lens[r] - 1400] = proj[r, :H * D].view(G, H // G, D).float().mean(1).bfloat16() * 4
        keys[r][lens[r] - 1 - 1500] = proj[r, :H * D].view(G, H // G, D).float().mean(1).bfloat16() * 6
    kv = view()
    kv.table_rows = torch.arange(3, dtype=torch.int32, device="cuda")
    ctx = _Ctx([1, 1, 1], [0, 1, 2], [n - 1 for n in lens])
    assert ops.attention_splits_keys(3, G, H // G, 1, max(lens))
    pd = proj.cuda()
    for cap in (25.0, 70.0, None):
        out = ops.paged_attention(pd[:, :H * D], kv, ctx, torch.empty(3, H * E, dtype=torch.bfloat16, device="cuda"), H, scale, window,
                                  torch.zeros(H, device="cuda"), cap or 0.0, None, pd[:, H * D:]).cpu().double()
        for r, n in enumerate(lens):
            want = _plain_token(proj[r, :H * D].view(H, D), keys[r], values[r], n - 1, scale, cap, window).reshape(-1)
            want = want * torch.sigmoid(proj[r, H * D:].double())
            assert (out[r] - want).abs().max() < 2e-2, (cap, r)


@gpu
@pytest.mark.parametrize("n_out,top,groups", [(8, 2, (2, 1)), (8, 3, (4, 2)), (6, 2, (6, 3)), (16, 5, (4, 3)), (5, 3, None), (4, 1, (1, 1)),
                                              (96, 6, (6, 2)), (200, 8, (100, 7)), (1024, 32, (8, 2)), (70, 2, (35, 1))])
def test_router_groups_count_as_their_two_best(n_out, top, groups):
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(n_out)
    z = 2.0 * torch.randn(37, n_out + 3)
    ids, weights = ops.moe_route(z.cuda(), None, top, n_out, "sigmoid", groups, False, 2, 1.7)
    s = torch.sigmoid(z[:, :n_out].double())
    want_ids, want_w = P.route(z[:, :n_out].double(), top, 1.7, groups)
    differs = 0
    for n in range(z.shape[0]):
        got = ids[n].tolist()
        assert (weights[n].cpu().double() - 1.7 * s[n][got]).abs().max() < 1e-5
        assert torch.allclose(s[n][got], s[n][want_ids[n]], atol=1e-6), (n, got, want_ids[n])
        if groups is not None:
            best = ops.moe_route(z[n:n + 1].cuda(), None, top, n_out, "sigmoid", groups)[0][0].tolist()
            differs += set(best) != set(got)
    if groups is not None and groups[1] < groups[0] and n_out // groups[0] > 1:
        assert differs > 0, "the inputs do not tell a group's best from its two best"
    with pytest.raises(ValueError):
        ops.moe_route(z.cuda(), None, top, n_out, "sigmoid", groups, False, 3)


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("N", [1, 5, 70, 600])
@pytest.mark.parametrize("W,ff,experts,top,groups,shared", [(64, 40, 6, 2, (3, 2), 24), (128, 64, 4, 1, (2, 1), 0), (96, 36, 8, 3, None, 52)])
def test_experts_weighted_by_scaled_scores(dtype, N, W, ff, experts, top, groups, shared):
    """The part alone, a few tokens and enough of them for the wide tiles; its sum made by itself and left to the caller."""
    from llm_infrence_engine_amd.config import PartSpec
    from llm_infrence_engine_amd.parts.base import Runtime, build_part

    torch.manual_seed(W + N)
    part = build_part("feed_forward", PartSpec("routed_experts", "m.", {
        "hidden_size": W, "expert_ff": ff, "experts": experts, "top": top, "activation": "clamped_glu", "limit": 0.9, "scores": "sigmoid",
        "correction": False, "groups": groups, "group_top": 2, "weight_scale": 1.6, "shared_ff": shared,
        "shared_limit": 1.3 if shared else None, "shared_gate": False}))
    w = {s.name: (torch.randn(s.shape) * (2.0 / math.sqrt(s.shape[-1]))).to(dtype) for s in part.tensor_specs()}
    part.load(lambda s: w[s.name].cuda(), Runtime(torch.device("cuda:0"), dtype))
    h = torch.randn(N, W).to(dtype)
    wd = {k: v.double() for k, v in w.items()}
    z = h.double() @ wd["m.router"].T
    ids, weights = P.route(z, top, 1.6, groups)
    outs = [P.expert(h.double(), wd, f"m.e{e}.", 0.9) for e in range(experts)]
    want = torch.stack([sum(a * outs[e][t] for e, a in zip(ids[t], weights[t])) for t in range(N)])
    if shared:
        want = want + P.expert(h.double(), wd, "m.shared.", 1.3)
    if N <= 5:
        mlp = {"router": {"top": top, "scale": 1.6}, "expert": {"limit": 0.9}, "shared": {"limit": 1.3} if shared else None}
        if groups:
            mlp["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
        assert torch.allclose(want, P.routed_experts(h.double(), wd, "m.", mlp), atol=1e-9)
    got = part.forward(h.cuda(), None).cpu().double()
    base, rows, g = part.forward_deferred(h.cuda(), None)
    left = (rows.view(N, top, W) * g[:, :, None]).sum(1).cpu().double() + (base.cpu().double() if base is not None else 0)
    tol = 3e-5 if dtype == torch.float32 else 2e-2
    # a token whose choice is a close call may go the other way in another precision
    for out in (got, left):
        err = (out - want).abs().max(1).values / (1 + want.abs().max(1).values)
        assert (err < tol).float().mean() > 0.97, float(err.max())


# ================================================================================================ whole models
def rounded_forward(cfg, w, toks):
    exact = P.forward(cfg, w, toks)
    return exact, float((P.forward(cfg, w, toks, act_dtype=torch.bfloat16) - exact).abs().max())


LENGTHS = {"P": [5, 61, 2, 130, 33, 48], "Q": [1, 9, 90, 47, 110, 64], "R": [3, 26, 70, 17, 2, 41, 60, 33],
           "S": [70, 3, 150, 50, 97, 33], "T": [40, 2, 140, 17, 66, 90, 35]}


@pytest.fixture(scope="module", params=list(SHAPES))
def shape(request, tmp_path_factory):
    name = request.param
    cfg = SHAPES[name]
    weights = random_weights(cfg, seed=SEEDS[name])
    # what a layer has no use for may be in a checkpoint all the same
    unused = {f"l{i}.mix.vmix": torch.tensor(0.9).bfloat16() for i, x in enumerate(cfg["layers"])
              if x["mixer"]["v_mix"] and f"l{i}.mix.vmix" not in weights}
    folder = write_model(tmp_path_factory.mktemp("kisusun" + name), cfg, dict(weights, **unused))
    reqs = requests_for(cfg["vocab"], LENGTHS[name], seed=ord(name))
    w64 = {k: v.double() for k, v in weights.items()}
    want, noise = {}, {}
    for rid, toks in reqs.items():
        want[rid], noise[rid] = rounded_forward(cfg, w64, toks)
        want[rid] = want[rid].numpy()
    return name, cfg, folder, reqs, want, noise


def _compare(got, want, noise, dtype):
    assert got
    for (rid, pos), row in got.items():
        err = np.abs(row.astype(np.float64) - want[rid][pos]).max()
        bound = F32_ATOL if dtype == "float32" else BF16_NOISE * max(noise[rid], 0.02)
        assert err < bound, f"request {rid} position {pos}: max |dlogit| {err:.3e} >= {bound:.3e}"


@gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("mode", ["whole", "bulk_then_single", "changing_portions", "mixed"])
def test_replay_against_plain(shape, tmp_path, dtype, mode):
    name, cfg, folder, reqs, want, noise = shape
    page = PAGES[name]
    up = lambda n: -(-n // 64) * 64
    if mode == "mixed":
        # room for the two longest requests only: pages and request rows are handed out again and again
        max_tokens = sum(sorted(up(len(t)) for t in reqs.values())[-2:])
        steps = traces.mixed(reqs, max_tokens, seed=3, max_live=4, tail=20)
    else:
        max_tokens = max(up(len(t)) for t in reqs.values())
        steps = {"whole": traces.whole, "bulk_then_single": lambda r: traces.bulk_then_single(r, tail=45),
                 "changing_portions": traces.changing_portions}[mode](reqs)
    runner = _replay(folder, dtype, steps, tmp_path / "out", max_tokens, page)
    _compare(traces.collect(steps, tmp_path / "out", cfg["vocab"]), want, noise, dtype)
    if mode == "mixed":
        assert all(g.allocator.pages_granted_again() > 0 for g in runner.manager.groups)


@gpu
def test_portions_and_batches_change_nothing_in_32_bit(shape, tmp_path):
    """The logits at a position do not depend on how the prompt was cut or on what else was in the batch, beyond
    rounding: whole against portions against mixed, directly (not through the oracle)."""
    name, cfg, folder, reqs, want, noise = shape
    page = PAGES[name]
    up = lambda n: -(-n // 64) * 64
    outs = {}
    total = sum(up(len(t)) for t in reqs.values())
    for mode, steps in (("whole", traces.whole(reqs)), ("portions", traces.changing_portions(reqs, sizes=(2, 3, 2, 31, 5, 2))),
                        ("mixed", traces.mixed(reqs, total, seed=9, tail=10))):
        _replay(folder, "float32", steps, tmp_path / mode, total, page)
        outs[mode] = traces.collect(steps, tmp_path / mode, cfg["vocab"])
    for mode in ("portions", "mixed"):
        for key, row in outs[mode].items():
            assert np.abs(row - outs["whole"][key]).max() < 3e-4, (mode, key)


@gpu
def test_one_row_and_few_pages_serve_every_request_in_turn(shape):
    """An engine with a single request row and pages for one request: every request gets the pages its predecessor left, in
    portions, and must see none of the old keys."""
    from llm_infrence_engine_amd.engine.batch import StepEntry
    from llm_infrence_engine_amd.engine.runner import load_runner

    name, cfg, folder, reqs, want, noise = shape
    page = PAGES[name]
    longest = max(len(t) for t in reqs.values())
    runner = load_runner(folder, dtype="float32", page_size=page, num_pages=-(-longest // page) + 1, max_requests=1,
                         max_len=-(-longest // page) * page)
    for rid, toks in reqs.items():
        cut = max(1, len(toks) // 2)
        got = [runner.step([StepEntry(rid, toks[:cut], list(range(cut)))]).cpu().numpy()]
        assert runner.manager.row(rid) == 0
        if cut < len(toks):
            got.append(runner.step([StepEntry(rid, toks[cut:], list(range(len(toks) - cut)))]).cpu().numpy())
        runner.free_request(rid)
        assert np.abs(np.concatenate(got) - want[rid]).max() < F32_ATOL, rid
    runner.manager.check_invariants()
    assert all(g.allocator.pages_granted_again() > 0 for g in runner.manager.groups)


def _marked_model(dim, vdim, window, seed=1):
    """One layer whose queries all look for marked tokens (ids from 90 on): such a token's key has one large entry past the
    rotated ones, which every query has too, so it takes nearly the whole softmax wherever it is seen."""
    cfg = config(97, 64, 1e-5, 1.0, 0.5, [attention(4, 2, dim, vdim, 10.0 / dim, dense(64), (10000.0, dim // 2, 4.0), window, 40.0)])
    weights = random_weights(cfg, seed=seed)
    common, mark = torch.linalg.qr(torch.randn(64, 2, generator=torch.Generator().manual_seed(2)))[0].T * 8.0
    emb = weights["embed"].float()
    emb = emb - torch.outer(emb @ common, common) / 64 - torch.outer(emb @ mark, mark) / 64 + 2.0 * common
    emb[90:] += 4.0 * mark
    q, k = weights["l0.mix.q"].float() * 0.2, weights["l0.mix.k"].float() * 0.2
    for t, heads, direction in ((q, 4, common), (k, 2, mark)):
        for h in range(heads):
            t[h * dim + dim - 1] = direction
    for n, t in (("embed", emb), ("l0.mix.q", q), ("l0.mix.k", k)):
        weights[n] = t.bfloat16().contiguous()
    return cfg, weights


@gpu
@pytest.mark.parametrize("dim,vdim", [(24, 16), (32, 32), (64, 32), (128, 128)])
@pytest.mark.parametrize("window,back", [(None, 400), (64, 63), (50, 49), (17, 16), (2, 1)])
def test_far_tokens_and_window_edges(tmp_path, dim, vdim, window, back):
    """A marked token ``back`` places back moves the last logits, one place further back (where there is a window) not at all: in
    the plain model and equally in the engine, in whole prompts, in portions and decoded token by token."""
    cfg, weights = _marked_model(dim, vdim, window)
    folder = write_model(tmp_path / "m", cfg, weights)
    w64 = {k_: v.double() for k_, v in weights.items()}
    rng = np.random.default_rng(5)
    n = back + 25
    plain = [int(t) for t in rng.integers(0, 90, n)]
    reqs, want, noise = {}, {}, {}
    for rid, at, token in (("none", 0, plain[0]), ("in_a", n - 1 - back, 91), ("in_b", n - 1 - back, 95), ("out", n - 2 - back, 92)):
        reqs[rid] = list(plain)
        reqs[rid][at] = token
        want[rid], noise[rid] = rounded_forward(cfg, w64, reqs[rid])
        want[rid] = want[rid].numpy()
    last = {rid: w[n - 1] for rid, w in want.items()}
    assert np.abs(last["in_a"] - last["in_b"]).max() > 0.2 and np.abs(last["in_a"] - last["none"]).max() > 0.2
    if window is not None:
        assert np.array_equal(last["out"], last["none"])
    room = 4 * (-(-n // 64) * 64)
    for mode, steps in (("whole", traces.whole(reqs)), ("single", traces.bulk_then_single(reqs, tail=min(n - 2, 300))),
                        ("portions", traces.changing_portions(reqs)), ("mixed", traces.mixed(reqs, room, seed=4, tail=20))):
        for dtype in ("float32", "bfloat16"):
            if mode == "single" and dtype == "bfloat16" and back > 100 and dim != 64:
                continue
            _replay(folder, dtype, steps, tmp_path / (mode + dtype), room, 16)
            _compare(traces.collect(steps, tmp_path / (mode + dtype), 97), want, noise, dtype)


@gpu
def test_first_tokens_feel_the_sink(tmp_path):
    """The first tokens of a sequence see few keys, and the one in the denominator weighs most there: at position 0 the weight of
    the only key is a sigmoid of its score."""
    cfg, weights = _marked_model(32, 32, 8)
    folder = write_model(tmp_path / "m", cfg, weights)
    w64 = {k_: v.double() for k_, v in weights.items()}
    reqs = {f"r{i}": t for i, t in enumerate([[3], [91], [5, 92], [93, 6, 7], [8, 9, 94, 95]])}
    for dtype in ("float32", "bfloat16"):
        for mode, steps in (("whole", traces.whole(reqs)), ("single", traces.bulk_then_single(reqs, tail=3))):
            _replay(folder, dtype, steps, tmp_path / (mode + dtype), 64, 16)
            got = traces.collect(steps, tmp_path / (mode + dtype), 97)
            for (rid, pos), row in got.items():
                exact, noise = rounded_forward(cfg, w64, reqs[rid])
                assert np.abs(row - exact[pos].numpy()).max() < (F32_ATOL if dtype == "float32" else BF16_NOISE * max(noise, 0.02))


@gpu
def test_long_decoding_passes_windows_and_pages(tmp_path):
    """Six hundred tokens decoded one by one behind a prompt of two: windows pass over decoded tokens again and again, and the
    windowed layers' pages are given back and used again."""
    cfg = SHAPES["S"]
    weights = random_weights(cfg, seed=SEEDS["S"])
    folder = write_model(tmp_path / "m", cfg, weights)
    toks = requests_for(cfg["vocab"], [602], 8)["r0"]
    exact, noise = rounded_forward(cfg, {k: v.double() for k, v in weights.items()}, toks)
    steps = traces.bulk_then_single({"a": toks, "b": toks[:300]}, tail=600)       # (one after the other)
    for dtype in ("float32", "bfloat16"):
        runner = _replay(folder, dtype, steps, tmp_path / dtype, 640, 16)
        _compare(traces.collect(steps, tmp_path / dtype, cfg["vocab"]), {"a": exact.numpy(), "b": exact.numpy()},
                 {"a": noise, "b": noise}, dtype)
        windowed = [g for g in runner.manager.groups if g.key.window is not None]
        assert windowed and all(g.allocator.pages_granted_again() > 0 for g in windowed)


@gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(shape, dtype):
    """``LLM.generate``: scheduler, prompt portions, continuous batching, graphs in bfloat16.  Every emitted token is
    the plain model's choice at its place, or within rounding of it."""
    import llm_infrence_engine_amd as eng

    name, cfg, folder, reqs, want, noise = shape
    weights = {k: v.double() for k, v in random_weights(cfg, seed=SEEDS[name]).items()}
    prompts = [toks[:max(1, len(toks) // 3)] for toks in list(reqs.values())[:4]]
    llm = eng.LLM(str(folder), dtype=dtype, block_size=PAGES[name], max_len=128, max_seqs=3, max_prefill_chunk=7)
    outs = llm.generate(prompts, eng.SamplingParams(max_new_tokens=40))
    slack = 2 * F32_ATOL if dtype == "float32" else None
    for p, o in zip(prompts, outs):
        assert len(o.token_ids) == 40 and o.finish_reason == "length"
        logits = P.forward(cfg, weights, p + o.token_ids)[len(p) - 1:-1]
        for t, row in zip(o.token_ids, logits):
            gap = float(row.max() - row[t])
            assert gap <= (slack if slack is not None else BF16_NOISE * max(max(noise.values()), 0.02)), (name, dtype, gap)
    m = llm.engine.runner.manager
    m.check_invariants()
    assert all(g.allocator.num_in_use() == 0 for g in m.groups) and m.num_requests() == 0
    if dtype == "bfloat16":
        # four decode steps to a graph launch, each fed the token the one before chose on the device: the same tokens
        del llm
        several = eng.LLM(str(folder), dtype=dtype, block_size=PAGES[name], max_len=128, max_seqs=3, max_prefill_chunk=7,
                          decode_steps_per_launch=4)
        again = several.generate(prompts, eng.SamplingParams(max_new_tokens=40))
        assert [o.token_ids for o in again] == [o.token_ids for o in outs]


@gpu
def test_command_line_generates(shape):
    import subprocess
    import sys

    from tests.conftest import ROOT

    name, cfg, folder, reqs, want, noise = shape
    if name != "P":
        pytest.skip("one shape is enough for the command line")
    r = subprocess.run([sys.executable, "-m", "llm_infrence_engine_amd", "--model", str(folder), "--dtype", "float32",
                        "--prompt-ids", "5,17,3", "--max-new-tokens", "4"], cwd=ROOT, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]


# ================================================================================================ arrangements together
@gpu
def test_a_normed_sum_is_carried_out_before_an_arrangement_that_knows_none():
    """A layer that hands on a normed sum, followed by one of the usual arrangement and by the last norm: the model settles what
    the next reader cannot."""
    from llm_infrence_engine_amd.kernels import ops
    from llm_infrence_engine_amd.parts.blocks import NormedAddend, PostNormResidual, PreNormResidual
    from llm_infrence_engine_amd.parts.model import Model
    from llm_infrence_engine_amd.parts.norms import RMSNorm
    from llm_infrence_engine_amd.parts.streams import HyperConnectedPreNorm, SummedStreams

    assert PostNormResidual.settles_writes and HyperConnectedPreNorm.settles_writes and SummedStreams.settles_writes
    assert not PreNormResidual.settles_writes and not RMSNorm.settles_writes
    norm = RMSNorm("", 64, 1e-5)
    norm.weight = torch.ones(64, device="cuda")
    x, y = torch.randn(3, 64), torch.randn(3, 64)
    want = x.double() + P.rms_norm(y.double(), torch.ones(64).double(), 1e-5)
    xd = x.cuda()
    assert Model._settled(xd, NormedAddend(y.cuda(), norm), norm) is None
    assert (xd.cpu().double() - want).abs().max() < 1e-5
    kept = NormedAddend(y.cuda(), norm)
    assert Model._settled(xd, kept, PostNormResidual) is kept and Model._settled(xd, None, norm) is None
    delta = torch.randn(3, 64, device="cuda")
    assert Model._settled(xd, delta, norm) is delta
