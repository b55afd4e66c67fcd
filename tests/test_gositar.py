"""The Gositar design against the plain implementation in ``tests/plain/gositar_plain.py``: every mechanism alone, then
whole models of several small shapes replayed whole, token by token, in portions and in mixed batches (32-bit and bfloat16
through graphs), and greedy generation through the engine's own entry point."""
import copy
import math

import numpy as np
import pytest
import torch
import torch.nn.functional as F

from tests import traces
from tests.plain import gositar_plain as P
from tests.test_gidurax import BF16_NOISE, F32_ATOL, _Ctx, _replay, requests_for, write_model

gpu = pytest.mark.gpu


# ================================================================================================ configurations
def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, limit, experts, top, groups=None, shared=None):
    d = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if groups is not None:
        d["router"]["groups"] = dict(zip(("count", "keep"), groups))
    if shared is not None:
        d["shared"] = dict(zip(("ff", "limit"), shared))
    return d


def attention(kind, heads, dim, rot_dim, vdim, kv_rank, scale, base, mlp, scaling=None):
    rot = {"base": base, "dims": rot_dim}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": kind, "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
                                                "kv_rank": kv_rank, "scale": scale, "rot": rot}}


A1, A2 = "latent_attention", "latent_attention_2"


def config(vocab, width, streams, eps, layers):
    return {"architecture": "Gositar", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers}


# Shapes that differ in every size and in the order of their layers: one to nine streams; both mixers with values wider and
# narrower than keys, latents of any size; frequency scaling with the ramp inside the pairs, outside them and absent; a
# layer without a feed-forward; experts with and without groups, with and without a shared one, one group that holds all,
# groups of one expert; one head; pages of 4 to 16.
SHAPES = {
    "P": config(211, 96, 3, 1e-5, [
        attention(A1, 5, 12, 8, 20, 28, 0.22, 10000.0, moe(40, 1.2, 6, 2, (3, 2), (24, 0.8)), (4.0, 64, 8.0, 1.0)),
        attention(A2, 3, 24, 6, 16, 40, 0.18, 500.0, dense(72)),
        attention(A2, 2, 16, 12, 10, 18, 0.25, 2000.0, None, (2.0, 32, 4.0, 0.5))]),
    "Q": config(130, 72, 1, 3e-6, [
        attention(A2, 1, 20, 4, 36, 50, 0.2, 100.0, dense(40), (16.0, 16, 2.0, 2.0)),
        attention(A1, 4, 10, 10, 14, 33, 0.3, 10000.0, moe(28, 2.0, 5, 3, None, None))]),
    "R": config(97, 100, 9, 1e-6, [
        attention(A1, 2, 18, 14, 26, 21, 0.25, 3000.0, moe(36, 0.7, 8, 3, (8, 4), (52, 3.0)), (3.0, 128, 16.0, 1.0)),
        attention(A1, 3, 8, 2, 12, 16, 0.4, 50.0, dense(64))]),
}
# latents and rotated parts that the matrix cores take in bfloat16, two cache groups, widths of whole pieces
SHAPES["S"] = config(257, 160, 4, 1e-5, [
    attention(A2, 6, 32, 32, 48, 192, 0.16, 10000.0, dense(192), (8.0, 256, 32.0, 1.0)),
    attention(A1, 5, 64, 64, 72, 64, 0.12, 50000.0, moe(64, 1.5, 12, 4, (4, 2), (96, 1.1)), (2.0, 128, 16.0, 1.0)),
    attention(A2, 6, 32, 32, 48, 192, 0.16, 10000.0, moe(64, 1.5, 4, 1, (1, 1), None))])
SHAPES["T"] = config(301, 128, 2, 1e-5, [
    attention(A1, 9, 32, 32, 32, 128, 0.2, 10000.0, moe(32, 0.9, 16, 5, (4, 3), (64, 1.4))),
    attention(A2, 3, 96, 64, 64, 256, 0.1, 1000000.0, dense(128), (40.0, 64, 32.0, 1.0))])
PAGES = {"P": 16, "Q": 8, "R": 4, "S": 16, "T": 16}
SEEDS = {"P": 1, "Q": 11, "R": 2, "S": 79, "T": 42}      # (choices of experts that do not rest on rounding)


def tensor_shapes(cfg):
    """Names and shapes, stated here from the design (not asked of the product)."""
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        H, D, R, E, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        for q in (1, 2) if mlp is not None else (1,):
            out.update({f"{p}norm{q}": (W,), f"{p}hc{q}.in": (S,), f"{p}hc{q}.out": (S,), f"{p}hc{q}.mix": (S, S)})
        a = p + "mix."
        out.update({a + "q": (H * (D + R), W), a + "dkv": (C + R, W), a + "dkv.norm": (C,), a + "uk": (H * D, C),
                    a + "uv": (H * E, C), a + "o": (W, H * E)})
        if layer["type"] == A1:
            out[a + "g"] = (H, W)
        f = p + "mlp."
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            out.update({f + "up": (mlp["ff"], W), f + "down": (W, mlp["ff"])})
            continue
        n, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        for e in range(n):
            out.update({f"{f}e{e}.gate": (ff, W), f"{f}e{e}.up": (ff, W), f"{f}e{e}.down": (W, ff)})
        out.update({f + "router": (n, W), f + "correction": (n,)})
        if mlp.get("shared"):
            s = mlp["shared"]["ff"]
            out.update({f + "shared.gate": (s, W), f + "shared.up": (s, W), f + "shared.down": (W, s)})
    return out


def random_weights(cfg, seed, dtype=torch.bfloat16):
    """Weights large enough that every mechanism moves the logits: scores of order one, gates half open, clamps that are
    reached, corrections that change choices.  Every token has a kind that its embedding leans towards and that the routers
    read, so that a choice of experts hardly ever rests on rounding."""
    g = torch.Generator().manual_seed(seed)
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    kinds = 6
    dirs = torch.linalg.qr(torch.randn(W, kinds, generator=g))[0].T              # [kinds, W], orthonormal
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g)
        if name.endswith(("norm1", "norm2", "final.norm", "dkv.norm")):
            t = 1.0 + 0.2 * r
        elif name == "embed":
            t = 0.6 * r + math.sqrt(W) * dirs[torch.arange(V) % kinds]
        elif leaf == "in":
            t = 1.0 / S + 0.2 * r / math.sqrt(S)
        elif leaf == "out":
            t = 0.7 + 0.3 * r
        elif leaf == "mix":
            t = 0.9 * torch.eye(S) + 0.25 * r / S
        elif leaf == "router":
            n = shape[0]
            rank = torch.stack([torch.randperm(n, generator=g) for _ in range(kinds)], dim=1).float()   # [n, kinds]
            t = (rank / max(1, n - 1) * 4.0 - 2.0) @ dirs / math.sqrt(W) * 1.2 + 0.02 * r / math.sqrt(W)
        elif leaf == "correction":
            t = 0.15 * r - 0.1
        else:
            t = r * (1.3 / math.sqrt(shape[-1]))
        w[name] = t
    return {name: t.to(dtype).contiguous() for name, t in w.items()}


# ================================================================================================ the oracle's own pins
def test_plain_pieces_against_library_routines():
    torch.manual_seed(0)
    x = torch.randn(9, 6, dtype=torch.float64)
    w = torch.randn(6, dtype=torch.float64)
    assert torch.allclose(P.layer_norm(x, w, 1e-5), F.layer_norm(x, (6,), w, None, 1e-5), atol=1e-12)
    assert torch.allclose(P.rms_norm(x, w, 1e-5), F.rms_norm(x, (6,), w, 1e-5), atol=1e-12)
    assert torch.allclose(P.relu_squared(x), F.relu(x) ** 2, atol=1e-12)
    # inside its limits the clamped form is a sigmoid-weighted product, outside the limit's own value
    g, u = torch.tensor([0.5, 9.0, -9.0]).double(), torch.tensor([0.25, 9.0, -9.0]).double()
    got = P.clamped_glu(g, u, 1.5)
    want = [0.5 * torch.sigmoid(torch.tensor(0.851, dtype=torch.float64)) * 1.25,
            1.5 * torch.sigmoid(torch.tensor(1.702 * 1.5, dtype=torch.float64)) * 2.5,
            -9.0 * torch.sigmoid(torch.tensor(-9.0 * 1.702, dtype=torch.float64)) * -0.5]
    assert all(abs(float(a) - float(b)) < 1e-12 for a, b in zip(got, want))
    # the rotation is a complex product with gain exp(i p f); both pairings; the rest stays
    f = torch.tensor([1.0, 0.1], dtype=torch.float64)
    v = torch.randn(5, 2, 7, dtype=torch.float64)
    pos = torch.tensor([0, 1, 2, 50, 1000])
    turn = torch.polar(torch.full((5, 2), 1.3, dtype=torch.float64), pos[:, None] * f[None, :])[:, None, :]
    for inter, iu, iv in ((True, [0, 2], [1, 3]), (False, [0, 1], [2, 3])):
        got = P.rotate(v, pos, f, 1.3, inter)
        z = torch.complex(v[..., iu], v[..., iv]) * turn
        assert torch.allclose(got[..., iu], z.real, atol=1e-12) and torch.allclose(got[..., iv], z.imag, atol=1e-12)
        assert torch.equal(got[..., 4:], v[..., 4:])
    q, k, vv = (torch.randn(7, 2, 5, dtype=torch.float64) for _ in range(3))
    ref = F.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1), vv.transpose(0, 1), is_causal=True, scale=0.3)
    assert torch.allclose(P.causal_attention(q, k, vv, 0.3), ref.transpose(0, 1), atol=1e-12)


def test_plain_frequencies_of_yarn():
    f, gain = P.yarn(8, 10000.0)
    assert gain == 1.0 and torch.allclose(f, 10000.0 ** (-torch.arange(4, dtype=torch.float64) / 4))
    sc = {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}
    f0, _ = P.yarn(64, 10000.0)
    fs, gain = P.yarn(64, 10000.0, sc)
    assert abs(gain - (0.1 * math.log(8.0) + 1.0)) < 1e-15
    turns = 4096 * f0 / (2 * math.pi)                   # how often a pair turns within the original length
    assert torch.allclose(fs[turns > 64], f0[turns > 64]) and torch.allclose(fs[turns < 0.5], f0[turns < 0.5] / 8.0)
    mid = (turns < 16) & (turns > 2)
    assert mid.any() and bool(((fs[mid] < f0[mid]) & (fs[mid] > f0[mid] / 8.0)).all())
    # a factor of one changes nothing; equal ends make a step, not a division by zero
    one, gain = P.yarn(16, 500.0, {"factor": 1.0, "original": 64, "fast": 8.0, "slow": 1.0})
    assert gain == 1.0 and torch.allclose(one, P.yarn(16, 500.0)[0])
    step, _ = P.yarn(16, 500.0, {"factor": 4.0, "original": 1, "fast": 8.0, "slow": 8.0})
    assert torch.isfinite(step).all()


@pytest.mark.parametrize("dims,base,scaling", [
    (32, 10000.0, None), (64, 500000.0, (8.0, 4096, 32.0, 1.0)), (6, 50.0, (3.0, 128, 16.0, 1.0)), (16, 500.0, (4.0, 1, 8.0, 8.0)),
    (12, 2000.0, (2.0, 32, 4.0, 0.5)), (4, 100.0, (16.0, 16, 2.0, 2.0)), (2, 10.0, (5.0, 1000, 64.0, 0.25)), (32, 1e6, (1.0, 64, 32.0, 1.0))])
def test_frequencies_of_the_product(dims, base, scaling):
    from llm_infrence_engine_amd.parts.positions import yarn_frequencies

    sc = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    f, gain = yarn_frequencies(dims, base, sc)
    want, want_gain = P.yarn(dims, base, sc)
    assert torch.allclose(f, want, rtol=1e-12, atol=0) and abs(gain - want_gain) < 1e-12


def test_plain_streams_and_router():
    X = torch.arange(12, dtype=torch.float64).view(3, 2, 2)
    M = torch.tensor([[1.0, 0.0, 2.0], [0.0, 1.0, 0.0], [0.5, 0.0, 0.0]], dtype=torch.float64)     # [from, to]
    y = torch.ones(2, 2, dtype=torch.float64)
    got = P.write_streams(X, M, torch.tensor([1.0, 0.0, 3.0], dtype=torch.float64), y)
    assert torch.equal(got[0], X[0] + 0.5 * X[2] + y) and torch.equal(got[1], X[1]) and torch.equal(got[2], 2 * X[0] + 3 * y)
    assert torch.equal(P.read_streams(X, torch.tensor([1.0, -1.0, 0.5], dtype=torch.float64)), X[0] - X[1] + 0.5 * X[2])
    # the best group is the one with the largest single choice score, also where all of them are negative; a strong expert of
    # a group that is not kept is out; weights come from the scores without the correction
    z = torch.log(torch.tensor([[0.4, 0.1, 0.3, 0.2]], dtype=torch.float64))
    ids, w = P.route(z, torch.tensor([-2.0, -0.9, -1.0, -3.0], dtype=torch.float64), 2, (2, 1))
    assert ids == [[2, 3]] and abs(w[0][0] - 0.6) < 1e-12 and abs(w[0][1] - 0.4) < 1e-12
    ids, w = P.route(z, None, 2, None)
    assert ids == [[0, 2]] and abs(w[0][0] - 4 / 7) < 1e-12
    ids, _ = P.route(z, torch.tensor([-2.0, -0.9, -1.0, -3.0], dtype=torch.float64), 2, (2, 2))
    assert ids == [[2, 1]]


def test_config_reads_every_size_and_refuses_what_it_does_not_know():
    from llm_infrence_engine_amd.cache import CacheLayout
    from llm_infrence_engine_amd.config import ConfigError, config_from_dict, preset
    from llm_infrence_engine_amd.parts.model import Model

    for name, cfg in SHAPES.items():
        c = config_from_dict(copy.deepcopy(cfg))
        assert type(c).__name__ == "GositarConfig" and c.to_dict() == cfg
        model = Model(c.to_spec())
        assert {s.name: tuple(s.shape) for s in model.tensor_specs()} == tensor_shapes(cfg)
        assert model.graph_safe() is True and hash(c.to_spec()) == hash(config_from_dict(copy.deepcopy(cfg)).to_spec())
        for layer, (kv, state, _) in zip(cfg["layers"], model.run_needs()):
            m = layer["mixer"]
            assert state is None and kv.window is None
            assert [(t.name, t.heads, t.width) for t in kv.tensors][:2] == [("c", 1, m["kv_rank"]), ("kr", 1, m["rot_dim"])]
        # equal needs share a group
        assert len(CacheLayout(model.run_needs()).group_keys) == len({(x["mixer"]["kv_rank"], x["mixer"]["rot_dim"]) for x in cfg["layers"]})
    for change in (lambda c: c["layers"][0].__setitem__("type", "something_else"),
                   lambda c: c["layers"][0]["mixer"].pop("kv_rank"),
                   lambda c: c["layers"][0]["mixer"].pop("scale"),
                   lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 7),
                   lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 10),
                   lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"),
                   lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 7),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("groups", {"count": 4, "keep": 1}),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("groups", {"count": 6, "keep": 1}),
                   lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"),
                   lambda c: c["layers"][1]["mlp"].pop("ff"),
                   lambda c: c["layers"][1]["mlp"].__setitem__("kind", "sparse"),
                   lambda c: c.pop("streams"),
                   lambda c: c.__setitem__("streams", 0)):
        bad = copy.deepcopy(SHAPES["P"])
        change(bad)
        with pytest.raises(ConfigError):
            config_from_dict(bad)
    for size in ("0.5b", "7b"):
        c = config_from_dict(preset(f"gositar-{size}"))
        assert c.streams == 4 and len(Model(c.to_spec()).layers) == len(c.layers)


def test_parts_refuse_what_they_cannot_do():
    from llm_infrence_engine_amd.parts.base import build_part
    from llm_infrence_engine_amd.config import PartSpec

    experts = {"hidden_size": 32, "expert_ff": 16, "experts": 6, "top": 2}
    with pytest.raises(ValueError):
        build_part("feed_forward", PartSpec("routed_experts", "", dict(experts, activation="clamped_glu")))            # no limit
    with pytest.raises(ValueError):
        build_part("feed_forward", PartSpec("routed_experts", "", dict(experts, groups=(4, 1))))
    with pytest.raises(ValueError):
        build_part("feed_forward", PartSpec("routed_experts", "", dict(experts, top=3, groups=(3, 1))))
    with pytest.raises(ValueError):
        build_part("stream_link", PartSpec("stream_link", "", {"streams": 33}))
    with pytest.raises(ValueError):
        build_part("position", PartSpec("rotary_pairs", "", {"width": 8, "dims": 8, "theta": 100.0, "pairing": "quarter"}))
    # a checkpoint's second norm and link of a layer without a feed-forward may be there and are not asked for
    from llm_infrence_engine_amd.config import config_from_dict

    spec = config_from_dict(copy.deepcopy(SHAPES["P"])).to_spec()
    assert set(spec.ignorable) == {"l2.norm2", "l2.hc2.in", "l2.hc2.out", "l2.hc2.mix"}


def test_random_weights_mode_keeps_the_streams_apart():
    from llm_infrence_engine_amd.config import config_from_dict
    from llm_infrence_engine_amd.parts.model import Model
    from llm_infrence_engine_amd.weights.random_init import random_tensors

    t = random_tensors(Model(config_from_dict(copy.deepcopy(SHAPES["S"])).to_spec()).tensor_specs(), seed=3)
    m = t["l1.hc2.mix"].float()
    assert (m - torch.eye(4)).abs().max() < 0.15 and (m - torch.eye(4)).abs().max() > 0
    assert (t["l0.hc1.in"].float() - 1.0).abs().max() < 0.6


def test_plain_model_prefix_property():
    """The plain model is causal: the logits of a prefix do not change when tokens follow."""
    cfg = SHAPES["R"]
    w = {k: v.double() for k, v in random_weights(cfg, 5).items()}
    toks = requests_for(cfg["vocab"], [23], 1)["r0"]
    full = P.forward(cfg, w, toks)
    assert torch.allclose(P.forward(cfg, w, toks[:9]), full[:9], atol=1e-9)


# ================================================================================================ kernels alone
@gpu
@pytest.mark.parametrize("S,W", [(1, 64), (2, 98), (3, 96), (4, 3584), (5, 100), (6, 36), (7, 256), (8, 1030), (9, 128), (20, 77)])
def test_streams_written_and_read_in_one_pass(S, W):
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(S)
    N, top = 11, 3
    x0 = torch.randn(N, S, W)
    mix, b, a = torch.randn(S, S), torch.randn(S), torch.randn(S)
    w, bias = 1 + 0.2 * torch.randn(W), 0.3 * torch.randn(W)
    base = {torch.float32: torch.randn(N, W), torch.bfloat16: torch.randn(N, W).bfloat16()}
    part, weights = torch.randn(N * top, W), torch.rand(N, top)
    routed = (part.view(N, top, W).double() * weights.double()[:, :, None]).sum(1)
    cases = [(base[torch.float32], base[torch.float32].double()), (base[torch.bfloat16], base[torch.bfloat16].double()),
             ((None, part, weights), routed), ((base[torch.bfloat16], part, weights), base[torch.bfloat16].double() + routed)]
    X = x0.double().transpose(0, 1)
    dev = lambda y: tuple(t.cuda() if t is not None else None for t in y) if isinstance(y, tuple) else y.cuda()
    rows = torch.tensor([7, 0, 10, 7], dtype=torch.int32, device="cuda")
    for i, (y, yd) in enumerate(cases):
        new = P.write_streams(X, mix.double(), b.double(), yd)
        u = P.read_streams(new, a.double())
        norms = {"layer": P.layer_norm(u, w.double(), 1e-5), "rms": P.rms_norm(u, w.double(), 1e-5), None: u}
        for kind, want in norms.items():
            for dtype in (torch.float32, torch.bfloat16):
                x = x0.cuda()
                bb = bias.cuda() if kind is not None and i % 2 else None
                out = torch.empty(N, W, dtype=dtype, device="cuda")
                ops.streams_step(x, write=(dev(y), mix.cuda(), b.cuda()), read=(a.cuda(), kind, w.cuda(), bb, 1e-5, out))
                ref = want + bias.double() if bb is not None else want
                scale = 1 + float(ref.abs().max())
                assert (x.cpu().double() - new.transpose(0, 1)).abs().max() < 2e-5 * (1 + S), (kind, i)
                assert (out.cpu().double() - ref).abs().max() < (3e-5 if dtype == torch.float32 else 6e-3) * scale, (kind, i, dtype)
        # chosen rows, nothing kept
        x = x0.cuda()
        out = torch.empty(4, W, dtype=torch.float32, device="cuda")
        ops.streams_step(x, write=(dev(y), mix.cuda(), b.cuda()), read=(a.cuda(), "layer", w.cuda(), None, 1e-5, out), rows=rows,
                         write_back=False)
        assert torch.equal(x.cpu(), x0)
        assert (out.cpu().double() - norms["layer"][rows.cpu().long()]).abs().max() < 1e-4
        # a write alone, a read alone
        ops.streams_step(x, write=(dev(y), mix.cuda(), b.cuda()))
        assert (x.cpu().double() - new.transpose(0, 1)).abs().max() < 2e-5 * (1 + S)
        kept = x.clone()
        out = ops.streams_step(x, read=(a.cuda(), "layer", w.cuda(), None, 1e-5, torch.empty(N, W, device="cuda")))
        assert torch.equal(x, kept) and (out.cpu().double() - norms["layer"]).abs().max() < 2e-4
    with pytest.raises(ValueError):
        ops.streams_step(x, write=(dev(y), mix.cuda(), b.cuda()), rows=rows)


@gpu
def test_embedding_into_every_stream():
    from llm_infrence_engine_amd.kernels import ops

    table = torch.randn(19, 52).bfloat16()
    ids = torch.tensor([3, 18, 0, 3], dtype=torch.int32)
    out = ops.embed(ids.cuda(), table.cuda(), torch.empty(4, 5, 52, device="cuda"))
    assert torch.equal(out.cpu(), table.float()[ids.long()][:, None, :].expand(4, 5, 52))


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("half", [False, True])
@pytest.mark.parametrize("C,R,dims,H", [(28, 8, 8, 5), (64, 32, 32, 4), (33, 10, 6, 3), (192, 64, 64, 2), (50, 4, 4, 1)])
def test_rotation_and_store_in_one_launch(dtype, half, C, R, dims, H):
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(C)
    N, page, P_ = 13, 4, 9
    gain = 1.21
    inv = (300.0 ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)).float()
    pos = torch.tensor([0, 1, 2, 3, 4, 15, 16, 17, 400, 401, 1000, 4095, 9], dtype=torch.int32)
    wide = torch.randn(N, 7 + C + R + 3).to(dtype)
    kv = wide[:, 7:7 + C + R]
    q = torch.randn(N, H, R + 11).to(dtype)
    w = 1 + 0.1 * torch.randn(C)
    slots = torch.tensor([5, 9, -1, 20, 21, 22, 23, 30, 31, 4, 6, 7, 8], dtype=torch.int32)
    kvd, qd = kv.double(), q.double()
    rot = lambda x: P.rotate(x, pos, inv.double(), gain, not half)
    c_pages = torch.full((P_, 1, page, C), 7.0, dtype=dtype, device="cuda")
    r_pages = torch.full((P_, 1, page, R), 7.0, dtype=dtype, device="cuda")
    ct = torch.full((P_, 1, C, page), 7.0, dtype=dtype, device="cuda")
    dst = torch.full((N, H, R + 2), 7.0, dtype=dtype, device="cuda")
    ops.latent_prepare(pos.cuda(), inv.cuda(), gain, half, kv=(wide.cuda()[:, 7:7 + C + R], w.cuda(), 1e-6, slots.cuda(), c_pages, r_pages, ct),
                       q=(q.cuda()[:, :, 11:], dst[:, :, 1:R + 1]))
    tol = 3e-4 if dtype == torch.float32 else 5e-2          # (angles are float: thousands of radians at the far positions)
    assert (dst[:, :, 1:R + 1].cpu().double() - rot(qd[:, :, 11:])).abs().max() < tol
    assert (dst[:, :, 0] == 7).all() and (dst[:, :, R + 1] == 7).all()
    c, kr = P.rms_norm(kvd[:, :C], w.double(), 1e-6), rot(kvd[:, C:])
    cp, rp = c_pages.cpu().double().view(P_ * page, C), r_pages.cpu().double().view(P_ * page, R)
    used = set()
    for n, s in enumerate(slots.tolist()):
        if s < 0:
            continue
        used.add(s)
        assert (cp[s] - c[n]).abs().max() < tol and (rp[s] - kr[n]).abs().max() < tol
        assert torch.equal(ct[s // page, 0, :, s % page], c_pages[s // page, 0, s % page])
    for s in range(P_ * page):
        if s not in used:
            assert (cp[s] == 7).all() and (rp[s] == 7).all()


@gpu
@pytest.mark.parametrize("N", [1, 16, 17, 128, 129, 300])
@pytest.mark.parametrize("H,I,J,gate", [(3, 32, 37, None), (5, 64, 80, "head"), (2, 96, 512, "value"), (4, 512, 128, "head"), (1, 160, 16, None)])
def test_per_head_maps_on_the_matrix_cores(N, H, I, J, gate):
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(N + I)
    x = torch.randn(N, H, I + 8).bfloat16()[:, :, 8:]
    m = torch.randn(H, J, I).bfloat16()
    g = {None: None, "head": torch.randn(N, H).bfloat16(), "value": torch.randn(N, H * J).bfloat16()}[gate]
    out = torch.full((N, H, J + 3), 5.0, dtype=torch.bfloat16, device="cuda")
    xd = torch.randn(N, H, I + 8).bfloat16()
    xd[:, :, 8:] = x
    assert ops.head_maps_transposed(torch.bfloat16, I, H * (I + 8), I + 8)
    ops.head_matmul(xd.cuda()[:, :, 8:], m.cuda(), out[:, :, :J], gate=g.cuda() if g is not None else None, transposed=True)
    want = torch.stack([x[:, h].double() @ m[h].double().T for h in range(H)], dim=1)
    if gate == "head":
        want = want * torch.sigmoid(g.double())[:, :, None]
    elif gate == "value":
        want = want * torch.sigmoid(g.double()).view(N, H, J)
    err = (out[:, :, :J].cpu().double() - want).abs() / (math.sqrt(I) + want.abs())
    assert err.max() < 5e-3 and (out[:, :, J:] == 5).all()
    # the vector kernel's per-head gate, both types
    for dtype in (torch.float32, torch.bfloat16):
        o = torch.empty(N, H, J, dtype=dtype, device="cuda")
        ops.head_matmul(x.to(dtype).cuda(), m.to(dtype).transpose(1, 2).contiguous().cuda(), o,
                        gate=g.to(dtype).cuda() if g is not None else None)
        err = (o.cpu().double() - want).abs() / (math.sqrt(I) + want.abs())
        assert err.max() < (1e-5 if dtype == torch.float32 else 5e-3)


def _latent_pages(lens, C, R, page, dtype, seed, stale=9.0):
    """Pages in no order, full of what earlier users left, holding random latents and key parts of requests; the rows, and a
    view with the transposed copy where the matrix cores would have it."""
    from llm_infrence_engine_amd.parts.base import KVView

    g = torch.Generator().manual_seed(seed)
    need = sum(-(-n // page) for n in lens)
    order = [int(p) + 1 for p in torch.randperm(need + 3, generator=g)]
    c_pages = torch.full((need + 4, 1, page, C), stale, dtype=dtype)
    r_pages = torch.full((need + 4, 1, page, R), stale, dtype=dtype)
    table = torch.zeros(len(lens) + 1, max(-(-n // page) for n in lens) + 2, dtype=torch.int32)
    rows = []
    for r, n in enumerate(lens):
        c, kr = torch.randn(n, C, generator=g).to(dtype), torch.randn(n, R, generator=g).to(dtype)
        rows.append([c, kr])
        for p in range(-(-n // page)):
            table[r, p] = order.pop()
    def fill():
        for r, (c, kr) in enumerate(rows):
            for p in range(-(-c.shape[0] // page)):
                part = slice(p * page, min(c.shape[0], (p + 1) * page))
                c_pages[table[r, p], 0, :part.stop - part.start] = c[part]
                r_pages[table[r, p], 0, :part.stop - part.start] = kr[part]
        kv = KVView({"c": c_pages.cuda(), "kr": r_pages.cuda()}, {"c": False, "kr": False}, table.cuda(), None, True, None, None)
        if dtype == torch.bfloat16 and page % 16 == 0:
            kv.pages["ct"] = kv.pages["c"].transpose(2, 3).contiguous()
            kv.transposed["ct"] = True
        return kv
    return rows, fill


def _plain_latent(q, c, kr, t, scale):
    """q [H, C + R] of the token at position t: softmax over the keys 0..t, [H, C]."""
    keys = torch.cat([c[:t + 1], kr[:t + 1]], dim=1).double()
    s = q.double() @ keys.T * scale
    p = torch.softmax(s, dim=1)
    return p @ c[:t + 1].double()


@gpu
@pytest.mark.parametrize("dtype,C,R,H,page", [
    (torch.float32, 40, 6, 3, 4), (torch.bfloat16, 50, 10, 5, 8), (torch.bfloat16, 64, 32, 4, 16), (torch.bfloat16, 64, 64, 9, 32),
    (torch.bfloat16, 128, 32, 14, 16), (torch.bfloat16, 128, 64, 17, 16), (torch.bfloat16, 192, 32, 6, 16), (torch.bfloat16, 192, 64, 3, 48),
    (torch.bfloat16, 256, 32, 14, 16), (torch.bfloat16, 256, 64, 5, 16), (torch.bfloat16, 384, 32, 7, 16), (torch.bfloat16, 384, 64, 20, 16),
    (torch.bfloat16, 512, 32, 4, 64), (torch.bfloat16, 512, 64, 28, 16)])
def test_attention_over_all_latents_with_one_loud_key(dtype, C, R, H, page):
    """Full attention, no window and no sink.  In request 0 one far key (a page's last slot) answers one head so loudly that
    its latent is the result: portions long enough for the staged kernel, short ones, and single decoded tokens whose keys
    are spread over blocks, at contexts around page and key-block borders; a key at the token's own place is seen, the one
    after it (stored already) is not."""
    from llm_infrence_engine_amd.kernels import ops

    lens = [613, 37, 1]
    scale = 0.5 / math.sqrt(C + R)
    rows, fill = _latent_pages(lens, C, R, page, dtype, seed=C + R)
    loud = page * 5 - 1                            # a page's last slot, far back
    ahead = 600                                    # and a key that is in the cache before its turn has come
    for at in (loud, ahead):
        rows[0][0][at] = 0.05 * rows[0][0][at]
        rows[0][0][at, 0] = 30.0
    kv = fill()
    before = dict(ops.launches)

    def run(entries, tol):
        """entries: (request, first position, tokens)"""
        ctx = _Ctx([n for _, _, n in entries], [r for r, _, _ in entries], starts=[s for _, s, _ in entries])
        kv.table_rows = torch.tensor([r for r, _, _ in entries], dtype=torch.int32, device="cuda")
        q = torch.randn(ctx.num_tokens, H, C + R).to(dtype)
        q[:, 0] = 0.1 * q[:, 0]
        q[:, 0, 0] = 2.0 * math.sqrt(C + R)        # head 0 listens for the loud keys
        out = ops.latent_attention(q.cuda(), kv, ctx, torch.empty(ctx.num_tokens, H, C, dtype=dtype, device="cuda"), scale).cpu()
        at = 0
        for r, s, n in entries:
            for t in range(s, s + n):
                want = _plain_latent(q[at], rows[r][0], rows[r][1], t, scale)
                err = (out[at].double() - want).abs().max()
                assert err < tol * (1 + float(want.abs().max())), (r, t, float(err))
                if r == 0 and loud <= t < ahead and t < loud + 200:
                    assert out[at, 0, 0] > 20.0, t
                at += 1

    tol = 2e-5 if dtype == torch.float32 else 1.5e-2
    run([(0, 0, 613)], tol)                                            # a whole prompt
    run([(1, 5, 32), (0, 300, 17), (2, 0, 1)], tol)                    # portions of unequal requests
    run([(0, 598, 2)], tol)                                            # a short one, right before the loud key ahead
    for t in sorted({0, 1, 15, 16, 31, 32, 33, 63, 64, loud - 1, loud, loud + 1, 127, 128, 129, 511, 512, 599, 600, 612}):
        run([(0, t, 1)], tol)
    run([(0, 612, 1), (1, 36, 1), (2, 0, 1)], tol)                     # a batch of single tokens
    matrix = dtype == torch.bfloat16 and ops.latent_mfma_sizes(C, R)
    count = lambda k: ops.launches.get(k, 0) - before.get(k, 0)
    assert (count("latent_attention_mfma") > 0) == matrix and (count("latent_attention_split") > 0) == matrix


@gpu
@pytest.mark.parametrize("C,R,H", [(64, 32, 4), (256, 32, 14), (512, 64, 28)])
def test_long_portions_fill_the_chip_and_long_contexts_are_split(C, R, H):
    """The widest blocks (eight tiles each) need many columns: a portion of 1,500 tokens behind 100 others; and a context of
    5,000 keys decoded by one token."""
    from llm_infrence_engine_amd.kernels import ops

    lens, scale = [1600, 5001], 0.6 / math.sqrt(C + R)
    rows, fill = _latent_pages(lens, C, R, 16, torch.bfloat16, seed=1)
    kv = fill()
    n = 1500 if H > 4 else 1600
    ctx = _Ctx([n], [0], starts=[1600 - n])
    kv.table_rows = torch.tensor([0], dtype=torch.int32, device="cuda")
    q = torch.randn(n, H, C + R).bfloat16()
    out = ops.latent_attention(q.cuda(), kv, ctx, torch.empty(n, H, C, dtype=torch.bfloat16, device="cuda"), scale).cpu()
    for i in [0, 1, 2, 31, 777, n - 2, n - 1]:
        want = _plain_latent(q[i], rows[0][0], rows[0][1], 1600 - n + i, scale)
        assert (out[i].double() - want).abs().max() < 1.5e-2 * (1 + float(want.abs().max())), i
    kv.table_rows = torch.tensor([1], dtype=torch.int32, device="cuda")
    ctx = _Ctx([1], [1], starts=[5000])
    assert ops.latent_splits(1, H, 1, 5001, None) > 1
    out = ops.latent_attention(q[:1].cuda(), kv, ctx, torch.empty(1, H, C, dtype=torch.bfloat16, device="cuda"), scale).cpu()
    want = _plain_latent(q[0], rows[1][0], rows[1][1], 5000, scale)
    assert (out[0].double() - want).abs().max() < 1.5e-2 * (1 + float(want.abs().max()))


@gpu
@pytest.mark.parametrize("n_out,top,groups,correction", [(8, 2, (2, 1), True), (8, 3, (8, 4), True), (12, 4, (4, 2), True), (16, 5, None, True),
                                                         (5, 3, None, False), (4, 1, (1, 1), True), (96, 6, (6, 2), True), (200, 8, (100, 7), True),
                                                         (1024, 32, (4, 1), True), (70, 2, (35, 1), False)])
def test_router_within_groups(n_out, top, groups, correction):
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(n_out)
    z = 2.0 * torch.randn(37, n_out + 3)
    corr = 0.2 * torch.randn(n_out) - 0.5 if correction else None              # choice scores below zero
    for scores in ("softmax", "sigmoid"):
        for normalise in (True, False):
            ids, weights = ops.moe_route(z.cuda(), corr.cuda() if correction else None, top, n_out, scores, groups, normalise)
            s = torch.softmax(z[:, :n_out].double(), 1) if scores == "softmax" else torch.sigmoid(z[:, :n_out].double())
            if scores == "softmax":
                want_ids, want_w = P.route(z[:, :n_out].double(), corr.double() if correction else None, top, groups)
            for n in range(z.shape[0]):
                got = ids[n].tolist()
                picked = s[n][got]
                w = picked / (picked.sum() + 1e-20) if normalise else picked
                assert (weights[n].cpu().double() - w).abs().max() < 1e-5
                if scores == "softmax":
                    choice = s[n] + (corr.double() if correction else 0)
                    # equal choices up to float rounding of the scores
                    assert torch.allclose(choice[got], choice[want_ids[n]], atol=1e-6), (n, got, want_ids[n])
                if groups is not None:
                    size = n_out // groups[0]
                    assert len({e // size for e in got}) <= groups[1] and len(set(got)) == top
    with pytest.raises(ValueError):
        ops.moe_route(z.cuda(), None, top, n_out, "softmax", (n_out - 1, 1) if n_out > 4 else (3, 1))


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("N", [1, 5, 70, 700])
@pytest.mark.parametrize("W,ff,experts,top,shared", [(64, 40, 6, 2, 24), (128, 64, 4, 1, 0), (96, 36, 8, 3, 52)])
def test_clamped_experts_with_a_shared_one(dtype, N, W, ff, experts, top, shared):
    """The part alone, a few tokens and enough of them for the wide tiles; its sum made by itself and left to the caller."""
    from llm_infrence_engine_amd.config import PartSpec
    from llm_infrence_engine_amd.parts.base import Runtime, build_part

    torch.manual_seed(W + N)
    part = build_part("feed_forward", PartSpec("routed_experts", "m.", {
        "hidden_size": W, "expert_ff": ff, "experts": experts, "top": top, "activation": "clamped_glu", "limit": 0.9, "normalise": True,
        "groups": (2, 1), "shared_ff": shared, "shared_limit": 1.3 if shared else None, "shared_gate": False}))
    w = {s.name: (torch.randn(s.shape) * (2.0 / math.sqrt(s.shape[-1]) if len(s.shape) == 2 else 0.1)).to(dtype) for s in part.tensor_specs()}
    keep = lambda s: w[s.name].cuda().float() if s.role == "bias" else w[s.name].cuda()
    part.load(keep, Runtime(torch.device("cuda:0"), dtype))
    h = torch.randn(N, W).to(dtype)
    mlp = {"router": {"top": top, "groups": {"count": 2, "keep": 1}}, "expert": {"limit": 0.9},
           "shared": {"limit": 1.3} if shared else None}
    wd = {k: v.double() for k, v in w.items()}
    ids, weights = P.route(h.double() @ wd["m.router"].T, wd["m.correction"], top, (2, 1))
    outs = [P.expert(h.double(), wd, f"m.e{e}.", 0.9) for e in range(experts)]
    want = torch.stack([sum(a * outs[e][t] for e, a in zip(ids[t], weights[t])) for t in range(N)])
    if shared:
        want = want + P.expert(h.double(), wd, "m.shared.", 1.3)
    if N <= 5:
        assert torch.allclose(want, P.routed_experts(h.double(), wd, "m.", mlp), atol=1e-9)
    got = part.forward(h.cuda(), None).cpu().double()
    base, rows, g = part.forward_deferred(h.cuda(), None)
    left = (rows.view(N, top, W) * g[:, :, None]).sum(1).cpu().double() + (base.cpu().double() if base is not None else 0)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    # a token whose choice is a close call may go the other way in another precision
    z = torch.softmax(h.double() @ wd["m.router"].T, 1) + wd["m.correction"]
    groups = z.view(N, 2, experts // 2).max(2).values
    kept = torch.where((groups[:, 0] > groups[:, 1])[:, None], z[:, :experts // 2], z[:, experts // 2:]).sort(1, descending=True).values
    gap = (groups[:, 0] - groups[:, 1]).abs()
    if top < experts // 2:
        gap = torch.minimum(gap, kept[:, top - 1] - kept[:, top])
    clear = gap > 1e-5
    assert clear.float().mean() > 0.95
    for out in (got, left):
        err = (out - want).abs().max(1).values / (1 + want.abs().max(1).values)
        assert err[clear].max() < tol, float(err[clear].max())


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("N,W,ff", [(1, 64, 40), (9, 128, 192), (64, 72, 88), (200, 128, 256), (300, 100, 60)])
def test_squared_relu_feed_forward(dtype, N, W, ff):
    from llm_infrence_engine_amd.config import PartSpec
    from llm_infrence_engine_amd.kernels import ops
    from llm_infrence_engine_amd.parts.base import Runtime, build_part

    torch.manual_seed(N)
    x = torch.cat([torch.randn(N * ff - 3) * 2, torch.tensor([0.0, -0.0, -5.0])]).to(dtype)
    got = ops.relu2(x.cuda(), torch.empty_like(x, device="cuda")).cpu().double()
    assert ((got - P.relu_squared(x.double())).abs() / (1 + got)).max() < (1e-6 if dtype == torch.float32 else 5e-3)
    part = build_part("feed_forward", PartSpec("dense_act", "m.", {"hidden_size": W, "intermediate_size": ff, "activation": "relu2"}))
    w = {s.name: (torch.randn(s.shape) * (1.5 / math.sqrt(s.shape[-1]))).to(dtype) for s in part.tensor_specs()}
    assert set(w) == {"m.up", "m.down"}
    part.load(lambda s: w[s.name].cuda(), Runtime(torch.device("cuda:0"), dtype))
    h = torch.randn(N, W).to(dtype)
    want = P.dense(h.double(), {k: v.double() for k, v in w.items()}, "m.")
    out = part.forward(h.cuda(), None).cpu().double()
    assert ((out - want).abs().max() / (1 + want.abs().max())) < (2e-5 if dtype == torch.float32 else 1.5e-2)


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
    folder = write_model(tmp_path_factory.mktemp("gositar" + name), cfg, weights)
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


@gpu
@pytest.mark.parametrize("kind,kv_rank,rot_dim", [(A1, 24, 8), (A2, 24, 8), (A1, 128, 32), (A2, 64, 32)])
def test_far_token_reaches_the_end(tmp_path, kind, kv_rank, rot_dim):
    """A token 400 places back still moves the last logits through the cache, in the plain model and equally in the engine,
    whole and decoded token by token over hundreds of steps: the far token's key is what every query looks for."""
    layer = attention(kind, 2, 32, rot_dim, 24, kv_rank, 0.3, 10000.0, dense(64), (4.0, 128, 16.0, 1.0))
    cfg = config(97, 64, 2, 1e-5, [layer])
    weights = random_weights(cfg, seed=1)
    # every token carries `common`, which the first entry of each head's query reads; ids from 90 on carry `far`, which the
    # latent's first entry reads and each head's first key entry takes from there
    common, far = torch.randn(2, 64, generator=torch.Generator().manual_seed(2))
    emb = weights["embed"].float() + 2.0 * common
    emb[90:] += 4.0 * far
    q, dkv, uk = (weights["l0.mix." + n].float() for n in ("q", "dkv", "uk"))
    dkv[0] = far / 8
    for h in range(2):
        q[h * (32 + rot_dim)] = common * 20 / 64
        uk[h * 32] = 0.0
        uk[h * 32, 0] = 1.0
    for n, t in (("embed", emb), ("l0.mix.q", q), ("l0.mix.dkv", dkv), ("l0.mix.uk", uk)):
        weights[n] = t.bfloat16().contiguous()
    folder = write_model(tmp_path / "m", cfg, weights)
    w64 = {k_: v.double() for k_, v in weights.items()}
    rng = np.random.default_rng(5)
    a = [int(t) for t in rng.integers(0, 90, 420)]
    a[7] = 91
    b = list(a)
    b[7] = 95
    la, lb = P.forward(cfg, w64, a)[-1].numpy(), P.forward(cfg, w64, b)[-1].numpy()
    assert np.abs(la - lb).max() > 0.1, "the test's weights do not show the far token"
    reqs = {"a": a, "b": b}
    for mode, steps in (("whole", traces.whole(reqs)), ("single", traces.bulk_then_single(reqs, tail=380))):
        _replay(folder, "float32", steps, tmp_path / mode, 2 * 448, 16)
        got = traces.collect(steps, tmp_path / mode, 97)
        assert np.abs(got[("a", 419)] - la).max() < 5e-4 and np.abs(got[("b", 419)] - lb).max() < 5e-4
    steps = traces.bulk_then_single(reqs, tail=40)
    _replay(folder, "bfloat16", steps, tmp_path / "bf16", 2 * 448, 16)
    got = traces.collect(steps, tmp_path / "bf16", 97)
    noise = max(rounded_forward(cfg, w64, t)[1] for t in reqs.values())
    assert np.abs(got[("a", 419)] - la).max() < BF16_NOISE * max(noise, 0.02) and np.abs(got[("b", 419)] - lb).max() < BF16_NOISE * max(noise, 0.02)


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


@gpu
@pytest.mark.parametrize("M", [1, 7, 16, 33, 64, 70, 300])
@pytest.mark.parametrize("N,K", [(96, 64), (130, 72), (512, 896), (2050, 128), (64, 1032)])
def test_activations_as_epilogues_of_the_products(M, N, K):
    """The squared relu and the clamped gate in every kernel that has them: few rows (three kernels, whichever takes the
    shape) and the tiled product of many."""
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(M + N)
    a, w = torch.randn(M, K).bfloat16(), (torch.randn(N, K) * 2 / math.sqrt(K)).bfloat16()
    z = a.double() @ w.double().T
    limit, alpha = 1.3, 1.702
    g, u = torch.clamp(z[:, ::2], max=limit), torch.clamp(z[:, 1::2], -limit, limit)
    want = {ops.EPI_RELU2: P.relu_squared(z), ops.EPI_CLAMPED: g * torch.sigmoid(alpha * g) * (u + 1)}
    numbers = torch.tensor([limit, alpha], device="cuda")
    ad, wd = a.cuda(), w.cuda()
    for epi, ref in want.items():
        outs = []
        if M <= ops.SKINNY_MAX_ROWS:
            outs.append(ops.gemm_skinny(ad, wd, numbers if epi == ops.EPI_CLAMPED else None, epi))
        if K % 64 == 0:
            outs.append(ops.gemm_tiled(ad, wd, epi, limit, alpha))
        for out in outs:
            err = (out.cpu().double() - ref).abs() / (1 + ref.abs())
            assert out.shape == ref.shape and err.max() < 1e-2, (epi, float(err.max()))


@gpu
@pytest.mark.parametrize("N,K,ff,experts,top", [(3, 64, 24, 4, 2), (90, 96, 40, 6, 2), (900, 96, 64, 4, 2), (1200, 128, 160, 4, 2)])
def test_clamped_gate_as_epilogue_of_the_grouped_product(N, K, ff, experts, top):
    """Small tiles, tiles of 128 rows (K no multiple of 64) and the tiled kernel's (K a multiple of 64), against the product
    and the gate in two steps."""
    from llm_infrence_engine_amd.kernels import ops

    torch.manual_seed(N)
    h = torch.randn(N, K).bfloat16()
    w = (torch.randn(experts, 2 * ff, K) * 2 / math.sqrt(K)).bfloat16()
    ids = torch.stack([torch.randperm(experts)[:top] for _ in range(N)]).int()
    for tile in (ops.moe_tile_rows(), ops.moe_wide_tile_rows(), ops.moe_widest_tile_rows()):
        if tile == ops.moe_widest_tile_rows() and K % 64:
            continue
        rows, tile_expert = ops.moe_align(ids.cuda(), experts, tile)
        out = torch.full((rows.numel(), ff), 7.0, dtype=torch.bfloat16, device="cuda")
        ops.grouped_gemm(h.cuda(), w.cuda(), rows, tile_expert, out, gather_div=top, act="clamped_glu", limit=0.8, alpha=1.702)
        seen = 0
        for p, item in enumerate(rows.tolist()):
            if item < 0:
                assert (out[p] == 7.0).all()
                continue
            e = int(ids.view(-1)[item])
            if item % 7 and N > 100:        # (a sample of the rows)
                seen += 1
                continue
            z = h[item // top].double() @ w[e].double().T
            g, u = torch.clamp(z[::2], max=0.8), torch.clamp(z[1::2], -0.8, 0.8)
            ref = g * torch.sigmoid(1.702 * g) * (u + 1)
            assert ((out[p].cpu().double() - ref).abs() / (1 + ref.abs())).max() < 1e-2
            seen += 1
        assert seen == N * top
    with pytest.raises(ops.UnsupportedShape):
        ops.grouped_gemm(h.float().cuda(), w.float().cuda(), *ops.moe_align(ids.cuda(), experts),
                         torch.empty(ops.moe_align(ids.cuda(), experts)[0].numel(), ff, device="cuda"), gather_div=top, act="clamped_glu",
                         limit=0.8, alpha=1.702)
