"""The Redirax family in the rollout engine against the plain oracle
(tests/redirax_oracle.py): attention with biases and turned neighbour pairs
beside linear attention with fixed decays, the normed half sum of the two,
residual streams and the tanh norm, the routed clamped experts with their
gated shared expert, layers that run another layer's weights; whole prompts
against token-by-token decoding, portions down to two tokens, unequal
batches, reuse of pages and slots, keys far behind and at page and tile
borders, a recurrence that remembers its first token over chunk borders,
first tokens, long decoding, odd sizes, the checkpoint-folder loader, the
trace replay entry point and greedy generation through the engine's
scheduler.

Every case runs on the CPU tier (PyTorch forms of the ops, fp32) and, marked
``gpu``, on the HIP kernels in fp32 and bf16.  Configurations are small and
made here; weights are random with a fixed seed (bf16-representable), or
built so that one key or one token is loud where random weights would hide a
fault.
"""
import copy
import io
import json
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import redirax_oracle as O  # noqa: E402

from polyrl_amd.models.hybrid import (redirax_config_from_json,  # noqa: E402
                                      redirax_config_to_json)
from polyrl_amd.rollout.engine import Engine, SamplingParams  # noqa: E402
from polyrl_amd.rollout.hybrid_model import HybridInferenceModel  # noqa: E402

CPU = ("cpu", torch.float32)
GPU32 = pytest.param(("cuda", torch.float32), marks=pytest.mark.gpu)
GPU16 = pytest.param(("cuda", torch.bfloat16), marks=pytest.mark.gpu)
TARGETS = [CPU, GPU32, GPU16]
VOCAB = 83


def mixer(heads=4, kv=2, dim=16, vdim=12, rot=8, base=60.0, factor=2.5,
          scale=0.3, rh=3, rdim=10, rvdim=14, decay=None):
    decay = decay or [0.5 + 0.49 * (i + 1) / rh for i in range(rh)]
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "scale": scale, "rot": {"base": base, "dims": rot,
                                    "scaling": {"factor": factor}}}
    return {"left": left, "right": {"heads": rh, "dim": rdim, "vdim": rvdim,
                                    "decay": decay}}


def dense(n=24):
    return {"kind": "dense", "ff": n}


def moe(n=20, experts=5, top=2, limit=1.1, shared=28, slimit=0.7):
    f = {"kind": "moe", "expert": {"ff": n, "limit": limit},
         "router": {"experts": experts, "top": top}}
    if shared:
        f["shared"] = {"ff": shared, "limit": slimit}
    return f


def config(layers, width=40, streams=3, cap=6.0, eps=1e-5):
    """``layers``: (mixer, mlp) pairs, or the index of the layer whose
    weights a layer runs."""
    out = []
    for L in layers:
        if isinstance(L, int):
            out.append(dict(copy.deepcopy(out[L]), weights_of=L))
        else:
            out.append({"type": "parallel", "mixer": copy.deepcopy(L[0]),
                        "mlp": copy.deepcopy(L[1])})
    c = {"architecture": "Redirax", "vocab": VOCAB, "width": width,
         "streams": streams, "layers": out, "norm": {"eps": eps}}
    if cap:
        c["logit_softcap"] = cap
    return c


FULL = config([(mixer(), moe()), (mixer(heads=3, kv=3, dim=12, vdim=20,
                                        rot=12, rh=1, rdim=16, rvdim=8),
                                  None), 0, (mixer(heads=6, kv=1, rot=6,
                                                   factor=1.0, rh=5, rdim=6,
                                                   rvdim=9), dense(32)), 1, 0])
# sizes that take the vector loads, the matrix cores and the fused experts
WIDE = config([(mixer(heads=4, kv=2, dim=32, vdim=64, rot=32, scale=0.15,
                      rh=2, rdim=48, rvdim=72), moe(n=64, shared=32)),
               (mixer(heads=2, kv=1, dim=24, vdim=136, rot=20, rh=3, rdim=20,
                      rvdim=64), dense(48)), 0], width=96, streams=2)


def engine(cfg, W, target, tokens=512, slots=4, page=4, **kw):
    dev, dt = target
    e = Engine(redirax_config_from_json(cfg), device=dev, dtype=dt,
               page_size=page, kv_token_capacity=tokens,
               max_running_requests=slots,
               max_num_batched_tokens=kw.pop("budget", 1 << 20), **kw)
    e.model.load_state_dict(W)
    return e


def close(got, want, target, what="", deep=False):
    """Logit rows agree: error (mean removed, RMS over the vocabulary) over
    the oracle's own spread.  In models with a router (``deep``) bf16 may
    turn a close choice of experts on some rows, so there one row in ten may
    be off by more than the limit; fp32 is the sharp comparison."""
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape, f"{what}: {got.shape} vs {want.shape}"
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / want.std(-1).clamp_min(1e-6)
    say = f"{what}: {float(err.max()):.3g} at row {int(err.argmax())}"
    if target[1] == torch.float32:
        assert float(err.max()) < 2e-4, say
    elif not deep:
        assert float(err.max()) < 0.12, say
    else:
        assert float(err.median()) < 0.05, say
        assert int((err > 0.12).sum()) <= max(2, err.numel() // 10), say


def toks(n, seed=0, avoid=()):
    g = torch.Generator().manual_seed(seed)
    t = torch.randint(0, VOCAB, (n,), generator=g).tolist()
    return [x if x not in avoid else (x + 7) % VOCAB for x in t]


def run(e, rid, t, want=None, end=True):
    want = list(range(len(t))) if want is None else want
    return e.step_forced([(rid, t, want)], [rid] if end else [])


def decode_after(e, rid, t, cut):
    rows = [e.step_forced([(rid, t[:cut], list(range(cut)))], [])]
    rows += [e.step_forced([(rid, [x], [0])], []) for x in t[cut:]]
    e.step_forced([], [rid])
    return torch.cat(rows)


def in_portions(e, rid, t, sizes):
    rows, at, i = [], 0, 0
    while at < len(t):
        n = min(sizes[i % len(sizes)], len(t) - at)
        rows.append(e.step_forced([(rid, t[at:at + n], list(range(n)))], []))
        at += n
        i += 1
    e.step_forced([], [rid])
    return torch.cat(rows)


# ------------------------------------------------------- mechanisms alone
ALONE = [
    ("plain", mixer(), None, {}),
    ("one-head-each", mixer(heads=1, kv=1, dim=4, vdim=3, rot=2, rh=1, rdim=3,
                            rvdim=2), None, dict(width=24)),
    ("all-rotated-factor-one", mixer(rot=16, factor=1.0), None, {}),
    ("no-rotation", mixer(rot=0), None, {}),
    ("odd-sizes", mixer(heads=3, kv=3, dim=11, vdim=7, rot=6, rh=7, rdim=5,
                        rvdim=3), None, dict(width=26)),
    ("one-kv-head-wide-values", mixer(heads=5, kv=1, dim=8, vdim=48, rot=4),
     None, {}),
    ("big-heads", mixer(heads=2, kv=1, dim=136, vdim=72, rot=34, scale=0.1,
                        rh=1, rdim=130, rvdim=70), None, {}),
    ("values-200", mixer(heads=2, kv=2, dim=48, vdim=200, rot=48, rh=2,
                         rdim=96, rvdim=128), None, {}),
    ("values-256", mixer(heads=2, kv=1, dim=128, vdim=256, rot=64, scale=0.1,
                         rh=1, rdim=64, rvdim=192), None, {}),
    ("key-300", mixer(rh=2, rdim=300, rvdim=20), None, {}),
    ("decays-zero-and-one", mixer(rh=2, decay=[0.0, 1.0]), None, {}),
    ("one-stream", mixer(), dense(), dict(streams=1)),
    ("four-streams", mixer(), dense(30), dict(streams=4, width=36)),
    ("six-streams", mixer(), dense(30), dict(streams=6, width=37)),
    ("ten-streams", mixer(), dense(), dict(streams=10)),
    ("no-cap", mixer(), dense(18), dict(cap=0)),
    ("experts", mixer(), moe(), {}),
    ("experts-32", mixer(), moe(n=32, shared=64), dict(width=64)),
    ("experts-no-shared", mixer(), moe(shared=0), {}),
    ("experts-one-of-one", mixer(), moe(experts=1, top=1), {}),
    ("experts-all", mixer(), moe(experts=3, top=3, limit=0.3, slimit=2.0),
     {}),
]


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name,m,f,kw", ALONE, ids=[a[0] for a in ALONE])
def test_mechanism_alone(target, name, m, f, kw):
    cfg = config([(m, f)], **kw)
    W = O.random_weights(cfg, seed=3)
    t = toks(37, seed=1)
    e = engine(cfg, W, target)
    want = O.forward(cfg, W, t)
    deep = f is not None and f["kind"] == "moe"
    close(run(e, "a", t), want, target, name, deep)
    close(in_portions(e, "b", t, (2, 5, 1)), want, target,
          name + " in portions", deep)


@pytest.mark.parametrize("target", TARGETS)
def test_logit_cap(target):
    W = None
    for cap in (0.5, 0.0):
        cfg = config([(mixer(), None)], cap=cap)
        W = W or O.random_weights(cfg, seed=5)
        t = toks(12, seed=2)
        got = run(engine(cfg, W, target), "a", t)
        close(got, O.forward(cfg, W, t), target, f"cap {cap}")
        assert (float(got.abs().max()) <= 0.5) == (cap > 0)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("cfg", [FULL, WIDE], ids=["full", "wide"])
def test_residual_after_every_layer(target, cfg):
    W = O.random_weights(cfg, seed=7)
    t = toks(17, seed=2)
    e = engine(cfg, W, target)
    e.model.capture_layers = []
    run(e, "a", t)
    want = []
    O.forward(cfg, W, t, collect=want)
    assert len(e.model.capture_layers) == len(want) == len(cfg["layers"])
    for i, got in enumerate(e.model.capture_layers):
        d = (got.double().cpu() - want[i]).abs() / want[i].abs().max()
        if target[1] == torch.float32:
            assert float(d.max()) < 2e-5, f"layer {i}: {float(d.max()):.3g}"
        else:
            d = d.max(-1).values
            assert int((d > 0.1).sum()) <= 2, f"layer {i}: {d}"


@pytest.mark.parametrize("target", TARGETS)
def test_constants_and_choices_show(target):
    """Where random weights might hide a fault: what the engine computes is
    the oracle with these settings, and each other reading of the design
    moves the logits far beyond the tolerance."""
    cfg = config([(mixer(), moe(limit=0.4, slimit=0.3))], streams=2)
    W = O.random_weights(cfg, seed=9)
    t = toks(30, seed=8)
    want = O.forward(cfg, W, t)
    close(run(engine(cfg, W, target), "a", t), want, target, deep=True)

    def moved(change):
        c, w = copy.deepcopy(cfg), dict(W)
        change(c["layers"][0], w)
        d = (O.forward(c, w, t) - want).pow(2).mean(-1).sqrt()
        return float((d / want.std(-1)).max())

    def swap(name):
        def go(L, w):
            w[name] = w[name].t().contiguous()
        return go
    left = lambda L: L["mixer"]["left"]
    for what, change in {
            "mix read as [to, from]": swap("l0.hc1.mix"),
            "rotation factor": lambda L, w: left(L)["rot"]["scaling"].update(
                factor=1.0),
            "rotation base": lambda L, w: left(L)["rot"].update(base=600.0),
            "rotated size": lambda L, w: left(L)["rot"].update(dims=6),
            "limit": lambda L, w: L["mlp"]["expert"].update(limit=0.5),
            "shared limit": lambda L, w: L["mlp"]["shared"].update(limit=0.4),
            "top": lambda L, w: L["mlp"]["router"].update(top=1),
            "router bias": lambda L, w: w.update(
                {"l0.mlp.router.b": -w["l0.mlp.router.b"]}),
            "shared gate": lambda L, w: w.update(
                {"l0.mlp.shared.sg": -w["l0.mlp.shared.sg"]}),
            "decay order": lambda L, w: L["mixer"]["right"]["decay"].reverse(),
            "output bias": lambda L, w: w.update(
                {"l0.mix.left.o.b": -w["l0.mix.left.o.b"]}),
            "key bias": lambda L, w: w.update(
                {"l0.mix.left.k.b": -w["l0.mix.left.k.b"]})}.items():
        assert moved(change) > 2e-3, f"test model hides: {what}"


# ---------------------------------------------- schedules give one answer
@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("cfg", [FULL, WIDE], ids=["full", "wide"])
def test_prefill_decode_and_portions_agree_with_oracle(target, cfg):
    W = O.random_weights(cfg, seed=11)
    t = toks(83, seed=3)
    want = O.forward(cfg, W, t)
    e = engine(cfg, W, target, page=4)
    close(run(e, "whole", t), want, target, "whole", deep=True)
    close(decode_after(e, "dec", t, 1), want, target, "token by token",
          deep=True)
    close(decode_after(e, "dec9", t, 9), want, target, "prefill 9 + decode",
          deep=True)
    for sizes in ((2,), (3, 2, 7), (16, 5), (4,), (13, 1, 1, 2), (11,),
                  (64, 19), (33, 32, 18)):
        close(in_portions(e, f"p{sizes}", t, sizes), want, target,
              f"portions {sizes}", deep=True)
    assert e.kv.free_pages == e.kv.num_pages


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("cfg", [FULL, WIDE], ids=["full", "wide"])
def test_unequal_batch_matches_each_alone(target, cfg):
    W = O.random_weights(cfg, seed=13)
    seqs = {"a": toks(33, seed=4), "b": toks(2, seed=5), "c": toks(19, seed=6),
            "d": toks(1, seed=7)}
    want = {k: O.forward(cfg, W, v) for k, v in seqs.items()}
    e = engine(cfg, W, target, page=4)
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    plan = [{"a": 5, "b": 2, "c": 1, "d": 1}, {"a": 1, "c": 9},
            {"c": 1, "a": 20}, {"a": 1, "c": 8}, {"a": 6}]
    for step in plan:
        entries, end = [], []
        for k, n in step.items():
            entries.append((k, seqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(seqs[k]):
                end.append(k)
        out = e.step_forced(entries, end)
        o = 0
        for k, n in step.items():
            got[k].append(out[o:o + n])
            o += n
    for k in seqs:
        assert at[k] == len(seqs[k])
        close(torch.cat(got[k]), want[k], target, f"request {k}", deep=True)


@pytest.mark.parametrize("target", TARGETS)
def test_pages_and_slots_are_reused_clean(target):
    """A pool of 6 pages and 2 slots serves a stream of requests: every page
    and slot is handed out again with another request's rows and states in
    it."""
    W = O.random_weights(FULL, seed=17)
    e = engine(FULL, W, target, tokens=24, slots=2, page=4)
    for i, n in enumerate((21, 7, 13, 24, 3, 10)):
        t = toks(n, seed=20 + i)
        got = decode_after(e, f"r{i}", t, max(1, n - 3)) if i % 2 else \
            run(e, f"r{i}", t)
        close(got, O.forward(FULL, W, t), target, f"request {i}", deep=True)
        assert e.kv.free_pages == e.kv.num_pages
    a, b = toks(11, seed=40), toks(12, seed=41)
    e.step_forced([("a", a[:6], []), ("b", b[:2], [])], [])
    ga = e.step_forced([("a", a[6:], list(range(5)))], ["a"])
    c = toks(9, seed=42)                     # takes a's pages and slot
    gc = e.step_forced([("c", c, list(range(9))),
                        ("b", b[2:], list(range(10)))], ["c", "b"])
    close(ga, O.forward(FULL, W, a)[6:], target, "a", deep=True)
    close(gc[:9], O.forward(FULL, W, c), target, "c in a's pages", deep=True)
    close(gc[9:], O.forward(FULL, W, b)[2:], target, "b after a pause",
          deep=True)


# --------------------------------------------------- weights of another layer
@pytest.mark.parametrize("target", TARGETS)
def test_shared_weights_have_caches_and_states_of_their_own(target):
    """Two layers on one set of tensors: rows and states per layer run, one
    copy of the weights, and not the result of one layer's cache read
    twice."""
    cfg = config([(mixer(), dense()), 0, 0])
    W = O.random_weights(cfg, seed=19)
    assert not any(k.startswith(("l1.", "l2.")) for k in W)
    e = engine(cfg, W, target)
    assert e.model.layers[0] is e.model.layers[1] is e.model.layers[2]
    assert sorted(e.kv.rows) == [0, 1, 2]
    assert sorted(k for k in e.states.tensors) == [
        (i, "right.S") for i in range(3)]
    t = toks(41, seed=6)
    want = O.forward(cfg, W, t)
    close(run(e, "a", t), want, target, "whole")
    close(decode_after(e, "b", t, 7), want, target, "decoded")
    close(in_portions(e, "c", t, (3, 9)), want, target, "portions")
    one = config([(mixer(), dense())])
    d = (want - O.forward(one, W, t)).pow(2).mean(-1).sqrt() / want.std(-1)
    assert float(d.max()) > 0.1


def test_weights_of_is_checked():
    cfg = config([(mixer(), dense()), 0, (mixer(rh=2), None)])
    redirax_config_from_json(cfg)
    chain = copy.deepcopy(cfg)
    chain["layers"].append(dict(copy.deepcopy(chain["layers"][1]),
                                weights_of=1))
    c = redirax_config_from_json(chain)
    assert [L.weights_of for L in c.layers] == [None, 0, None, 0]
    bad = copy.deepcopy(cfg)
    bad["layers"][1]["weights_of"] = 2
    with pytest.raises(ValueError, match="differs"):
        redirax_config_from_json(bad)
    circle = copy.deepcopy(cfg)
    circle["layers"][0]["weights_of"] = 1
    with pytest.raises(ValueError, match="circle"):
        redirax_config_from_json(circle)
    ahead = copy.deepcopy(cfg)
    ahead["layers"][0]["weights_of"] = 1
    del ahead["layers"][1]["weights_of"]
    c = redirax_config_from_json(ahead)
    m = HybridInferenceModel(c, device="cpu", dtype=torch.float32)
    assert m.layers[0] is m.layers[1] and "l1.norm1" in m._name_map \
        and "l0.norm1" not in m._name_map


# ------------------------------------- keys at borders made visible: loud key
LOUD = 5


def _loud_model(m, width=32):
    """One layer; channel 0 of the normed input is (nearly) one for every
    token, channel 1 for token LOUD only."""
    cfg = config([(m, None)], width=width, streams=2)
    W = O.random_weights(cfg, seed=23)
    W["embed"][:, 0] = 4.0
    W["embed"][:, 1] = 0.0
    W["embed"][LOUD, 1] = 4.0
    W["l0.hc1.in"][:] = 0.5
    W["l0.norm1.alpha"] = torch.tensor(1.0)
    for c in (0, 1):
        W["l0.norm1"][c] = 1.0
        W["l0.norm1.b"][c] = 0.0
    return cfg, W


def _loud_attention(dim=16, vdim=16, rot=8):
    """The last (unrotated) entry of every query head reads the constant
    channel, that of every key head LOUD's channel, and the linear
    attention's share is zero: whoever sees LOUD's key puts nearly all its
    weight on it."""
    cfg, W = _loud_model(mixer(dim=dim, vdim=vdim, rot=rot, scale=1.0))
    p = "l0.mix.left."
    for n, heads, ch in (("q", 4, 0), ("k", 2, 1)):
        for a in range(heads):
            W[p + n][a * dim + dim - 1] = 0.0
            W[p + n][a * dim + dim - 1, ch] = 4.0
            W[p + n + ".b"][a * dim + dim - 1] = 0.0
    W["l0.mix.right.out"].zero_()
    return cfg, W


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("where,vdim", [
    (0, 16), (1, 16), (3, 16), (4, 16), (15, 16), (16, 16), (31, 16),
    (32, 16), (63, 16), (64, 16), (65, 16), (100, 16), (127, 144), (128, 144)])
def test_loud_key_far_behind_and_at_borders(target, where, vdim):
    """LOUD at the start, at page, key-tile and row-tile borders, seen by
    every later token up to 300 positions on and by none before it: in one
    prompt, decoded, across cuts right behind it and in portions."""
    cfg, W = _loud_attention(vdim=vdim)
    n = 300 if where < 4 else where + 45
    t = toks(n, seed=9 + where, avoid=(LOUD,))
    t[where] = LOUD
    want = O.forward(cfg, W, t)
    t2 = list(t)
    t2[where] = LOUD + 1
    d = (want - O.forward(cfg, W, t2)).abs().max(-1).values
    assert float(d[where:].min()) > 0.3, "test model hides the key"
    assert where == 0 or float(d[:where].max()) < 1e-9
    e = engine(cfg, W, target, page=4, tokens=1024)
    close(run(e, "whole", t), want, target, "prompt")
    close(decode_after(e, "dec", t, n - 6), want, target, "decoded")
    for cut in (where + 1, where + 2):
        rows = [e.step_forced([("p", t[:cut], list(range(cut)))], []),
                e.step_forced([("p", t[cut:], list(range(n - cut)))], ["p"])]
        close(torch.cat(rows), want, target, f"cut at {cut}")
    close(in_portions(e, "por", t, (64, 2, 63, 3)), want, target,
          "in portions")


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("shift", [1, 2, 7, 60])
def test_rotation_picks_the_key_at_its_distance(target, shift):
    """Scores made of one turned pair only, the query's pair turned ahead by
    a fixed angle: the weight goes to keys near one distance, so a position
    that is one off, a pair read in the other layout or a wrong frequency
    moves the logits."""
    import math
    f = 1.0 / 40.0
    m = mixer(heads=1, kv=1, dim=4, vdim=16, rot=2, base=10.0, factor=40.0,
              scale=4.0)
    cfg, W = _loud_model(m)
    p = "l0.mix.left."
    for n, ang in (("q", 0.0), ("k", shift * f)):
        W[p + n][:] = 0.0
        W[p + n + ".b"][:] = 0.0
        W[p + n + ".b"][0], W[p + n + ".b"][1] = \
            5 * math.cos(ang), 5 * math.sin(ang)
    W = {k: v.bfloat16().float() for k, v in W.items()}
    W["l0.mix.right.out"].zero_()
    t = toks(90, seed=12)
    want = O.forward(cfg, W, t)
    off = copy.deepcopy(cfg)
    off["layers"][0]["mixer"]["left"]["rot"]["scaling"]["factor"] = 41.0
    d = (want - O.forward(off, W, t)).abs().max()
    assert float(d) > 0.01, "test model hides the frequency"
    e = engine(cfg, W, target)
    close(run(e, "a", t), want, target, "prompt")
    close(decode_after(e, "b", t, 60), want, target, "decoded")


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("rdim,rvdim", [(24, 20), (7, 5), (64, 68)])
def test_recurrence_remembers_its_first_token(target, rdim, rvdim):
    """Keys that only token LOUD writes and decays next to one: LOUD as the
    first token still rules the logits 300 tokens later, so a state that is
    lost, restarted or decayed once too often at a cut, at a chunk border or
    in a slot that is used again shows.  The pool has one slot."""
    cfg, W = _loud_model(mixer(rh=2, rdim=rdim, rvdim=rvdim,
                               decay=[0.9999, 0.995]))
    p = "l0.mix.right."
    W[p + "k"].zero_()
    W[p + "k"][:, 1] = 2.0
    W[p + "q"][:, 0] = 1.0
    W["l0.mix.left.out"].zero_()
    n = 300
    t = [LOUD] + toks(n - 1, seed=33, avoid=(LOUD,))
    t2 = [LOUD + 1] + t[1:]
    want = O.forward(cfg, W, t)
    d = (want - O.forward(cfg, W, t2)).abs().max(-1).values
    assert float(d[-20:].max()) > 0.2 * float(want[-1].std()), \
        "test model forgets its first token"
    faster = copy.deepcopy(cfg)
    faster["layers"][0]["mixer"]["right"]["decay"] = [0.9999, 0.9949]
    d = (want - O.forward(faster, W, t)).abs().max()
    assert float(d) > 2e-3, "test model hides the decay"
    e = engine(cfg, W, target, page=4, tokens=320, slots=1)
    close(run(e, "whole", t), want, target, "one portion")
    close(decode_after(e, "dec", t, n - 5), want, target, "decoded")
    for sizes in ((2, 70, 1, 129), (63, 65), (64,), (128, 1, 2)):
        close(in_portions(e, f"p{sizes}", t, sizes), want, target,
              f"portions {sizes}")
    close(in_portions(e, "twos", t[:40], (2,)), want[:40], target, "in twos")


@pytest.mark.parametrize("target", TARGETS)
def test_fast_decays_over_chunk_borders(target):
    """Heads that forget within a few tokens beside heads that keep all: the
    newest token's share is as right in row 64 as in row 63."""
    cfg = config([(mixer(rh=4, rdim=32, rvdim=32,
                         decay=[0.05, 0.3, 0.9, 1.0]), None)], width=48)
    W = O.random_weights(cfg, seed=29)
    W["l0.mix.left.out"].zero_()
    t = toks(200, seed=30)
    want = O.forward(cfg, W, t)
    e = engine(cfg, W, target)
    close(run(e, "a", t), want, target, "whole")
    close(in_portions(e, "b", t, (65, 64, 63, 2)), want, target, "portions")


@pytest.mark.parametrize("target", TARGETS)
def test_long_portion_beside_short_ones(target):
    """A 280-token portion in one batch with a 3-token and a 1-token
    request."""
    cfg = config([(mixer(), dense()), (mixer(rdim=16, rvdim=16), None)])
    W = O.random_weights(cfg, seed=35)
    a, b, c = toks(281, seed=36), toks(3, seed=37), toks(2, seed=38)
    e = engine(cfg, W, target, page=4, tokens=512)
    e.step_forced([("c", c[:1], [])], [])
    got = e.step_forced([("b", b, [0, 1, 2]), ("a", a[:280], [0, 100, 279]),
                         ("c", c[1:], [0])], ["b", "c"])
    last = e.step_forced([("a", a[280:], [0])], ["a"])
    wa = O.forward(cfg, W, a)
    close(got[:3], O.forward(cfg, W, b), target, "short")
    close(torch.cat([got[3:6], last]), wa[[0, 100, 279, 280]], target, "long")
    close(got[6:], O.forward(cfg, W, c)[1:], target, "single")


@pytest.mark.parametrize("target", TARGETS)
def test_large_batch_of_prompts(target):
    """Prompts of 1 100 rows in one step: many chunks, many row tiles, and
    experts that get hundreds of rows."""
    cfg = config([(mixer(heads=2, kv=1, dim=8, vdim=8, rot=8, rh=2, rdim=8,
                         rvdim=8), moe(n=32, experts=3, top=1, shared=32))],
                 width=32, streams=2)
    W = O.random_weights(cfg, seed=43)
    a, b, c = toks(700, seed=44), toks(385, seed=45), toks(15, seed=46)
    e = engine(cfg, W, target, page=16, tokens=2048)
    wa, wb, wc = ([3, 63, 64, 65, 699], [0, 65, 384], [0, 14])
    got = e.step_forced([("a", a, wa), ("b", b, wb), ("c", c, wc)],
                        ["a", "b", "c"])
    want = torch.cat([O.forward(cfg, W, s)[w] for s, w in
                      ((a, wa), (b, wb), (c, wc))])
    close(got, want, target, deep=True)


@pytest.mark.parametrize("target", TARGETS)
def test_first_tokens_and_long_decoding(target):
    W = O.random_weights(FULL, seed=31)
    e = engine(FULL, W, target)
    for n in (1, 2, 3, 4):
        t = toks(n, seed=50 + n)
        close(run(e, f"s{n}", t), O.forward(FULL, W, t), target, f"len {n}",
              deep=True)
    t = toks(160, seed=55)
    close(decode_after(e, "long", t, 2), O.forward(FULL, W, t), target,
          "158 decoded tokens", deep=True)


# ------------------------------------- loader, replay entry, generation
def _save(tmp_path, cfg, W):
    from safetensors.torch import save_file
    d = tmp_path / "ckpt"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.bfloat16().contiguous() for k, v in W.items()},
              str(d / "model.safetensors"))
    return str(d)


def test_config_round_trip():
    c = redirax_config_from_json(FULL)
    assert c.streams == 3 and c.norm_kind == "tanh"
    assert c.layers[1].ff is None and c.layers[3].ff.act == "relu"
    assert [L.weights_of for L in c.layers] == [None, None, 0, None, 1, 0]
    r = c.layers[0].mixer.left.rope
    assert r.interleaved and r.linear and r.factor == 2.5
    f = c.layers[0].ff
    assert (f.limit, f.shared_limit, f.shared_ff) == (1.1, 0.7, 28)
    assert redirax_config_from_json(redirax_config_to_json(c)) == c
    for path, value in ((("left", "kv_heads"), 3), (("left", "heads"), 5)):
        bad = copy.deepcopy(FULL)
        bad["layers"][0]["mixer"][path[0]][path[1]] = value
        with pytest.raises((AssertionError, ValueError)):
            redirax_config_from_json(bad)
    bad = copy.deepcopy(FULL)
    bad["layers"][0]["mixer"]["right"]["decay"] = [0.5]
    with pytest.raises(ValueError, match="one decay per head"):
        redirax_config_from_json(bad)


@pytest.mark.parametrize("cfg", [FULL, WIDE], ids=["full", "wide"])
def test_tensor_names(cfg):
    W = O.random_weights(cfg, seed=1)
    m = HybridInferenceModel(redirax_config_from_json(cfg), device="cpu",
                             dtype=torch.float32)
    assert set(m._name_map) == set(W)
    m.load_state_dict(W)
    for k, v in W.items():
        assert torch.equal(m._name_map[k].reshape(v.shape), v), k
    lost = dict(W)
    del lost["l0.hc2.out"]
    with pytest.raises(KeyError, match="l0.hc2.out"):
        m.load_state_dict(lost)


@pytest.mark.parametrize("target", [CPU, GPU32])
def test_folder_loader_and_trace_replay(target, tmp_path, monkeypatch, capsys):
    from polyrl_amd.models import get_model_config
    from polyrl_amd.rollout import trace_replay
    W = O.random_weights(FULL, seed=37)
    path = _save(tmp_path, FULL, W)
    c = get_model_config(path)
    assert c.arch == "redirax" and c.num_hidden_layers == 6
    a, b = toks(13, seed=60), toks(6, seed=61)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:8], "want": [7]},
                                {"id": "b", "tokens": b, "want": [0, 5]}],
         "end": ["b"]},
        {"step": 1, "entries": [{"id": "a", "tokens": a[8:9], "want": []}],
         "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[9:], "want": [3]}],
         "end": ["a"]},
    ]
    monkeypatch.setattr(sys, "stdin",
                        io.StringIO("\n".join(map(json.dumps, steps)) + "\n"))
    out = tmp_path / "out"
    rc = trace_replay.main(["--model", path, "--dtype", "float32", "--out",
                            str(out), "--max-tokens", "128", "--device",
                            target[0]])
    assert rc == 0
    assert capsys.readouterr().out.split() == ["done", "0", "done", "1",
                                               "done", "2"]
    import numpy as np
    wa, wb = O.forward(FULL, W, a), O.forward(FULL, W, b)
    g0 = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4")
                          .reshape(3, -1))
    close(g0, torch.stack([wa[7], wb[0], wb[5]]), target, "step 0", deep=True)
    assert not (out / "1.f32").exists()
    g2 = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4")
                          .reshape(1, -1))
    close(g2, wa[12:13], target, "step 2", deep=True)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("cfg", [FULL, WIDE], ids=["full", "wide"])
def test_greedy_generation_through_the_scheduler(target, cfg):
    """Engine.generate: admission, chunked prompts (token budget of 8),
    mixed steps, sampling at temperature 0, pages and slots released."""
    if target[0] == "cuda":
        from polyrl_amd.ops import seq
        assert seq.seq_extension_loaded()
    W = O.random_weights(cfg, seed=41)
    e = engine(cfg, W, target, slots=3, budget=8)
    prompts = [toks(n, seed=70 + n) for n in (11, 2, 17, 5)]
    outs = e.generate(prompts, SamplingParams(temperature=0.0,
                                              max_new_tokens=5), "g")
    wrong = 0
    for p, o in zip(prompts, outs):
        ids = list(p)
        for got_tok in o.output_ids:
            logits = O.forward(cfg, W, ids)[-1]
            top2 = logits.topk(2).values
            tie = 1e-3 if target[1] == torch.float32 else \
                0.25 * float(logits.std())
            if float(top2[0] - top2[1]) > tie:      # skip near ties
                wrong += got_tok != int(logits.argmax())
            ids.append(got_tok)
        assert len(o.output_ids) == 5 and o.finish_reason == "length"
    # bf16: a close choice of experts may turn one token
    assert wrong <= (0 if target[1] == torch.float32 else 1)
    assert e.kv.free_pages == e.kv.num_pages
    assert e.states.free_slots == e.states.num_slots


def test_registry_preset_runs_and_resumes_memory():
    from polyrl_amd.models import get_model_config
    c = get_model_config("redirax-debug")
    e = Engine(c, device="cpu", dtype=torch.float32, page_size=4,
               kv_token_capacity=64, max_running_requests=2)
    e.model.init_random(seed=1)
    t = toks(9, seed=90)
    a = run(e, "a", t)
    assert a.shape == (9, c.vocab_size) and torch.isfinite(a).all()
    e.release_memory()
    assert not e.kv.rows
    e.resume_memory()
    torch.testing.assert_close(run(e, "b", t), a)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_decode_graph_replays_match_eager_steps(dtype):
    """Pure decode steps replay a captured graph once their batch size has
    recurred: 40 greedy tokens (eager sampling, copies and a host sync
    between the replays) equal the run with every launch issued eagerly,
    also after the batch shrinks to another size.  (In fp32 the experts take
    a host decision, so there the stack is dense.)"""
    cfg = WIDE if dtype == torch.bfloat16 else config(
        [(mixer(), dense()), (mixer(rvdim=16), None), 0])
    W = O.random_weights(cfg, seed=47)
    prompts = [toks(n, seed=80 + n) for n in (9, 3, 14)]
    new = (40, 17, 40)
    outs = {}
    for graphs in (False, True):
        e = engine(cfg, W, ("cuda", dtype), slots=3)
        assert e.enable_hybrid_graphs and e.model.graph_safe_decode(3)
        e.enable_hybrid_graphs = graphs
        for i, (p, n) in enumerate(zip(prompts, new)):
            e.add_request(f"g-{i}", p, SamplingParams(temperature=0.0,
                                                      max_new_tokens=n))
        got = {}
        while e.has_work():
            for o in e.step():
                got[o.rid] = o
        outs[graphs] = [got[f"g-{i}"] for i in range(3)]
        assert sorted(e._graphs) == ([2, 3] if graphs else [])
        assert e.states.free_slots == e.states.num_slots
    for a, b in zip(outs[False], outs[True]):
        assert a.output_ids == b.output_ids
        torch.testing.assert_close(torch.tensor(a.output_logprobs),
                                   torch.tensor(b.output_logprobs),
                                   rtol=1e-5, atol=1e-5)
