"""Bulitar through the engine against the plain implementation (tests/plain_bulitar.py).

Configurations are made here, with sizes that differ from one another wherever the design lets them (query and key/value
head counts, head size and value size either way round, rotations of a part of the head and of the whole, with and without
stretched frequencies, chunks of a page and a half, of a page, of a few tokens and none, taps from one to five, states wider than
high and higher than wide, inner sizes from one to more than sixteen, experts of which a token runs one, some and all, loops that begin
with the first layer, end with the last, run once, twice and three times, layers without a feed-forward).  Host tests run the
engine's own parts, cache and step function on the CPU with the torch operations of tests/torch_backend.py; GPU tests run the
HIP kernels, each kernel against the torch operation of the same name and the whole model in the four trace families, in
float32 (tight) and bfloat16.
"""
import json
import math

import pytest
import torch

import plain_bulitar as plain
import trace_util
from torch_backend import TorchBackend
import torch_backend as ref

from mini_inference_engine_amd.cache import CacheManager, GroupSpec
from mini_inference_engine_amd.config import BulitarConfig, ConfigError, EngineConfig, load_model_config
from mini_inference_engine_amd.engine.batch import StepRow
from mini_inference_engine_amd.engine.runner import ModelRunner
from mini_inference_engine_amd.kernels.api import BiasedBranch
from mini_inference_engine_amd.parts import LayerNorm, RMSNorm, RotaryYarn
from mini_inference_engine_amd.replay.trace import replay
from mini_inference_engine_amd.weights import random_tensors


def rot(dims, base=100.0, factor=None, original=64, fast=8.0, slow=1.0):
    d = dict(base=base, dims=dims)
    if factor is not None:
        d["scaling"] = dict(factor=factor, original=original, fast=fast, slow=slow)
    return d


def att(heads, kv_heads, dim, vdim=None, scale=None, conv=3, rotation=None, chunk=None):
    d = dict(heads=heads, kv_heads=kv_heads, dim=dim, scale=scale if scale is not None else dim ** -0.5,
             rot=rotation or rot(dim, factor=4.0))
    if conv is not None:
        d["conv"] = conv
    if vdim is not None:
        d["vdim"] = vdim
    if chunk is not None:
        d["mask"] = dict(size=chunk)
    return d


def delta(heads, kv_heads, dim, vdim, conv=4, ranks=(6, 5)):
    d = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, decay_rank=ranks[0], gate_rank=ranks[1])
    if conv is not None:
        d["conv"] = conv
    return d


def moe(experts, top, ff, scale=1.5):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, scale=scale))


def layer(mixer, mlp):
    return dict(type="channel_delta" if "decay_rank" in mixer else "attention", mixer=mixer, mlp=mlp)


def loop(start, stop, times):
    return dict(start=start, stop=stop, times=times)


def model(vocab, width, eps, layers, loop=None, emb=1.0):
    d = dict(architecture="Bulitar", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=emb), layers=layers)
    if loop is not None:
        d["loop"] = loop
    return d


A_ATT = att(6, 2, 16, vdim=24, chunk=24, rotation=rot(12, base=50.0, factor=4.0))
A_DELTA = delta(4, 2, 16, 24, ranks=(12, 7))
CFG_A = model(211, 64, 1e-5, [layer(A_ATT, moe(5, 2, 48)), layer(A_DELTA, moe(7, 3, 32, scale=0.8)), layer(A_ATT, None),
                              layer(A_DELTA, None), layer(A_ATT, moe(5, 2, 48))], loop(1, 4, 3), emb=3.0)
# the loop begins with the first layer; chunks of a page and none; plain rotation; one expert a token; a state of one row a column
CFG_B = model(150, 48, 1e-3, [layer(att(4, 4, 24, vdim=8, chunk=16, conv=4, rotation=rot(24)), moe(4, 1, 40)),
                              layer(delta(3, 1, 40, 8, conv=2, ranks=(20, 33)), moe(3, 3, 24)),
                              layer(att(4, 1, 8, conv=None, rotation=rot(4, factor=3.0)), moe(6, 2, 16, scale=3.0)),
                              layer(delta(2, 2, 8, 48, conv=5, ranks=(1, 1)), None)], loop(0, 2, 2))
# sizes the kernels' vector paths do not like: nothing a multiple of 8, an odd vocabulary; the loop runs once, to the last layer
CFG_C = model(101, 70, 1e-6, [layer(delta(2, 1, 10, 13, conv=1, ranks=(3, 17)), moe(5, 5, 26)),
                              layer(att(3, 1, 10, vdim=14, conv=1, chunk=5, rotation=rot(6, factor=2.0)), None),
                              layer(delta(5, 5, 7, 6, conv=3), moe(9, 2, 18)),
                              layer(att(6, 3, 18, vdim=6, conv=2, chunk=1), moe(3, 1, 22))], loop(2, 4, 1), emb=0.5)
# wider heads and states, eight query heads on one key head, chunks longer than most requests, no loop
CFG_D = model(333, 96, 1e-4, [layer(delta(4, 1, 100, 72, ranks=(24, 16)), moe(9, 3, 32)),
                              layer(att(8, 1, 40, vdim=56, conv=4, chunk=100), moe(6, 2, 48)),
                              layer(delta(2, 2, 64, 130, conv=3, ranks=(16, 48)), None),
                              layer(att(4, 2, 64, chunk=70, rotation=rot(32, base=1000.0, factor=16.0, original=128)), moe(9, 3, 32))], emb=7.0)
CONFIGS = {"A": (CFG_A, 3), "B": (CFG_B, 4), "C": (CFG_C, 6), "D": (CFG_D, 8)}


def shape_weights(cfg, seed, sharp=True):
    """Random weights shaped so that faults show: products keep the scale of their input, norm weights, biases and step vectors are
    far from their resting values, convolutions look back as much as at the token itself, decays range from fast to slow, routers
    are decisive and their corrections move the choice.  ``sharp`` False leaves scores and routers at unit scale: the bfloat16 runs
    use it, because spread scores amplify the rounding of 8-bit values as much as they amplify faults."""
    w = random_tensors(cfg, seed, torch.float32, std=1.0)
    g = torch.Generator().manual_seed(seed + 100)
    draw = lambda v: torch.randn(v.shape, generator=g)        # noqa: E731
    for k, v in w.items():
        if k.endswith((".q.b", ".k.b", ".v.b", ".o.b", ".correction")):
            v.copy_(draw(v) * 0.4)
        elif k == "loop.step":
            v.copy_(draw(v))
        elif k.endswith(".conv"):
            v.copy_(draw(v) * v.shape[-1] ** -0.5)
        elif k.endswith(".A_log"):
            v.copy_(draw(v))
        elif k.endswith(".dt_bias"):
            v.copy_(draw(v) * 2.0 - 2.0)
        elif "norm" in k:
            v.copy_(1.0 + 0.4 * draw(v))
        elif v.dim() >= 2:
            v.mul_(v.shape[-1] ** -0.5)
        if k.endswith(".router") and sharp:
            v.mul_(3.0)
    if sharp:
        for k, v in w.items():
            if k.endswith(".mix.q") and k[:-1] + "o.b" in w:
                v.mul_(1.5)
    return w


def make(name, dtype=torch.float32, sharp=True):
    raw, seed = CONFIGS[name]
    cfg = BulitarConfig.from_dict(raw)
    return raw, cfg, {k: v.to(dtype) for k, v in shape_weights(cfg, seed, sharp).items()}


def expected_logits(raw, weights, prompts):
    wf = {k: v.float() for k, v in weights.items()}
    return {rid: plain.forward(raw, wf, toks) for rid, toks in prompts.items()}


def host_runner(cfg, weights, pages=64, rows=8, tokens=256, slots=None):
    return ModelRunner(cfg, weights=weights, dtype="float32", device="cpu", backend=TorchBackend(torch.float32),
                       num_pages=pages, max_rows=rows, max_step_tokens=tokens, max_model_len=pages * 16, num_state_slots=slots)


def make_runner(device, cfg, w, pages, rows, tokens, dtype="float32"):
    if device == "cpu":
        return host_runner(cfg, w, pages=pages, rows=rows, tokens=tokens)
    return ModelRunner(cfg, weights=w, dtype=dtype, num_pages=pages, max_rows=rows, max_step_tokens=tokens,
                       max_model_len=(pages - 1) * 16)


# float32 against the float64 plain implementation: rounding, amplified by scores that are spread on purpose; a fault
# (a lost key, a chunk that is one position off, a lost state, a wrong expert) moves logits by a hundred times this
F32_TOL = 2e-4
# bfloat16: every sublayer rounds a handful of values to 8 bits
BF16_TOL_PER_LAYER = 1.5e-2

FAMILIES = {"whole": trace_util.whole, "decode_tail": lambda p: trace_util.decode_tail(p, 40),
            "portions": trace_util.portions, "mixed": lambda p: trace_util.mixed(p, 4, seed=5)}
LENGTHS = [3, 70, 1, 37, 90, 18, 49]


def compare_most(got, expected, tol, what, over=0.1, cap=1.0):
    """The bfloat16 comparison.  A token whose router scores nearly tie may choose another expert once values are rounded
    to 8 bits, and then its logits (and, weakly, those after it) differ by design, not by fault: at most ``over`` of the
    rows may exceed ``tol``, none may exceed ``cap`` of the logit scale or be other than finite."""
    errs = []
    for (rid, p), row in got.items():
        err = float((row.double().cpu() - expected[rid][p]).abs().max()) / float(expected[rid].abs().max())
        assert math.isfinite(err) and err <= cap, f"{what}: request {rid} position {p}: error {err:.3e} of the logit scale"
        errs.append(err)
    bad = sum(e > tol for e in errs)
    assert errs and bad <= over * len(errs), f"{what}: {bad} of {len(errs)} rows beyond {tol:.1e} of the logit scale (worst {max(errs):.1e})"
    return max(errs)


def layer_runs(raw):
    return len(plain.run_order(raw))


def run_family(name, family, tmp_path, device, dtype, tol):
    raw, cfg, weights = make(name, torch.float32 if dtype == "float32" else torch.bfloat16, sharp=dtype == "float32")
    prompts = trace_util.random_prompts(raw["vocab"], LENGTHS, seed=17)
    steps = FAMILIES[family](prompts)
    peak = trace_util.live_token_peak(steps)
    pages = peak // 16 + 1 + 4
    backend = TorchBackend(torch.float32) if device == "cpu" else None
    runner = ModelRunner(cfg, weights=weights, dtype=dtype, device=device, backend=backend, num_pages=pages, max_rows=4,
                         max_step_tokens=max(64, peak), max_model_len=(pages - 1) * 16, num_state_slots=5)
    if family == "mixed":
        assert peak < sum(-(-n // 64) * 64 for n in LENGTHS), "the pool must be smaller than all requests together"
    replay(runner, trace_util.to_lines(steps), str(tmp_path), lambda _: None, max_live=4)
    runner.cache.check()
    assert not runner.cache.live
    got = trace_util.read_outputs(str(tmp_path), steps, raw["vocab"])
    check = trace_util.compare if dtype == "float32" else compare_most
    return check(got, expected_logits(raw, weights, prompts), tol, f"bulitar {name}/{family}/{dtype}")


# ------------------------------------------------------------------------------------------- configuration
def test_config_round_trip_registry_and_sizes_from_tensor_shapes(tmp_path):
    from safetensors.torch import save_file
    for name in CONFIGS:
        raw, cfg, weights = make(name)
        assert BulitarConfig.from_dict(cfg.to_dict()) == cfg
        # the inner sizes of the low-rank products are in no key of a checkpoint's file: they come from its tensors
        bare = json.loads(json.dumps(raw))
        for entry in bare["layers"]:
            entry["mixer"].pop("decay_rank", None), entry["mixer"].pop("gate_rank", None)
        folder = tmp_path / name
        folder.mkdir()
        (folder / "config.json").write_text(json.dumps(bare))
        save_file({k: v.contiguous() for k, v in weights.items()}, str(folder / "model.safetensors"))
        loaded, arch = load_model_config(str(folder))
        assert loaded == cfg and arch.name == "Bulitar"
        with pytest.raises(ConfigError):
            BulitarConfig.from_dict(bare)
    a, b, c, d = (BulitarConfig.from_dict(CONFIGS[n][0]) for n in "ABCD")
    assert a.run_order() == [(0, None), (1, 0), (2, None), (3, None), (1, 1), (2, None), (3, None), (1, 2), (2, None), (3, None), (4, None)]
    assert b.run_order()[:4] == [(0, 0), (1, None), (0, 1), (1, None)] and c.run_order()[2:] == [(2, 0), (3, None)]
    assert d.loop is None and d.run_order() == [(i, None) for i in range(4)] and a.embedding_scale == 3.0
    assert a.layers[0].mixer.vdim == 24 and a.layers[0].mixer.chunk == 24 and a.layers[2].mlp is None
    assert b.layers[2].mixer.taps is None and b.layers[2].mixer.chunk is None and b.layers[0].mixer.rot.scaling is None
    assert (b.layers[1].mixer.decay_rank, b.layers[1].mixer.gate_rank) == (20, 33) and b.layers[2].mlp.scale == 3.0


@pytest.mark.parametrize("bad", [
    lambda c: c["layers"][0]["mixer"].update(kv_heads=4),                  # 6 query heads over 4 key heads
    lambda c: c["layers"][1]["mixer"].update(kv_heads=3),                  # 4 heads over 3
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18),              # more than the head
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3),
    lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0.0),
    lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"),
    lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
    lambda c: c["layers"][0]["mixer"].update(conv=0),
    lambda c: c["layers"][0]["mixer"].pop("scale"),
    lambda c: c["layers"][1]["mixer"].update(decay_rank=0),
    lambda c: c["layers"][1]["mixer"].update(gate_rank=True),
    lambda c: c["layers"][0]["mlp"]["router"].update(top=6),               # more than there are experts
    lambda c: c["layers"][0]["mlp"].update(kind="dense"),
    lambda c: c["layers"][0].update(type="mlstm"),
    lambda c: c["loop"].update(stop=6),
    lambda c: c["loop"].update(start=4),
    lambda c: c["loop"].update(times=0),
    lambda c: c["norm"].update(eps=0.0),
    lambda c: c.update(layers=[]),
])
def test_config_refuses_what_cannot_be_computed(bad):
    raw = json.loads(json.dumps(CFG_A))
    bad(raw)
    with pytest.raises(ConfigError):
        BulitarConfig.from_dict(raw)


def test_model_structure():
    _, cfg, weights = make("A")
    runner = host_runner(cfg, weights)
    m = runner.model
    assert tuple(weights["l0.mix.q.conv"].shape) == (96, 3) and tuple(weights["l0.mix.v.conv"].shape) == (48, 3)
    assert tuple(weights["l0.mix.v.b"].shape) == (48,) and tuple(weights["l0.mix.o.b"].shape) == (64,) and "l0.mix.q.norm" not in weights
    assert tuple(weights["l1.mix.q"].shape) == (32, 64) and tuple(weights["l1.mix.v"].shape) == (96, 64) and tuple(weights["l1.mix.b"].shape) == (4, 64)
    assert tuple(weights["l1.mix.a2"].shape) == (64, 12) and tuple(weights["l1.mix.g2"].shape) == (96, 7) and tuple(weights["l1.mix.norm"].shape) == (24,)
    assert tuple(weights["loop.in"].shape) == (64, 128) and tuple(weights["loop.step"].shape) == (3, 64)
    assert "l2.norm2" not in weights and "l2.mlp.router" not in weights and "l0.norm1.b" not in weights
    assert tuple(weights["l1.mlp.e6.gate"].shape) == (32, 64) and "l1.mlp.e7.gate" not in weights
    # every layer run has a cache of its own; one page group, for the chunk; a model with a state takes no padding tokens
    assert len(m.spec.schedule) == 11 and len(m.cache_entries) == 11 and m.page_groups == [24] and not m.padding_safe
    assert [call.turn for call in m.spec.schedule if call.entry is not None] == [0, 1, 2]
    assert len({id(call.entry) for call in m.spec.schedule if call.entry is not None}) == 1
    # the delta rule's rows of the input product start on multiples of 16, and its inner sizes are padded to them
    d = m.spec.layers[1].mixer
    assert (d.channels, d.beta_col, d.decay_col, d.gate_col, d.columns) == (160, 160, 176, 192, 208)
    assert tuple(d.w_in.shape) == (208, 64) and tuple(d.w_decay.shape) == (64, 16) and float(d.w_decay[:, 12:].abs().max()) == 0.0


# ------------------------------------------------------------------- the plain implementation against small sums by hand
def test_plain_rotation_and_mask_by_hand():
    # pairs that turn often keep their frequency, pairs that hardly turn are slowed down by the factor, the ramp lies between
    freqs, size = plain.yarn_frequencies(10000.0, 16, dict(factor=4.0, original=512, fast=8.0, slow=1.0))
    n = lambda t: 16 * math.log(512 / (2 * math.pi * t)) / (2 * math.log(10000.0))        # noqa: E731
    assert math.floor(n(8.0)) == 2 and math.ceil(n(1.0)) == 4
    for i, f in enumerate(freqs):
        share = 0.0 if i <= 2 else 0.5 if i == 3 else 1.0
        assert abs(f - 10000.0 ** (-2 * i / 16) * (share / 4.0 + 1 - share)) < 1e-12
    assert abs(size - (0.1 * math.log(4.0) + 1.0)) < 1e-12
    x = torch.randn(5, 2, 20, dtype=torch.float64)
    y = plain.turn_neighbours(x, torch.arange(5), freqs, size)
    assert torch.equal(y[..., 16:], x[..., 16:])
    a = 3 * freqs[5]
    assert abs(float(y[3, 1, 10] - size * (x[3, 1, 10] * math.cos(a) - x[3, 1, 11] * math.sin(a)))) < 1e-12
    assert abs(float(y[3, 1, 11] - size * (x[3, 1, 11] * math.cos(a) + x[3, 1, 10] * math.sin(a)))) < 1e-12
    seen = plain.visible(9, dict(size=3))
    assert [[j for j in range(9) if seen[i, j]] for i in (0, 2, 3, 7, 8)] == [[0], [0, 1, 2], [3], [6, 7], [6, 7, 8]]
    assert [j for j in range(9) if plain.visible(9, None)[7, j]] == list(range(8))
    ln = plain.layer_norm(torch.tensor([[1.0, 3.0]], dtype=torch.float64), torch.tensor([2.0, 5.0], dtype=torch.float64), 3.0)
    assert torch.allclose(ln, torch.tensor([[-1.0, 2.5]], dtype=torch.float64))


def test_engine_rotation_equals_the_plain_one():
    for dims, base, factor, original, fast, slow in ((16, 10000.0, 4.0, 512, 8.0, 1.0), (6, 20.0, 2.0, 1024, 4.0, 0.5), (48, 1e6, 1.0, 4096, 32.0, 1.0)):
        part = RotaryYarn(dims, base, factor, original, fast, slow, layout="interleaved")
        freqs, size = plain.yarn_frequencies(base, dims, dict(factor=factor, original=original, fast=fast, slow=slow))
        assert part.layout == "interleaved" and torch.allclose(part.frequencies(), torch.tensor(freqs, dtype=torch.float64), rtol=1e-12)
        assert abs(part.magnitude - size) < 1e-12
    assert RotaryYarn(8, 100.0, 2.0, 64, 8.0, 1.0).layout == "half"
    with pytest.raises(ValueError):
        RotaryYarn(8, 100.0, 2.0, 64, 8.0, 1.0, layout="thirds")


def test_plain_delta_rule_router_and_loop_by_hand():
    t = lambda *x: torch.tensor(x, dtype=torch.float64)        # noqa: E731
    # two key channels, one value: the state decays channel by channel, then the write replaces a share of what the key reads
    k = t(t(1, 0).tolist(), t(0.6, 0.8).tolist())[:, None, :]
    q, v = t([0, 1], [1, 1])[:, None, :], t([2], [5])[:, None, :]
    g = t([0.5, 0.5], [0.25, 0.5])[:, None, :]
    o, S = plain.delta_scan(q, k, v, g, t([1.0], [0.5]))
    assert float(o[0]) == 0.0                               # the first write is in channel 0, the query asks channel 1
    u = 0.5 * (5 - 0.6 * 0.25 * 2)                          # reads the decayed state
    assert torch.allclose(S[0, :, 0], t(0.25 * 2 + 0.6 * u, 0.8 * u)) and abs(float(o[1]) - float(S.sum())) < 1e-12
    assert torch.allclose(plain.unit(t([3.0, 4.0])), t([0.6, 0.8]), atol=1e-7)
    # decays by hand: one head of two channels
    W = {"m.a1": t([2.0]), "m.a2": t([1.0], [-1.0]), "m.dt_bias": t(0.0, 1.0), "m.A_log": t(math.log(3.0))}
    W["m.A_log"] = W["m.A_log"].view(1)
    dec = plain.channel_decay(t([0.5]), W, "m", 1, 2)
    sp = lambda z: math.log1p(math.exp(z))        # noqa: E731
    assert torch.allclose(dec[0, 0], t(math.exp(-3 * sp(1.0)), math.exp(-3 * sp(0.0))))
    # the convolution's last column is the token's own
    x = torch.arange(1.0, 5.0, dtype=torch.float64)[:, None]
    assert plain.short_conv(x, t([10.0, 1.0]))[:, 0].tolist() == [1.0, 12.0, 23.0, 34.0]
    # router: the correction moves the choice, not the weights, which are not made to sum to one
    W = {"m.router": torch.eye(3, dtype=torch.float64), "m.correction": t(0.0, -1.0, 0.0)}
    picked, share = plain.choose(t([1.0, 2.0, 0.5]), W, "m", 2, 2.5)
    assert picked.tolist() == [[0, 2]] and torch.allclose(share, 2.5 * torch.sigmoid(t([1.0, 0.5])))
    # before a pass: a product of stream and embedding, then the pass's vector
    W = {"loop.in": t([1.0, 10.0]), "loop.step": t([0.5], [7.0])}
    assert torch.equal(plain.begin_pass(t([3.0]), t([2.0]), W, 1), t([30.0]))
    assert plain.run_order(CFG_B) == [(0, 0), (1, None), (0, 1), (1, None), (2, None), (3, None)]


def test_router_margins_of_the_test_models():
    """The float32 comparisons are only fair if no token of the test prompts sits on a routing boundary."""
    for name in CONFIGS:
        raw, _, weights = make(name)
        margins = []
        for toks in trace_util.random_prompts(raw["vocab"], LENGTHS, seed=17).values():
            plain.forward(raw, weights, toks, margins=margins)
        assert margins and min(margins) > 1e-6, f"{name}: a token is routed with a margin of {min(margins):.1e}"


# ------------------------------------------------------------------------------------- mechanisms, one by one
def one_layer(mixer, mlp, width=32, vocab=50, eps=1e-5, **kw):
    return model(vocab, width, eps, [layer(mixer, mlp)], **kw)


MECHANISMS = {
    "attention": one_layer(att(4, 2, 8, vdim=12, chunk=6), None),
    "attention-all-keys": one_layer(att(2, 2, 16, vdim=4, conv=4), None),
    "attention-chunk-of-one": one_layer(att(2, 1, 8, chunk=1, conv=2), None),
    "attention-chunk-of-a-page": one_layer(att(2, 1, 8, chunk=16), None),
    "attention-no-convolution": one_layer(att(3, 1, 8, conv=None, rotation=rot(8), chunk=9), None),
    "attention-one-tap": one_layer(att(1, 1, 24, vdim=40, conv=1, rotation=rot(6, factor=3.0)), None),
    "attention-large-eps": one_layer(att(2, 1, 8, chunk=20), None, eps=0.5),
    "delta": one_layer(delta(4, 2, 8, 12), None),
    "delta-one-head-rank-one": one_layer(delta(1, 1, 20, 4, conv=2, ranks=(1, 1)), None),
    "delta-a-key-head-a-head": one_layer(delta(3, 3, 6, 10, conv=1, ranks=(17, 2)), None),
    "delta-no-convolution": one_layer(delta(2, 1, 5, 5, conv=None, ranks=(4, 40)), None),
    "delta-large-eps": one_layer(delta(2, 1, 8, 8), None, eps=0.5),
    "experts": one_layer(delta(1, 1, 8, 8), moe(6, 2, 24)),
    "experts-all-of-them": one_layer(delta(1, 1, 8, 8), moe(4, 4, 20, scale=1.0)),
    "experts-one-of-one": one_layer(delta(1, 1, 8, 8), moe(1, 1, 20, scale=0.3)),
    "loop-of-one-pass": one_layer(att(2, 1, 8, chunk=10), None, loop=loop(0, 1, 1)),
    "loop-of-four-passes": one_layer(delta(2, 1, 8, 8), moe(4, 2, 16), loop=loop(0, 1, 4), emb=2.0),
    "loop-in-the-middle": model(50, 32, 1e-5, [layer(att(2, 1, 8), None), layer(delta(1, 1, 8, 8), None), layer(att(2, 1, 8, chunk=7), None),
                                               layer(delta(1, 1, 8, 8), None)], loop(1, 3, 2), emb=5.0),
    "scaled-embedding": one_layer(att(2, 1, 8), None, emb=20.0),
}


@pytest.mark.parametrize("name", list(MECHANISMS))
def test_each_mechanism_alone_on_the_host(name):
    raw = MECHANISMS[name]
    cfg = BulitarConfig.from_dict(raw)
    weights = shape_weights(cfg, 1)
    runner = host_runner(cfg, weights, pages=8, rows=2, tokens=64)
    toks = trace_util.random_prompts(raw["vocab"], [49], seed=2)["r0"]
    want = plain.forward(raw, weights, toks)
    rc = runner.cache.open("a")
    pos, rows = 0, []
    for n in (11, 1, 2, 15, 20):                              # a portion, a single token, two tokens, the rest in two
        assert runner.cache.reserve(rc, pos, n)
        row = StepRow(rc, toks[pos:pos + n], pos, list(range(n)))
        rows.append(runner.forward_step([row]))
        runner.after_step([row])
        pos += n
    got = torch.cat(rows).double()
    assert float((got - want).abs().max()) < 2e-5 * float(want.abs().max())


def test_a_backend_that_leaves_the_adds_to_the_caller():
    """Biases, step vectors and branch outputs still reach the stream where no product adds into it."""
    raw, cfg, weights = make("A")
    runner = ModelRunner(cfg, weights=weights, dtype="float32", device="cpu", backend=TorchBackend(torch.float32, adds_in_place=False),
                         num_pages=16, max_rows=2, max_step_tokens=64, max_model_len=256)
    prompts = trace_util.random_prompts(raw["vocab"], [40], seed=2)
    got = trace_util.run_on_runner(runner, trace_util.portions(prompts))
    trace_util.compare(got, expected_logits(raw, weights, prompts), F32_TOL, "adds by the caller")


def test_a_pending_bias_reaches_every_reader_of_the_stream():
    ops = TorchBackend(torch.float32)
    g = torch.Generator().manual_seed(1)
    stream, y, b = torch.randn(5, 8, generator=g), torch.randn(5, 8, generator=g), torch.randn(8, generator=g)
    for norm in (LayerNorm(8, 1e-5, "n", has_bias=False), RMSNorm(8, 1e-5, "n")):
        norm.ops, norm.weight = ops, torch.randn(8, generator=g)
        for value in (y, None):
            total = stream + b if value is None else stream + y + b
            s = stream.clone()
            got = norm.forward(BiasedBranch(value, b), s)
            assert torch.allclose(s, total, atol=1e-6) and torch.allclose(got, norm.forward(None, total.clone()), atol=1e-5)
            s, rows = stream.clone(), torch.tensor([3, 1], dtype=torch.int32)
            got = norm.lazy(BiasedBranch(value, b), s, rows=rows).materialize()
            assert torch.allclose(got, norm.forward(None, total.clone())[rows.long()], atol=1e-5)
            assert torch.allclose(stream + BiasedBranch(value, b).float(), total, atol=1e-6)


def changed(raw, weights, toks, change):
    """How far the plain implementation's logits move, of their scale, when ``change`` is made to a copy of the weights."""
    other = {k: v.clone() for k, v in weights.items()}
    change(other)
    want = plain.forward(raw, weights, toks)
    return float((plain.forward(raw, other, toks) - want).abs().max()) / float(want.abs().max())


def test_every_mechanism_shows_in_the_logits_of_the_test_models():
    """The test weights are such that leaving a mechanism out would be seen far above the tolerances."""
    raw, _, weights = make("A")
    toks = trace_util.random_prompts(raw["vocab"], [60], seed=3)["r0"]
    zero = lambda name: (lambda w: w[name].zero_())            # noqa: E731
    for name in ("l0.mix.q.b", "l0.mix.k.b", "l2.mix.v.b", "l4.mix.o.b", "l1.mix.A_log", "l3.mix.dt_bias", "l1.mix.b", "l1.mix.a2", "l3.mix.g2",
                 "l1.mlp.correction", "loop.step"):
        assert changed(raw, weights, toks, zero(name)) > 20 * F32_TOL, f"{name} hardly shows"
    for name in ("l0.mix.q.conv", "l0.mix.v.conv", "l4.mix.k.conv", "l1.mix.q.conv", "l3.mix.v.conv"):
        assert changed(raw, weights, toks, lambda w: w[name][:, 0].zero_()) > 20 * F32_TOL, f"{name}: its furthest tap hardly shows"
    assert changed(raw, weights, toks, lambda w: w["loop.in"][:, 64:].zero_()) > 20 * F32_TOL, "the embedding in the loop hardly shows"
    assert changed(raw, weights, toks, lambda w: w["loop.step"].copy_(w["loop.step"][[0, 0, 2]])) > 20 * F32_TOL, "the pass's own vector hardly shows"


def test_prefill_equals_token_by_token_decoding():
    raw, cfg, weights = make("A")
    prompts = trace_util.random_prompts(raw["vocab"], [60], seed=21)
    whole = trace_util.run_on_runner(host_runner(cfg, weights), trace_util.whole(prompts))
    single = trace_util.run_on_runner(host_runner(cfg, weights), trace_util.decode_tail(prompts, 59))
    pairs = trace_util.run_on_runner(host_runner(cfg, weights), trace_util.portions(prompts, sizes=(2,)))
    scale = max(float(v.abs().max()) for v in whole.values())
    for key, row in whole.items():
        assert float((single[key] - row).abs().max()) < 2e-5 * scale, f"token by token differs at {key}"
        assert float((pairs[key] - row).abs().max()) < 2e-5 * scale, f"two by two differs at {key}"
    trace_util.compare(whole, expected_logits(raw, weights, prompts), F32_TOL, "whole")


# ------------------------------------------------------------------------------------------ whole models, host
@pytest.mark.parametrize("family", list(FAMILIES))
@pytest.mark.parametrize("name", list(CONFIGS))
def test_families_on_the_host(name, family, tmp_path):
    run_family(name, family, tmp_path, "cpu", "float32", F32_TOL)


def chunk_model(chunk):
    """One attention layer within chunks, a convolution of one tap and no feed-forward: the logits of a position are a function
    of its own token and the earlier ones of its chunk."""
    raw = one_layer(att(3, 1, 16, vdim=8, conv=1, chunk=chunk, scale=0.05), None, width=48, vocab=90)
    cfg = BulitarConfig.from_dict(raw)
    w = shape_weights(cfg, 5)
    w["embed"][89] = 4.0 * w["embed"][89].sign()              # the token that stands out; scores are close: every visible key has a share
    return raw, cfg, w


def chunk_runs(device, dtype="float32"):
    """A token that stands out is put on the last place of a chunk and the first of the next, on a page's last and the next's first
    slot, and at the very start, in a prompt's portion and for tokens decoded one by one.  Where it is visible it must move the
    logits; elsewhere the engine's logits must not move at all; both ways they follow the plain implementation."""
    for chunk in (20, 16, 33):
        raw, cfg, w = chunk_model(chunk)
        if dtype == "bfloat16":
            w = {k: v.to(torch.bfloat16) for k, v in w.items()}
        wf = {k: v.float() for k, v in w.items()}
        base = [t if t != 89 else 0 for t in trace_util.random_prompts(90, [75], seed=9)["r0"]]

        def run(tokens, cut):
            steps = [{"step": 0, "entries": [{"id": "x", "tokens": tokens[:cut], "want": list(range(cut))}], "end": []}]
            steps += [{"step": 1 + i, "entries": [{"id": "x", "tokens": tokens[cut + i:cut + i + 1], "want": [0]}], "end": []}
                      for i in range(len(tokens) - cut)]
            steps[-1]["end"] = ["x"]
            return {k: v.cpu() for k, v in trace_util.run_on_runner(make_runner(device, cfg, w, 8, 2, 80, dtype), steps).items()}

        for cut in (70, 18):                  # asked-for positions in the portion; the chunks' edges among decoded tokens
            plain_run = run(base, cut)
            for needle in (0, 15, 16, chunk - 1, chunk, 2 * chunk - 1, 2 * chunk, 47):
                tokens = list(base)
                tokens[needle] = 89
                want = plain.forward(raw, wf, tokens)
                got = run(tokens, cut)
                trace_util.compare(got, {"x": want}, F32_TOL if dtype == "float32" else 2 * BF16_TOL_PER_LAYER, f"chunk {chunk}, needle at {needle}, portion of {cut}")
                for p in range(75):
                    moved = float((got[("x", p)] - plain_run[("x", p)]).abs().max()) / float(want.abs().max())
                    if p >= needle and p // chunk == needle // chunk:
                        assert moved > 1e-3, f"chunk {chunk}: position {p} must see the token at {needle} (portion of {cut})"
                    else:
                        assert moved == 0.0 if device == "cuda" else moved < 2e-7, \
                            f"chunk {chunk}: position {p} must not see the token at {needle} (portion of {cut}): {moved:.1e}"


def test_keys_at_the_edges_of_the_chunks_on_the_host():
    chunk_runs("cpu")


def far_key_runs(device):
    """One key far back (hundreds of positions, through a dozen pages) is made to decide the attention's output: token 63 has
    the key that token 62, the last one, asks for.  The key stands at a page's last slot, at the next page's first, at the chunk's
    first place and at the very first position; one place before the chunk it decides nothing."""
    for chunk in (None, 300, 100):
        raw = one_layer(att(2, 1, 16, scale=1.0, conv=1, rotation=rot(4, base=1e6), chunk=chunk), None, width=32, vocab=64)
        cfg = BulitarConfig.from_dict(raw)
        w = shape_weights(cfg, 7)
        along = torch.ones(16)
        along[:4] = 0.0                                       # the pairs that turn stay out of it
        w["embed"][:, :2] = 0.0
        w["embed"][62, 1], w["embed"][63, 0] = 20.0, 20.0
        for x in "qk":
            w[f"l0.mix.{x}"].zero_()
            w[f"l0.mix.{x}.b"].copy_(torch.randn(w[f"l0.mix.{x}.b"].shape, generator=torch.Generator().manual_seed(3)))
            w[f"l0.mix.{x}.conv"].fill_(1.0)
        w["l0.mix.q"][:, 1] = 30 * along.repeat(2)
        w["l0.mix.k"][:, 0], w["l0.mix.k"][:, 1] = 30 * along, -30 * along
        toks = [t % 62 for t in trace_util.random_prompts(64, [230], seed=9)["r0"]]
        toks[-1] = 62
        for needle in (0, 31, 32, 199, 200, 207, 208):
            tokens = list(toks)
            tokens[needle] = 63
            want = plain.forward(raw, w, tokens)
            steps = [{"step": 0, "entries": [{"id": "x", "tokens": tokens[:190], "want": [189]}], "end": []}]
            steps += [{"step": 1 + i, "entries": [{"id": "x", "tokens": tokens[190 + i:191 + i], "want": [0]}], "end": []}
                      for i in range(40)]
            steps[-1]["end"] = ["x"]
            got = {k: v.cpu() for k, v in trace_util.run_on_runner(make_runner(device, cfg, w, 16, 2, 192), steps).items()}
            trace_util.compare(got, {"x": want}, F32_TOL, f"chunk {chunk}: far key at {needle}")
            moved = float((plain.forward(raw, w, toks)[-1] - want[-1]).abs().max()) / float(want.abs().max())
            if chunk != 100 or needle >= 200:
                assert moved > 1e-2, "the far key must matter to the last position for this test to mean anything"
            else:
                assert moved == 0.0


def test_a_far_key_and_the_first_token_are_seen():
    far_key_runs("cpu")


def test_state_slots_and_pages_are_used_again():
    """Five requests, one after another, through a runner with one usable state slot and pages for one request: each must
    start from an empty state and see no key of the one before."""
    raw, cfg, weights = make("A")
    prompts = trace_util.random_prompts(raw["vocab"], [40, 33, 40, 7, 25], seed=3)
    runner = ModelRunner(cfg, weights=weights, dtype="float32", device="cpu", backend=TorchBackend(torch.float32),
                         num_pages=4, max_rows=1, max_step_tokens=64, max_model_len=48, num_state_slots=2)
    got = trace_util.run_on_runner(runner, trace_util.portions(prompts, sizes=(5, 2, 9)))
    trace_util.compare(got, expected_logits(raw, weights, prompts), F32_TOL, "reuse")
    states = [(k, t) for e in runner.storage.entries.values() for k, t in e.tensors.items() if k.split(".")[-1] in ("state", "tail")]
    assert len(states) == 5 + 2 * 6                           # attention runs: a tail each; delta runs: a state and a tail
    for _, t in states:
        t.fill_(-2.0)
    rc = runner.cache.open("fresh")
    assert all(float(t[rc.state_slot].abs().max()) == 0.0 for _, t in states)
    runner.cache.close(rc)


def test_pages_before_the_chunk_are_given_back():
    cm = CacheManager(16, [GroupSpec(24, 9, 0)], 3)
    rc = cm.open("a")
    assert cm.reserve(rc, 0, 120)
    cm.advance(rc, 120)
    assert sum(p != 0 for p in rc.tables[0]) == 2
    cm.close(rc)
    # a request that decodes far beyond its chunks keeps what a chunk touches only
    raw = one_layer(att(2, 1, 8, chunk=30), None)
    cfg = BulitarConfig.from_dict(raw)
    w = shape_weights(cfg, 2)
    prompts = trace_util.random_prompts(50, [150], seed=1)
    runner = ModelRunner(cfg, weights=w, dtype="float32", device="cpu", backend=TorchBackend(torch.float32), num_pages=7,
                         max_rows=1, max_step_tokens=64, max_model_len=160)          # six usable pages of 16 for 150 tokens
    got = trace_util.run_on_runner(runner, trace_util.portions(prompts, sizes=(20, 3, 1, 30)))
    trace_util.compare(got, expected_logits(raw, w, prompts), F32_TOL, "pages given back")


def test_long_decoding_carries_the_state():
    """Two hundred tokens one by one through slow decays: what the first tokens wrote is still in the states at the end."""
    raw = one_layer(delta(2, 1, 16, 6, conv=2), None, loop=loop(0, 1, 2))
    cfg = BulitarConfig.from_dict(raw)
    w = shape_weights(cfg, 4)
    w["l0.mix.A_log"].fill_(-6.0)
    w["l0.mix.b"].mul_(0.1)
    prompts = trace_util.random_prompts(50, [200], seed=6)
    got = trace_util.run_on_runner(host_runner(cfg, w, pages=16, rows=1, tokens=64), trace_util.decode_tail(prompts, 199))
    want = expected_logits(raw, w, prompts)
    trace_util.compare(got, want, F32_TOL, "long decoding")
    short = plain.forward(raw, w, prompts["r0"][60:])
    moved = float((short[-1] - want["r0"][-1]).abs().max()) / float(want["r0"].abs().max())
    assert moved > 1e-3, "the first sixty tokens must still matter at the end for this test to mean anything"


def test_batched_rows_equal_rows_alone():
    raw, cfg, weights = make("A")
    prompts = trace_util.random_prompts(raw["vocab"], [21, 5, 34, 1, 50], seed=12)
    alone = {}
    for rid, toks in prompts.items():
        alone.update(trace_util.run_on_runner(host_runner(cfg, weights), trace_util.decode_tail({rid: toks}, 1)))
    runner = host_runner(cfg, weights)
    ents = [{"id": rid, "tokens": toks[:-1], "want": list(range(len(toks) - 1))} for rid, toks in prompts.items() if len(toks) > 1]
    last = [{"id": rid, "tokens": toks[-1:], "want": [0]} for rid, toks in prompts.items()]
    got = trace_util.run_on_runner(runner, [{"step": 0, "entries": ents, "end": []}, {"step": 1, "entries": last, "end": list(prompts)}])
    assert set(got) == set(alone)
    for key, row in alone.items():
        assert float((got[key] - row).abs().max()) < 2e-5 * float(row.abs().max())


def generate(name, device, dtype, lengths=(9, 30, 2, 17, 23), budget=32, blocks=24, **engine):
    from mini_inference_engine_amd import LLMEngine, SamplingParams
    raw, cfg, weights = make(name, torch.float32 if dtype == "float32" else torch.bfloat16, sharp=dtype == "float32")
    prompts = list(trace_util.random_prompts(raw["vocab"], list(lengths), seed=4).values())
    ecfg = EngineConfig(num_blocks=blocks, max_num_seqs=3, max_num_batched_tokens=budget, max_model_len=max(128, max(lengths) + 32), **engine)
    kw = dict(device="cpu", backend=TorchBackend(torch.float32)) if device == "cpu" else {}
    eng = LLMEngine(cfg, ecfg, dtype=dtype, verbose=False, weights=weights, **kw)
    outs = eng.generate(prompts, SamplingParams(max_tokens=30, ignore_eos=True))          # through a chunk's edge
    wf = {k: v.float() for k, v in weights.items()}
    beyond = total = 0
    for prompt, out in zip(prompts, outs):
        ids = list(prompt) + list(out.output_ids)
        assert len(out.output_ids) == 30
        logits = plain.forward(raw, wf, ids)
        for i, tok in enumerate(out.output_ids):
            row = logits[len(prompt) + i - 1]
            slack = (F32_TOL if dtype == "float32" else 2 * BF16_TOL_PER_LAYER * layer_runs(raw)) * float(row.abs().max())
            beyond += float(row.max() - row[tok]) > slack
            total += 1
    # bfloat16: a token whose router nearly ties may run another expert (see compare_most)
    assert beyond <= (0 if dtype == "float32" else 0.1 * total), f"{beyond} of {total} tokens are not the plain implementation's choice"
    return eng


def test_greedy_generation_through_the_scheduler_on_the_host():
    eng = generate("A", "cpu", "float32", use_hip_graphs=False)
    assert eng.num_steps > 30, "five requests under three slots and a budget of 32 tokens come in several waves"


# ----------------------------------------------------------------------------------------------- GPU: kernels
def _rand(shape, dtype, g, scale=1.0):
    return (torch.randn(shape, generator=g) * scale).to(dtype).cuda()


@pytest.fixture(scope="module")
def hip():
    from mini_inference_engine_amd.kernels.hip_backend import HipBackend
    return {torch.float32: HipBackend(torch.float32), torch.bfloat16: HipBackend(torch.bfloat16)}


def close(a, b, tol, what):
    assert bool(torch.isfinite(a.double()).all()), f"{what}: not finite"
    err = float((a.double().cpu() - b.double().cpu()).abs().max()) / max(1e-9, float(b.double().abs().max()))
    assert err <= tol, f"{what}: {err:.3e} of the scale, tolerance {tol:.1e}"


TOL = {torch.float32: 2e-6, torch.bfloat16: 1e-2}


def step_of(rows, slots=None):
    from test_labirax import step_of as make_step
    step = make_step(rows, slots)
    step.num_decode_rows = sum(1 for n in rows if n == 1)
    return step


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_biased_projections_through_a_convolution_kernel(hip, dtype):
    """Rows of one token, of fewer tokens than the convolution looks back, and of many, over tails that hold something; biases before
    the convolution; both pairings; norms after the rotation and before it; sizes that fill no wave."""
    ops, g = hip[dtype], torch.Generator().manual_seed(41)
    for (rows, Hq, Hkv, dim, vdim, K, nf, layout, norm, bias) in (
            ([1, 1, 1], 6, 2, 16, 24, 3, 6, "interleaved", "turned", True), ([37, 1, 2], 3, 3, 24, 8, 4, 12, "interleaved", "turned", True),
            ([2, 3, 1, 70], 4, 1, 10, 14, 5, 3, "interleaved", "turned", True), ([64], 16, 4, 64, 64, 2, 32, "interleaved", "turned", False),
            ([1, 1], 2, 1, 130, 70, 4, 20, "interleaved", "turned", True), ([9, 1], 1, 1, 8, 8, 1, 0, "half", "turned", True),
            ([1, 1, 1], 3, 1, 12, 20, 7, 6, "interleaved", "turned", True), ([80, 3], 4, 2, 48, 80, 3, 9, "half", "turned", True),
            ([70, 1], 5, 5, 18, 6, 2, 9, "interleaved", "head", True), ([1, 1], 2, 2, 20, 4, 2, 3, "interleaved", None, True),
            ([300], 10, 2, 56, 72, 4, 13, "interleaved", "turned", True)):
        T, P = sum(rows), -(-max(dim, vdim) // 16) * 16
        C, q_col = (Hq + Hkv) * dim + Hkv * vdim, 5
        sums = _rand((T, q_col + C + 3), torch.float32, g, 2.0)
        col_bias = _rand((q_col + C + 3,), torch.float32, g) if bias else None
        taps = _rand((C, K), torch.float32, g)
        tail = _rand((len(rows) + 2, max(1, K - 1), C), torch.float32, g)
        qn, kn = (_rand((dim,), torch.float32, g) + 1, _rand((dim,), torch.float32, g) + 1) if norm == "head" else (None, None)
        inv_freq = (50.0 ** -(torch.arange(nf, dtype=torch.float32) / nf)).cuda() if nf else None
        positions = (torch.arange(T, dtype=torch.int32) * 3 + 5).cuda()
        pages, page = T // 16 + 3, 16
        slots = torch.randperm((pages - 1) * page, generator=g)[:T].to(torch.int32).cuda() + page
        if len(rows) == 1:
            slots = (torch.arange(T, dtype=torch.int32) + page).cuda()          # a row's tokens in slots one after another
        kc, vc = torch.full((pages, Hkv, page, P), 7.0, dtype=dtype).cuda(), torch.full((pages, Hkv, P, page), 7.0, dtype=dtype).cuda()
        kw, vw = kc.clone(), vc.clone()
        step = step_of(rows)
        cols = (q_col, q_col + Hq * dim, q_col + (Hq + Hkv) * dim)
        t1, t2 = tail.clone(), tail.clone()
        opts = dict(col_bias=col_bias, norm_per_head=norm == "head", norm_turned=norm == "turned", rotation_scale=1.3)
        want = ref.ref_qkv_finish(sums, *cols, Hq, Hkv, dim, vdim, P, positions, inv_freq, layout, kw, vw, slots, qn, kn, 1e-2, None, dtype,
                                  conv=(taps, t2, step.host["row_start"], step.host["state_slots"]), **opts)
        got = ops.qkv_finish(sums, *cols, Hq, Hkv, dim, vdim, P, positions, inv_freq, layout, kc, vc, slots, q_norm=qn, k_norm=kn, eps=1e-2,
                             conv=(taps, t1, step), **opts)
        what = f"rows {rows}, {Hq}/{Hkv} heads of {dim}/{vdim}, {K} taps, {layout}, norm {norm}"
        tol = 1e-5 if dtype == torch.float32 else TOL[dtype]
        close(got, want, tol, f"queries, {what}")
        close(kc, kw, tol, f"keys, {what}")
        close(vc, vw, tol, f"values, {what}")
        close(t1, t2, 1e-6, f"tails, {what}")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_norm_embedding_and_stream_kernels(hip, dtype):
    """Layer norms without a bias, with a vector that is added to every row of the stream, in place and of gathered rows; the
    embedding's second place; the stream's copy.  Widths on both the vector and the plain path."""
    ops, g = hip[dtype], torch.Generator().manual_seed(42)
    for (T, W) in ((1, 64), (37, 70), (5, 320), (130, 2048), (3, 4096), (2, 5000), (9, 33)):
        stream, x = _rand((T, W), torch.float32, g, 3.0) + 1.5, _rand((T, W), dtype, g)
        w, b, v = _rand((W,), torch.float32, g) + 1, _rand((W,), torch.float32, g), _rand((W,), torch.float32, g)
        rows = torch.tensor([T - 1, 0], dtype=torch.int32).cuda()
        for xx, bias, vec in ((x, None, None), (x, None, v), (None, None, v), (None, b, None), (x, b, v)):
            s1, s2 = stream.clone(), stream.clone()
            what = f"{T}x{W}, add {xx is not None}, bias {bias is not None}, vector {vec is not None}"
            close(ops.add_layernorm(xx, s1, w, bias, 1e-2, out_dtype=torch.float32, rows=rows, x_bias=vec),
                  ref.ref_add_layernorm(xx, s2, w, bias, 1e-2, torch.float32, rows, vec), 2e-6, f"gathered rows {what}")
            assert torch.equal(s1, stream)
            close(ops.add_layernorm(xx, s1, w, bias, 1e-2, x_bias=vec), ref.ref_add_layernorm(xx, s2, w, bias, 1e-2, dtype, None, vec), TOL[dtype], what)
            close(s1, s2, 1e-6, f"the stream, {what}")
            wide = torch.zeros(T, 2 * W + 8, dtype=dtype).cuda()
            s1 = stream.clone()
            ops.stream_copy(xx, s1, wide[:, 8:8 + W], x_bias=vec)
            close(wide[:, 8:8 + W], ref.ref_stream_copy(xx, stream, vec, torch.empty(T, W, dtype=dtype).cuda()), TOL[dtype], f"stream_copy {what}")
            assert torch.equal(s1, stream) and float(wide[:, :8].abs().max()) == 0.0 and float(wide[:, 8 + W:].abs().max()) == 0.0
        s1, s2 = stream.clone(), stream.clone()
        close(ops.branch_layernorm_add(x, s1, w, None, 1e-3, next_norm=(v, None, 1e-3)), ref.ref_branch_layernorm_add(x, s2, w, None, 1e-3, (v, None, 1e-3), dtype),
              TOL[dtype], f"branch norms without biases {T}x{W}")
        close(s1, s2, 2e-6, "the stream after the branch")
        table, ids = _rand((50, W), dtype, g), torch.randint(0, 50, (T,), generator=g, dtype=torch.int32).cuda()
        pair = torch.zeros(T, 2 * W, dtype=dtype).cuda()
        got = ops.embedding(ids, table, scale=2.5, copy=pair[:, W:])
        close(got, ref.ref_embedding(ids, table, 2.5), 1e-7, "embedding")
        assert torch.equal(pair[:, W:], got.to(dtype)) and float(pair[:, :W].abs().max()) == 0.0


@pytest.mark.gpu
def test_sigmoid_router_kernel(hip):
    ops, g = hip[torch.bfloat16], torch.Generator().manual_seed(43)
    for (T, E, top) in ((1, 5, 2), (37, 12, 12), (130, 64, 4), (9, 128, 16), (70, 200, 3), (3, 1, 1)):
        z, c = _rand((T, E + 3), torch.float32, g, 2.0)[:, :E], _rand((E,), torch.float32, g, 0.4)
        for scale, renormalise, bias in ((2.5, False, None), (1.0, True, None), (0.7, True, _rand((E,), torch.float32, g))):
            got, share = ops.route_topk(z, bias, top, over="sigmoid", choice_bias=c, renormalise=renormalise, scale=scale)
            want, wshare = ref.ref_route_topk(z, bias, top, "sigmoid", c, renormalise, scale)
            assert torch.equal(got.cpu(), want.cpu()), f"{T} tokens, {top} of {E}"
            close(share, wshare, 1e-6, f"shares, {T} tokens, {top} of {E}")
    got, share = ops.route_topk(z, None, 1, over="all", scale=3.0)
    close(share, 3.0 * torch.ones_like(share), 1e-6, "a factor on softmax shares")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_chunked_softmax_kernels(hip, dtype):
    """Decode rows and portions over random pages against the torch operation: chunks of one position, of a page, of no multiple of
    one, longer than the contexts; beside a window; rows that begin at a chunk's first and last place; contexts split over workgroups."""
    from test_mutusun import AttentionCase
    ops, g = hip[dtype], torch.Generator().manual_seed(44)
    rows = [(0, 1), (5, 1), (23, 1), (63, 1), (64, 1), (79, 1), (80, 1), (200, 1), (700, 1), (0, 50), (17, 31), (63, 2), (79, 2), (100, 130), (0, 300),
            (400, 70)]
    for (Hq, Hkv, P, chunk, window) in ((6, 2, 16, 24, None), (3, 3, 32, 16, None), (4, 1, 16, 1, None), (2, 2, 48, 80, None), (8, 2, 64, 100, None),
                                        (4, 4, 128, 33, None), (16, 4, 64, 640, None), (40, 1, 64, 64, None), (4, 2, 256, 50, None), (8, 4, 64, 2000, None),
                                        (4, 2, 64, 50, 20), (10, 2, 80, 80, None)):
        case = AttentionCase(rows, Hkv, P, dtype, g)
        q = _rand((case.num_tokens, Hq * P), dtype, g)
        args = (q, Hq, Hkv, P, case.k, case.v)
        want = ref.ref_paged_attention(*args, case.block_tables, case.token_row, case.positions, P ** -0.5, window, torch.float32, chunk=chunk)
        what = f"heads {Hq}/{Hkv} of {P}, chunk {chunk}, window {window}"
        close(ops.paged_attention(*args, case.group, case.step, P ** -0.5, window, chunk=chunk), want, 1e-5 if dtype == torch.float32 else 1.5e-2, what)
        if dtype == torch.bfloat16:
            close(ops.paged_attention(*args, case.group, case.step, P ** -0.5, window, chunk=chunk, force_generic=True), want, 1.5e-2, f"32-bit kernel, {what}")
            for splits in (1, 3):
                close(ops.paged_attention(*args, case.group, case.step, P ** -0.5, window, chunk=chunk, num_splits=splits), want, 1.5e-2, f"{splits} splits, {what}")


def delta_case(rows, H, G, d, dv, ra, rg, g, slow=False):
    T, up = sum(rows), lambda n: -(-n // 16) * 16        # noqa: E731
    u = _rand((T, 2 * G * d + H * dv + 5), torch.float32, g)
    beta_col, decay_col = 3, up(3 + H)
    gate_col = decay_col + up(ra)
    sums = _rand((T, gate_col + up(rg)), torch.float32, g)
    w_decay, w_gate = torch.zeros(H * d, up(ra)).cuda(), torch.zeros(H * dv, up(rg)).cuda()
    w_decay[:, :ra], w_gate[:, :rg] = _rand((H * d, ra), torch.float32, g, ra ** -0.5), _rand((H * dv, rg), torch.float32, g, rg ** -0.5)
    rate = torch.exp(_rand((H,), torch.float32, g) * (1.0 if not slow else 0.1) - (6.0 if slow else 0.0))
    bias = _rand((H * d,), torch.float32, g, 3.0) - 1.0
    nw = _rand((dv,), torch.float32, g) + 1
    state = _rand((len(rows) + 2, H, d, dv), torch.float32, g, 0.5)
    args = (u, 2, 2 + G * d, 2 + 2 * G * d, sums, beta_col, decay_col, gate_col, H, G, d, dv, w_decay, rate, bias, w_gate, d ** -0.5, nw, 1e-5)
    return args, state


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gated_delta_kernel(hip, dtype):
    """Whole rows and (bfloat16 mode) rows in chunks, queries and keys shared by heads, states of sizes that fill no tile, wider than
    high and higher than wide, slots that hold something, decays from so fast that a product over a chunk underflows to hardly any,
    single-token rows beside long ones."""
    ops, g = hip[dtype], torch.Generator().manual_seed(45)
    for (rows, H, G, d, dv, ra, rg, slow) in (([1, 1, 1], 4, 2, 16, 32, 12, 7, False), ([37, 1, 5], 6, 3, 24, 8, 16, 33, False), ([200], 5, 1, 7, 6, 3, 1, False),
                                              ([1, 1, 130, 70, 64, 65, 2], 4, 4, 48, 64, 20, 16, False), ([300, 2], 2, 1, 128, 64, 24, 24, True),
                                              ([200], 2, 2, 128, 128, 8, 8, False), ([9], 1, 1, 250, 40, 5, 5, False), ([1, 90], 1, 1, 200, 256, 16, 16, False),
                                              ([3, 190], 3, 1, 100, 200, 64, 40, True), ([1, 1], 2, 1, 256, 256, 8, 8, False), ([400], 8, 8, 40, 24, 20, 28, True),
                                              ([1, 257], 3, 3, 64, 72, 17, 100, False), ([1, 1, 1, 1], 2, 1, 128, 128, 16, 128, False)):
        args, state = delta_case(rows, H, G, d, dv, ra, rg, g, slow)
        step = step_of(rows)
        s1, s2 = state.clone(), state.clone()
        got = ops.gated_delta(*args, s1, step)
        want = ref.ref_gated_delta(*args, s2, step.host["row_start"], step.host["state_slots"], dtype)
        what = f"rows {rows}, {H} heads of {d} x {dv}"
        close(s1, s2, 2e-5, f"gated delta: state, {what}")
        close(got, want, 5e-5 if dtype == torch.float32 else 1e-2, f"gated delta, {what}")
        assert torch.equal(s1[0], state[0]) and torch.equal(s1[-1], state[-1]), "slots of no row are left alone"


@pytest.mark.gpu
def test_gated_delta_in_chunks_with_keys_that_repeat(hip):
    """The worst case for a chunk's inverse: every token has the same key and writes it whole, with next to no decay; and the
    opposite: decays of e^-40 a token."""
    ops, g = hip[torch.bfloat16], torch.Generator().manual_seed(46)
    for kind in ("repeat", "fast"):
        rows = [200]
        args, state = delta_case(rows, 2, 1, 32, 16, 8, 8, g)
        args = list(args)
        if kind == "repeat":
            args[0][:, 2 + 32:2 + 64] = args[0][0, 2 + 32:2 + 64]
            args[4][:, 3:5] = 9.0                              # beta next to 1
            args[13].fill_(1e-4)
        else:
            args[13].fill_(20.0)
            args[14].fill_(2.0)
        step = step_of(rows)
        s1, s2 = state.clone(), state.clone()
        got = ops.gated_delta(*args, s1, step)
        want = ref.ref_gated_delta(*args, s2, step.host["row_start"], step.host["state_slots"], torch.bfloat16)
        close(s1, s2, 5e-5, f"{kind}: state")
        close(got, want, 1e-2, f"{kind}: outputs")


# ------------------------------------------------------------------------------------------- GPU: whole models
@pytest.mark.gpu
@pytest.mark.parametrize("family", list(FAMILIES))
@pytest.mark.parametrize("name", list(CONFIGS))
def test_families_float32(name, family, tmp_path):
    run_family(name, family, tmp_path, "cuda", "float32", F32_TOL)


@pytest.mark.gpu
@pytest.mark.parametrize("family", list(FAMILIES))
@pytest.mark.parametrize("name", list(CONFIGS))
def test_families_bfloat16(name, family, tmp_path):
    raw, _ = CONFIGS[name]
    run_family(name, family, tmp_path, "cuda", "bfloat16", BF16_TOL_PER_LAYER * layer_runs(raw))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_keys_at_the_edges_of_the_chunks(dtype):
    chunk_runs("cuda", dtype)


@pytest.mark.gpu
def test_a_far_key_and_the_first_token_are_seen_by_the_kernels():
    far_key_runs("cuda")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_in_chunks_of_the_recurrence(dtype):
    """Prompts of several hundred tokens, whole and in uneven portions: the recurrence runs in chunks side by side in bfloat16 and
    token by token in float32; several chunks of the attention end within the prompts."""
    raw, cfg, weights = make("D", torch.float32 if dtype == "float32" else torch.bfloat16, sharp=dtype == "float32")
    prompts = trace_util.random_prompts(raw["vocab"], [400, 129], seed=8)
    want = expected_logits(raw, weights, prompts)
    for steps in (trace_util.whole(prompts), trace_util.portions(prompts, sizes=(130, 2, 65, 64, 200))):
        runner = ModelRunner(cfg, weights=weights, dtype=dtype, num_pages=40, max_rows=2, max_step_tokens=512, max_model_len=39 * 16)
        got = {k: v.cpu() for k, v in trace_util.run_on_runner(runner, steps).items()}
        if dtype == "float32":
            trace_util.compare(got, want, F32_TOL, "long prompts")
        else:
            compare_most(got, want, BF16_TOL_PER_LAYER * layer_runs(raw), "long prompts")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(dtype):
    eng = generate("A", "cuda", dtype)
    assert eng.num_graph_steps > 0, "decode steps run as captured graphs"


@pytest.mark.gpu
def test_captured_prompt_portions_run_the_recurrence_in_chunks():
    """Prompts in portions of exactly the step's budget of 128 tokens: the captured step of such a portion is replayed for
    portion after portion of several requests, each going on from its own states."""
    eng = generate("D", "cuda", "bfloat16", lengths=(256, 384, 130, 256), budget=128, blocks=80)
    assert eng.num_graph_steps > 0 and eng.runner.portion_graphs[-1].tokens == 128


# --------------------------------------------------------------------------------------------- the command line
def test_random_model_of_the_named_size_is_what_the_loader_reads(tmp_path):
    from safetensors.torch import load_file
    from test_labirax import run_cli
    folder = str(tmp_path / "m")
    run_cli("random-model", "--shape", "bulitar-tiny", "--seed", "3", "--dtype", "float32", "--out", folder)
    cfg, arch = load_model_config(folder)
    assert arch.name == "Bulitar" and len(cfg.layers) == 3 and cfg.loop.times == 2
    stored = load_file(folder + "/model.safetensors")
    raw = json.loads(open(folder + "/config.json").read())
    runner = host_runner(cfg, stored, pages=8, rows=2, tokens=64)
    toks = trace_util.random_prompts(raw["vocab"], [40], seed=1)
    got = trace_util.run_on_runner(runner, trace_util.portions(toks, sizes=(9, 2, 20)))
    trace_util.compare(got, expected_logits(raw, stored, toks), F32_TOL, "the named size")


@pytest.mark.gpu
def test_generate_from_the_command_line(tmp_path):
    from safetensors.torch import load_file
    from test_labirax import run_cli
    folder = str(tmp_path / "m")
    run_cli("random-model", "--shape", "bulitar-tiny", "--seed", "3", "--dtype", "float32", "--out", folder)
    prompts = [[5, 17, 3, 200, 41], list(range(20, 54)), [7]]
    args = ["generate", "--model", folder, "--dtype", "float32", "--max-tokens", "6", "--ignore-eos", "--num-blocks", "24", "--quiet"]
    for p in prompts:
        args += ["--prompt-ids", ",".join(map(str, p))]
    lines = [json.loads(line) for line in run_cli(*args).stdout.splitlines() if line.startswith("{")]
    raw, stored = json.loads(open(folder + "/config.json").read()), load_file(folder + "/model.safetensors")
    assert [r["prompt_len"] for r in lines] == [len(p) for p in prompts]
    for prompt, rec in zip(prompts, lines):
        ids = list(prompt)
        assert len(rec["output_ids"]) == 6
        for tok in rec["output_ids"]:
            row = plain.forward(raw, stored, ids)[-1]
            assert float(row.max() - row[tok]) <= 1e-5 * float(row.abs().max()), f"token {tok} after {len(ids)} tokens"
            ids.append(tok)
