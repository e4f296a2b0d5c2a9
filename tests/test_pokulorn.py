"""Pokulorn through the engine against the plain implementation (tests/plain_pokulorn.py).

Configurations are made here, with sizes that differ from one another wherever the design lets them (query and key/value
head counts, head size and value size either way round, rotations of a part of the head, with and without stretched
frequencies, windows of a page and a half, of a page and of one key, kept first tokens of none, one, a page and more, taps from
one to five, state groups from one to one a head, norm parts that cut through heads, factors on both sides, layers that mix
values beside layers that do not, layers without a feed-forward).  Host tests run the engine's own parts, cache and step
function on the CPU with the torch operations of tests/torch_backend.py; GPU tests run the HIP kernels, each kernel
against the torch operation of the same name and the whole model in the four trace families, in float32 (tight) and
bfloat16.
"""
import json
import math

import pytest
import torch

import plain_pokulorn as plain
import trace_util
from torch_backend import TorchBackend
import torch_backend as ref

from mini_inference_engine_amd.cache import CacheManager, GroupSpec
from mini_inference_engine_amd.config import ConfigError, EngineConfig, PokulornConfig, load_model_config
from mini_inference_engine_amd.engine.batch import StepRow
from mini_inference_engine_amd.engine.runner import ModelRunner
from mini_inference_engine_amd.parts import RotaryYarn
from mini_inference_engine_amd.replay.trace import replay
from mini_inference_engine_amd.weights import random_tensors


def rot(dims, base=100.0, factor=None, original=64, fast=8.0, slow=1.0):
    d = dict(base=base, dims=dims)
    if factor is not None:
        d["scaling"] = dict(factor=factor, original=original, fast=fast, slow=slow)
    return d


def att(heads, kv_heads, dim, vdim=None, scale=None, conv=3, rotation=None, window=None, keep=None, v_mix=None):
    d = dict(heads=heads, kv_heads=kv_heads, dim=dim, scale=scale if scale is not None else dim ** -0.5,
             rot=rotation or rot(dim, factor=4.0))
    if conv is not None:
        d["conv"] = conv
    if vdim is not None:
        d["vdim"] = vdim
    if window is not None:
        d["mask"] = dict(size=window) if keep is None else dict(size=window, keep_first=keep)
    if v_mix is not None:
        d["v_mix"] = v_mix
    return d


def ssm(heads, vdim, state, groups=1, conv=4, norm_groups=1):
    return dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)


def pair(left, right, left_scale=0.5, right_scale=0.5):
    return dict(left=left, right=right, left_scale=left_scale, right_scale=right_scale)


def mem(heads, dim, vdim=None, cap=15.0):
    d = dict(heads=heads, dim=dim, gate_cap=cap)
    if vdim is not None:
        d["vdim"] = vdim
    return d


def dense(ff, limit=2.0):
    return dict(kind="dense", ff=ff, limit=limit)


def layer(kind, mixer, mlp):
    return dict(type=kind, mixer=mixer, mlp=mlp)


def model(vocab, width, eps, layers):
    return dict(architecture="Pokulorn", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)


A_ATT = att(6, 2, 16, vdim=24, window=24, keep=3, v_mix=True, rotation=rot(12, base=50.0, factor=4.0))
A_PAIR = pair(att(4, 2, 24, vdim=16, conv=2, rotation=rot(24, factor=8.0, original=32)), ssm(6, 8, 20, groups=3, conv=4, norm_groups=4), 0.7, 1.3)
A_MEM = mem(3, 16, vdim=24, cap=8.0)
CFG_A = model(211, 64, 1e-5, [layer("attention", A_ATT, dense(96)),
                              layer("mlstm", A_MEM, dense(80, 1.5)),
                              layer("parallel", A_PAIR, dense(96)),
                              layer("attention", A_ATT, None),
                              layer("mlstm", A_MEM, None),
                              layer("attention", A_ATT, dense(112))])
# a layer that does not mix before the first that does; a window of a page; kept tokens over two pages; plain rotation
B_PLAIN = att(4, 4, 8, window=16, keep=20, conv=4, rotation=rot(8))
B_MIX = att(4, 1, 24, vdim=8, window=40, keep=1, v_mix=True, conv=5)
CFG_B = model(150, 48, 1e-3, [layer("attention", B_PLAIN, dense(56, 0.7)),
                              layer("parallel", pair(att(2, 2, 16, conv=3, scale=0.3), ssm(4, 16, 12, groups=4, conv=2, norm_groups=1), 2.0, 0.25), None),
                              layer("attention", B_MIX, dense(40)),
                              layer("attention", att(4, 4, 16, v_mix=False, conv=None, rotation=rot(4, factor=3.0)), dense(40)),   # no window, no convolution
                              layer("attention", B_MIX, None)])
# sizes the kernels' vector paths do not like: nothing a multiple of 8, an odd vocabulary, one head of everything
CFG_C = model(101, 70, 1e-6, [layer("parallel", pair(att(3, 1, 10, vdim=14, conv=1, rotation=rot(6, factor=2.0)), ssm(5, 6, 7, conv=3, norm_groups=3), 1.0, 1.0), dense(50, 9.0)),
                              layer("mlstm", mem(1, 10, vdim=13, cap=3.0), dense(26)),
                              layer("attention", att(3, 3, 18, vdim=6, window=5, keep=2, conv=2, v_mix=True), None),
                              layer("mlstm", mem(3, 5), dense(18)),
                              layer("attention", att(6, 3, 14, vdim=6, window=1, keep=0, v_mix=True, conv=4), dense(22))])
# wider heads and states, eight query heads on one key head, a window longer than most requests, kept tokens beyond a step
CFG_D = model(333, 96, 1e-4, [layer("parallel", pair(att(8, 1, 40, vdim=56, conv=4), ssm(2, 64, 48, conv=4, norm_groups=2), 0.6, 1.5), dense(128)),
                              layer("attention", att(4, 2, 64, window=70, keep=66, v_mix=True, rotation=rot(32, base=1000.0, factor=16.0, original=128)), dense(64)),
                              layer("mlstm", mem(2, 40, vdim=72), dense(64)),
                              layer("attention", att(8, 2, 32, vdim=64, window=100, keep=5, v_mix=True), dense(96))])
CONFIGS = {"A": (CFG_A, 3), "B": (CFG_B, 4), "C": (CFG_C, 6), "D": (CFG_D, 8)}


def shape_weights(cfg, seed, sharp=True):
    """Random weights shaped so that faults show: products keep the scale of their input, norm weights, sinks and mixing
    shares are far from their resting values, convolutions look back as much as at the token itself, decays and gates
    range from fast to slow, feed-forward values reach their limits.  ``sharp`` also spreads the attention scores; the
    bfloat16 runs leave them at unit scale, because spread scores amplify the rounding of 8-bit values as much as they
    amplify faults."""
    w = random_tensors(cfg, seed, torch.float32, std=1.0)
    g = torch.Generator().manual_seed(seed + 100)
    draw = lambda v: torch.randn(v.shape, generator=g)        # noqa: E731
    for k, v in w.items():
        if k.endswith(".vmix"):
            v.copy_(0.4 + 0.3 * draw(v))
        elif k.endswith(".sink"):
            v.copy_(draw(v) + (1.0 if sharp else 0.0))
        elif k.endswith((".q.conv", ".k.conv", ".v.conv", ".right.conv")):
            v.copy_(draw(v) * v.shape[-1] ** -0.5)
        elif k.endswith("conv.b"):
            v.copy_(draw(v) * 0.3)
        elif k.endswith(".A_log"):
            v.copy_(draw(v))
        elif k.endswith(".dt_bias"):
            v.copy_(draw(v) - 2.0)
        elif k.endswith(".f.b"):
            v.copy_(draw(v) * 2.0 + 2.0)
        elif k.endswith(".i.b"):
            v.copy_(draw(v) * 2.0)
        elif k.endswith(".D"):
            v.copy_(1.0 + 0.5 * draw(v))
        elif "norm" in k:
            v.copy_(1.0 + 0.4 * draw(v))
            if sharp and k.endswith(".q.norm"):
                v.mul_(2.0)
        elif v.dim() >= 2:
            v.mul_(v.shape[-1] ** -0.5)
    return w


def make(name, dtype=torch.float32, sharp=True):
    raw, seed = CONFIGS[name]
    cfg = PokulornConfig.from_dict(raw)
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
# (a lost key, a window that is one position off, a lost state, a sink left out) moves logits by a hundred times this
F32_TOL = 2e-4
# bfloat16: every sublayer rounds a handful of values to 8 bits.  Nearly all rows stay within a hundredth of the logit scale a
# layer; a head's norm amplifies the rounding of the few rows where a memory's output nearly cancels (so do the torch
# operations on the CPU when they round to bfloat16 at the same places), so a twentieth of the rows may go to three times that.
BF16_TOL_PER_LAYER = 1e-2

FAMILIES = {"whole": trace_util.whole, "decode_tail": lambda p: trace_util.decode_tail(p, 40),
            "portions": trace_util.portions, "mixed": lambda p: trace_util.mixed(p, 4, seed=5)}
LENGTHS = [3, 70, 1, 37, 90, 18, 49]


def compare_bf16(got, expected, tol, what):
    errs = {k: float((row.double().cpu() - expected[k[0]][k[1]]).abs().max()) / float(expected[k[0]].abs().max()) for k, row in got.items()}
    worst = max(errs, key=lambda k: errs[k] if math.isfinite(errs[k]) else math.inf)
    assert math.isfinite(errs[worst]) and errs[worst] <= 3 * tol, f"{what}: {worst}: error {errs[worst]:.3e} of the logit scale"
    over = sum(e > tol for e in errs.values())
    assert over <= 0.05 * len(errs), f"{what}: {over} of {len(errs)} rows beyond {tol:.1e} of the logit scale"
    return errs[worst]


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
    check = trace_util.compare if dtype == "float32" else compare_bf16
    return check(got, expected_logits(raw, weights, prompts), tol, f"pokulorn {name}/{family}/{dtype}")


# ------------------------------------------------------------------------------------------- configuration
def test_config_round_trip_and_registry(tmp_path):
    for name in CONFIGS:
        raw, cfg, _ = make(name)
        assert PokulornConfig.from_dict(cfg.to_dict()) == cfg
        (tmp_path / "config.json").write_text(json.dumps(raw))
        loaded, arch = load_model_config(str(tmp_path))
        assert loaded == cfg and arch.name == "Pokulorn"
    a, b, c = (PokulornConfig.from_dict(CONFIGS[n][0]) for n in "ABC")
    assert a.first_value_layer() == 0 and b.first_value_layer() == 2 and c.first_value_layer() == 2
    assert a.layers[0].mixer.vdim == 24 and a.layers[0].mixer.keep_first == 3 and a.layers[3].mlp is None
    assert b.layers[3].mixer.window is None and b.layers[3].mixer.taps is None and b.layers[0].mixer.rot.scaling is None
    assert c.layers[3].mixer.vdim == 5 and c.layers[4].mixer.keep_first == 0


@pytest.mark.parametrize("bad", [
    lambda c: c["layers"][0]["mixer"].update(kv_heads=4),                  # 6 query heads over 4 key heads
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18),              # more than the head
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3),
    lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0.0),
    lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("original"),
    lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
    lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1),
    lambda c: c["layers"][0]["mixer"].update(conv=0),
    lambda c: c["layers"][3]["mixer"].update(vdim=16),                     # mixes values of another size than the first layer's
    lambda c: c["layers"][1]["mixer"].update(gate_cap=0.0),
    lambda c: c["layers"][2]["mixer"]["right"].update(groups=4),           # 6 heads in 4 groups
    lambda c: c["layers"][2]["mixer"]["right"].update(norm_groups=5),      # 48 numbers in 5 parts
    lambda c: c["layers"][2]["mixer"]["left"].update(v_mix=True),
    lambda c: c["layers"][0]["mlp"].update(limit=0.0),
    lambda c: c["layers"][0]["mlp"].update(kind="moe"),
    lambda c: c["layers"][0].update(type="conv"),
    lambda c: c.update(layers=[]),
])
def test_config_refuses_what_cannot_be_computed(bad):
    raw = json.loads(json.dumps(CFG_A))
    bad(raw)
    with pytest.raises(ConfigError):
        PokulornConfig.from_dict(raw)


def test_model_structure():
    _, cfg, weights = make("A")
    runner = host_runner(cfg, weights)
    m = runner.model
    assert tuple(weights["l0.mix.q.conv"].shape) == (96, 3) and tuple(weights["l0.mix.v.conv"].shape) == (48, 3)
    assert tuple(weights["l0.mix.q.norm"].shape) == (16,) and tuple(weights["l0.mix.vmix"].shape) == () and tuple(weights["l0.mix.sink"].shape) == (6,)
    assert tuple(weights["l2.mix.right.in"].shape) == (2 * 48 + 2 * 60 + 6, 64) and tuple(weights["l2.mix.right.conv"].shape) == (168, 4)
    assert tuple(weights["l2.mix.left.g"].shape) == (64, 64) and "l2.mix.left.sink" not in weights and "l2.mix.left.vmix" not in weights
    assert tuple(weights["l1.mix.norm"].shape) == (72,) and tuple(weights["l1.mix.i"].shape) == (3, 64)
    assert "l3.norm2" not in weights and "l3.mlp.gate" not in weights and "l4.norm1" in weights
    # two page groups: the window of 24 beside three kept tokens (two layers share it), every key for the side of the pair
    assert sorted(zip(m.page_groups, m.page_group_keeps), key=str) == [(24, 3), (None, 0)]
    assert not m.padding_safe, "a model with a state takes no padding tokens"
    # a pair's sides share one product each way
    block = m.spec.layers[2]
    assert block.mixer.w_in.shape[0] == block.mixer.left.w_in.shape[0] + block.mixer.right.w_in.shape[0]
    assert tuple(block.mixer.w_o.shape) == (64, 64 + 48)


# ------------------------------------------------------------------- the plain implementation against small sums by hand
def test_plain_rotation_and_mask_by_hand():
    # pairs that turn often keep their frequency, pairs that hardly turn are slowed down by the factor, the ramp lies between
    freqs, size = plain.yarn_frequencies(10000.0, 16, dict(factor=4.0, original=512, fast=8.0, slow=1.0))
    n = lambda t: 16 * math.log(512 / (2 * math.pi * t)) / (2 * math.log(10000.0))        # noqa: E731
    assert math.floor(n(8.0)) == 2 and math.ceil(n(1.0)) == 4
    straight = [10000.0 ** (-2 * i / 16) for i in range(8)]
    for i, f in enumerate(freqs):
        share = 0.0 if i <= 2 else 0.5 if i == 3 else 1.0
        assert abs(f - straight[i] * (share / 4.0 + 1 - share)) < 1e-12
    assert abs(size - (0.1 * math.log(4.0) + 1.0)) < 1e-12
    x = torch.randn(5, 2, 20, dtype=torch.float64)
    y = plain.turn_halves(x, torch.arange(5), freqs, size)
    assert torch.equal(y[..., 16:], x[..., 16:])
    a = 3 * freqs[5]
    assert abs(float(y[3, 1, 5] - size * (x[3, 1, 5] * math.cos(a) - x[3, 1, 13] * math.sin(a)))) < 1e-12
    assert abs(float(y[3, 1, 13] - size * (x[3, 1, 13] * math.cos(a) + x[3, 1, 5] * math.sin(a)))) < 1e-12
    seen = plain.visible(9, dict(size=3, keep_first=2))
    assert [j for j in range(9) if seen[7, j]] == [0, 1, 5, 6, 7] and [j for j in range(9) if seen[1, j]] == [0, 1]
    assert [j for j in range(9) if plain.visible(9, dict(size=3))[7, j]] == [5, 6, 7]
    w = plain.sink_softmax(torch.zeros(1, 2, 2, dtype=torch.float64), plain.visible(2, None), torch.tensor([math.log(2.0)], dtype=torch.float64))
    assert torch.allclose(w[0], torch.tensor([[1 / 3, 0.0], [0.25, 0.25]], dtype=torch.float64))


def test_engine_rotation_equals_the_plain_one():
    for dims, base, factor, original, fast, slow in ((16, 10000.0, 4.0, 512, 8.0, 1.0), (32, 500.0, 16.0, 64, 32.0, 1.0), (6, 20.0, 2.0, 1024, 4.0, 0.5),
                                                     (48, 1e6, 1.0, 4096, 32.0, 1.0)):
        part = RotaryYarn(dims, base, factor, original, fast, slow)
        freqs, size = plain.yarn_frequencies(base, dims, dict(factor=factor, original=original, fast=fast, slow=slow))
        assert torch.allclose(part.frequencies(), torch.tensor(freqs, dtype=torch.float64), rtol=1e-12)
        assert abs(part.magnitude - size) < 1e-12


def test_plain_recurrences_by_hand():
    one = torch.ones(1, 1, 1, dtype=torch.float64)
    # a state space of one number: S = e^-(rate dt) S + dt b x
    y, S = plain.ssm_scan(2 * one.expand(2, 1, 1), one.expand(2, 1, 1) * 3, one.expand(2, 1, 1), torch.full((2, 1), 0.5, dtype=torch.float64),
                          torch.tensor([math.log(2.0)], dtype=torch.float64), torch.tensor([0.25], dtype=torch.float64))
    assert abs(float(y[0]) - 3.5) < 1e-12 and abs(float(y[1]) - (3 * math.exp(-1.0) + 3 + 0.5)) < 1e-12 and abs(float(S) - 3 * (1 + math.exp(-1.0))) < 1e-12
    # a memory of one number: the maximum starts at 0, the denominator is at least exp(-m)
    i, f = torch.tensor([[-1.0], [2.0]], dtype=torch.float64), torch.tensor([[-0.5], [-0.1]], dtype=torch.float64)
    o, (S, n, m) = plain.mlstm_scan(0.1 * one.expand(2, 1, 1), one.expand(2, 1, 1), 5 * one.expand(2, 1, 1), i, f)
    m1 = -0.5                                              # max(-0.5 + 0, -1)
    s1 = math.exp(-1.0 - m1)
    assert abs(float(o[0]) - 0.5 * s1 / (max(0.1 * s1, math.exp(-m1)) + 1e-6)) < 1e-12
    s2 = math.exp(-0.1 + m1 - 2.0) * s1 + 1.0              # the new maximum is the input gate
    assert abs(float(o[1]) - 0.5 * s2 / (max(0.1 * s2, math.exp(-2.0)) + 1e-6)) < 1e-12 and float(m) == 2.0 and abs(float(n) - s2) < 1e-12
    # the convolution's last column is the token's own
    u = torch.arange(1.0, 5.0, dtype=torch.float64)[:, None]
    assert plain.short_conv(u, torch.tensor([[10.0, 1.0]], dtype=torch.float64))[:, 0].tolist() == [1.0, 12.0, 23.0, 34.0]
    g = plain.grouped_rms(torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=torch.float64), 2, 0.0)
    assert torch.allclose(g, torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=torch.float64) / torch.tensor([12.5, 12.5, 2.0, 2.0], dtype=torch.float64).sqrt())


# ------------------------------------------------------------------------------------- mechanisms, one by one
def one_layer(kind, mixer, mlp, width=32, vocab=50, eps=1e-5):
    return model(vocab, width, eps, [layer(kind, mixer, mlp)])


MECHANISMS = {
    "attention": one_layer("attention", att(4, 2, 8, vdim=12, window=6, keep=2), None),
    "attention-all-keys": one_layer("attention", att(2, 2, 16, vdim=4, conv=4), None),
    "attention-window-of-one": one_layer("attention", att(2, 1, 8, window=1, keep=1, conv=2), None),
    "attention-window-keeps-nothing": one_layer("attention", att(2, 1, 8, window=7, keep=0), None),
    "attention-no-convolution": one_layer("attention", att(3, 1, 8, conv=None, rotation=rot(8), window=9, keep=17), None),
    "attention-no-convolution-values-mixed": model(50, 32, 1e-5, [layer("attention", att(2, 1, 8, v_mix=True, conv=None, rotation=rot(8)), None)] * 2),
    "attention-one-tap": one_layer("attention", att(1, 1, 24, vdim=40, conv=1, rotation=rot(6, factor=3.0)), None),
    "values-mixed": model(50, 32, 1e-5, [layer("attention", att(2, 1, 8, vdim=12, v_mix=True, window=5, keep=1), None),
                                         layer("attention", att(4, 1, 16, vdim=12, v_mix=True, conv=2), None)]),
    "pair": one_layer("parallel", pair(att(2, 1, 8, vdim=12), ssm(2, 6, 5), 0.3, 1.7), None),
    "pair-groups-and-parts": one_layer("parallel", pair(att(2, 2, 8, conv=2), ssm(6, 4, 3, groups=3, conv=3, norm_groups=8)), None),
    "pair-a-group-a-head": one_layer("parallel", pair(att(1, 1, 16), ssm(3, 10, 12, groups=3, conv=1, norm_groups=3), 1.0, 1.0), None),
    "mlstm": one_layer("mlstm", mem(2, 8, vdim=12), None),
    "mlstm-low-cap": one_layer("mlstm", mem(1, 20, vdim=4, cap=1.0), None),
    "clamped-feed-forward": one_layer("mlstm", mem(1, 8), dense(24, 0.5)),
    "feed-forward-hardly-clamped": one_layer("mlstm", mem(1, 8), dense(20, 50.0)),
}


@pytest.mark.parametrize("name", list(MECHANISMS))
def test_each_mechanism_alone_on_the_host(name):
    raw = MECHANISMS[name]
    cfg = PokulornConfig.from_dict(raw)
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
    for name in ("l0.mix.sink", "l3.mix.vmix", "l5.mix.vmix", "l2.mix.right.D", "l2.mix.right.conv.b", "l2.mix.right.dt_bias", "l1.mix.f.b", "l1.mix.i.b"):
        assert changed(raw, weights, toks, zero(name)) > 20 * F32_TOL, f"{name} hardly shows"
    assert changed(raw, weights, toks, zero("l0.mix.vmix")) == 0.0, "the first layer that mixes has nothing to mix with"
    for name in ("l0.mix.q.conv", "l0.mix.v.conv", "l2.mix.left.k.conv", "l2.mix.right.conv"):
        assert changed(raw, weights, toks, lambda w: w[name][:, 0].zero_()) > 20 * F32_TOL, f"{name}: its furthest tap hardly shows"


def test_prefill_equals_token_by_token_decoding():
    raw, cfg, weights = make("A")
    prompts = trace_util.random_prompts(raw["vocab"], [60], seed=21)
    whole = trace_util.run_on_runner(host_runner(cfg, weights), trace_util.whole(prompts))
    single = trace_util.run_on_runner(host_runner(cfg, weights), trace_util.decode_tail(prompts, 59))
    pairs = trace_util.run_on_runner(host_runner(cfg, weights), trace_util.portions(prompts, sizes=(2,)))
    scale = max(float(v.abs().max()) for v in whole.values())
    for key, row in whole.items():
        assert float((single[key] - row).abs().max()) < 1e-5 * scale, f"token by token differs at {key}"
        assert float((pairs[key] - row).abs().max()) < 1e-5 * scale, f"two by two differs at {key}"
    trace_util.compare(whole, expected_logits(raw, weights, prompts), F32_TOL, "whole")


# ------------------------------------------------------------------------------------------ whole models, host
@pytest.mark.parametrize("family", list(FAMILIES))
@pytest.mark.parametrize("name", list(CONFIGS))
def test_families_on_the_host(name, family, tmp_path):
    run_family(name, family, tmp_path, "cpu", "float32", F32_TOL)


def window_model(keep):
    """One attention layer with a window of 20 keys (a page and a quarter) beside ``keep`` kept ones, a convolution of one tap
    and no feed-forward: the logits of a position are a function of its own token, the 19 before it and the kept ones."""
    raw = one_layer("attention", att(3, 1, 16, vdim=8, conv=1, window=20, keep=keep, scale=0.5), None, width=48, vocab=90)
    cfg = PokulornConfig.from_dict(raw)
    w = shape_weights(cfg, 5)
    w["l0.mix.sink"].fill_(-3.0)
    w["l0.mix.q.norm"].mul_(0.2)                              # scores close to one another: every visible key has a share
    w["embed"][89] = 4.0 * w["embed"][89].sign()              # the token that stands out
    return raw, cfg, w


def window_runs(device):
    """A token that stands out is put just inside and just outside the window of the positions asked for, on the last kept
    place and the one after it, and on a page's last and next first slot, in a prompt's portion and for tokens decoded one
    by one.  Where it is visible, it must move the logits; elsewhere the engine's logits must not move at all; both ways
    they follow the plain implementation."""
    for keep in (0, 3, 18):
        raw, cfg, w = window_model(keep)
        base = [t if t != 89 else 0 for t in trace_util.random_prompts(90, [75], seed=9)["r0"]]

        def run(tokens, cut):
            steps = [{"step": 0, "entries": [{"id": "x", "tokens": tokens[:cut], "want": list(range(cut))}], "end": []}]
            steps += [{"step": 1 + i, "entries": [{"id": "x", "tokens": tokens[cut + i:cut + i + 1], "want": [0]}], "end": []}
                      for i in range(len(tokens) - cut)]
            steps[-1]["end"] = ["x"]
            return {k: v.cpu() for k, v in trace_util.run_on_runner(make_runner(device, cfg, w, 8, 2, 80), steps).items()}

        for cut in (70, 42):                  # asked-for positions in the portion; the window's edge among decoded tokens
            plain_run = run(base, cut)
            for needle in (40, 41, 47, 48, 0, 2, 3, 15, 16, 17, 18):
                tokens = list(base)
                tokens[needle] = 89
                want = plain.forward(raw, w, tokens)
                got = run(tokens, cut)
                trace_util.compare(got, {"x": want}, F32_TOL, f"keep {keep}, needle at {needle}, portion of {cut}")
                for p in range(75):
                    moved = float((got[("x", p)] - plain_run[("x", p)]).abs().max()) / float(want.abs().max())
                    if p >= needle and (p <= needle + 19 or needle < keep):
                        assert moved > 2e-6, f"keep {keep}: position {p} must see the token at {needle} (portion of {cut})"
                    else:
                        assert moved < 2e-7, f"keep {keep}: position {p} must not see the token at {needle} (portion of {cut}): {moved:.1e}"


def test_keys_at_the_edges_of_the_window_and_of_the_kept_tokens_on_the_host():
    window_runs("cpu")


def far_key_runs(device):
    """One key far back (hundreds of positions, through a dozen pages) is made to decide the attention's output: token 63 has
    the key that token 62, the last one, asks for, and 62's own key points the other way.  The key stands at a page's last
    slot, at the next page's first, and at the very first position, for the full attention of a pair; and among the kept
    tokens of a window that is long past."""
    for kind in ("parallel", "attention"):
        a = att(2, 1, 16, scale=0.4, conv=1, rotation=rot(4, base=1e6))
        if kind == "attention":
            a.update(mask=dict(size=30, keep_first=37))
        raw = one_layer(kind, a if kind == "attention" else pair(a, ssm(1, 4, 4), 1.0, 0.01), None, width=32, vocab=64)
        cfg = PokulornConfig.from_dict(raw)
        w = shape_weights(cfg, 7)
        p = "l0.mix" if kind == "attention" else "l0.mix.left"
        along = torch.ones(16)
        along[0] = along[2] = 0.0                             # the pair that turns fast stays out of it
        w["embed"][:, :2] = 0.0
        w["embed"][62, 1], w["embed"][63, 0] = 20.0, 20.0
        w[f"{p}.q"].zero_()
        w[f"{p}.q"][:, 1] = along.repeat(2)
        w[f"{p}.k"][:, 0], w[f"{p}.k"][:, 1] = 10 * along, -10 * along
        for x in "qk":
            w[f"{p}.{x}.conv"].fill_(1.0)
            w[f"{p}.{x}.norm"].fill_(2.5)
        toks = [t % 62 for t in trace_util.random_prompts(64, [230], seed=9)["r0"]]
        toks[-1] = 62
        for needle in (31, 32, 0, 36):
            tokens = list(toks)
            tokens[needle] = 63
            want = plain.forward(raw, w, tokens)
            steps = [{"step": 0, "entries": [{"id": "x", "tokens": tokens[:190], "want": [189]}], "end": []}]
            steps += [{"step": 1 + i, "entries": [{"id": "x", "tokens": tokens[190 + i:191 + i], "want": [0]}], "end": []}
                      for i in range(40)]
            steps[-1]["end"] = ["x"]
            got = {k: v.cpu() for k, v in trace_util.run_on_runner(make_runner(device, cfg, w, 16, 2, 192), steps).items()}
            trace_util.compare(got, {"x": want}, F32_TOL, f"{kind}: far key at {needle}")
            moved = float((plain.forward(raw, w, toks)[-1] - want[-1]).abs().max()) / float(want.abs().max())
            assert moved > 1e-2, "the far key must matter to the last position for this test to mean anything"


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
    states = [(k, t) for e in runner.storage.entries.values() for k, t in e.tensors.items()
              if k.split(".")[-1] in ("state", "tail", "normaliser", "maximum")]
    assert len(states) == 3 + 2 * 3 + 3                       # attention: a tail; memory: three; the pair: two tails and a state
    for _, t in states:
        t.fill_(-2.0)
    rc = runner.cache.open("fresh")
    assert all(float(t[rc.state_slot].abs().max()) == 0.0 for _, t in states)
    runner.cache.close(rc)


def test_pages_before_the_window_are_given_back_and_the_kept_ones_stay():
    cm = CacheManager(16, [GroupSpec(24, 9, 20), GroupSpec(None, 9)], 3)
    rc = cm.open("a")
    assert cm.reserve(rc, 0, 120)
    cm.advance(rc, 120)                                       # the next query sees 97 .. and 0 .. 19: pages 0, 1, 6, 7
    assert [p != 0 for p in rc.tables[0]] == [True, True, False, False, False, False, True, True] and all(rc.tables[1])
    cm.check()
    cm.close(rc)
    cm.check()
    assert cm.num_free(0) == 8
    # a request that decodes far beyond its window keeps what its window touches and the kept tokens' page only
    raw = one_layer("attention", att(2, 1, 8, window=30, keep=5), None)
    cfg = PokulornConfig.from_dict(raw)
    w = shape_weights(cfg, 2)
    prompts = trace_util.random_prompts(50, [150], seed=1)
    runner = ModelRunner(cfg, weights=w, dtype="float32", device="cpu", backend=TorchBackend(torch.float32), num_pages=7,
                         max_rows=1, max_step_tokens=64, max_model_len=160)          # six usable pages of 16 for 150 tokens
    got = trace_util.run_on_runner(runner, trace_util.portions(prompts, sizes=(20, 3, 1, 30)))
    trace_util.compare(got, expected_logits(raw, w, prompts), F32_TOL, "pages given back")


def test_long_decoding_carries_the_state():
    """Two hundred tokens one by one through slow decays: what the first tokens wrote is still in the states at the end."""
    for kind, mixer in (("mlstm", mem(2, 8, vdim=12)), ("parallel", pair(att(1, 1, 8), ssm(2, 6, 8), 0.05, 1.0))):
        raw = one_layer(kind, mixer, None)
        cfg = PokulornConfig.from_dict(raw)
        w = shape_weights(cfg, 4)
        if kind == "mlstm":
            w["l0.mix.f.b"].fill_(9.0)
        else:
            w["l0.mix.right.A_log"].fill_(-5.0)
        prompts = trace_util.random_prompts(50, [200], seed=6)
        got = trace_util.run_on_runner(host_runner(cfg, w, pages=16, rows=1, tokens=64), trace_util.decode_tail(prompts, 199))
        want = expected_logits(raw, w, prompts)
        trace_util.compare(got, want, F32_TOL, "long decoding")
        other = dict(r0=[(prompts["r0"][0] + 1) % 50] + prompts["r0"][1:])
        moved = float((expected_logits(raw, w, other)["r0"][-1] - want["r0"][-1]).abs().max()) / float(want["r0"].abs().max())
        assert moved > 1e-4, "the first token must still matter at the end for this test to mean anything"


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
        assert float((got[key] - row).abs().max()) < 1e-5 * float(row.abs().max())


def generate(name, device, dtype, lengths=(9, 30, 2, 17, 23), budget=32, blocks=24, **engine):
    from mini_inference_engine_amd import LLMEngine, SamplingParams
    raw, cfg, weights = make(name, torch.float32 if dtype == "float32" else torch.bfloat16, sharp=dtype == "float32")
    prompts = list(trace_util.random_prompts(raw["vocab"], list(lengths), seed=4).values())
    ecfg = EngineConfig(num_blocks=blocks, max_num_seqs=3, max_num_batched_tokens=budget, max_model_len=max(128, max(lengths) + 32), **engine)
    kw = dict(device="cpu", backend=TorchBackend(torch.float32)) if device == "cpu" else {}
    eng = LLMEngine(cfg, ecfg, dtype=dtype, verbose=False, weights=weights, **kw)
    outs = eng.generate(prompts, SamplingParams(max_tokens=30, ignore_eos=True))          # through a window's edge
    wf = {k: v.float() for k, v in weights.items()}
    for prompt, out in zip(prompts, outs):
        ids = list(prompt) + list(out.output_ids)
        assert len(out.output_ids) == 30
        logits = plain.forward(raw, wf, ids)
        for i, tok in enumerate(out.output_ids):
            row = logits[len(prompt) + i - 1]
            slack = (F32_TOL if dtype == "float32" else 2 * BF16_TOL_PER_LAYER * len(raw["layers"])) * float(row.abs().max())
            assert float(row.max() - row[tok]) <= slack, f"token {i} of a request is not the plain implementation's choice"
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
    return make_step(rows, slots)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_projections_through_a_convolution_kernel(hip, dtype):
    """Rows of one token, of fewer tokens than the convolution looks back, and of many, over tails that hold something;
    values left for and mixed with another layer's; sizes that fill no wave."""
    ops, g = hip[dtype], torch.Generator().manual_seed(31)
    for (rows, Hq, Hkv, dim, vdim, K, nf, norm, share) in (([1, 1, 1], 6, 2, 16, 24, 3, 6, True, "out"), ([37, 1, 2], 3, 3, 24, 8, 4, 12, True, "mix"),
                                                          ([2, 3, 1, 70], 4, 1, 10, 14, 5, 3, True, None), ([64], 16, 4, 64, 64, 2, 32, False, "mix"),
                                                          ([1, 1], 2, 1, 130, 70, 4, 20, True, "out"), ([9, 1], 1, 1, 8, 8, 1, 0, True, None),
                                                          ([1, 1, 1], 3, 1, 12, 20, 7, 6, True, None)):
        T, P = sum(rows), -(-max(dim, vdim) // 16) * 16
        C, q_col = (Hq + Hkv) * dim + Hkv * vdim, 5
        sums = _rand((T, q_col + C + 3), torch.float32, g, 2.0)
        taps = _rand((C, K), torch.float32, g)
        tail = _rand((len(rows) + 2, max(1, K - 1), C), torch.float32, g)
        qn, kn = (_rand((dim,), torch.float32, g) + 1, _rand((dim,), torch.float32, g) + 1) if norm else (None, None)
        inv_freq = (50.0 ** -(torch.arange(nf, dtype=torch.float32) / nf)).cuda() if nf else None
        positions = (torch.arange(T, dtype=torch.int32) * 3 + 5).cuda()
        pages, page = T // 16 + 3, 16
        slots = torch.randperm((pages - 1) * page, generator=g)[:T].to(torch.int32).cuda() + page
        kc, vc = torch.full((pages, Hkv, page, P), 7.0, dtype=dtype).cuda(), torch.full((pages, Hkv, P, page), 7.0, dtype=dtype).cuda()
        kw, vw = kc.clone(), vc.clone()
        step = step_of(rows)
        other = _rand((T, Hkv * vdim), torch.float32, g)
        out1, out2 = torch.zeros(T, Hkv * vdim).cuda(), torch.zeros(T, Hkv * vdim).cuda()
        kws = lambda o: dict(values_out=o) if share == "out" else dict(value_mix=(0.3, other)) if share == "mix" else {}        # noqa: E731
        cols = (q_col, q_col + Hq * dim, q_col + (Hq + Hkv) * dim)
        t1, t2 = tail.clone(), tail.clone()
        want = ref.ref_qkv_finish(sums, *cols, Hq, Hkv, dim, vdim, P, positions, inv_freq, "half", kw, vw, slots, qn, kn, 1e-5, None, dtype,
                                  norm_per_head=True, rotation_scale=1.3, conv=(taps, t2, step.host["row_start"], step.host["state_slots"]), **kws(out2))
        got = ops.qkv_finish(sums, *cols, Hq, Hkv, dim, vdim, P, positions, inv_freq, "half", kc, vc, slots, q_norm=qn, k_norm=kn, eps=1e-5,
                             norm_per_head=True, rotation_scale=1.3, conv=(taps, t1, step), **kws(out1))
        what = f"rows {rows}, {Hq}/{Hkv} heads of {dim}/{vdim}, {K} taps"
        tol = 1e-5 if dtype == torch.float32 else TOL[dtype]
        close(got, want, tol, f"queries, {what}")
        close(kc, kw, tol, f"keys, {what}")
        close(vc, vw, tol, f"values, {what}")
        if share == "out":
            close(out1, out2, 2e-6, f"values left, {what}")
        assert torch.equal(t1, t2), f"tails, {what}"


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_short_convolution_gate_and_clamped_unit_kernels(hip, dtype):
    ops, g = hip[dtype], torch.Generator().manual_seed(32)
    for (rows, C, K, act) in (([1, 1, 1], 48, 4, "silu"), ([37, 1, 2], 70, 3, "silu"), ([2, 3, 1, 70], 333, 6, "none"), ([130], 512, 2, "silu"), ([5], 16, 1, "silu")):
        T = sum(rows)
        x = _rand((T, C + 9), torch.float32, g)
        taps, bias = _rand((C, K), torch.float32, g), _rand((C,), torch.float32, g)
        tail = _rand((len(rows) + 2, max(1, K - 1), C), torch.float32, g)
        step = step_of(rows)
        t1, t2 = tail.clone(), tail.clone()
        got = ops.short_conv(x, 4, C, taps, bias, t1, step, activation=act)
        want = ref.ref_short_conv(x, 4, C, taps, bias, t2, step.host["row_start"], step.host["state_slots"], act)
        close(got, want, 2e-6, f"short_conv rows {rows}, {K} taps")
        assert torch.equal(t1, t2), f"tails, rows {rows}, {K} taps"
    for (T, H, dv, P) in ((1, 3, 24, 32), (37, 2, 14, 16), (130, 8, 64, 64), (5, 16, 128, 128)):
        o, gate = _rand((T, H * P), dtype, g), _rand((T, H * dv + 6), torch.float32, g, 2.0)
        want = ref.ref_gate_heads(o, gate, 4, H, dv, P, 0.7, dtype)
        close(ops.gate_heads(o, gate, 4, H, dv, P, scale=0.7), want, TOL[dtype], f"gate_heads {T}x{H}x{dv}")
        wide = torch.zeros(T, H * dv + 16, dtype=dtype).cuda()
        ops.gate_heads(o, gate, 4, H, dv, P, out=wide[:, 8:8 + H * dv], scale=0.7)
        close(wide[:, 8:8 + H * dv], want, TOL[dtype], "gate_heads into columns")
        assert float(wide[:, :8].abs().max()) == 0.0 and float(wide[:, 8 + H * dv:].abs().max()) == 0.0
    for (T, W, I) in ((1, 64, 48), (9, 72, 40), (16, 128, 112), (37, 64, 50), (130, 96, 64), (300, 70, 36)):
        x, w = _rand((T, W), dtype, g), _rand((2 * I, W), dtype, g, 3 * W ** -0.5)
        for limit, alpha, shift in ((2.0, 1.702, 1.0), (0.5, 1.0, 0.0)):
            gu = ref.ref_linear(x, w, None, torch.float32).double()
            close(ops.linear_clamped_glu(x, w, I, limit, alpha, shift), ref.ref_clamped_glu(gu, I, limit, alpha, shift), 1e-5 if dtype == torch.float32 else 1e-2,
                  f"clamped unit {T}x{W}->{I}")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_state_space_kernel(hip, dtype):
    """Whole rows and (bfloat16 mode) rows in chunks, groups from one to one a head, states of sizes that fill no tile, slots
    that hold something, decays from fast to slow, norm parts that cut through heads."""
    ops, g = hip[dtype], torch.Generator().manual_seed(33)
    for (rows, H, G, N, dv, parts) in (([1, 1, 1], 4, 2, 16, 32, 2), ([37, 1, 5], 6, 3, 24, 8, 4), ([200], 5, 1, 7, 6, 3), ([130, 70, 1, 64, 65], 4, 4, 48, 64, 1),
                                       ([300, 2], 2, 1, 128, 64, 2), ([9], 1, 1, 300, 40, 1), ([3, 190], 3, 1, 132, 100, 1), ([70], 2, 2, 20, 200, 5)):
        T, inner = sum(rows), H * dv
        u = _rand((T, inner + 2 * G * N + 4), torch.float32, g)
        b_col, c_col = inner, inner + G * N
        sums = _rand((T, 4 + inner + H), torch.float32, g)
        dt_bias, rate, skip = _rand((H,), torch.float32, g) - 1, torch.exp(_rand((H,), torch.float32, g)), _rand((H,), torch.float32, g)
        nw = _rand((inner,), torch.float32, g) + 1
        state = _rand((len(rows) + 2, H, N, dv), torch.float32, g, 0.5)
        step = step_of(rows)
        s1, s2 = state.clone(), state.clone()
        got = ops.state_space(u, b_col, c_col, sums, 4, 4 + inner, H, G, N, dv, dt_bias, rate, skip, parts, nw, 1e-5, s1, step, scale=0.8)
        want = ref.ref_state_space(u, b_col, c_col, sums, 4, 4 + inner, H, G, N, dv, dt_bias, rate, skip, parts, nw, 1e-5, s2,
                                   step.host["row_start"], step.host["state_slots"], 0.8, dtype)
        close(s1, s2, 1e-5, f"state space: state, rows {rows}")
        close(got, want, 2e-5 if dtype == torch.float32 else 1e-2, f"state space rows {rows}, {H} heads of {N} x {dv}")
        assert torch.equal(s1[0], state[0]) and torch.equal(s1[-1], state[-1]), "slots of no row are left alone"
        wide = torch.zeros(T, inner + 8, dtype=dtype).cuda()
        ops.state_space(u, b_col, c_col, sums, 4, 4 + inner, H, G, N, dv, dt_bias, rate, skip, parts, nw, 1e-5, state.clone(), step, out=wide[:, 8:], scale=0.8)
        assert torch.equal(wide[:, 8:], got) and float(wide[:, :8].abs().max()) == 0.0


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_matrix_memory_kernel(hip, dtype):
    """As above for the matrix memory: gates at both ends of their cap, a running maximum that rises and falls, rows longer
    than one round of the maximum's scan."""
    ops, g = hip[dtype], torch.Generator().manual_seed(34)
    for (rows, H, d, dv, cap, spread) in (([1, 1, 1], 2, 16, 32, 15.0, 3.0), ([37, 1, 5], 3, 24, 8, 4.0, 8.0), ([200], 1, 10, 14, 15.0, 3.0),
                                          ([130, 70, 1, 64, 65], 4, 48, 64, 12.0, 10.0), ([300, 2], 2, 64, 128, 15.0, 3.0), ([9], 1, 260, 72, 15.0, 1.0),
                                          ([3, 190], 1, 130, 300, 8.0, 5.0), ([1100], 1, 8, 12, 15.0, 4.0)):
        T, nk, nv = sum(rows), H * d, H * dv
        cols = dict(q=3, k=3 + nk, v=3 + 2 * nk, g=3 + 2 * nk + nv, i=3 + 2 * nk + 2 * nv, f=3 + 2 * nk + 2 * nv + H)
        sums = _rand((T, cols["f"] + H + 2), torch.float32, g)
        sums[:, cols["i"]:cols["i"] + 2 * H] *= spread
        ib, fb, nw = _rand((H,), torch.float32, g), _rand((H,), torch.float32, g) + 2, _rand((nv,), torch.float32, g) + 1
        slots = len(rows) + 2
        state, norm, top = _rand((slots, H, d, dv), torch.float32, g, 0.5), _rand((slots, H, d), torch.float32, g), _rand((slots, H), torch.float32, g)
        step = step_of(rows)
        first, second = [t.clone() for t in (state, norm, top)], [t.clone() for t in (state, norm, top)]
        got = ops.mlstm(sums, cols, H, d, dv, ib, fb, cap, d ** -0.5, nw, 1e-5, *first, step, scale=1.2)
        want = ref.ref_mlstm(sums, cols, H, d, dv, ib, fb, cap, d ** -0.5, nw, 1e-5, *second, step.host["row_start"], step.host["state_slots"], 1.2, dtype)
        what = f"rows {rows}, {H} heads of {d} x {dv}"
        for a, b, name in zip(first, second, ("memory", "normaliser", "maximum")):
            close(a, b, 2e-5, f"{name}, {what}")
        close(got, want, 5e-5 if dtype == torch.float32 else 1e-2, f"mlstm {what}")
        assert all(torch.equal(a[0], b[0]) and torch.equal(a[-1], b[-1]) for a, b in zip(first, (state, norm, top))), "slots of no row are left alone"


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_kept_first_keys_and_head_sink_kernels(hip, dtype):
    """Decode rows and portions over random pages against the torch operation: kept tokens of none to several blocks, windows
    shorter and longer than they are, rows that begin among the kept tokens, before and after the window leaves them,
    grouped heads, contexts split over workgroups."""
    from test_mutusun import AttentionCase
    ops, g = hip[dtype], torch.Generator().manual_seed(35)
    rows = [(0, 1), (5, 1), (23, 1), (63, 1), (64, 1), (200, 1), (700, 1), (0, 50), (17, 31), (63, 2), (100, 130), (0, 300), (400, 70)]
    for (Hq, Hkv, P, window, keep, sinks) in ((6, 2, 16, 24, 3, True), (3, 3, 32, 16, 20, True), (4, 1, 16, 40, 1, False), (2, 2, 48, 1, 66, True),
                                              (8, 2, 64, 100, 130, True), (4, 4, 128, 33, 32, False), (16, 4, 64, 140, 64, True), (8, 4, 64, None, 0, True),
                                              (4, 2, 256, 50, 9, True), (4, 2, 64, 50, 0, True)):
        case = AttentionCase(rows, Hkv, P, dtype, g)
        q = _rand((case.num_tokens, Hq * P), dtype, g)
        sink = _rand((Hq,), torch.float32, g, 2.0) + 1.0 if sinks else None
        args = (q, Hq, Hkv, P, case.k, case.v)
        want = ref.ref_paged_attention(*args, case.block_tables, case.token_row, case.positions, P ** -0.5, window, torch.float32, sink=sink, keep_first=keep)
        kw = dict(sink=sink, keep_first=keep)
        what = f"heads {Hq}/{Hkv} of {P}, window {window}, {keep} kept"
        got = ops.paged_attention(*args, case.group, case.step, P ** -0.5, window, **kw)
        close(got, want, 1e-5 if dtype == torch.float32 else 1.5e-2, what)
        if dtype == torch.bfloat16:
            close(ops.paged_attention(*args, case.group, case.step, P ** -0.5, window, force_generic=True, **kw), want, 1.5e-2, f"32-bit kernel, {what}")
            for splits in (1, 3):
                close(ops.paged_attention(*args, case.group, case.step, P ** -0.5, window, num_splits=splits, **kw), want, 1.5e-2, f"{splits} splits, {what}")


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
    run_family(name, family, tmp_path, "cuda", "bfloat16", BF16_TOL_PER_LAYER * len(raw["layers"]))


@pytest.mark.gpu
def test_keys_at_the_edges_of_the_window_and_of_the_kept_tokens():
    window_runs("cuda")


@pytest.mark.gpu
def test_a_far_key_and_the_first_token_are_seen_by_the_kernels():
    far_key_runs("cuda")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_in_chunks_of_the_recurrences(dtype):
    """Prompts of several hundred tokens, whole and in uneven portions: the recurrences run in chunks side by side in
    bfloat16 and whole in float32; the windows end long before the prompts do."""
    raw, cfg, weights = make("D", torch.float32 if dtype == "float32" else torch.bfloat16, sharp=dtype == "float32")
    prompts = trace_util.random_prompts(raw["vocab"], [400, 129], seed=8)
    want = expected_logits(raw, weights, prompts)
    for steps in (trace_util.whole(prompts), trace_util.portions(prompts, sizes=(130, 2, 65, 64, 200))):
        runner = ModelRunner(cfg, weights=weights, dtype=dtype, num_pages=40, max_rows=2, max_step_tokens=512, max_model_len=39 * 16)
        got = {k: v.cpu() for k, v in trace_util.run_on_runner(runner, steps).items()}
        if dtype == "float32":
            trace_util.compare(got, want, F32_TOL, "long prompts")
        else:
            compare_bf16(got, want, BF16_TOL_PER_LAYER * len(raw["layers"]), "long prompts")


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(dtype):
    eng = generate("A", "cuda", dtype)
    assert eng.num_graph_steps > 0, "decode steps run as captured graphs"


@pytest.mark.gpu
def test_captured_prompt_portions_run_the_recurrences_in_chunks():
    """Prompts in portions of exactly the step's budget of 128 tokens: the captured step of such a portion is replayed for
    portion after portion of several requests, each going on from its own states."""
    eng = generate("D", "cuda", "bfloat16", lengths=(256, 384, 130, 256), budget=128, blocks=80)
    assert eng.num_graph_steps > 0 and eng.runner.portion_graphs[-1].tokens == 128


# --------------------------------------------------------------------------------------------- the command line
def test_random_model_of_the_named_size_is_what_the_loader_reads(tmp_path):
    from safetensors.torch import load_file
    from test_labirax import run_cli
    folder = str(tmp_path / "m")
    run_cli("random-model", "--shape", "pokulorn-tiny", "--seed", "3", "--dtype", "float32", "--out", folder)
    cfg, arch = load_model_config(folder)
    assert arch.name == "Pokulorn" and [layer.mlp is None for layer in cfg.layers] == [False] * 5 + [True]
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
    run_cli("random-model", "--shape", "pokulorn-tiny", "--seed", "3", "--dtype", "float32", "--out", folder)
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
