"""The Figotar design in the serving engine against the float64 oracle (tests/oracles): small
configurations with random weights written as model folders (config.json + model.safetensors),
loaded through the engine's own registry and driven through its step function (``feed``), its
scheduler (``generate``) and the replay command line.  The CPU runs use the op library's torch
references, the GPU runs (marked) the HIP kernels; both in float32 (sharp) and bfloat16.

Weights are rounded to bfloat16 as stored, so product and oracle see the same numbers.
"""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

from distributed_llm_amd.engine.llm_engine import BS, LLMEngine
from distributed_llm_amd.engine.sampling import SamplingParams
from oracles import figotar_oracle as orc

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ----------------------------------------------------------------------------- model folders

def ff(n=20):
    return {"kind": "dense", "ff": n}


def attn(heads=4, kv_heads=2, dim=8, vdim=6, scale=0.4, size=9, temp=(0.4, 7), mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size:
        m["mask"] = {"size": size}
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def latent(heads=3, dim=6, rot=4, vdim=10, rank=12, q_rank=14, base=100.0, scale=0.4, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": scale,
                      "rot": {"dims": rot, "base": base}}}


def mlstm(heads=3, dim=5, vdim=9, cap=6.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def make_cfg(layers, width=24, vocab=40, eps=1e-5):
    return {"architecture": "Figotar", "norm": {"eps": eps}, "vocab": vocab, "width": width, "layers": json.loads(json.dumps(layers))}


def make_weights(cfg, seed=0, qk_gain=1.0, sink=1.0, igate=0.0, fgate=2.0, gate_gain=1.0):
    g = torch.Generator().manual_seed(seed)
    W, wd = {}, cfg["width"]
    r = lambda *s, k=1.0: torch.randn(*s, generator=g) * k
    lin = lambda o, i, k=1.0: r(o, i, k=k / math.sqrt(i))
    W["embed"], W["head"], W["final.norm"] = r(cfg["vocab"], wd), lin(cfg["vocab"], wd), 0.2 * r(wd)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if L.get("mlp") else ()):
            W[p + n] = 0.3 * r(wd) - 0.1
        W[p + "mix.o"] = lin(wd, H * dv)
        if L["type"] == "attention":
            G = m["kv_heads"]
            for n, c, k in (("q", H * d, qk_gain), ("k", G * d, qk_gain), ("v", G * dv, 1.0)):
                W[p + "mix." + n], W[p + f"mix.{n}.b"] = lin(c, wd, k), 0.4 * r(c)
            W[p + "mix.g"] = lin(H, wd, 1.5)
        elif L["type"] == "latent_attention":
            rd, rank, qr = m["rot_dim"], m["kv_rank"], m["q_rank"]
            W[p + "mix.dq"], W[p + "mix.dq.norm"] = lin(qr, wd), 1 + 0.3 * r(qr)
            W[p + "mix.uq"] = lin(H * (d + rd), qr, qk_gain)
            W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = lin(rank + rd, wd), 1 + 0.3 * r(rank)
            W[p + "mix.uk"], W[p + "mix.uv"] = lin(H * d, rank, qk_gain), lin(H * dv, rank)
            W[p + "mix.g"], W[p + "mix.sink"] = lin(H, wd, 1.5), sink + 0.5 * r(H)
        else:
            W[p + "mix.q"], W[p + "mix.k"], W[p + "mix.v"] = lin(H * d, wd), lin(H * d, wd), lin(H * dv, wd)
            W[p + "mix.g"], W[p + "mix.norm"] = lin(H * dv, wd, 1.5), 1 + 0.3 * r(H * dv)
            W[p + "mix.i"], W[p + "mix.i.b"] = lin(H, wd, gate_gain), igate + 0.5 * r(H)
            W[p + "mix.f"], W[p + "mix.f.b"] = lin(H, wd, gate_gain), fgate + 0.5 * r(H)
        if L.get("mlp"):
            n = L["mlp"]["ff"]
            for name, o, k in (("gate", n, wd), ("up", n, wd), ("down", wd, n)):
                W[p + "mlp." + name], W[p + f"mlp.{name}.b"] = lin(o, k), 0.3 * r(o)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}


def write_model(path, cfg, W):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(W, os.path.join(path, "model.safetensors"))
    return str(path)


def engine(path, device, dtype, rows=3, tokens=256):
    return LLMEngine(path, device=device, dtype=dtype, max_num_seqs=rows, max_model_len=tokens,
                     num_kv_blocks=(tokens + BS - 1) // BS, prefix_cache=False)


def close(got, want, dtype, what=""):
    """Row-wise error after removing the mean, relative to the logits' spread."""
    want = want.to(torch.float32)
    d = got.float() - want
    d = d - d.mean(-1, keepdim=True)
    spread = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    rows = d.pow(2).mean(-1).sqrt() / spread
    limit = 3e-4 if dtype == torch.float32 else 0.12      # bfloat16: rounding at these widths gives 0.01 to 0.05
    assert float(rows.max()) < limit, f"{what}: relative error {float(rows.max()):.3g} at row {int(rows.argmax())}"


# every mixer, with and without a feed-forward; sizes differ from layer to layer
FULL = [mlstm(mlp=ff()), attn(mlp=ff(28)), latent(mlp=ff()), attn(heads=6, kv_heads=3, dim=6, vdim=10, size=21, temp=(0.2, 16)),
        mlstm(heads=2, dim=18, vdim=20, cap=3.0), latent(heads=5, dim=4, rot=6, vdim=4, rank=8, q_rank=9, base=5000.0, mlp=ff(33))]

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]


def toks(n, vocab=40, seed=0):
    g = torch.Generator().manual_seed(100 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


@pytest.fixture(scope="module")
def full_model(tmp_path_factory):
    cfg = make_cfg(FULL)
    W = make_weights(cfg, seed=1)
    return write_model(tmp_path_factory.mktemp("full"), cfg, W), cfg, W


_WANT = {}


def full_want(full_model, t):
    key = tuple(t)
    if key not in _WANT:
        _WANT[key] = orc.forward(t, full_model[2], full_model[1])
    return _WANT[key]


# ----------------------------------------------------------------------------- each mechanism alone

SINGLE = {
    "attention": ([attn()], {}), "attention-with-ff": ([attn(mlp=ff(31))], {}),
    "attention-ungrouped": ([attn(heads=3, kv_heads=3, dim=5, vdim=9, size=4)], {}),
    "attention-one-kv-head": ([attn(heads=4, kv_heads=1, dim=6, vdim=4, size=30)], {}),
    "attention-one-head": ([attn(heads=1, kv_heads=1, dim=7, vdim=5)], {}),
    "attention-no-window": ([attn(size=0)], {}), "attention-window-one": ([attn(size=1)], {}), "attention-window-two": ([attn(size=2)], {}),
    "attention-window-beyond": ([attn(size=1000)], {}), "attention-no-temperature": ([attn(temp=None)], {}),
    "attention-temperature-every-token": ([attn(temp=(0.5, 1), size=20)], {}), "attention-cooling": ([attn(temp=(-0.2, 5))], {}),
    "attention-wide-heads": ([attn(heads=2, kv_heads=1, dim=72, vdim=130, scale=0.1, size=16)], {}),
    "attention-many-heads": ([attn(heads=36, kv_heads=2, dim=4, vdim=3)], {}), "attention-seven-heads": ([attn(heads=7, kv_heads=7, dim=4, vdim=3, size=33)], {}),
    "latent": ([latent()], {}), "latent-with-ff": ([latent(mlp=ff(7))], {}),
    "latent-one-head": ([latent(heads=1, dim=9, rot=2, vdim=3, rank=5, q_rank=3)], {}),
    "latent-many-heads": ([latent(heads=20, dim=4, rot=8, vdim=8, rank=16)], {}),
    "latent-wide": ([latent(heads=2, dim=40, rot=24, vdim=72, rank=136, q_rank=50, scale=0.15)], {}),
    "latent-mostly-rotated": ([latent(heads=2, dim=2, rot=16, vdim=4, rank=6, base=20.0)], {}),
    "mlstm": ([mlstm()], {}), "mlstm-with-ff": ([mlstm(mlp=ff())], {}), "mlstm-one-head": ([mlstm(heads=1, dim=3, vdim=2)], {}),
    "mlstm-wide": ([mlstm(heads=2, dim=70, vdim=40, cap=15.0)], {}), "mlstm-tight-cap": ([mlstm(cap=0.5)], {}),
    "mlstm-strong-input-gates": ([mlstm(cap=12.0)], {"igate": 5.0, "gate_gain": 3.0}), "mlstm-forgetful": ([mlstm(cap=12.0)], {"fgate": -4.0}),
    "large-eps": ([attn(mlp=ff()), latent(), mlstm()], {"eps": 0.3}),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_mechanism_alone(tmp_path, device, dtype, name):
    layers, kw = SINGLE[name]
    kw = dict(kw)
    cfg = make_cfg(layers, **({"eps": kw.pop("eps")} if "eps" in kw else {}))
    W = make_weights(cfg, seed=3, **kw)
    eng = engine(write_model(tmp_path / "m", cfg, W), device, dtype)
    t = toks(43)
    want = orc.forward(t, W, cfg)
    got = [eng.feed([("a", t[:37], list(range(37)))])] + [eng.feed([("a", t[i:i + 1], [0])]) for i in range(37, 43)]
    close(torch.cat(got), want, dtype, name)


def test_layer_stream_matches(full_model):
    """The stream after every layer, not only the logits."""
    path, cfg, W = full_model
    eng = engine(path, "cpu", torch.float32)
    t = toks(29, seed=7)
    taps = []
    orc.forward(t, W, cfg, taps)
    eng.model.tap = []
    eng.feed([("a", t, [0])], ["a"])
    assert len(eng.model.tap) == len(taps) == len(FULL)
    for i, (a, b) in enumerate(zip(eng.model.tap, taps)):
        assert torch.allclose(a.double(), b, atol=3e-4, rtol=1e-4), f"layer {i}"


@pytest.mark.parametrize("coef,every", [(0.1, 8), (-0.05, 1), (2.0, 100), (0.7, 4096), (0.3, 2.5)])
def test_query_factors(coef, every):
    """The table of query factors, one number per position, at and around every step of the floor."""
    from distributed_llm_amd.models.configs import figotar_config
    from distributed_llm_amd.models.registry import build_model
    cfg = figotar_config(make_cfg([attn(temp=(coef, every))]))
    m = build_model(cfg, device="cpu", dtype=torch.float32)
    m.ensure_positions(5000)
    (tab,) = m._qtab.values()
    assert tab.numel() >= 5000 and tab.dtype == torch.float32
    want = torch.tensor([orc.temperature(p, {"coef": coef, "every": every}) for p in range(5000)], dtype=torch.float64)
    assert torch.allclose(tab[:5000].double(), want, atol=1e-6)
    if every == 8:
        assert tab[6] == 1.0 and tab[7] > 1.0 and tab[7] == tab[14] and tab[15] > tab[14]


# ----------------------------------------------------------------------------- cutting the prompt

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[50], [1] * 50, [2] * 25, [17, 2, 15, 1, 1, 3, 11], [16, 16, 16, 2], [9, 9, 9, 9, 9, 5], [3, 47], [49, 1]])
def test_portions_and_decoding(full_model, device, dtype, cuts):
    if device == "cpu" and dtype == torch.bfloat16 and len(cuts) > 8:
        pytest.skip("bfloat16 matrix products on the CPU are slow; the GPU run covers this case")
    eng = engine(full_model[0], device, dtype)
    t = toks(50, seed=1)
    got, at = [], 0
    for n in cuts:
        got.append(eng.feed([("r", t[at:at + n], list(range(n)))], ["r"] if at + n == len(t) else []))
        at += n
    close(torch.cat(got), full_want(full_model, t), dtype, f"cuts {cuts[:4]}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_and_long_decoding(full_model, device, dtype):
    """Positions 0, 1, 2 on their own, then 150 single-token steps past several page borders and
    every layer's window."""
    if device == "cpu" and dtype == torch.bfloat16:
        pytest.skip("bfloat16 matrix products on the CPU are slow; the GPU run covers this case")
    eng = engine(full_model[0], device, dtype)
    t = toks(153, seed=2)
    want = full_want(full_model, t)
    got = [eng.feed([("r", t[i:i + 1], [0])]) for i in range(len(t))]
    close(torch.cat(got[:3]), want[:3], dtype, "first tokens")
    close(torch.cat(got), want, dtype, "long decoding")
    for n in (1, 2):      # a whole request of one and of two tokens
        close(eng.feed([("s", t[:n], list(range(n)))], ["s"]), want[:n], dtype, f"{n}-token request")


# ----------------------------------------------------------------------------- batches, rows, pages

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("expand_min", [1, 10 ** 9])      # latent layers: keys and values of every portion made from latents, or never
def test_mixed_batches_and_reuse(full_model, monkeypatch, device, dtype, expand_min):
    """Unequal requests share steps (portions beside single tokens); more requests than batch rows
    and more tokens than pages pass through, so rows, state slots and pages are used again."""
    from distributed_llm_amd.ops import seqmix
    monkeypatch.setattr(seqmix, "LATENT_EXPAND_MIN", expand_min)
    eng = engine(full_model[0], device, dtype, rows=3, tokens=112)       # 7 pages of 16
    lens = [40, 9, 33, 1, 21, 30, 5]
    reqs = {f"q{i}": toks(n, seed=10 + i) for i, n in enumerate(lens)}
    at = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    waiting, live = list(reqs), []
    pattern, step = [7, 1, 2, 1, 16, 1, 3, 1], 0
    while waiting or live:
        used = sum((len(reqs[k]) + BS - 1) // BS for k in live)
        while waiting and len(live) < 3 and used + (len(reqs[waiting[0]]) + BS - 1) // BS <= 7:
            used += (len(reqs[waiting[0]]) + BS - 1) // BS
            live.append(waiting.pop(0))
        entries, end = [], []
        for j, k in enumerate(live):
            if step % 5 == 3 and j == 1:      # a live request left out of the step
                continue
            n = min(pattern[(step + 3 * j) % len(pattern)], len(reqs[k]) - at[k])
            entries.append((k, reqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        out = eng.feed(entries, end)
        o = 0
        for k, tk, _ in entries:
            got[k].append(out[o:o + len(tk)])
            o += len(tk)
        live = [k for k in live if k not in end]
        step += 1
    for k in reqs:
        close(torch.cat(got[k]), full_want(full_model, reqs[k]), dtype, k)
    assert eng.bm.num_free_blocks() == 7 and len(eng._free_rows) == 3


# ----------------------------------------------------------------------------- window edges, distance, far keys, sinks, memory

def _needle(cfg, W, n, pos_a, pos_b, fill=0):
    """The token whose place (position ``pos_a`` instead of ``pos_b``) moves the oracle's last logits
    most, and that movement relative to the logits' spread."""
    best = (0.0, 1)
    for tok in range(1, 12):
        a, b = [fill] * n, [fill] * n
        a[pos_a], b[pos_b] = tok, tok
        la, lb = orc.forward(a, W, cfg)[-1], orc.forward(b, W, cfg)[-1]
        best = max(best, (float((la - lb).std() / la.std()), tok))
    return best


def _prompt_decode_cut(eng, t, cut, what, want):
    """The whole prompt in one step; then cut at ``cut``, the rest as a portion, the last token alone."""
    n = len(t)
    close(eng.feed([("w", t, list(range(n)))], ["w"]), want, torch.float32, f"prompt, {what}")
    got = [eng.feed([("c", t[:cut], list(range(cut)))])] if cut else []
    if n - 1 > cut:
        got.append(eng.feed([("c", t[cut:n - 1], list(range(n - 1 - cut)))]))
    got.append(eng.feed([("c", t[n - 1:], [0])], ["c"]))
    close(torch.cat(got), want, torch.float32, f"cut and decoded, {what}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,n", [(2, 42), (15, 45), (16, 48), (17, 60), (63, 126), (64, 100), (65, 131), (100, 130)])
def test_window_edges(tmp_path, device, size, n):
    """A prompt of one repeated token with one other token placed on the oldest position the last
    position sees or just before it, chosen and scaled so that the row's weight lies on it (twelve heads:
    the last ones hardly fall with the distance): a window that is one key off moves the logits."""
    cfg = make_cfg([attn(heads=12, kv_heads=3, dim=8, vdim=5, scale=2.0, size=size, temp=(0.5, 32))], width=16)
    edge = n - size
    for seed in range(size, size + 1000, 100):      # the first weights that show the edge
        W = make_weights(cfg, seed=seed, qk_gain=2.0)
        move, tok = _needle(cfg, W, n, edge, edge - 1)
        if move > 0.1:
            break
    assert move > 0.1, "the test's weights do not show the edge"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32)
    for at in (edge - 1, edge, min(edge + 1, n - 2)):
        t = [0] * n
        t[at] = tok
        _prompt_decode_cut(eng, t, at, f"other token at {at} of {n}", orc.forward(t, W, cfg))
    t = [0] * n
    t[edge] = tok
    got = [eng.feed([("d", t[:n - 4], list(range(n - 4)))])] + [eng.feed([("d", t[i:i + 1], [0])]) for i in range(n - 4, n)]
    close(torch.cat(got), orc.forward(t, W, cfg), torch.float32, "the edge decoded")


@pytest.mark.parametrize("device", DEVICES)
def test_scores_fall_with_the_distance(tmp_path, device):
    """Without a window: identical keys at every distance, so that only the slopes tell them apart; a slope
    counted from one token off, or with the heads in another order, shows."""
    cfg = make_cfg([attn(heads=6, kv_heads=2, dim=6, vdim=6, size=0, temp=None, scale=0.05)], width=16)
    W = make_weights(cfg, seed=4)
    t = [3] * 90
    t[0] = t[40] = 5
    want = orc.forward(t, W, cfg)
    old = orc.slope
    try:
        orc.slope = lambda h, H: old(h + 1, H)
        moved = orc.forward(t, W, cfg)
    finally:
        orc.slope = old
    assert float((moved - want).std() / want.std()) > 0.01, "the test's weights do not show the slopes"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32)
    _prompt_decode_cut(eng, t, 37, "slopes", want)


@pytest.mark.parametrize("device", DEVICES)
def test_temperature_steps(tmp_path, device):
    """A strong temperature whose step falls on page borders and portion starts: a floor taken one position
    early or late moves the rows beside it."""
    cfg = make_cfg([attn(heads=4, kv_heads=4, dim=8, vdim=6, scale=0.2, size=40, temp=(1.0, 16))], width=16)
    W = make_weights(cfg, seed=7)
    t = toks(70, seed=3)
    want = orc.forward(t, W, cfg)
    old = orc.temperature
    try:
        orc.temperature = lambda p, qt: old(p - 1, qt)
        late = orc.forward(t, W, cfg)
    finally:
        orc.temperature = old
    for p in (15, 31, 47):
        assert float((late[p] - want[p]).std() / want[p].std()) > 0.005, "the test's weights do not show the step"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32)
    for cut in (14, 15, 16, 47):
        _prompt_decode_cut(eng, t, cut, f"cut at {cut}", want)
    got = [eng.feed([("d", t[:13], list(range(13)))])] + [eng.feed([("d", t[i:i + 1], [0])]) for i in range(13, 70)]
    close(torch.cat(got), want, torch.float32, "steps decoded")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("expand_min", [1, 10 ** 9])
@pytest.mark.parametrize("n", [15, 16, 17, 63, 64, 65, 130, 330])
def test_far_keys_of_the_latent_attention(tmp_path, monkeypatch, device, n, expand_min):
    """A softmax so sharp that one key, far back among repeated ones and on either side of a page (16)
    or key-tile (32, 64) border, carries a row; prompts and decoded rows."""
    from distributed_llm_amd.ops import seqmix
    monkeypatch.setattr(seqmix, "LATENT_EXPAND_MIN", expand_min)
    cfg = make_cfg([latent(heads=2, dim=8, rot=2, vdim=5, rank=10, base=1e4, scale=2.0)], width=16)
    for seed in range(n, n + 500, 100):
        W = make_weights(cfg, seed=seed, qk_gain=2.0)
        moves = []
        for tok in range(1, 12):
            t = [0] * n
            a = orc.forward(t, W, cfg)[-1]
            t[1] = tok
            moves.append((float((orc.forward(t, W, cfg)[-1] - a).std() / a.std()), tok))
        move, tok = max(moves)
        if move > 0.1:
            break
    assert move > 0.1, "the test's weights do not show the far key"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32, tokens=512)
    for at in sorted({1, n // 2, n - 2}):
        t = [0] * n
        t[at] = tok
        _prompt_decode_cut(eng, t, at, f"other token at {at} of {n}", orc.forward(t, W, cfg))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("expand_min", [1, 10 ** 9])
@pytest.mark.parametrize("sink", [-6.0, 0.0, 4.0, 30.0])
def test_the_sink_takes_weight(tmp_path, monkeypatch, device, sink, expand_min):
    """The sink's score against small ones: from no share of a row's denominator to nearly all of it; not
    scaled, counted once however the keys are split.  The layer's norm hides a common factor, so two
    heads have sinks far apart."""
    from distributed_llm_amd.ops import seqmix
    monkeypatch.setattr(seqmix, "LATENT_EXPAND_MIN", expand_min)
    cfg = make_cfg([latent(heads=2, scale=0.2)], width=16)
    W = make_weights(cfg, seed=2)
    W["l0.mix.sink"] = torch.tensor([sink, -20.0], dtype=torch.bfloat16)
    t = toks(40, seed=3)
    want = orc.forward(t, W, cfg)
    W0 = dict(W)
    W0["l0.mix.sink"] = torch.tensor([-40.0, -20.0], dtype=torch.bfloat16)      # next to no sink
    without = orc.forward(t, W0, cfg)
    assert (float((want - without).std() / want.std()) > 0.03) == (sink > -6.0), "the test's sink does not show"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32)
    _prompt_decode_cut(eng, t, 33, f"sink {sink}", want)


@pytest.mark.parametrize("device", DEVICES)
def test_far_memory_of_the_mlstm(tmp_path, device):
    """Forget gates near one and one strong input early on: its trace is still in the memory hundreds of
    tokens later, across portions and single tokens; a lost or stale state would show."""
    cfg = make_cfg([mlstm(heads=2, dim=6, vdim=7, cap=12.0)], width=16)
    W = make_weights(cfg, seed=6, fgate=9.0, igate=-1.0, gate_gain=2.0)
    n = 300
    moves = []
    for tok in range(1, 12):
        t = [0] * n
        a = orc.forward(t, W, cfg)[-1]
        t[2] = tok
        moves.append((float((orc.forward(t, W, cfg)[-1] - a).std() / a.std()), tok))
    move, tok = max(moves)
    assert move > 0.02, "the test's weights do not show the memory"
    t = [0] * n
    t[2] = tok
    want = orc.forward(t, W, cfg)
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32, rows=1, tokens=512)
    other = toks(20, seed=8)
    for what in ("first use of the slot", "slot used again"):
        got, at = [], 0
        for m in (2, 1, 2, 130, 1, 1, 16, 15, 100, 31, 1):
            got.append(eng.feed([("m", t[at:at + m], list(range(m)))], ["m"] if at + m == n else []))
            at += m
        assert at == n
        close(torch.cat(got), want, torch.float32, what)
        eng.feed([("o", other, [0])], ["o"])


# ----------------------------------------------------------------------------- the engine's own entry points

def greedy_ok(prompt, out, W, cfg, n):
    """Every generated token is the oracle's arg-max after the tokens before it (the sampler reads
    logits rounded to bfloat16, so a token within that rounding of the best counts)."""
    assert len(out) == n
    lg = orc.forward(prompt + out[:-1], W, cfg)[len(prompt) - 1:]
    for row, t in zip(lg, out):
        top = float(row.max())
        assert float(row[t]) >= top - abs(top) * 2.0 ** -7, (t, int(row.argmax()))


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation(full_model, device):
    """``generate`` (scheduler, admission, prefill, decode steps, sampler) continues prompts as the
    oracle's arg-max does; more prompts than batch rows, so rows and state slots turn over."""
    path, cfg, W = full_model
    eng = engine(path, device, torch.float32, rows=2)
    prompts = [toks(n, seed=20 + n) for n in (5, 23, 1, 12)]
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=8, temperature=0.0, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o.error is None
        greedy_ok(p, o.token_ids, W, cfg, 8)
    # the sampler on this model's logits
    sp = SamplingParams(max_new_tokens=6, temperature=0.9, top_p=0.9, top_k=20, ignore_eos=True)
    for o in eng.generate(prompts[:2], sp):
        assert o.error is None and len(o.token_ids) == 6 and all(0 <= x < cfg["vocab"] for x in o.token_ids)


@pytest.mark.parametrize("device", DEVICES)
def test_prefix_cache_of_a_model_without_recurrent_layers(tmp_path, device):
    """Attention layers alone keep no state outside their pages, so prompts may share whole pages."""
    cfg = make_cfg([attn(size=20), latent(mlp=ff())])
    W = make_weights(cfg, seed=9)
    eng = LLMEngine(write_model(tmp_path / "m", cfg, W), device=device, dtype=torch.float32, max_num_seqs=2, max_model_len=256,
                    num_kv_blocks=16, prefix_cache=True)
    base = toks(40, seed=60)
    for p in (base, base[:33] + toks(4, seed=61), base, base[:17]):
        o = eng.generate([p], SamplingParams(max_new_tokens=6, temperature=0.0, ignore_eos=True))[0]
        assert o.error is None
        greedy_ok(p, o.token_ids, W, cfg, 6)


def test_replay_command_line(full_model, tmp_path):
    """bin/trace_run on a model folder: steps from standard input, logits files, ``done`` lines."""
    path, cfg, W = full_model
    a, b = toks(21, seed=1), toks(6, seed=2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:18], "want": [0, 17]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[18:19], "want": []}, {"id": "b", "tokens": b, "want": [5]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[19:], "want": [1]}], "end": ["a"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "64", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = orc.forward(a, W, cfg), orc.forward(b, W, cfg)
    read = lambda k, n: torch.from_numpy(np.fromfile(out / f"{k}.f32", dtype="<f4").reshape(n, -1))
    close(read(0, 2), wa[[0, 17]], torch.float32, "step 0")
    close(read(1, 1), wb[[5]], torch.float32, "step 1")
    close(read(2, 1), wa[[20]], torch.float32, "step 2")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_unaligned_sizes(tmp_path, device, dtype):
    """Width, vocabulary and head sizes that no 16-byte vector or 64-wide tile divides: every kernel's
    scalar tail and the library-GEMM routes; generation samples from an unaligned vocabulary."""
    layers = [attn(heads=5, kv_heads=5, dim=6, vdim=7, size=11, mlp=ff(9)), latent(heads=3, dim=5, rot=2, vdim=3, rank=7, q_rank=5, mlp=ff(11)),
              mlstm(heads=5, dim=7, vdim=3), latent(heads=7, dim=3, rot=6, vdim=9, rank=10), attn(heads=3, kv_heads=1, dim=10, vdim=3, size=7)]
    cfg = make_cfg(layers, width=21, vocab=37)
    W = make_weights(cfg, seed=6)
    eng = engine(write_model(tmp_path / "m", cfg, W), device, dtype)
    t = toks(42, vocab=37, seed=3)
    want = orc.forward(t, W, cfg)
    got = [eng.feed([("a", t[:33], list(range(33)))])] + [eng.feed([("a", t[i:i + 1], [0])]) for i in range(33, 42)]
    close(torch.cat(got), want, dtype, "unaligned")
    if dtype == torch.float32:
        out = eng.generate([t[:7]], SamplingParams(max_new_tokens=5, temperature=0.0, ignore_eos=True))[0]
        greedy_ok(t[:7], out.token_ids, W, cfg, 5)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("expand_min", [1, 32, 10 ** 9])
def test_aligned_sizes_take_the_matrix_core_paths(tmp_path, monkeypatch, dtype, expand_min):
    """Sizes that the matrix-core kernels and the tuned GEMMs take (bf16), against the oracle; prompt
    portions, decoding and mixed steps; windows that leave whole key tiles out."""
    from distributed_llm_amd.ops import seqmix
    monkeypatch.setattr(seqmix, "LATENT_EXPAND_MIN", expand_min)
    layers = [attn(heads=4, kv_heads=2, dim=32, vdim=64, scale=0.18, size=40, temp=(0.2, 64), mlp=ff(128)),
              latent(heads=4, dim=32, rot=16, vdim=64, rank=64, q_rank=64, scale=0.15, mlp=ff(64)),
              mlstm(heads=4, dim=32, vdim=32, mlp=ff(64)), attn(heads=8, kv_heads=1, dim=48, vdim=40, scale=0.14, size=130, temp=(0.1, 50)),
              latent(heads=2, dim=64, rot=32, vdim=32, rank=160, q_rank=128, scale=0.1), attn(heads=2, kv_heads=2, dim=128, vdim=96, scale=0.09, size=7)]
    cfg = make_cfg(layers, width=128, vocab=64)
    # (an mLSTM's first output is v times the sign of k . q: weights that bring it near zero make bfloat16
    # rounding visible there, with these it is not)
    W = make_weights(cfg, seed=9)
    eng = engine(write_model(tmp_path / "m", cfg, W), "cuda", dtype, tokens=512)
    a, b = toks(250, vocab=64, seed=1), toks(90, vocab=64, seed=2)
    wa, wb = orc.forward(a, W, cfg), orc.forward(b, W, cfg)
    ga = [eng.feed([("a", a[:200], list(range(200)))])]
    out = eng.feed([("a", a[200:201], [0]), ("b", b[:70], list(range(70)))])
    ga.append(out[:1])
    gb = [out[1:]]
    for i in range(20):
        out = eng.feed([("a", a[201 + i:202 + i], [0]), ("b", b[70 + i:71 + i], [0])])
        ga.append(out[:1])
        gb.append(out[1:])
    ga.append(eng.feed([("a", a[221:], list(range(29)))], ["a"]))
    close(torch.cat(ga), wa, dtype, "a")
    close(torch.cat(gb), wb, dtype, "b")


def test_registry_reads_config(full_model):
    from distributed_llm_amd.models.configs import DenseSpec, HybridConfig, QTempSpec, RopeSpec, config_from_dir, figotar_config
    path, cfg, W = full_model
    c = config_from_dir(path)
    assert isinstance(c, HybridConfig) and c.family == "figotar" and c.n_layers == len(cfg["layers"])
    assert c.pre_norm and c.post_norm and c.norm_offset and not c.parallel_ff and not c.tied_head
    m = c.layers[1].mixer
    assert m.kind == "biased_attention" and m.paged and not m.recurrent and m.head_gate and (m.window, m.scale) == (9, 0.4)
    assert m.q_temp == QTempSpec(0.4, 7.0) and m.slopes == (0.25, 0.0625, 2.0 ** -6, 2.0 ** -8)
    m = c.layers[2].mixer
    assert m.kind == "latent_attention" and m.rot == RopeSpec(4, 100.0) and m.head_gate and m.sinks and m.rot_half
    assert (m.q_rank, m.rot_dim, m.kv_rank) == (14, 4, 12)
    m = c.layers[0].mixer
    assert m.kind == "mlstm" and m.recurrent and not m.paged and m.gate_cap == 6.0
    assert c.layers[0].mlp == DenseSpec(20, act="gelu_glu", bias=True) and c.layers[3].mlp is None
    assert c.num_params() == sum(v.numel() for v in W.values())
    for layer, key, value in ((1, "kv_heads", 3), (2, "rot_dim", 6), (1, "q_temp", {"coef": 1.0, "every": 0})):
        bad = json.loads(json.dumps(cfg))
        bad["layers"][layer]["mixer"][key] = value
        with pytest.raises(ValueError):
            figotar_config(bad)
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["type"] = "mamba9"
    with pytest.raises(ValueError):
        figotar_config(bad)


@pytest.mark.parametrize("device", DEVICES)
def test_random_weights(device):
    """The seeded random tensors that benchmarks use have the checkpoint's names and sizes."""
    from distributed_llm_amd.models.configs import figotar_config
    from distributed_llm_amd.models.registry import build_model
    raw = make_cfg(FULL)
    cfg = figotar_config(raw)
    m = build_model(cfg, device=device, dtype=torch.float32)
    names = m._random(0, 0.02)
    want = make_weights(raw)
    assert {k: tuple(v.shape) for k, v in names.items()} == {k: tuple(v.shape) for k, v in want.items()}
    assert sum(v.numel() for v in names.values()) == cfg.num_params()
    twice = sum(L["uv"].numel() for L in m.layers if "uv" in L)      # the value up-projections are kept in two layouts
    slopes = sum(L["slopes"].numel() for L in m.layers if "slopes" in L)
    assert m.weight_bytes() == 4 * (cfg.num_params() + twice + slopes)
    assert m.decode_read_bytes() == 4 * (cfg.num_params() + slopes - m.embed.numel() - cfg.hidden)
