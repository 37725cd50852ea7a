"""The Gosavik decoder as a spec of parts.

Token embedding; a residual of several streams that a sublayer reads through one weighted sum and an RMS norm and that
its result joins through a mixing matrix; blocks of a mixer and a dense feed-forward W2 gelu_tanh(W1 h). What a mixer
reads is mixed with the row before it, channel by channel. A mixer is attention over a latent inside a window (queries
from a latent of their own, slowed long waves, a learned sink, a gate per channel), or grouped-query attention with
biases, a short convolution on queries, keys and values, keys and values turned by position, and a learned sink. A run of
layers may be passed several times with the same tensors and a cache of its own each time. At the end the streams are
added up, normed and multiplied by an output table of its own.

Tensor names: `embed`, `head`, `final.norm`, and per layer i `l<i>.norm1`, `l<i>.norm2`, `l<i>.shift`,
`l<i>.hc1.in/.out/.mix`, `l<i>.hc2.in/.out/.mix`, `l<i>.mlp.up`, `l<i>.mlp.down` and `l<i>.mix.*` (`dq`, `dq.norm`,
`uq`, `dkv`, `dkv.norm`, `uk`, `uv`, `sink`, `g`, `o`; or `q`, `k`, `v` with `.b` and `.conv` each, `sink`, `o`, `o.b`).
"""
from __future__ import annotations

from ..config.gosavik_config import GosavikConfig
from ..config.model_config import ARCHITECTURES, Architecture
from ..parts.spec import LayerCall, LayerSpec, ModelSpec, PartSpec, StageSpec

NO_CONTEXT_LIMIT = 1 << 30      # nothing in the design bounds a sequence's length


def _norm(cfg, name, read=None):
    """An RMS norm of the weighted sum of the streams (without weights: of their plain sum)."""
    return PartSpec("norm", "streams_rmsnorm",
                    {"width": cfg.width, "streams": cfg.streams, "eps": cfg.norm_eps, "weighted": read is not None},
                    {"gain": name, **({"read": read} if read is not None else {})})


def _connection(cfg, pre):
    return PartSpec("connection", "stream_mix", {"streams": cfg.streams}, {"mix": pre + "mix", "out": pre + "out"})


def _rot(m):
    rot = m.get("rot") or {}
    dims = int(rot.get("dims", 0))
    sc = rot.get("scaling") if dims else None
    return {"rot_dims": dims, "rot_base": float(rot.get("base", 10000.0)),
            "rot_slowed": (sc["factor"], sc["original"], sc["fast"], sc["slow"]) if sc else None}


def _latent(cfg, m, pre):
    params = {"width": cfg.width, "n_heads": m["heads"], "dim": m["dim"], "rot_dim": m["rot_dim"], "value_dim": m["vdim"],
              "rank": m["kv_rank"], "q_rank": m["q_rank"], "scale": m["scale"], "eps": cfg.norm_eps,
              "window": (m.get("mask") or {}).get("size", 0), "pair_half": True, "sink": True, "gate": True, **_rot(m)}
    names = {k: pre + k for k in ("dq", "uq", "dkv", "uk", "uv", "sink", "o")}
    names.update(dq_norm=pre + "dq.norm", dkv_norm=pre + "dkv.norm", gate=pre + "g")
    return PartSpec("mixer", "latent_attention", params, names)


def _attention(cfg, m, pre):
    params = {"width": cfg.width, "n_heads": m["heads"], "n_kv_heads": m["kv_heads"], "key_dim": m["dim"],
              "value_dim": m["vdim"], "taps": m["conv"], "scale": m["scale"], "turn_base": float(m["rot"]["base"]),
              "window": (m.get("mask") or {}).get("size", 0), **_rot(m)}
    names = {k: pre + k for k in ("q", "k", "v", "o", "sink")}
    for k in ("q", "k", "v"):
        names.update({k + "_bias": pre + k + ".b", k + "_conv": pre + k + ".conv"})
    names["o_bias"] = pre + "o.b"
    return PartSpec("mixer", "convolved_attention", params, names)


def _block(cfg, entry, i):
    pre = f"l{i}."
    mixer = (_latent if entry["type"] == "latent_attention" else _attention)(cfg, entry["mixer"], pre + "mix.")
    parts = {"mixer_norm": _norm(cfg, pre + "norm1", pre + "hc1.in"), "mixer": mixer, "mixer_connection": _connection(cfg, pre + "hc1."),
             "mixer_shift": PartSpec("row_shift", "previous_row", {"width": cfg.width}, {"amount": pre + "shift"})}
    if entry.get("mlp") is not None:
        parts["feed_forward_norm"] = _norm(cfg, pre + "norm2", pre + "hc2.in")
        parts["feed_forward"] = PartSpec("feed_forward", "activated_dense",
                                         {"width": cfg.width, "hidden": entry["mlp"]["ff"], "act": "gelu_tanh"},
                                         {"up": pre + "mlp.up", "down": pre + "mlp.down"})
        parts["feed_forward_connection"] = _connection(cfg, pre + "hc2.")
    return LayerSpec("hyper_stream32", parts, {"streams": cfg.streams})


def build_spec(cfg: GosavikConfig) -> ModelSpec:
    layers = tuple(_block(cfg, entry, i) for i, entry in enumerate(cfg.layers))
    ignorable = []
    for i, entry in enumerate(cfg.layers):     # a layer without a feed-forward has nothing around one; a file may carry it
        if entry.get("mlp") is None:
            ignorable += [f"l{i}.norm2", f"l{i}.hc2.*"]
    stage = StageSpec(name="trunk", lag=0, input=PartSpec("stage_input", "scaled_token_embedding", {"scale": 1.0}),
                      calls=tuple(LayerCall(i) for i in cfg.run_order()), out_norm=_norm(cfg, "final.norm"))
    return ModelSpec(d_model=cfg.width, vocab_size=cfg.vocab, max_context=NO_CONTEXT_LIMIT, layers=layers,
                     stages=(stage,), embedding="embed", lm_head="head", eos_token_id=-1, ignorable=tuple(ignorable))


ARCHITECTURES.register("Gosavik", Architecture("Gosavik", GosavikConfig, build_spec))
