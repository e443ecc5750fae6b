"""The model registry: what a config.json or a dimensions object is, and which loader, cache spec, engine and runner serve it.

``MI355XARWorker`` asks it for everything that differs between model families; the scheduler, the block pool, the sampler and the engine
loop are the same for all of them.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Callable

import torch

from .config import TalkerDims
from .decoder_config import PARSERS, DecoderDims, dims_from_config, read_config


@dataclass(frozen=True)
class ModelEntry:
    name: str
    dims_type: type
    matches: Callable[[dict], bool]                    # config.json contents
    parse: Callable[[dict, int], Any]                  # (config, max_model_len) -> dims
    load: Callable[[str, Any], tuple[dict, dict]]      # (path, dims) -> (weights, extras)
    random: Callable[[Any, int], dict]                 # (dims, seed) -> weights
    kv_cache_dtype: str                                # default of make_config
    cache_spec: Callable[[Any, Any, int], dict]        # (dims, worker config, tp size) -> {layer name: spec}
    build_engine: Callable[[Any, int], Any]            # (worker, num_blocks) -> engine
    build_runner: Callable[[Any], Any]                 # worker (engine built) -> runner


@dataclass(frozen=True)
class RowCacheSpec:
    """One layer's share of a cache block: block_size rows of (padded) width `width` -- latents, or keys and values side by side."""
    block_size: int
    width: int
    dtype: torch.dtype

    @property
    def page_size_bytes(self) -> int:
        return self.block_size * self.width * torch.empty((), dtype=self.dtype).element_size()


def _talker() -> ModelEntry:
    def parse(cfg, max_model_len):
        from .checkpoint import dims_from_hf_config
        return dims_from_hf_config(cfg, max_model_len=max_model_len)

    def load(path, dims):
        from .checkpoint import check_against_dims, load_talker_checkpoint
        w, extras = load_talker_checkpoint(path)
        check_against_dims(w, dims)
        return w, extras

    def random(dims, seed):
        from .weights import make_weights
        return make_weights(dims, seed=seed)

    def cache_spec(dims, cfg, tp):
        from .worker import AttentionSpec
        store = {"bf16": torch.bfloat16, "auto": torch.bfloat16, "fp16": torch.float16, "float16": torch.float16, "half": torch.float16,
                 "fp8": torch.uint8, "fp8_e4m3": torch.uint8, "int8": torch.int8}[cfg.kv_cache_dtype]
        hkv = max(dims.kv_heads // tp, 1)
        spec = AttentionSpec(block_size=int(cfg.block_size), num_kv_heads=hkv, head_size=dims.head_dim, dtype=store,
                             scale_bytes_per_token=2 * hkv * 4 if cfg.kv_cache_dtype == "int8" else 0)
        return {f"model.layers.{l}.self_attn.attn": spec for l in range(dims.layers)}

    return ModelEntry("talker", TalkerDims, lambda c: "talker_config" in c or "code_predictor_config" in c, parse, load, random, "fp8", cache_spec,
                      lambda worker, nb: worker._build_talker_engine(nb), lambda worker: worker._build_talker_runner())


def _decoder() -> ModelEntry:
    def load(path, dims):
        from .checkpoint import load_decoder_checkpoint
        return load_decoder_checkpoint(path, dims), {}

    def random(dims, seed):
        from .weights import make_decoder_weights
        return make_decoder_weights(dims, seed=seed)

    def cache_spec(dims, cfg, tp):
        from .decoder_mixers import ELEM, cache_row_widths
        e = ELEM[cfg.dtype]
        rows = {l: sum(cache_row_widths(dims, l, e.code)) for l in range(dims.num_layers)}
        return {f"model.layers.{l}.mixer": RowCacheSpec(int(cfg.block_size), w, e.torch) for l, w in rows.items() if w}

    def build_engine(worker, num_blocks):
        from .decoder_engine import DecoderEngine
        cfg = worker.vllm_config
        if worker.tp_size > 1:
            raise ValueError("decoder-only models run one replica per GPU (tensor_parallel_size = 1)")
        eng = DecoderEngine(worker.dims, worker._weights, dtype=cfg.dtype, kv_dtype=cfg.kv_cache_dtype, num_blocks=num_blocks, block_size=cfg.block_size,
                            max_batch=cfg.max_num_seqs, device=str(worker.device))
        worker._weights = None
        return eng

    def build_runner(worker):
        from .decoder_runner import DecoderModelRunner
        cfg = worker.vllm_config
        return DecoderModelRunner(worker.engine, use_graphs=not getattr(cfg, "enforce_eager", False),
                                  async_scheduling=bool(getattr(cfg, "async_scheduling", False)))

    return ModelEntry("decoder", DecoderDims, lambda c: c.get("architecture") in PARSERS, dims_from_config, load, random, "auto", cache_spec,
                      build_engine, build_runner)


REGISTRY: tuple[ModelEntry, ...] = (_decoder(), _talker())


def entry_for_config(cfg: dict) -> ModelEntry | None:
    return next((e for e in REGISTRY if e.matches(cfg)), None)


def entry_for_dims(dims) -> ModelEntry:
    for e in REGISTRY:
        if isinstance(dims, e.dims_type):
            return e
    raise TypeError(f"no model family serves {type(dims).__name__}")


def dims_of_model_dir(path: str, max_model_len: int = 4096):
    """Dimensions from a model directory's config.json, by whatever family claims it (an unclaimed one is read as a talker's: its parts may
    sit at the top level)."""
    cfg = read_config(path)
    e = entry_for_config(cfg)
    if e is None and "architecture" in cfg:
        raise ValueError(f"{path}: architecture {cfg['architecture']!r} is not served (known: {sorted(PARSERS)} and the talker checkpoints)")
    return (e or entry_for_dims_type(TalkerDims)).parse(cfg, max_model_len)


def entry_for_dims_type(t: type) -> ModelEntry:
    return next(e for e in REGISTRY if e.dims_type is t)
