"""A worker and its scheduler around a model directory or a dimensions object: the engine-core loop, ready for ``add_request`` / ``run``."""
from __future__ import annotations

from .scheduler import MI355XARScheduler, TalkerStageEngine
from .worker import MI355XARWorker, make_config


def serve(model, *, weights: dict | None = None, dtype: str = "bfloat16", num_blocks: int = 1024, block_size: int = 16, max_num_seqs: int = 64,
          max_model_len: int = 4096, max_num_batched_tokens: int = 8192, async_scheduling: bool = False, enforce_eager: bool = False) -> TalkerStageEngine:
    """model: a checkpoint directory (config.json decides the family) or a dimensions object with `weights` (None: random ones)."""
    kw = dict(model_path=model) if isinstance(model, str) else dict(model=model.with_(max_model_len=max_model_len), weights=weights)
    cfg = make_config(**kw, dtype=dtype, block_size=block_size, max_num_seqs=max_num_seqs, num_gpu_blocks_override=num_blocks, enforce_eager=enforce_eager,
                      async_scheduling=async_scheduling, max_model_len=max_model_len)
    worker = MI355XARWorker(cfg)
    worker.init_device()
    worker.load_model()
    worker.initialize_from_config(None)
    worker.compile_or_warm_up_model()
    sched = MI355XARScheduler(num_blocks=num_blocks, block_size=block_size, max_num_seqs=max_num_seqs, max_num_batched_tokens=max_num_batched_tokens,
                              max_model_len=worker.dims.max_model_len, async_scheduling=async_scheduling)
    return TalkerStageEngine(worker, sched)
