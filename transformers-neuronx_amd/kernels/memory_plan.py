"""What the linear memories' kernels launch by: a step planner (`engine.batch`) that such a mixer brings with it.

Runs of MEMORY_LONG tokens or more go chunk by chunk, the others token by token. `ctx.plan[...]`:
`memory_chunk_run`, `memory_chunk_begin`  for every chunk of MEMORY_CHUNK tokens its run and its first token in the run
`memory_long_run`, `memory_long_first`    the runs that go by chunks, and the number of each one's first chunk
"""
import numpy as np

MEMORY_CHUNK = 64
MEMORY_LONG = 24


def memory_plan(run_lens: np.ndarray, cached: np.ndarray, page_size: int):
    chunk_run, chunk_begin, long_run, long_first = [], [], [], []
    for i in np.nonzero(run_lens >= MEMORY_LONG)[0]:
        long_run.append(int(i))
        long_first.append(len(chunk_run))
        for begin in range(0, int(run_lens[i]), MEMORY_CHUNK):
            chunk_run.append(int(i))
            chunk_begin.append(begin)
    arrays = {"memory_chunk_run": chunk_run, "memory_chunk_begin": chunk_begin, "memory_long_run": long_run,
              "memory_long_first": long_first}
    return {k: np.array(v, dtype=np.int32) for k, v in arrays.items()}, {}
