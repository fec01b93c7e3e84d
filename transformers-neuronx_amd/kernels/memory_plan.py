"""What the linear memories' kernels launch by: a step planner (`engine.batch`) that such a mixer brings with it.

Runs of MEMORY_LONG tokens or more go chunk by chunk, the others token by token (measured for 32 heads of 128 x 128 and 64
of 128 x 64: a run of 64 tokens takes 17 to 21 us token by token and 22 to 25 by chunks, one of 128 tokens 28 to 37 and 23 to
29). `ctx.plan[...]`:
`memory_chunk_run`, `memory_chunk_begin`  for every chunk of MEMORY_CHUNK tokens its run and its first token in the run
`memory_long_run`, `memory_long_first`    the runs that go by chunks, and the number of each one's first chunk
and on the host, `ctx.plan_host["memory_walk_most"]`: the most tokens of a run that goes token by token.
"""
import numpy as np

MEMORY_CHUNK = 64
MEMORY_LONG = 80


def memory_plan(run_lens: np.ndarray, cached: np.ndarray, page_size: int, least: int = MEMORY_LONG):
    chunk_run, chunk_begin, long_run, long_first = [], [], [], []
    for i in np.nonzero(run_lens >= least)[0]:
        long_run.append(int(i))
        long_first.append(len(chunk_run))
        for begin in range(0, int(run_lens[i]), MEMORY_CHUNK):
            chunk_run.append(int(i))
            chunk_begin.append(begin)
    arrays = {"memory_chunk_run": chunk_run, "memory_chunk_begin": chunk_begin, "memory_long_run": long_run,
              "memory_long_first": long_first}
    return {k: np.array(v, dtype=np.int32) for k, v in arrays.items()}, {"memory_walk_most": least - 1}
