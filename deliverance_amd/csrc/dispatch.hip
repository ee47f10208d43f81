// Which kernel form a step of a given shape takes, where the host and the layer loop of run_step.hip must agree.
#include "common.h"

// Decode attention splits a (sequence, head) pair's keys over workgroups when the pairs alone leave most
// of the chip idle and the context is long: shares of at least 1,024 keys, as many as bring the
// workgroups to about 512, 32 at most.  The choice reads the step's shape only (pairs and the width of
// the block table), so that a recorded step keeps it.
extern "C" int da_decode_splits(int n_seqs, int n_heads, int max_blocks, int page) {
  const long by_keys = ((long)max_blocks * page) / 1024;
  const long pairs = (long)n_seqs * n_heads;
  const long by_fill = 512 / (pairs > 0 ? pairs : 1);
  long n = by_keys < by_fill ? by_keys : by_fill;
  if (n > 32) n = 32;
  return n >= 2 ? (int)n : 1;
}

// Measured on MI355X inside the model: the fused norm + product kernel wins up to 16 rows (one row tile)
// and a width of 1,024, by 10 to 15 % of a decode step; up to 8 rows (which take half the LDS, so that the
// workgroups still run side by side) up to a width of 2,048: up to 1,280 with 16 columns a workgroup, beyond
// with 32 from 5 rows on (every workgroup reads and normalises all rows again, and at a width of 1,600 that is
// 2.5 us of vector work a compute unit; with 32 columns half as many workgroups do it).  Never for a vocabulary.
extern "C" int da_can_fuse_ln(int n_rows, int K, int N) {
  const bool fits = (n_rows <= 16 && K <= 1024) || (n_rows <= 8 && K <= 2048);
  return n_rows > 0 && fits && K % 8 == 0 && N <= 16384;
}
