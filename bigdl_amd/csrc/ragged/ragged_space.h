// Argument block shared by the two kernels of the state space recurrence (token by token in ragged_delta.hip, long bfloat16
// portions on the matrix cores in ragged_space.hip).
#pragma once
#include "ragged_common.h"

struct SpaceArgs {
  const void* dt;        // step logits: row t, column h of a [rows, lddt] matrix of type T
  int64_t lddt;
  const float* dt_bias;  // [H]
  const float* rate;     // [H]
  const float* D;        // [H]
  int b0, c0;            // columns of the inputs' matrix where B and C begin
  float* sum_log;        // [B, H] or null (matrix-core kernel): the sum of a sequence's log decays
  int keep_end;          // 1: the last state goes back to the state array (always so token by token)
};
