// Arguments shared by the gated delta rule kernels (delta.hip, delta_chunk.hip).
#pragma once
#include "common.h"

struct DeltaArgs {
    ProjSrc u;             // the layer's input projection: step sizes, decays and output gates
    int b_at, a_at, g_at;  // their first columns
    const float* dt_bias;  // [heads]
    const float* a_neg;    // -exp(A_log) [heads]
    const float* norm;     // [P]
    float eps, q_scale;
    int ldx, xk, xv;       // convolved rows: stride, first columns of k and v (q at 0)
    int ldo, col, width;   // output rows
    int heads, kv_heads, P, N, N4;
};
