// The forms in which a sublayer's result reaches the kernel that sums it into the stream.
#pragma once
#include "common.h"

// A mixture's result as its experts' unsummed rows: out[t] = add[t] + scale * sum_k weights[t, k] * y[pair_row[t top + k]].
struct ExpertSum {
    const float* y;             // [sorted rows, H]; null: the result comes as ordinary rows
    const int* pair_row;        // [T, top]
    const float* weights;       // [T, top] or null
    const void* add;            // [T, H] of the activation dtype, or null
    int top;
    float scale;
};

// Two results that meet weighted: out[t] = sa a[t] + sb b[t] (rows of the activation dtype).
struct PairSum {
    const void* a;
    const void* b;
    float sa, sb;
};
