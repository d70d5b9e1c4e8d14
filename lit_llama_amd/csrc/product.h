// Internal (NOT part of the C ABI): products of hybrid layers whose operand needs no norm.
#pragma once
#include "common.h"

struct mi355_product {
    int dtype;            // of x and of the weights
    const void* x;        // [M, ldx]; bf16: whole 128-column units, zero from column K on
    int64_t ldx;
    int M;
    void* y;
    int64_t ldy;
    int y_dtype;
    int epi;              // MI355_EPI_* (f32 models: STORE)
    float alpha, limit;
    int slice_rows;       // see mi355_linear_args
    int64_t slice_stride;
    void* ws;             // of mi355_linear_gemm
    uint64_t ws_bytes;
};

// The weight-streaming kernel up to 8 rows, the tiled product above it (and where its LDS has no room for the operand); f32: the exact
// generic kernel.  hybrid.hip
int mi355_product_run(const mi355_product& p, const mi355_proj& w, hipStream_t s);
// mi355_linear_fast of up to 8 products in one launch (bf16 operands without norm, STORE; they differ in w, x, y and N alone).  gemv.hip
int mi355_linear_fast_jobs(const mi355_linear_args* a, int count, mi355_stream_t stream);
// does a product of M rows take the tiled kernel?
bool mi355_product_wide(const mi355_proj& w, int M, int R);
