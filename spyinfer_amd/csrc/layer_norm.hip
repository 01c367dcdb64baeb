// Layer norms (the mean taken off, a bias behind) of rows that reach the stream:
//   out[t]  = base[t] + (y[t] - mean) / sqrt(var + eps) * w + b     (var: the mean squared deviation; out may be base)
//   copy[t] = the same in the activation dtype, for the products that read the stream (optional)
// and of the stream itself (base == null): out[r] = (x - mean) / sqrt(var + eps) * w + b in the activation dtype, at picked
// rows if `rows` is given.
// The result y comes as rows of the activation dtype, as a weighted pair of such rows (PairSum), or as a mixture's unsummed
// rows (ExpertSum), formed here, so that neither sum is a pass of its own nor rounded.  All arithmetic is float32; the
// deviations are squared behind the mean, not their sums of squares subtracted.
#include "common.h"
#include "result_rows.h"
#include <math.h>

enum { LN_ROWS = 0, LN_PAIR = 1, LN_EXPERTS = 2 };

struct LnResult {
    const void* y;
    PairSum pair;
    ExpertSum ex;
};

// One value of the result.
template <typename TA, int FORM>
__device__ __forceinline__ float ln_value(const LnResult& res, int t, int i, int H) {
    const size_t at = (size_t)t * H + i;
    if constexpr (FORM == LN_ROWS) return to_f32<TA>(reinterpret_cast<const TA*>(res.y)[at]);
    else if constexpr (FORM == LN_PAIR)
        return fmaf(res.pair.sa, to_f32<TA>(reinterpret_cast<const TA*>(res.pair.a)[at]), res.pair.sb * to_f32<TA>(reinterpret_cast<const TA*>(res.pair.b)[at]));
    else {
        const ExpertSum& ex = res.ex;
        float v = 0.f;
        for (int k = 0; k < ex.top; ++k) {
            const int row = ex.pair_row[(size_t)t * ex.top + k];
            if (row >= 0) v = fmaf((ex.weights ? ex.weights[(size_t)t * ex.top + k] : 1.f) * ex.scale, ex.y[(size_t)row * H + i], v);
        }
        return ex.add ? v + to_f32<TA>(reinterpret_cast<const TA*>(ex.add)[at]) : v;
    }
}

// One block per row.  PASSES > 0: the row (H % 4 == 0, 16-byte aligned, at most 4 PASSES values a thread) is read once and
// kept in registers; 0: any row, read again for every pass.
template <typename TA, typename TW, int PASSES, int FORM>
__global__ void layer_norm_residual_kernel(float* out, TA* __restrict__ copy, const float* base, LnResult res,
                                           const TW* __restrict__ w, const TW* __restrict__ b, float eps, int H) {
    __shared__ float red[16], red2[16];
    const int t = blockIdx.x;
    const size_t off = (size_t)t * H;
    if constexpr (PASSES > 0) {
        float yv[PASSES][4], xv[PASSES][4], wv[PASSES][4], bv[PASSES][4];
        // (what does not depend on the sums is asked for ahead of them: the stream's old values, both vectors)
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) yv[p][e] = 0.f;
            if (i < H) {
                if constexpr (FORM == LN_ROWS) Vec4<TA>::load(reinterpret_cast<const TA*>(res.y) + off + i, yv[p]);
                if constexpr (FORM == LN_PAIR) {
                    float a4[4], b4[4];
                    Vec4<TA>::load(reinterpret_cast<const TA*>(res.pair.a) + off + i, a4);
                    Vec4<TA>::load(reinterpret_cast<const TA*>(res.pair.b) + off + i, b4);
#pragma unroll
                    for (int e = 0; e < 4; ++e) yv[p][e] = fmaf(res.pair.sa, a4[e], res.pair.sb * b4[e]);
                }
                Vec4<float>::load(base + off + i, xv[p]);
                Vec4<TW>::load(w + i, wv[p]);
                Vec4<TW>::load(b + i, bv[p]);
            }
        }
        if constexpr (FORM == LN_EXPERTS) {
            const ExpertSum& ex = res.ex;
            for (int k = 0; k < ex.top; ++k) {
                const int row = ex.pair_row[(size_t)t * ex.top + k];
                if (row < 0) continue;
                const float wt = (ex.weights ? ex.weights[(size_t)t * ex.top + k] : 1.f) * ex.scale;
                const float* src = ex.y + (size_t)row * H;
#pragma unroll
                for (int p = 0; p < PASSES; ++p) {
                    const int i = (p * blockDim.x + threadIdx.x) * 4;
                    if (i < H) {
                        float v[4];
                        Vec4<float>::load(src + i, v);
#pragma unroll
                        for (int e = 0; e < 4; ++e) yv[p][e] = fmaf(wt, v[e], yv[p][e]);
                    }
                }
            }
            if (ex.add) {
#pragma unroll
                for (int p = 0; p < PASSES; ++p) {
                    const int i = (p * blockDim.x + threadIdx.x) * 4;
                    if (i < H) {
                        float v[4];
                        Vec4<TA>::load(reinterpret_cast<const TA*>(ex.add) + off + i, v);
#pragma unroll
                        for (int e = 0; e < 4; ++e) yv[p][e] += v[e];
                    }
                }
            }
        }
        float s = 0.f;
#pragma unroll
        for (int p = 0; p < PASSES; ++p)
#pragma unroll
            for (int e = 0; e < 4; ++e) s += yv[p][e];
        const float mean = block_sum(s, red) / (float)H;
        s = 0.f;
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < H) {
#pragma unroll
                for (int e = 0; e < 4; ++e) { yv[p][e] -= mean; s = fmaf(yv[p][e], yv[p][e], s); }
            }
        }
        const float r = 1.0f / sqrtf(block_sum(s, red2) / (float)H + eps);
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < H) {
                float v[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] = xv[p][e] + fmaf(yv[p][e] * r, wv[p][e], bv[p][e]);
                Vec4<float>::store(out + off + i, v);
                if (copy) Vec4<TA>::store(copy + off + i, v);
            }
        }
    } else {
        float s = 0.f;
        for (int i = threadIdx.x; i < H; i += blockDim.x) s += ln_value<TA, FORM>(res, t, i, H);
        const float mean = block_sum(s, red) / (float)H;
        s = 0.f;
        for (int i = threadIdx.x; i < H; i += blockDim.x) { const float v = ln_value<TA, FORM>(res, t, i, H) - mean; s = fmaf(v, v, s); }
        const float r = 1.0f / sqrtf(block_sum(s, red2) / (float)H + eps);
        for (int i = threadIdx.x; i < H; i += blockDim.x) {
            const float v = base[off + i] + fmaf((ln_value<TA, FORM>(res, t, i, H) - mean) * r, to_f32<TW>(w[i]), to_f32<TW>(b[i]));
            out[off + i] = v;
            if (copy) copy[off + i] = from_f32<TA>(v);
        }
    }
}

template <typename TA, typename TW, int FORM>
static void ln_launch(float* out, TA* copy, const float* base, const LnResult& res, const TW* w, const TW* b, float eps, int T, int H,
                      bool pieces, hipStream_t st) {
    const int threads = H >= 4096 ? 512 : (H >= 1024 ? 256 : (H >= 512 ? 128 : 64));
    const int passes = pieces ? (H / 4 + threads - 1) / threads : 0;
#define LN(P) layer_norm_residual_kernel<TA, TW, P, FORM><<<T, threads, 0, st>>>(out, copy, base, res, w, b, eps, H)
    if (passes == 0 || passes > 8) LN(0);
    else if (passes == 1) LN(1);
    else if (passes == 2) LN(2);
    else if (passes <= 4) LN(4);
    else LN(8);
#undef LN
}

// dtype: of y (or a and b, or add) and of copy alike, the activation dtype; exactly one of y, a (with b) and ex_y is given.
extern "C" int spy_layer_norm_residual(float* out, void* copy, const float* base, int dtype, const void* y, const void* a, const void* b2,
                                       float sa, float sb, const float* ex_y, const int* pair_row, const float* weights, const void* add,
                                       int top, float scale, const void* w, const void* b, int w_dtype, float eps, int T, int H,
                                       hipStream_t st) {
    SPY_REQUIRE(T > 0 && H > 0 && out && base && w && b, "spy_layer_norm_residual: empty operand");
    SPY_REQUIRE((y != nullptr) + (a != nullptr) + (ex_y != nullptr) == 1 && (!a == !b2), "spy_layer_norm_residual: the result as rows, as a pair or as experts' rows, one of them");
    SPY_REQUIRE(!ex_y || (pair_row && top > 0), "spy_layer_norm_residual: experts' rows without their places");
    const LnResult res = {y, {a, b2, sa, sb}, {ex_y, pair_row, weights, add, top, scale}};
    const uintptr_t bits = (uintptr_t)out | (uintptr_t)copy | (uintptr_t)base | (uintptr_t)y | (uintptr_t)a | (uintptr_t)b2 | (uintptr_t)ex_y |
                           (uintptr_t)add | (uintptr_t)w | (uintptr_t)b;
    const bool pieces = H % 4 == 0 && bits % 16 == 0;
    SPY_DISPATCH(dtype, TA, SPY_DISPATCH(w_dtype, TW, {
        if (y) ln_launch<TA, TW, LN_ROWS>(out, (TA*)copy, base, res, (const TW*)w, (const TW*)b, eps, T, H, pieces, st);
        else if (a) ln_launch<TA, TW, LN_PAIR>(out, (TA*)copy, base, res, (const TW*)w, (const TW*)b, eps, T, H, pieces, st);
        else ln_launch<TA, TW, LN_EXPERTS>(out, (TA*)copy, base, res, (const TW*)w, (const TW*)b, eps, T, H, pieces, st);
    }));
    SPY_CHECK_LAUNCH("spy_layer_norm_residual");
    return 0;
}

// out[r] = the layer norm of x[rows ? rows[r] : r]; one block per row.  PASSES as above.
template <typename TW, typename TO, int PASSES>
__global__ void layer_norm_kernel(TO* __restrict__ out, const float* __restrict__ x, const TW* __restrict__ w, const TW* __restrict__ b,
                                  float eps, const int* __restrict__ rows, int T, int H) {
    __shared__ float red[16], red2[16];
    const int r = blockIdx.x;
    const int t = rows ? rows[r] : r;
    TO* o = out + (size_t)r * H;
    if (t < 0 || t >= T) {       // never the case for a checked batch; write zeros rather than read outside
        for (int i = threadIdx.x; i < H; i += blockDim.x) o[i] = from_f32<TO>(0.f);
        return;
    }
    const float* row = x + (size_t)t * H;
    float s = 0.f;
    if constexpr (PASSES > 0) {
        float v[PASSES][4], wv[PASSES][4], bv[PASSES][4];
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[p][e] = 0.f;
            if (i < H) { Vec4<float>::load(row + i, v[p]); Vec4<TW>::load(w + i, wv[p]); Vec4<TW>::load(b + i, bv[p]); }
#pragma unroll
            for (int e = 0; e < 4; ++e) s += v[p][e];
        }
        const float mean = block_sum(s, red) / (float)H;
        s = 0.f;
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < H) {
#pragma unroll
                for (int e = 0; e < 4; ++e) { v[p][e] -= mean; s = fmaf(v[p][e], v[p][e], s); }
            }
        }
        const float q = 1.0f / sqrtf(block_sum(s, red2) / (float)H + eps);
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < H) {
                float y[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) y[e] = fmaf(v[p][e] * q, wv[p][e], bv[p][e]);
                Vec4<TO>::store(o + i, y);
            }
        }
        return;
    }
    for (int i = threadIdx.x; i < H; i += blockDim.x) s += row[i];
    const float mean = block_sum(s, red) / (float)H;
    s = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) { const float v = row[i] - mean; s = fmaf(v, v, s); }
    const float q = 1.0f / sqrtf(block_sum(s, red2) / (float)H + eps);
    for (int i = threadIdx.x; i < H; i += blockDim.x) o[i] = from_f32<TO>(fmaf((row[i] - mean) * q, to_f32<TW>(w[i]), to_f32<TW>(b[i])));
}

extern "C" int spy_layer_norm(void* out, int out_dtype, const float* x, const void* w, const void* b, int w_dtype, float eps, const int* rows,
                              int n_out, int T, int H, hipStream_t st) {
    SPY_REQUIRE(n_out > 0 && T > 0 && H > 0 && (rows || n_out == T), "spy_layer_norm: %d rows of %d", n_out, T);
    const int threads = H >= 4096 ? 512 : (H >= 1024 ? 256 : (H >= 512 ? 128 : 64));
    const bool pieces = H % 4 == 0 && (((uintptr_t)out | (uintptr_t)x | (uintptr_t)w | (uintptr_t)b) % 16) == 0;
    const int passes = pieces ? (H / 4 + threads - 1) / threads : 0;
#define LNK(P) layer_norm_kernel<TW, TO, P><<<n_out, threads, 0, st>>>((TO*)out, x, (const TW*)w, (const TW*)b, eps, rows, T, H)
    SPY_DISPATCH(w_dtype, TW, SPY_DISPATCH(out_dtype, TO, {
        if (passes == 0 || passes > 8) LNK(0);
        else if (passes == 1) LNK(1);
        else if (passes == 2) LNK(2);
        else if (passes <= 4) LNK(4);
        else LNK(8);
    }));
#undef LNK
    SPY_CHECK_LAUNCH("spy_layer_norm");
    return 0;
}
