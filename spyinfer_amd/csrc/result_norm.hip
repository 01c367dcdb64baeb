// Layers that norm a sublayer's RESULT as well as the next sublayer's input, in one pass over the row:
//   x = resid[t] + y[t] / sqrt(mean(y[t]^2) + eps_y) * wy          (wy float32: the result's norm weight, with whatever learned
//   out[r] = x / sqrt(mean(x^2) + eps) * w                          vector scales the result multiplied into it)
// rows == null: every row, and x goes back to the stream; else row rows[r] only, and the stream stays as it is.
// The result y comes as rows of the activation dtype, or as the experts' unsummed rows of a mixture: y[t] = add[t] + scale *
// sum_k weight[t, k] * Y[pair_row[t top + k]] (no weights: all one; no add: nothing), so that neither the mixture's sum nor
// its rounding to the activation dtype is a pass of its own.  All arithmetic is float32.
#include "common.h"
#include "result_rows.h"
#include <math.h>

// One block per row.  PASSES > 0: the row (H % 4 == 0, 16-byte aligned, at most 4 PASSES values a thread) is read once and
// kept in registers; 0: any row, read again for every pass.
template <typename TA, typename TW, int PASSES, bool EXPERTS>
__global__ void result_norm_kernel(float* __restrict__ resid, const TA* __restrict__ y, ExpertSum ex, const float* __restrict__ wy,
                                   float eps_y, const TW* __restrict__ w, float eps, TA* __restrict__ out, const int* __restrict__ rows,
                                   int T, int H) {
    __shared__ float red[16];
    const int r = blockIdx.x;
    int t = r;
    if (rows) {
        t = rows[r];
        if (t < 0 || t >= T) {   // never the case for a checked batch; write zeros rather than read outside
            for (int i = threadIdx.x; i < H; i += blockDim.x) out[(size_t)r * H + i] = from_f32<TA>(0.f);
            return;
        }
    }
    float* x = resid + (size_t)t * H;
    const TA* yr = EXPERTS ? nullptr : y + (size_t)t * H;
    const TA* ar = (EXPERTS && ex.add) ? reinterpret_cast<const TA*>(ex.add) + (size_t)t * H : nullptr;
    TA* o = out + (size_t)r * H;
    if constexpr (PASSES > 0) {
        float yv[PASSES][4], xv[PASSES][4];
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) { yv[p][e] = 0.f; xv[p][e] = 0.f; }
            if (i < H) {
                Vec4<float>::load(x + i, xv[p]);
                if (!EXPERTS) Vec4<TA>::load(yr + i, yv[p]);
            }
        }
        if constexpr (EXPERTS) {
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
            if (ar) {
#pragma unroll
                for (int p = 0; p < PASSES; ++p) {
                    const int i = (p * blockDim.x + threadIdx.x) * 4;
                    if (i < H) {
                        float v[4];
                        Vec4<TA>::load(ar + i, v);
#pragma unroll
                        for (int e = 0; e < 4; ++e) yv[p][e] += v[e];
                    }
                }
            }
        }
        float ss = 0.f;
#pragma unroll
        for (int p = 0; p < PASSES; ++p)
#pragma unroll
            for (int e = 0; e < 4; ++e) ss = fmaf(yv[p][e], yv[p][e], ss);
        // (both weights are asked for ahead of the sums that they wait for)
        float av[PASSES][4], bv[PASSES][4];
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < H) { Vec4<float>::load(wy + i, av[p]); Vec4<TW>::load(w + i, bv[p]); }
        }
        ss = block_sum(ss, red);
        const float sy = 1.0f / sqrtf(ss / (float)H + eps_y);
        ss = 0.f;
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < H) {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    xv[p][e] += (sy * yv[p][e]) * av[p][e];
                    ss = fmaf(xv[p][e], xv[p][e], ss);
                }
                if (!rows) Vec4<float>::store(x + i, xv[p]);
            }
        }
        ss = block_sum(ss, red);
        const float sx = 1.0f / sqrtf(ss / (float)H + eps);
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < H) {
                float v[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] = (sx * xv[p][e]) * bv[p][e];
                Vec4<TA>::store(o + i, v);
            }
        }
    } else {
        auto result = [&](int i) {
            float v = 0.f;
            if constexpr (EXPERTS) {
                for (int k = 0; k < ex.top; ++k) {
                    const int row = ex.pair_row[(size_t)t * ex.top + k];
                    if (row >= 0) v = fmaf((ex.weights ? ex.weights[(size_t)t * ex.top + k] : 1.f) * ex.scale, ex.y[(size_t)row * H + i], v);
                }
                if (ar) v += to_f32<TA>(ar[i]);
            } else {
                v = to_f32<TA>(yr[i]);
            }
            return v;
        };
        float ss = 0.f;
        for (int i = threadIdx.x; i < H; i += blockDim.x) { const float v = result(i); ss = fmaf(v, v, ss); }
        ss = block_sum(ss, red);
        const float sy = 1.0f / sqrtf(ss / (float)H + eps_y);
        ss = 0.f;
        for (int i = threadIdx.x; i < H; i += blockDim.x) {
            const float v = x[i] + (sy * result(i)) * wy[i];
            if (!rows) x[i] = v;
            ss = fmaf(v, v, ss);
        }
        ss = block_sum(ss, red);
        const float sx = 1.0f / sqrtf(ss / (float)H + eps);
        for (int i = threadIdx.x; i < H; i += blockDim.x) {      // (a thread reads back what it wrote itself)
            const float v = rows ? x[i] + (sy * result(i)) * wy[i] : x[i];
            o[i] = from_f32<TA>((sx * v) * to_f32<TW>(w[i]));
        }
    }
}

template <typename TA, typename TW, bool EXPERTS>
static void result_norm_launch(float* resid, const TA* y, const ExpertSum& ex, const float* wy, float eps_y, const TW* w, float eps, TA* out,
                               const int* rows, int n_out, int T, int H, bool pieces, hipStream_t st) {
    const int threads = H >= 4096 ? 512 : (H >= 1024 ? 256 : (H >= 512 ? 128 : 64));
    const int passes = pieces ? (H / 4 + threads - 1) / threads : 0;
#define RN(P) result_norm_kernel<TA, TW, P, EXPERTS><<<n_out, threads, 0, st>>>(resid, y, ex, wy, eps_y, w, eps, out, rows, T, H)
    if (passes == 0 || passes > 8) RN(0);
    else if (passes == 1) RN(1);
    else if (passes == 2) RN(2);
    else if (passes <= 4) RN(4);
    else RN(8);
#undef RN
}

extern "C" int spy_result_norm(float* resid, const void* y, int y_dtype, const float* ex_y, const int* pair_row, const float* weights,
                               const void* add, int top, float scale, const float* wy, float eps_y, const void* w, int w_dtype, float eps,
                               void* out, const int* rows, int n_out, int T, int H, hipStream_t st) {
    // y_dtype: of y, of add and of the result alike (the activation dtype)
    SPY_REQUIRE(n_out > 0 && T > 0 && H > 0, "spy_result_norm: empty operand");
    SPY_REQUIRE((y != nullptr) != (ex_y != nullptr), "spy_result_norm: a result as rows or as experts' rows, one of them");
    SPY_REQUIRE(!ex_y || (pair_row && top > 0), "spy_result_norm: experts' rows without their places");
    SPY_REQUIRE(rows || n_out == T, "spy_result_norm: %d rows of %d", n_out, T);
    const ExpertSum ex = {ex_y, pair_row, weights, add, top, scale};
    const uintptr_t bits = (uintptr_t)resid | (uintptr_t)y | (uintptr_t)ex_y | (uintptr_t)add | (uintptr_t)wy | (uintptr_t)w | (uintptr_t)out;
    const bool pieces = H % 4 == 0 && bits % 16 == 0;
    SPY_DISPATCH(y_dtype, TA, SPY_DISPATCH(w_dtype, TW, {
        if (ex_y) result_norm_launch<TA, TW, true>(resid, (const TA*)y, ex, wy, eps_y, (const TW*)w, eps, (TA*)out, rows, n_out, T, H, pieces, st);
        else result_norm_launch<TA, TW, false>(resid, (const TA*)y, ex, wy, eps_y, (const TW*)w, eps, (TA*)out, rows, n_out, T, H, pieces, st);
    }));
    SPY_CHECK_LAUNCH("spy_result_norm");
    return 0;
}
