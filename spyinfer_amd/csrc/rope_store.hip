// Projection biases, rotation by angles formed in the kernel, and the store of keys and values into their pages, for
// attention layers whose heads are rotated in part and whose frequencies are rescaled (no table: the angle of pair j at
// position p is float(p) * freq[j], float32, and its cosine and sine come from the full-range functions).  The same for
// layers that norm every query and key head, with one map a head or several.  And what such layers do with the heads'
// results: a sigmoid gate, the difference of two maps.
//
// The projections come as rows of a wider product: [q heads | k heads | v heads] of `d` values each, `xs` values from
// one token's row to the next.  One wave per (token, head).  q -> q_out[t, h, :]; k -> K[page, h, off, :];
// v -> V[page, h, :, off] (values lie transposed in a page).
#include "common.h"
#include <math.h>

#define RS_MAX_D 512
#define RS_WAVES 4

template <typename TA, typename TW>
__global__ __launch_bounds__(RS_WAVES * 64) void bias_rope_store_kernel(
    const TA* __restrict__ x, long long xs, TA* __restrict__ q_out, int n_q, int n_kv, int d, const TW* __restrict__ bias,
    const float* __restrict__ freq, int rot, const int* __restrict__ positions, TA* __restrict__ kc, TA* __restrict__ vc, int P,
    int num_pages, const int* __restrict__ slots, float mag, float v_eps, int v_n, float qt_coef, int qt_every,
    const TA* __restrict__ v1, long long v1s, int v1d, float lam, int dv) {
    // v1 != null: values of another layer for the same tokens (head hv's at v1 + t v1s + hv v1d, dv of them); what is stored
    // is (1 - lam) v + lam v1 (float32, rounded once).
    // qt_every > 0: a query is multiplied by 1 + qt_coef ln(floor((position + 1) / qt_every) + 1), float32 (queries that grow
    // with the logarithm of the position, in steps of qt_every positions)
    const int t = blockIdx.x, lane = threadIdx.x & 63;
    const int h = blockIdx.y * RS_WAVES + (threadIdx.x >> 6);
    const int heads = n_q + 2 * n_kv;
    if (h >= heads) return;
    const TA* row = x + (size_t)t * xs + (size_t)h * d;
    const TW* b = bias ? bias + (size_t)h * d : nullptr;
    const bool is_q = h < n_q, is_k = !is_q && h < n_q + n_kv;
    int page = -1, off = 0;
    if (!is_q) {
        if (!slots) return;
        const int slot = slots[t];
        if (slot < 0 || slot >= num_pages * P) return;
        page = slot / P;
        off = slot - page * P;
    }
    if (!is_q && !is_k) {
        const int hv = h - n_q - n_kv;
        TA* dst = vc + ((size_t)page * n_kv + hv) * d * P + off;
        float r = 1.f;
        if (v_n > 0) {
            // the value head over its root mean square (its first v_n values: the rest is padding)
            float ss = 0.f;
            for (int j = lane; j < v_n; j += 64) {
                const float v = to_f32<TA>(row[j]) + (b ? to_f32<TW>(b[j]) : 0.f);
                ss = fmaf(v, v, ss);
            }
            r = 1.0f / sqrtf(wave_sum(ss) / (float)v_n + v_eps);
        }
        const TA* other = v1 ? v1 + (size_t)t * v1s + (size_t)hv * v1d : nullptr;
        for (int j = lane; j < d; j += 64) {
            float v = (to_f32<TA>(row[j]) + (b ? to_f32<TW>(b[j]) : 0.f)) * r;
            if (other && j < dv) v = (1.0f - lam) * v + lam * to_f32<TA>(other[j]);
            dst[(size_t)j * P] = from_f32<TA>(v);
        }
        return;
    }
    const int half = rot >> 1;
    const float p = (float)positions[t];
    const float qt = (is_q && qt_every > 0) ? 1.0f + qt_coef * logf((float)((positions[t] + 1) / qt_every) + 1.0f) : 1.0f;
    TA* dst = is_q ? q_out + ((size_t)t * n_q + h) * d : kc + (((size_t)page * n_kv + (h - n_q)) * P + off) * d;
    for (int j = lane; j < half; j += 64) {
        const float a = to_f32<TA>(row[j]) + (b ? to_f32<TW>(b[j]) : 0.f);
        const float c = to_f32<TA>(row[j + half]) + (b ? to_f32<TW>(b[j + half]) : 0.f);
        const float ang = p * freq[j];
        const float cs = cosf(ang) * mag, sn = sinf(ang) * mag;
        dst[j] = from_f32<TA>((a * cs - c * sn) * qt);
        dst[j + half] = from_f32<TA>((c * cs + a * sn) * qt);
    }
    for (int j = rot + lane; j < d; j += 64) dst[j] = from_f32<TA>((to_f32<TA>(row[j]) + (b ? to_f32<TW>(b[j]) : 0.f)) * qt);
}

// The same for many bfloat16 tokens, in 16-byte pieces (d % 8 == 0, rot % 16 == 0, P % 8 == 0, no value norm).  The first T blocks
// have a token's q and k heads each: the token's cosines and sines are formed once and lie in LDS for all its heads.  The
// others have 16 tokens of one value head each, which go through LDS, so that a dim's 8 tokens, which lie side by side in a
// page, leave in one store.
typedef __attribute__((__vector_size__(4 * sizeof(uint32_t)))) uint32_t rs_u32x4;
__device__ __forceinline__ void rs_widen(const rs_u32x4& r, float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) { v[2 * i] = __uint_as_float(r[i] << 16); v[2 * i + 1] = __uint_as_float(r[i] & 0xffff0000u); }
}
__device__ __forceinline__ rs_u32x4 rs_narrow(const float (&v)[8]) {
    return rs_u32x4{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7])};
}
// 16 tokens' values of one kv head, staged as rows of `ld`, into the pages: 8 tokens of a dim that lie side by side in a page
// leave in one store.  (P is a multiple of 8; the block has 256 threads.)
__device__ __forceinline__ void rs_values_to_pages(const bf16_t* tile, int ld, int d, int t0, int T, const int* __restrict__ slots,
                                                   bf16_t* __restrict__ vc, int P, int num_pages, int n_kv, int hv) {
    for (int i = threadIdx.x; i < 2 * d; i += 256) {
        const int tg = i / d, j = i - tg * d;                 // dim j of tokens t0 + 8 tg .. + 7
        const int tb = t0 + 8 * tg;
        if (tb >= T) continue;
        const int s0 = slots[tb];
        bool run = tb + 8 <= T && s0 >= 0 && s0 % 8 == 0 && s0 + 8 <= num_pages * P;
        if (run) {
#pragma unroll
            for (int e = 1; e < 8; ++e) run = run && slots[tb + e] == s0 + e;
        }
        const bf16_t* col = tile + 8 * tg * ld + j;
        if (run) {                                            // P is a multiple of 8: the 8 slots lie in one page
            rs_u32x4 w;
#pragma unroll
            for (int e = 0; e < 4; ++e) w[e] = (uint32_t)col[2 * e * ld] | ((uint32_t)col[(2 * e + 1) * ld] << 16);
            const int page = s0 / P, off = s0 - page * P;
            *reinterpret_cast<rs_u32x4*>(vc + (((size_t)page * n_kv + hv) * d + j) * P + off) = w;
        } else {
            for (int e = 0; e < 8 && tb + e < T; ++e) {
                const int slot = slots[tb + e];
                if (slot < 0 || slot >= num_pages * P) continue;
                const int page = slot / P, off = slot - page * P;
                vc[(((size_t)page * n_kv + hv) * d + j) * P + off] = col[e * ld];
            }
        }
    }
}
template <typename TW>
__global__ __launch_bounds__(256) void bias_rope_store_many_kernel(
    const bf16_t* __restrict__ x, long long xs, bf16_t* __restrict__ q_out, int T, int n_q, int n_kv, int d, const TW* __restrict__ bias,
    const float* __restrict__ freq, int rot, const int* __restrict__ positions, bf16_t* __restrict__ kc, bf16_t* __restrict__ vc, int P,
    int num_pages, const int* __restrict__ slots, float mag, float qt_coef, int qt_every, const bf16_t* __restrict__ v1, long long v1s, int v1d,
    float lam, int dv) {
    __shared__ __align__(16) bf16_t tile[16 * (RS_MAX_D + 8)];
    __shared__ float cs[RS_MAX_D / 2], sn[RS_MAX_D / 2];
    const int qk_heads = n_q + n_kv, d8 = d >> 3;
    if ((int)blockIdx.x < T) {
        const int t = blockIdx.x, half = rot >> 1, h8 = half >> 3;
        const int pos = positions[t];
        const float p = (float)pos;
        const float qt = qt_every > 0 ? 1.0f + qt_coef * logf((float)((pos + 1) / qt_every) + 1.0f) : 1.0f;
        for (int j = threadIdx.x; j < half; j += 256) {
            const float ang = p * freq[j];
            cs[j] = cosf(ang) * mag;
            sn[j] = sinf(ang) * mag;
        }
        __syncthreads();
        const int slot = slots ? slots[t] : -1;
        const bool stored = slot >= 0 && slot < num_pages * P;
        const int page = stored ? slot / P : 0, off = stored ? slot - page * P : 0;
        // units of a head: its rotated pairs of pieces, then the pieces that pass unchanged
        const int per = d8 - h8;
        for (int u = threadIdx.x; u < qk_heads * per; u += 256) {
            const int h = u / per, c = u - h * per;
            const bool is_q = h < n_q;
            if (!is_q && !stored) continue;
            const bf16_t* row = x + (size_t)t * xs + (size_t)h * d;
            const TW* b = bias ? bias + (size_t)h * d : nullptr;
            bf16_t* dst = is_q ? q_out + ((size_t)t * n_q + h) * d : kc + (((size_t)page * n_kv + (h - n_q)) * P + off) * d;
            const float f = is_q ? qt : 1.0f;
            const int ja = c < h8 ? 8 * c : rot + 8 * (c - h8);
            float a[8], y[8];
            rs_widen(*reinterpret_cast<const rs_u32x4*>(row + ja), a);
            if (b) {
#pragma unroll
                for (int e = 0; e < 8; ++e) a[e] += to_f32<TW>(b[ja + e]);
            }
            if (c < h8) {
                float o[8], z[8];
                rs_widen(*reinterpret_cast<const rs_u32x4*>(row + ja + half), o);
                if (b) {
#pragma unroll
                    for (int e = 0; e < 8; ++e) o[e] += to_f32<TW>(b[ja + half + e]);
                }
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const float c_ = cs[ja + e], s_ = sn[ja + e];
                    y[e] = (a[e] * c_ - o[e] * s_) * f;
                    z[e] = (o[e] * c_ + a[e] * s_) * f;
                }
                *reinterpret_cast<rs_u32x4*>(dst + ja + half) = rs_narrow(z);
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) y[e] = a[e] * f;
            }
            *reinterpret_cast<rs_u32x4*>(dst + ja) = rs_narrow(y);
        }
        return;
    }
    // ---- values: 16 tokens of one kv head (blocks of this kind exist only with slots) -----------------------------
    const int vb = blockIdx.x - T;
    const int t0 = (vb / n_kv) * 16, hv = vb % n_kv, ld = d + 8;
    const TW* b = bias ? bias + (size_t)(qk_heads + hv) * d : nullptr;
    for (int i = threadIdx.x; i < 16 * d8; i += 256) {
        const int tt = i / d8, j0 = 8 * (i - tt * d8);
        if (t0 + tt >= T) continue;
        float v[8];
        rs_widen(*reinterpret_cast<const rs_u32x4*>(x + (size_t)(t0 + tt) * xs + (size_t)(qk_heads + hv) * d + j0), v);
        if (b) {
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] += to_f32<TW>(b[j0 + e]);
        }
        if (v1) {
            const bf16_t* o = v1 + (size_t)(t0 + tt) * v1s + (size_t)hv * v1d + j0;
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (j0 + e < dv) v[e] = (1.0f - lam) * v[e] + lam * bf16_to_f32(o[e]);
        }
        *reinterpret_cast<rs_u32x4*>(tile + tt * ld + j0) = rs_narrow(v);
    }
    __syncthreads();
    rs_values_to_pages(tile, ld, d, t0, T, slots, vc, P, num_pages, n_kv, hv);
}

extern "C" int spy_bias_rope_store(const void* x, long long xs, int dtype, void* q_out, int T, int n_q, int n_kv, int d,
                                   const void* bias, int b_dtype, const float* freq, int rot, const int* positions, void* kc,
                                   void* vc, int P, int num_pages, const int* slots, float mag, float v_eps, int v_n, float qt_coef, int qt_every,
                                   const void* v1, long long v1s, int v1d, float lam, int dv, hipStream_t st) {
    SPY_REQUIRE(T > 0 && n_q > 0 && n_kv > 0 && d > 0 && xs >= (long long)(n_q + 2 * n_kv) * d, "spy_bias_rope_store: bad sizes");
    SPY_REQUIRE(d <= RS_MAX_D, "spy_bias_rope_store: head size %d exceeds the supported %d", d, RS_MAX_D);
    SPY_REQUIRE(rot >= 0 && rot <= d && rot % 2 == 0 && (rot == 0 || freq), "spy_bias_rope_store: %d rotated dims do not fit a head of %d", rot, d);
    SPY_REQUIRE(!slots || (kc && vc && P > 0 && num_pages > 0), "spy_bias_rope_store: slots without a cache");
    SPY_REQUIRE(n_q + 2 * n_kv <= 65535 * RS_WAVES, "spy_bias_rope_store: too many heads");
    SPY_REQUIRE(v_n >= 0 && v_n <= d, "spy_bias_rope_store: a value norm over %d of %d values", v_n, d);
    SPY_REQUIRE(!v1 || (dv > 0 && dv <= d && v1d >= dv && v1s >= (long long)(n_kv - 1) * v1d + dv), "spy_bias_rope_store: the other layer's values do not fit");
    const uintptr_t bits = (uintptr_t)x | (uintptr_t)q_out | (uintptr_t)kc | (uintptr_t)vc;
    if (dtype == SPY_BF16 && T >= 64 && d % 8 == 0 && rot % 16 == 0 && xs % 8 == 0 && v_n == 0 && (!slots || P % 8 == 0) && bits % 16 == 0) {
        const long long blocks = (long long)T + (slots ? (long long)((T + 15) / 16) * n_kv : 0);
        SPY_REQUIRE(blocks < (1ll << 31), "spy_bias_rope_store: too many tokens");
        SPY_DISPATCH(b_dtype, TW, (bias_rope_store_many_kernel<TW><<<(unsigned)blocks, 256, 0, st>>>(
            (const bf16_t*)x, xs, (bf16_t*)q_out, T, n_q, n_kv, d, (const TW*)bias, freq, rot, positions, (bf16_t*)kc, (bf16_t*)vc, P, num_pages, slots,
            mag, qt_coef, qt_every, (const bf16_t*)v1, v1s, v1d, lam, dv)));
        SPY_CHECK_LAUNCH("spy_bias_rope_store");
        return 0;
    }
    const dim3 grid(T, (n_q + 2 * n_kv + RS_WAVES - 1) / RS_WAVES);
    SPY_DISPATCH(dtype, TA, SPY_DISPATCH(b_dtype, TW, (bias_rope_store_kernel<TA, TW><<<grid, RS_WAVES * 64, 0, st>>>(
        (const TA*)x, xs, (TA*)q_out, n_q, n_kv, d, (const TW*)bias, freq, rot, positions, (TA*)kc, (TA*)vc, P, num_pages, slots, mag, v_eps, v_n,
        qt_coef, qt_every, (const TA*)v1, v1s, v1d, lam, dv))));
    SPY_CHECK_LAUNCH("spy_bias_rope_store");
    return 0;
}

// ---- per-head norms, rotation and store, from heads as the projections give them (no padding) ---------------------------
// For layers that norm every query and key head (root mean square over its own `dim` values, one weight for all heads)
// ahead of the rotation, and for layers with several maps a head (differential attention): a map is a head of its own in
// the projection, normed and rotated by itself, while in the cache a kv head's maps lie one behind the other in ONE row of
// d >= maps dim values, so that a map's score is the product of that row with a query that is zero in the other maps'
// places.  One wave per (token, unit): n_q maps query units, n_kv maps key units, n_kv value units of dv values; units lie
// `hs` (values: `hv`) values apart from their first column on.  q -> q_out[t, unit, d]; k -> K[page, g, off, :]; v ->
// V[page, g, :, off], each filled up with zeros to d.  inter: pair j is dims (2 j, 2 j + 1) instead of (j, j + rot / 2).
struct NormRope {
    int n_q, n_kv, maps, dim, dv, d;
    long long q_off, k_off, v_off;
    int hs, hv, rot, inter, P, num_pages;
    float eps;
};
template <typename TA, typename TW>
__global__ __launch_bounds__(RS_WAVES * 64) void norm_rope_store_kernel(
    const TA* __restrict__ x, long long xs, TA* __restrict__ q_out, NormRope a, const TW* __restrict__ qw, const TW* __restrict__ kw,
    const float* __restrict__ freq, const int* __restrict__ positions, TA* __restrict__ kc, TA* __restrict__ vc, const int* __restrict__ slots) {
    const int t = blockIdx.x, lane = threadIdx.x & 63;
    int u = blockIdx.y * RS_WAVES + (threadIdx.x >> 6);
    const int nq = a.n_q * a.maps, nk = slots ? a.n_kv * a.maps : 0, nv = slots ? a.n_kv : 0;
    if (u >= nq + nk + nv) return;
    const TA* row = x + (size_t)t * xs;
    int page = 0, off = 0;
    if (u >= nq) {
        const int slot = slots[t];
        if (slot < 0 || slot >= a.num_pages * a.P) return;
        page = slot / a.P;
        off = slot - page * a.P;
    }
    if (u >= nq + nk) {
        const int g = u - nq - nk;
        const TA* src = row + a.v_off + (size_t)g * a.hv;
        TA* dst = vc + ((size_t)page * a.n_kv + g) * a.d * a.P + off;
        for (int j = lane; j < a.d; j += 64) dst[(size_t)j * a.P] = j < a.dv ? src[j] : from_f32<TA>(0.f);
        return;
    }
    const bool is_q = u < nq;
    if (!is_q) u -= nq;
    const int map = u % a.maps;
    const TA* src = row + (is_q ? a.q_off : a.k_off) + (size_t)u * a.hs;
    const TW* w = is_q ? qw : kw;
    TA* dst = is_q ? q_out + ((size_t)t * nq + u) * a.d : kc + (((size_t)page * a.n_kv + u / a.maps) * a.P + off) * a.d;
    float ss = 0.f;
    for (int j = lane; j < a.dim; j += 64) { const float v = to_f32<TA>(src[j]); ss = fmaf(v, v, ss); }
    const float r = 1.0f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
    TA* at = dst + map * a.dim;
    const int half = a.rot >> 1;
    const float p = (float)positions[t];
    for (int j = lane; j < half; j += 64) {
        const int ja = a.inter ? 2 * j : j, jb = a.inter ? 2 * j + 1 : j + half;
        const float v = (to_f32<TA>(src[ja]) * r) * to_f32<TW>(w[ja]), z = (to_f32<TA>(src[jb]) * r) * to_f32<TW>(w[jb]);
        const float ang = p * freq[j];
        const float cs = cosf(ang), sn = sinf(ang);
        at[ja] = from_f32<TA>(v * cs - z * sn);
        at[jb] = from_f32<TA>(z * cs + v * sn);
    }
    for (int j = a.rot + lane; j < a.dim; j += 64) at[j] = from_f32<TA>((to_f32<TA>(src[j]) * r) * to_f32<TW>(w[j]));
    // zeros: a query's other maps and its padding; a key's padding (by the wave of its last map)
    if (is_q) {
        for (int j = lane; j < a.d; j += 64)
            if (j < map * a.dim || j >= (map + 1) * a.dim) dst[j] = from_f32<TA>(0.f);
    } else if (map == a.maps - 1) {
        for (int j = a.maps * a.dim + lane; j < a.d; j += 64) dst[j] = from_f32<TA>(0.f);
    }
}

// The same for many bfloat16 tokens, in 16-byte pieces (dim, dv, d, the rotated dims and all columns multiples of 8; pairs
// (j, j + rot / 2): of 16).  The first T blocks have a token's query and key units each, L lanes a unit (L a power of two, one
// piece a lane), the token's cosines and sines once in LDS for all of them; the others have 16 tokens of one value head.
template <typename TW>
__global__ __launch_bounds__(256) void norm_rope_store_many_kernel(
    const bf16_t* __restrict__ x, long long xs, bf16_t* __restrict__ q_out, NormRope a, const TW* __restrict__ qw, const TW* __restrict__ kw,
    const float* __restrict__ freq, const int* __restrict__ positions, bf16_t* __restrict__ kc, bf16_t* __restrict__ vc,
    const int* __restrict__ slots, int T, int L) {
    __shared__ __align__(16) bf16_t tile[16 * (RS_MAX_D + 8)];
    __shared__ float cs[RS_MAX_D / 2], sn[RS_MAX_D / 2];
    const rs_u32x4 none = {0u, 0u, 0u, 0u};
    const int d8 = a.d >> 3;
    if ((int)blockIdx.x < T) {
        const int t = blockIdx.x, half = a.rot >> 1, c8 = a.dim >> 3;
        const float p = (float)positions[t];
        for (int j = threadIdx.x; j < half; j += 256) {
            const float ang = p * freq[j];
            cs[j] = cosf(ang);
            sn[j] = sinf(ang);
        }
        __syncthreads();
        const int slot = slots ? slots[t] : -1;
        const bool stored = slot >= 0 && slot < a.num_pages * a.P;
        const int page = stored ? slot / a.P : 0, off = stored ? slot - page * a.P : 0;
        const int nq = a.n_q * a.maps, units = nq + (stored ? a.n_kv * a.maps : 0);
        const int c = threadIdx.x & (L - 1), per = 256 / L;
        // (every lane of a unit goes round the loop together: the sums' exchanges stay inside the unit's L lanes)
        for (int u0 = threadIdx.x / L; u0 < units; u0 += per) {
            const bool is_q = u0 < nq;
            const int u = is_q ? u0 : u0 - nq, map = u % a.maps;
            const bf16_t* src = x + (size_t)t * xs + (is_q ? a.q_off : a.k_off) + (size_t)u * a.hs;
            const TW* w = is_q ? qw : kw;
            bf16_t* dst = is_q ? q_out + ((size_t)t * nq + u) * a.d : kc + (((size_t)page * a.n_kv + u / a.maps) * a.P + off) * a.d;
            float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (c < c8) rs_widen(*reinterpret_cast<const rs_u32x4*>(src + 8 * c), v);
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss = fmaf(v[e], v[e], ss);
            for (int o = L >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
            const float r = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
            if (c < c8) {
                const int j0 = 8 * c;
#pragma unroll
                for (int e = 0; e < 8; ++e) v[e] = (v[e] * r) * to_f32<TW>(w[j0 + e]);
                if (j0 < a.rot) {
                    float y[8];
                    if (a.inter) {
#pragma unroll
                        for (int e = 0; e < 8; e += 2) {
                            const float c_ = cs[(j0 + e) >> 1], s_ = sn[(j0 + e) >> 1];
                            y[e] = v[e] * c_ - v[e + 1] * s_;
                            y[e + 1] = v[e + 1] * c_ + v[e] * s_;
                        }
                    } else {
                        const bool low = j0 < half;
                        const int jo = low ? j0 + half : j0 - half, jj = low ? j0 : jo;
                        float o[8];
                        rs_widen(*reinterpret_cast<const rs_u32x4*>(src + jo), o);
#pragma unroll
                        for (int e = 0; e < 8; ++e) {
                            const float z = (o[e] * r) * to_f32<TW>(w[jo + e]), c_ = cs[jj + e], s_ = sn[jj + e];
                            y[e] = low ? v[e] * c_ - z * s_ : v[e] * c_ + z * s_;
                        }
                    }
#pragma unroll
                    for (int e = 0; e < 8; ++e) v[e] = y[e];
                }
                *reinterpret_cast<rs_u32x4*>(dst + map * a.dim + j0) = rs_narrow(v);
            }
            if (is_q) {                                           // zeros: a query's other maps and its padding; a key's padding
                for (int i = c; i < d8 - c8; i += L) *reinterpret_cast<rs_u32x4*>(dst + 8 * (i < map * c8 ? i : i + c8)) = none;
            } else if (map == a.maps - 1) {
                for (int i = a.maps * c8 + c; i < d8; i += L) *reinterpret_cast<rs_u32x4*>(dst + 8 * i) = none;
            }
        }
        return;
    }
    const int vb = blockIdx.x - T;
    const int t0 = (vb / a.n_kv) * 16, hv = vb % a.n_kv, ld = a.d + 8;
    for (int i = threadIdx.x; i < 16 * d8; i += 256) {
        const int tt = i / d8, j0 = 8 * (i - tt * d8);
        if (t0 + tt >= T) continue;
        *reinterpret_cast<rs_u32x4*>(tile + tt * ld + j0) =
            j0 < a.dv ? *reinterpret_cast<const rs_u32x4*>(x + (size_t)(t0 + tt) * xs + a.v_off + (size_t)hv * a.hv + j0) : none;
    }
    __syncthreads();
    rs_values_to_pages(tile, ld, a.d, t0, T, slots, vc, a.P, a.num_pages, a.n_kv, hv);
}

extern "C" int spy_norm_rope_store(const void* x, long long xs, int dtype, void* q_out, int T, int n_q, int n_kv, int maps, int dim, int dv,
                                   int d, long long q_off, long long k_off, long long v_off, int hs, int hv, const void* qw, const void* kw,
                                   int w_dtype, float eps, const float* freq, int rot, int inter, const int* positions, void* kc, void* vc,
                                   int P, int num_pages, const int* slots, hipStream_t st) {
    SPY_REQUIRE(T > 0 && n_q > 0 && n_kv > 0 && maps > 0 && dim > 0 && dv > 0 && d >= maps * dim && d >= dv && hs >= dim, "spy_norm_rope_store: bad sizes");
    SPY_REQUIRE(rot >= 0 && rot <= dim && rot % 2 == 0 && (rot == 0 || freq), "spy_norm_rope_store: %d rotated dims do not fit a head of %d", rot, dim);
    SPY_REQUIRE(qw && (!slots || kw), "spy_norm_rope_store: no norm weights");
    SPY_REQUIRE(q_off >= 0 && q_off + (long long)(n_q * maps - 1) * hs + dim <= xs, "spy_norm_rope_store: the queries' columns reach beyond the rows");
    SPY_REQUIRE(!slots || (kc && vc && P > 0 && num_pages > 0 && hv >= dv && k_off >= 0 && v_off >= 0 &&
                           k_off + (long long)(n_kv * maps - 1) * hs + dim <= xs && v_off + (long long)(n_kv - 1) * hv + dv <= xs),
                "spy_norm_rope_store: slots without a cache, or the keys' or values' columns reach beyond the rows");
    const int units = (n_q + (slots ? n_kv : 0)) * maps + (slots ? n_kv : 0);
    SPY_REQUIRE(units <= 65535 * RS_WAVES, "spy_norm_rope_store: too many heads");
    const NormRope a = {n_q, n_kv, maps, dim, dv, d, q_off, k_off, v_off, hs, hv, rot, inter, P, num_pages, eps};
    const uintptr_t bits = (uintptr_t)x | (uintptr_t)q_out | (uintptr_t)kc | (uintptr_t)vc;
    const long long columns = q_off | (slots ? k_off | v_off | hv : 0) | hs | xs;
    if (dtype == SPY_BF16 && T >= 64 && dim % 8 == 0 && dim <= 512 && d <= RS_MAX_D && d % 8 == 0 && dv % 8 == 0 && rot % (inter ? 8 : 16) == 0 && columns % 8 == 0 &&
        (!slots || P % 8 == 0) && bits % 16 == 0) {
        const long long blocks = (long long)T + (slots ? (long long)((T + 15) / 16) * n_kv : 0);
        SPY_REQUIRE(blocks < (1ll << 31), "spy_norm_rope_store: too many tokens");
        int L = 1;
        while (L < dim / 8) L <<= 1;
        SPY_DISPATCH(w_dtype, TW, (norm_rope_store_many_kernel<TW><<<(unsigned)blocks, 256, 0, st>>>(
            (const bf16_t*)x, xs, (bf16_t*)q_out, a, (const TW*)qw, (const TW*)kw, freq, positions, (bf16_t*)kc, (bf16_t*)vc, slots, T, L)));
        SPY_CHECK_LAUNCH("spy_norm_rope_store");
        return 0;
    }
    const dim3 grid(T, (units + RS_WAVES - 1) / RS_WAVES);
    SPY_DISPATCH(dtype, TA, SPY_DISPATCH(w_dtype, TW, (norm_rope_store_kernel<TA, TW><<<grid, RS_WAVES * 64, 0, st>>>(
        (const TA*)x, xs, (TA*)q_out, a, (const TW*)qw, (const TW*)kw, freq, positions, (TA*)kc, (TA*)vc, slots))));
    SPY_CHECK_LAUNCH("spy_norm_rope_store");
    return 0;
}

// ---- two maps of a head into one -----------------------------------------------------------------------------------------
// x [T, H, 2, d] (only the first dv values of a map's result count) -> out [T, H dv]: o = x1 - lam x2, over its root mean
// square (mean over the dv values, no weight), times `mult`.  One wave per (token, head).
template <typename TA, typename TO>
__global__ __launch_bounds__(RS_WAVES * 64) void map_difference_kernel(TO* __restrict__ out, const TA* __restrict__ x, int heads, int dv, int d,
                                                                       float lam, float eps, float mult) {
    const int i = blockIdx.x * RS_WAVES + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (i >= heads) return;
    const TA* a = x + (size_t)i * 2 * d;
    TO* o = out + (size_t)i * dv;
    float v[RS_MAX_D / 64];
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < RS_MAX_D / 64; ++e) {
        const int j = lane + 64 * e;
        v[e] = j < dv ? to_f32<TA>(a[j]) - lam * to_f32<TA>(a[d + j]) : 0.f;
        ss = fmaf(v[e], v[e], ss);
    }
    const float r = mult / sqrtf(wave_sum(ss) / (float)dv + eps);
#pragma unroll
    for (int e = 0; e < RS_MAX_D / 64; ++e) {
        const int j = lane + 64 * e;
        if (j < dv) o[j] = from_f32<TO>(v[e] * r);
    }
}

extern "C" int spy_map_difference(void* out, int out_dtype, const void* x, int dtype, int T, int H, int dv, int d, float lam, float eps,
                                  float mult, hipStream_t st) {
    SPY_REQUIRE(T > 0 && H > 0 && dv > 0 && d >= dv && d <= RS_MAX_D, "spy_map_difference: heads of %d in rows of %d (up to %d)", dv, d, RS_MAX_D);
    SPY_REQUIRE((long long)T * H < (1ll << 31) - RS_WAVES, "spy_map_difference: too many heads");
    const int heads = T * H;
    SPY_DISPATCH(dtype, TA, SPY_DISPATCH(out_dtype, TO, (map_difference_kernel<TA, TO><<<(heads + RS_WAVES - 1) / RS_WAVES, RS_WAVES * 64, 0, st>>>(
        (TO*)out, (const TA*)x, heads, dv, d, lam, eps, mult))));
    SPY_CHECK_LAUNCH("spy_map_difference");
    return 0;
}

// y[t, j] *= mult * sigmoid(g[t, j / per] + bias[j / per]) in place; the gate's rows may be part of a wider product (`gs`
// values from row to row); the bias may be absent.  per: columns of y that share one gate value (1: a gate per column;
// a head's size: one number per head).
template <typename TA, typename TW>
__global__ void sigmoid_gate_kernel(TA* __restrict__ y, const TA* __restrict__ g, long long gs, const TW* __restrict__ bias, float mult,
                                    int T, int N, int per) {
    const size_t total = (size_t)T * N;
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (size_t)gridDim.x * blockDim.x) {
        const size_t t = i / N, j = i - t * N;
        const size_t c = per > 1 ? j / per : j;
        const float gate = to_f32<TA>(g[t * gs + c]) + (bias ? to_f32<TW>(bias[c]) : 0.f);
        y[i] = from_f32<TA>(to_f32<TA>(y[i]) * mult / (1.0f + expf(-gate)));
    }
}

extern "C" int spy_sigmoid_gate(void* y, const void* g, long long gs, int dtype, const void* bias, int b_dtype, float mult, int T, int N,
                                int per, hipStream_t st) {
    SPY_REQUIRE(T > 0 && N > 0 && per > 0 && N % per == 0 && gs >= N / per, "spy_sigmoid_gate: bad sizes");
    const size_t total = (size_t)T * N;
    const unsigned blocks = (unsigned)((total + 255) / 256 > 65536 ? 65536 : (total + 255) / 256);
    SPY_DISPATCH(dtype, TA, SPY_DISPATCH(b_dtype, TW, (sigmoid_gate_kernel<TA, TW><<<blocks, 256, 0, st>>>((TA*)y, (const TA*)g, gs,
        (const TW*)bias, mult, T, N, per))));
    SPY_CHECK_LAUNCH("spy_sigmoid_gate");
    return 0;
}
