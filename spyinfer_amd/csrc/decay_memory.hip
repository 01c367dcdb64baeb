// Recurrences whose state is a matrix per head that decays by ONE number a token:
//
//     S_t = a_t S_(t-1) + b_t k_t v_t^T,      o_t = S_t^T q_t            S [d, dv] float32 in the request's slot
//
// with a either a constant of the head (retention: b = 1, q and k rotated by their position, k times a constant) or formed
// from a step size of the token (state spaces: dt = softplus(. + bias), a = exp(-rate_h dt), b = dt; q and k shared by the
// heads of a group).  Everything here is float32, whatever the operands' dtype.
//
// Steps of single tokens: one block per (entry, head) reads S once, writes it once and leaves the head's result
// (decay_memory_step_kernel).
//
// Steps with longer entries: with cum_t = sum of log a up to t inside a piece of 64 tokens,
//     o_t = exp(cum_t) S_in^T q_t + sum_(s <= t) exp(cum_t - cum_s) b_s (q_t . k_s) v_s
//     S_out = exp(cum_end) S_in + sum_s exp(cum_end - cum_s) b_s k_s v_s^T
// (all exponents <= 0), so all pieces' own contributions to the state come first, for all pieces at once (pieces_kernel),
// then a walk over an entry's pieces that adds up (fold_kernel: memory traffic only), then all pieces' results at once
// (results_kernel).  The products run on the matrix cores in float32 (v_mfma_f32_16x16x4_f32: products and sums are exact
// float32 arithmetic).  Lane layout of that instruction: lane l holds A[row l % 16][k = l / 16], B[k = l / 16][column
// l % 16], and of the result rows 4 (l / 16) .. + 3 of column l % 16.
//
// What happens to o: stored as float32; or normed over the head's dv values (root mean square, no weight), times
// silu(gate), rounded once; or (o + D_h v) silu(gate) stored as float32 for a norm over several heads (group_norm_kernel).
#include "common.h"
#include <math.h>

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float dm_f32x4_t;

enum { DM_PLAIN = 0, DM_NORM_GATE = 1, DM_SKIP_GATE = 2 };

struct DecayMemory {
    int H, per, d, dv;                       // heads, heads that share a q/k head, sizes
    long long qs, ks, vs, gs;                // values from a token's row to the next: q, k, v, gate
    float kscale;
    const float* log_decay;                  // [H] constant per head, or null:
    const float* dt;                         //   raw step sizes, rows of `dts` values,
    long long dts;
    const float* dt_bias;                    //   [H]
    const float* rate;                       //   [H]: a = exp(-rate dt)
    const float2* rot;                       // [T][dims / 2] cosine and sine of every token's angles, or null (no rotation)
    int half;                                // dims / 2; pairs (i, i + half)
    const float* skip;                       // D [H] (DM_SKIP_GATE)
    float eps;                               // (DM_NORM_GATE)
    int epi;
    const int* slot_ids;
    int num_slots;
    float* state;
    long long state_stride;
    int pieces8;                             // every row and head in 16-byte pieces of the operands: eight values at a time
};

__device__ __forceinline__ float dm_silu(float x) { return x / (1.0f + expf(-x)); }

// value i of a q or k row, rotated by the token's angles
template <typename TA>
__device__ __forceinline__ float dm_rotated(const TA* row, int i, const float2* rot, int half) {
    const float x = to_f32<TA>(row[i]);
    if (!rot || i >= 2 * half) return x;
    const int j = i < half ? i : i - half;
    const float o = to_f32<TA>(row[i < half ? i + half : j]);
    const float2 c = rot[j];
    return i < half ? x * c.x - o * c.y : x * c.x + o * c.y;
}

// eight neighbouring values from a 16-byte aligned place
template <typename TA>
__device__ __forceinline__ void dm_load8(const TA* p, float (&v)[8]) {
    if constexpr (sizeof(TA) == 2) {
        typedef __attribute__((__vector_size__(4 * sizeof(uint32_t)))) uint32_t u32x4_t;
        const u32x4_t r = *reinterpret_cast<const u32x4_t*>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) { v[2 * i] = __uint_as_float(r[i] << 16); v[2 * i + 1] = __uint_as_float(r[i] & 0xffff0000u); }
    } else {
        float lo[4], hi[4];
        Vec4<float>::load(reinterpret_cast<const float*>(p), lo);
        Vec4<float>::load(reinterpret_cast<const float*>(p) + 4, hi);
#pragma unroll
        for (int i = 0; i < 4; ++i) { v[i] = lo[i]; v[4 + i] = hi[i]; }
    }
}

// values i .. i + 7 of a q or k row (d values), rotated by the token's angles; `pieces8`: i, d and half are multiples of 8
template <typename TA>
__device__ __forceinline__ void dm_rotated8(const DecayMemory& m, const TA* row, int i, const float2* rot, float (&v)[8]) {
    if (!m.pieces8) {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = i + e < m.d ? dm_rotated<TA>(row, i + e, rot, m.half) : 0.f;
        return;
    }
    if (i >= m.d) {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = 0.f;
        return;
    }
    dm_load8<TA>(row + i, v);
    if (!rot || i >= 2 * m.half) return;
    const bool low = i < m.half;
    const int j = low ? i : i - m.half;
    float o[8];
    dm_load8<TA>(row + (low ? i + m.half : j), o);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        const float2 c = rot[j + e];
        v[e] = low ? v[e] * c.x - o[e] * c.y : v[e] * c.x + o[e] * c.y;
    }
}

// values j .. j + 7 of a head's dv values
template <typename TA>
__device__ __forceinline__ void dm_values8(const DecayMemory& m, const TA* row, int j, float (&v)[8]) {
    if (m.pieces8 && j < m.dv) { dm_load8<TA>(row + j, v); return; }
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = j + e < m.dv ? to_f32<TA>(row[j + e]) : 0.f;
}

// log of the decay and the write's factor of token t, head h
__device__ __forceinline__ void dm_scalars(const DecayMemory& m, int t, int h, float* la, float* b) {
    if (m.log_decay) { *la = m.log_decay[h]; *b = 1.0f; return; }
    const float dt = softplus_f(m.dt[(size_t)t * m.dts + h] + m.dt_bias[h]);
    *la = -m.rate[h] * dt;
    *b = dt;
}

// ---- the angles of a step's tokens, once for all heads (and all layers of one rotation) -----------------------------------
__global__ void rotation_angles_kernel(float2* __restrict__ out, const int* __restrict__ positions, const float* __restrict__ freq, int T, int half) {
    const size_t n = (size_t)T * half;
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) {
        const int t = (int)(i / half), j = (int)(i - (size_t)t * half);
        const float ang = (float)positions[t] * freq[j];
        out[i] = make_float2(cosf(ang), sinf(ang));
    }
}

extern "C" int spy_rotation_angles(void* out, const int* positions, const float* freq, int T, int half, hipStream_t st) {
    SPY_REQUIRE(T > 0 && half > 0 && freq && ((uintptr_t)out % 8) == 0, "spy_rotation_angles: empty operand");
    const size_t n = (size_t)T * half;
    const unsigned blocks = (unsigned)((n + 255) / 256 > 65536 ? 65536 : (n + 255) / 256);
    rotation_angles_kernel<<<blocks, 256, 0, st>>>((float2*)out, positions, freq, T, half);
    SPY_CHECK_LAUNCH("spy_rotation_angles");
    return 0;
}

// ---- steps of single tokens ------------------------------------------------------------------------------------------------
#define DS_THREADS 256
#define DS_MAX_D 256
#define DS_SLICE 128        // value channels of a block (V == 4)
#define DS_SLICE_1 8        // the same with V == 1
// Thread (row group, column group): V neighbouring columns, every RG-th row of S, all of them asked for ahead of the first
// use.  Entry s is token s.
template <typename TA, int V, int ROWS>
__global__ __launch_bounds__(DS_THREADS) void decay_memory_step_kernel(void* __restrict__ out, const TA* __restrict__ q, const TA* __restrict__ k,
                                                                       const TA* __restrict__ v, const TA* __restrict__ gate, DecayMemory m) {
    __shared__ float qs[DS_MAX_D], ks[DS_MAX_D], part[DS_THREADS * V], red[16];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    constexpr int SLICE = V == 4 ? DS_SLICE : DS_SLICE_1;
    const int j_lo = blockIdx.z * SLICE, cols = min(m.dv - j_lo, SLICE);
    const int nc = (cols + V - 1) / V, RG = DS_THREADS / nc;
    const int rg = tid / nc, c = tid - rg * nc;
    const int slot = m.slot_ids[t];
    if (slot < 0 || slot >= m.num_slots) return;
    float* S = m.state + (size_t)slot * m.state_stride + (size_t)h * m.d * m.dv + j_lo + c * V;
    const bool on = rg < RG;
    float sv[ROWS][V];
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
        const int r = rg + i * RG;
#pragma unroll
        for (int e = 0; e < V; ++e) sv[i][e] = 0.f;
        if (on && r < m.d) {
            if constexpr (V == 4) Vec4<float>::load(S + (size_t)r * m.dv, sv[i]);
            else sv[i][0] = S[(size_t)r * m.dv];
        }
    }
    const int hq = h / m.per;
    const float2* rot = m.rot ? m.rot + (size_t)t * m.half : nullptr;
    for (int i = tid; i < m.d; i += DS_THREADS) {
        qs[i] = dm_rotated<TA>(q + (size_t)t * m.qs + (size_t)hq * m.d, i, rot, m.half);
        ks[i] = dm_rotated<TA>(k + (size_t)t * m.ks + (size_t)hq * m.d, i, rot, m.half) * m.kscale;
    }
    float la, b;
    dm_scalars(m, t, h, &la, &b);
    const float a = expf(la);
    const TA* vr = v + (size_t)t * m.vs + (size_t)h * m.dv + j_lo;
    float bv[V], acc[V];
#pragma unroll
    for (int e = 0; e < V; ++e) {
        bv[e] = (on && c * V + e < cols) ? b * to_f32<TA>(vr[c * V + e]) : 0.f;
        acc[e] = 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
        const int r = rg + i * RG;
        if (on && r < m.d) {
            const float kr = ks[r], qr = qs[r];
#pragma unroll
            for (int e = 0; e < V; ++e) {
                sv[i][e] = fmaf(a, sv[i][e], kr * bv[e]);
                acc[e] = fmaf(sv[i][e], qr, acc[e]);
            }
            if constexpr (V == 4) Vec4<float>::store(S + (size_t)r * m.dv, sv[i]);
            else S[(size_t)r * m.dv] = sv[i][0];
        }
    }
    if (on) {
#pragma unroll
        for (int e = 0; e < V; ++e) part[(rg * nc + c) * V + e] = acc[e];
    }
    __syncthreads();
    // (cols <= DS_SLICE < DS_THREADS: a thread has one column of the result)
    float o = 0.f;
    if (tid < cols) {
        for (int g = 0; g < RG; ++g) o += part[g * nc * V + tid];
    }
    const size_t at = ((size_t)t * m.H + h) * m.dv + j_lo + tid;
    float gj = 0.f;
    if (m.epi != DM_PLAIN && tid < cols) gj = dm_silu(to_f32<TA>(gate[(size_t)t * m.gs + (size_t)h * m.dv + j_lo + tid]));
    if (m.epi == DM_NORM_GATE) {                    // (one slice: cols == dv, checked by the launcher)
        const float ss = block_sum(tid < cols ? o * o : 0.f, red);
        if (tid < cols) reinterpret_cast<TA*>(out)[at] = from_f32<TA>(o / sqrtf(ss / (float)m.dv + m.eps) * gj);
    } else if (tid < cols) {
        if (m.epi == DM_SKIP_GATE) o = fmaf(m.skip[h], to_f32<TA>(vr[tid]), o) * gj;
        reinterpret_cast<float*>(out)[at] = o;
    }
}

// ---- longer entries, in pieces of up to 64 tokens ----------------------------------------------------------------------------
#define DP_TOKENS 64
#define DP_THREADS 256
#define DP_LD (64 + 16)       // floats from one staged row of 64 values to the next: four rows beside each other lie in different banks

// cum[t] of the piece's tokens (inclusive) and b, by the block's first wave; la beyond the piece's end is 0.  The sums are
// double: what is used of them is differences, and one token that forgets nearly everything must not cost the others their
// decays' last digits.
__device__ __forceinline__ void dp_scan(const DecayMemory& m, int t0, int n, int h, double* cum, float* bs) {
    if (threadIdx.x < 64) {
        const int lane = threadIdx.x;
        float la = 0.f, b = 0.f;
        if (lane < n) dm_scalars(m, t0 + lane, h, &la, &b);
        double sum = (double)la;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const double up = __shfl_up(sum, o, 64);
            if (lane >= o) sum += up;
        }
        cum[lane] = sum;
        bs[lane] = b;
    }
}

// A piece's own contribution to the state: work[piece][h] [d][dv] = sum_s exp(cum_end - cum_s) b_s k_s v_s^T, and its whole
// decay exp(cum_end) in decay[piece][h].  Block z has a 64 x 64 part of it; wave w of it 16 rows.
template <typename TA>
__global__ __launch_bounds__(DP_THREADS) void decay_memory_pieces_kernel(float* __restrict__ work, float* __restrict__ decay, const TA* __restrict__ k,
                                                                         const TA* __restrict__ v, DecayMemory m, const int* __restrict__ piece_t0,
                                                                         const int* __restrict__ piece_t1) {
    __shared__ __align__(16) float ks[DP_TOKENS * DP_LD], vs[DP_TOKENS * DP_LD];
    __shared__ double cum[DP_TOKENS];
    __shared__ float bs[DP_TOKENS];
    const int piece = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int nd = (m.d + 63) / 64;
    const int i0 = (blockIdx.z % nd) * 64, j0 = (blockIdx.z / nd) * 64;
    const int t0 = piece_t0[piece], n = min(piece_t1[piece] - t0, DP_TOKENS);
    const int hq = h / m.per;
    dp_scan(m, t0, n, h, cum, bs);
    __syncthreads();
    const double end = cum[n - 1];
    const int rows = (n + 3) & ~3;
    for (int e = tid; e < rows * 16; e += DP_THREADS) {              // eight values of k's or of v's part of a row
        const int s = e >> 4, c = 8 * (e & 7);
        float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        float f = 0.f;
        if (s < n) {
            if (e & 8) {
                dm_values8<TA>(m, v + (size_t)(t0 + s) * m.vs + (size_t)h * m.dv, j0 + c, x);
                f = bs[s] * expf((float)(end - cum[s]));
            } else {
                dm_rotated8<TA>(m, k + (size_t)(t0 + s) * m.ks + (size_t)hq * m.d, i0 + c, m.rot ? m.rot + (size_t)(t0 + s) * m.half : nullptr, x);
                f = m.kscale;
            }
        }
        float* dst = ((e & 8) ? vs : ks) + s * DP_LD + c;
        const float lo[4] = {x[0] * f, x[1] * f, x[2] * f, x[3] * f}, hi[4] = {x[4] * f, x[5] * f, x[6] * f, x[7] * f};
        Vec4<float>::store(dst, lo);
        Vec4<float>::store(dst + 4, hi);
    }
    if (tid == 0 && blockIdx.z == 0) decay[(size_t)piece * m.H + h] = expf((float)end);
    __syncthreads();
    const int wave = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4;
    if (i0 + 16 * wave >= m.d) return;
    dm_f32x4_t acc[4];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) acc[jt] = dm_f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < rows; s += 4) {
        const float ka = ks[(s + g) * DP_LD + 16 * wave + r];
#pragma unroll
        for (int jt = 0; jt < 4; ++jt) acc[jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka, vs[(s + g) * DP_LD + 16 * jt + r], acc[jt], 0, 0, 0);
    }
    float* dst = work + ((size_t)piece * m.H + h) * m.d * m.dv;
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
        const int j = j0 + 16 * jt + r;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = i0 + 16 * wave + 4 * g + i;
            if (row < m.d && j < m.dv) dst[(size_t)row * m.dv + j] = acc[jt][i];
        }
    }
}

// Along an entry's pieces, element by element of the state: every piece's contribution is replaced by the state that the
// piece starts from, and the entry's last state goes to the request's slot.  Block z is a piece; the first of an entry walks.
// (Pieces are the grid's slowest dimension: blocks go to the dies in turn, and with every n-th block at work only some of
// the dies would have any.)
#define DF_AHEAD 8
template <int V>
__global__ __launch_bounds__(256) void decay_memory_fold_kernel(float* __restrict__ work, const float* __restrict__ decay, DecayMemory m,
                                                                const int* __restrict__ piece_entry, const int* __restrict__ piece_first, int n_pieces) {
    const int first = blockIdx.z, h = blockIdx.y;
    if (piece_first[first] != first) return;
    const int slot = m.slot_ids[piece_entry[first]];
    if (slot < 0 || slot >= m.num_slots) return;
    const size_t size = (size_t)m.d * m.dv, i = ((size_t)blockIdx.x * 256 + threadIdx.x) * V;
    if (i >= size) return;
    int last = first;
    while (last + 1 < n_pieces && piece_first[last + 1] == first) ++last;
    float* st = m.state + (size_t)slot * m.state_stride + (size_t)h * size + i;
    float S[V];
    if constexpr (V == 4) Vec4<float>::load(st, S); else S[0] = st[0];
    for (int p0 = first; p0 <= last; p0 += DF_AHEAD) {
        float L[DF_AHEAD][V], A[DF_AHEAD];
#pragma unroll
        for (int u = 0; u < DF_AHEAD; ++u) {
            const int p = min(p0 + u, last);
            const float* src = work + ((size_t)p * m.H + h) * size + i;
            if constexpr (V == 4) Vec4<float>::load(src, L[u]); else L[u][0] = src[0];
            A[u] = decay[(size_t)p * m.H + h];
        }
#pragma unroll
        for (int u = 0; u < DF_AHEAD; ++u) {
            if (p0 + u <= last) {
                float* dst = work + ((size_t)(p0 + u) * m.H + h) * size + i;
                if constexpr (V == 4) Vec4<float>::store(dst, S); else dst[0] = S[0];
#pragma unroll
                for (int e = 0; e < V; ++e) S[e] = fmaf(A[u], S[e], L[u][e]);
            }
        }
    }
    if constexpr (V == 4) Vec4<float>::store(st, S); else st[0] = S[0];
}

// A piece's results.  Wave w of a block has tokens 16 w .. + 15; block z has 16 NJ value channels.  Results lie transposed in
// the accumulators: lane (r, g) holds token r, channels 16 jt + 4 g .. + 3.
//   first o = S_in^T q, over d in slabs of 64 staged rows of S_in and of k (which serve the scores in the same pass);
//   then o *= exp(cum_t); then o += sum_s P^T_(s, t) v_s: the scores' tile leaves lane (r, g) with tokens s = 4 g + i of token
//   t = r, which is what it must supply when the four products of a tile take s in the order 4 g + i, i = 0 .. 3.
template <typename TA, int NJ>
__global__ __launch_bounds__(DP_THREADS) void decay_memory_results_kernel(void* __restrict__ out, const float* __restrict__ work, const TA* __restrict__ q,
                                                                          const TA* __restrict__ k, const TA* __restrict__ v, const TA* __restrict__ gate,
                                                                          DecayMemory m, const int* __restrict__ piece_entry,
                                                                          const int* __restrict__ piece_t0, const int* __restrict__ piece_t1) {
    constexpr int KLD = 64 + 4, SLD = 16 * NJ + 16, VLD = 16 * NJ + 4;
    __shared__ __align__(16) float ks[DP_TOKENS * KLD], sv[64 * SLD];
    __shared__ double cum[DP_TOKENS];
    __shared__ float bs[DP_TOKENS];
    const int piece = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, j0 = blockIdx.z * 16 * NJ;
    const int t0 = piece_t0[piece], n = min(piece_t1[piece] - t0, DP_TOKENS);
    const int hq = h / m.per;
    const int slot = m.slot_ids[piece_entry[piece]];
    if (slot < 0 || slot >= m.num_slots) return;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int tl = 16 * wave + r;                                    // this lane's token inside the piece
    const bool mine = 16 * wave < n, tok = tl < n;
    dp_scan(m, t0, n, h, cum, bs);
    const float* S = work + ((size_t)piece * m.H + h) * m.d * m.dv;
    const int rows = min((n + 15) & ~15, DP_TOKENS);
    dm_f32x4_t acc[NJ], sc[4];
#pragma unroll
    for (int jt = 0; jt < NJ; ++jt) acc[jt] = dm_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < 4; ++st) sc[st] = dm_f32x4_t{0.f, 0.f, 0.f, 0.f};
    const TA* qrow = q + (size_t)(t0 + (tok ? tl : 0)) * m.qs + (size_t)hq * m.d;
    const float2* qrot = m.rot ? m.rot + (size_t)(t0 + (tok ? tl : 0)) * m.half : nullptr;
    // Inside a slab, step st of the products takes dim 16 g + st from lane (r, g), so that a lane's 16 values of its query lie
    // side by side in memory; in LDS, dim i of the slab has the place 4 (i % 16) + i / 16 (k: column, S_in: row).
    for (int i0 = 0; i0 < m.d; i0 += 64) {
        const int steps = min(16, m.d - i0);                         // dims 16 g + st of this slab exist up to here for g = 0
        __syncthreads();                                             // the slab before has been read
        for (int e = tid; e < rows * 8; e += DP_THREADS) {
            const int s = e >> 3, c = e & 7;
            float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (s < n) dm_rotated8<TA>(m, k + (size_t)(t0 + s) * m.ks + (size_t)hq * m.d, i0 + 8 * c, m.rot ? m.rot + (size_t)(t0 + s) * m.half : nullptr, x);
            float* dst = ks + s * KLD + 32 * (c & 1) + (c >> 1);
#pragma unroll
            for (int i = 0; i < 8; ++i) dst[4 * i] = x[i] * m.kscale;
        }
        for (int e = tid; e < 64 * 4 * NJ; e += DP_THREADS) {
            const int i = e / (4 * NJ), c = 4 * (e - i * (4 * NJ));
            float x[4] = {0.f, 0.f, 0.f, 0.f};
            if (i0 + i < m.d) {
                const float* src = S + (size_t)(i0 + i) * m.dv + j0 + c;
                if (m.pieces8) { if (j0 + c < m.dv) Vec4<float>::load(src, x); }
                else {
#pragma unroll
                    for (int u = 0; u < 4; ++u) x[u] = j0 + c + u < m.dv ? src[u] : 0.f;
                }
            }
            Vec4<float>::store(sv + (4 * (i & 15) + (i >> 4)) * SLD + c, x);
        }
        float qf[16];
        {
            float lo[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, hi[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (tok) {
                dm_rotated8<TA>(m, qrow, i0 + 16 * g, qrot, lo);
                dm_rotated8<TA>(m, qrow, i0 + 16 * g + 8, qrot, hi);
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) { qf[i] = lo[i]; qf[8 + i] = hi[i]; }
        }
        __syncthreads();
        if (mine) {
#pragma unroll
            for (int st = 0; st < 16; ++st) {
                if (st < steps) {
#pragma unroll
                    for (int jt = 0; jt < NJ; ++jt) acc[jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[(4 * st + g) * SLD + 16 * jt + r], qf[st], acc[jt], 0, 0, 0);
#pragma unroll
                    for (int tile = 0; tile < 4; ++tile)
                        if (tile <= wave) sc[tile] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(16 * tile + r) * KLD + 4 * st + g], qf[st], sc[tile], 0, 0, 0);
                }
            }
        }
    }
    __syncthreads();
    for (int e = tid; e < rows * 2 * NJ; e += DP_THREADS) {
        const int s = e / (2 * NJ), c = 8 * (e - s * (2 * NJ));
        float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (s < n) dm_values8<TA>(m, v + (size_t)(t0 + s) * m.vs + (size_t)h * m.dv, j0 + c, x);
        const float lo[4] = {x[0], x[1], x[2], x[3]}, hi[4] = {x[4], x[5], x[6], x[7]};
        Vec4<float>::store(sv + s * VLD + c, lo);
        Vec4<float>::store(sv + s * VLD + c + 4, hi);
    }
    __syncthreads();
    if (!mine) return;                                               // (no barrier behind this)
    const double ct = cum[tok ? tl : n - 1];
    const float et = expf((float)ct);
#pragma unroll
    for (int jt = 0; jt < NJ; ++jt) acc[jt] *= et;
#pragma unroll
    for (int tile = 0; tile < 4; ++tile) {
        if (tile <= wave) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int s = 16 * tile + 4 * g + i;
                const float p = (s <= tl && s < n) ? sc[tile][i] * (bs[s] * expf((float)(ct - cum[s]))) : 0.f;
#pragma unroll
                for (int jt = 0; jt < NJ; ++jt) acc[jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[s * VLD + 16 * jt + r], p, acc[jt], 0, 0, 0);
            }
        }
    }
    const int t = t0 + tl;
    float scale = 1.f;
    if (m.epi == DM_NORM_GATE) {                                     // (one block has the whole head, checked by the launcher)
        float ss = 0.f;
#pragma unroll
        for (int jt = 0; jt < NJ; ++jt)
#pragma unroll
            for (int i = 0; i < 4; ++i) ss = fmaf(acc[jt][i], acc[jt][i], ss);        // (channels beyond dv are zero)
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        scale = 1.0f / sqrtf(ss / (float)m.dv + m.eps);
    }
    if (!tok) return;
    const TA* gr = m.epi != DM_PLAIN ? gate + (size_t)t * m.gs + (size_t)h * m.dv : nullptr;
    const float D = m.epi == DM_SKIP_GATE ? m.skip[h] : 0.f;
#pragma unroll
    for (int jt = 0; jt < NJ; ++jt) {
        const int jb = j0 + 16 * jt + 4 * g;
        const size_t at = ((size_t)t * m.H + h) * m.dv + jb;
        float y[4], gv[4] = {0.f, 0.f, 0.f, 0.f};
        if (gr) {
            if (m.pieces8) { if (jb < m.dv) Vec4<TA>::load(gr + jb, gv); }
            else {
#pragma unroll
                for (int i = 0; i < 4; ++i) gv[i] = jb + i < m.dv ? to_f32<TA>(gr[jb + i]) : 0.f;
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            y[i] = acc[jt][i];
            if (m.epi == DM_NORM_GATE) y[i] = (y[i] * scale) * dm_silu(gv[i]);
            if (m.epi == DM_SKIP_GATE) y[i] = fmaf(D, sv[tl * VLD + jb + i - j0], y[i]) * dm_silu(gv[i]);
        }
        if (m.pieces8) {
            if (jb < m.dv) {
                if (m.epi == DM_NORM_GATE) Vec4<TA>::store(reinterpret_cast<TA*>(out) + at, y);
                else Vec4<float>::store(reinterpret_cast<float*>(out) + at, y);
            }
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (jb + i >= m.dv) continue;
                if (m.epi == DM_NORM_GATE) reinterpret_cast<TA*>(out)[at + i] = from_f32<TA>(y[i]);
                else reinterpret_cast<float*>(out)[at + i] = y[i];
            }
        }
    }
}

// out[t, :] = o / rms(o) over each of `groups` equal runs of N values, times w (null: none), times silu(gate[t, :]) (null:
// none; rows `gs` values apart); one block per (token, run)
// PASSES > 0: the run (its values in 16-byte pieces, at most 4 PASSES a thread) is read once and kept in registers.
template <typename TA, typename TW, int PASSES>
__global__ void group_norm_kernel(TA* __restrict__ out, const float* __restrict__ o, const TW* __restrict__ w, const TA* __restrict__ gate,
                                  long long gs, float eps, int groups, int N) {
    __shared__ float red[16];
    const int t = blockIdx.x, g = blockIdx.y, n = N / groups;
    const float* row = o + (size_t)t * N + (size_t)g * n;
    const TW* wr = w ? w + (size_t)g * n : nullptr;
    TA* dst = out + (size_t)t * N + (size_t)g * n;
    const TA* gr = gate ? gate + (size_t)t * gs + (size_t)g * n : nullptr;
    float ss = 0.f;
    if constexpr (PASSES > 0) {
        float v[PASSES][4], wv[PASSES][4], gv[PASSES][4];
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) { v[p][e] = 0.f; wv[p][e] = 1.f; }
            if (i < n) {
                Vec4<float>::load(row + i, v[p]);
                if (wr) Vec4<TW>::load(wr + i, wv[p]);
                if (gr) Vec4<TA>::load(gr + i, gv[p]);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) ss = fmaf(v[p][e], v[p][e], ss);
        }
        const float r = 1.0f / sqrtf(block_sum(ss, red) / (float)n + eps);
#pragma unroll
        for (int p = 0; p < PASSES; ++p) {
            const int i = (p * blockDim.x + threadIdx.x) * 4;
            if (i < n) {
                float y[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) y[e] = (v[p][e] * r) * wv[p][e] * (gr ? dm_silu(gv[p][e]) : 1.0f);
                Vec4<TA>::store(dst + i, y);
            }
        }
        return;
    }
    for (int i = threadIdx.x; i < n; i += blockDim.x) ss = fmaf(row[i], row[i], ss);
    const float r = 1.0f / sqrtf(block_sum(ss, red) / (float)n + eps);
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        float y = (row[i] * r) * (wr ? to_f32<TW>(wr[i]) : 1.0f);
        if (gr) y *= dm_silu(to_f32<TA>(gr[i]));
        dst[i] = from_f32<TA>(y);
    }
}

extern "C" int spy_group_norm(void* out, int dtype, const float* o, const void* w, int w_dtype, const void* gate, long long gs, float eps, int T,
                              int groups, int N, hipStream_t st) {
    SPY_REQUIRE(T > 0 && groups > 0 && N > 0 && N % groups == 0 && groups <= 65535, "spy_group_norm: %d groups of %d values", groups, N);
    SPY_REQUIRE(!gate || gs >= N, "spy_group_norm: the gate's rows are too short");
    const int n = N / groups, threads = n >= 1024 ? 256 : (n >= 512 ? 128 : 64);
    const bool pieces = n % 4 == 0 && gs % 4 == 0 && (((uintptr_t)out | (uintptr_t)o | (uintptr_t)w | (uintptr_t)gate) % 16) == 0;
    const int passes = pieces ? (n / 4 + threads - 1) / threads : 0;
#define GN(P) group_norm_kernel<TA, TW, P><<<dim3(T, groups), threads, 0, st>>>((TA*)out, o, (const TW*)w, (const TA*)gate, gs, eps, groups, N)
    SPY_DISPATCH(dtype, TA, SPY_DISPATCH(w_dtype, TW, {
        if (passes == 0 || passes > 8) GN(0);
        else if (passes == 1) GN(1);
        else if (passes == 2) GN(2);
        else if (passes <= 4) GN(4);
        else GN(8);
    }));
#undef GN
    SPY_CHECK_LAUNCH("spy_group_norm");
    return 0;
}

// q, k: rows of heads of d (head h of H reads head h / per), v and gate: rows of H heads of dv.  single != 0: every entry is
// one token (entry s is token s).  Otherwise pieces (int32 [4][n_pieces]: entry, first row, end row, index of the entry's
// first piece; at most 64 rows each) with work [n_pieces][H][d][dv] and decay [n_pieces][H] as scratch.
// out: [T, H dv], float32 (epi 0 and 2) or of the operands' dtype (epi 1: dv at most 128).
extern "C" int spy_decay_memory(void* out, const void* q, long long qs, const void* k, long long ks, const void* v, long long vs, const void* gate,
                                long long gs, int dtype, int H, int per, int d, int dv, float kscale, const float* log_decay, const float* dt,
                                long long dts, const float* dt_bias, const float* rate, const void* rot, int half, const float* skip, float eps,
                                int epi, float* state, long long state_stride, const int* slot_ids, int num_slots, int S, int T, int single,
                                const int* pieces, int n_pieces, float* work, float* decay, hipStream_t st) {
    SPY_REQUIRE(S > 0 && T > 0 && H > 0 && per > 0 && H % per == 0 && d > 0 && dv > 0 && num_slots > 0, "spy_decay_memory: empty operand");
    SPY_REQUIRE(d <= DS_MAX_D && dv <= 4096 && H <= 65535, "spy_decay_memory: heads of %d x %d (key size up to %d)", d, dv, DS_MAX_D);
    SPY_REQUIRE(state_stride >= (long long)H * d * dv && qs >= (long long)(H / per) * d && ks >= (long long)(H / per) * d && vs >= (long long)H * dv,
                "spy_decay_memory: the state or the rows are too short");
    SPY_REQUIRE(log_decay || (dt && dt_bias && rate && dts >= H), "spy_decay_memory: no decay");
    SPY_REQUIRE(half >= 0 && 2 * half <= d && (!rot || half > 0), "spy_decay_memory: %d rotated pairs of a head of %d", half, d);
    SPY_REQUIRE(epi >= 0 && epi <= 2 && (epi == DM_PLAIN || (gate && gs >= (long long)H * dv)) && (epi != DM_SKIP_GATE || skip) &&
                (epi != DM_NORM_GATE || dv <= DS_SLICE), "spy_decay_memory: epilogue %d with heads of %d", epi, dv);
    const uintptr_t bits = (uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)gate | (uintptr_t)work | (uintptr_t)out;
    const bool pieces8 = d % 8 == 0 && dv % 8 == 0 && half % 8 == 0 && ((qs | ks | vs | gs) & 7) == 0 && bits % 16 == 0;
    const DecayMemory m = {H, per, d, dv, qs, ks, vs, gs, kscale, log_decay, dt, dts, dt_bias, rate, (const float2*)rot, half, skip, eps, epi,
                           slot_ids, num_slots, state, state_stride, pieces8 ? 1 : 0};
    const bool v4 = dv % 4 == 0 && state_stride % 4 == 0 && ((uintptr_t)state % 16) == 0 && ((uintptr_t)work % 16) == 0;
    if (single) {
        SPY_REQUIRE(S == T, "spy_decay_memory: %d tokens of %d entries", T, S);
        // (a norm over the head needs the head in one block: values that cannot be read four at a time are normed by a pass of its own)
        SPY_REQUIRE(epi != DM_NORM_GATE || v4 || dv <= DS_SLICE_1, "spy_decay_memory: a head of %d values cannot be normed in a block", dv);
        const int slice = v4 ? DS_SLICE : DS_SLICE_1;
        const dim3 grid(S, H, (dv + slice - 1) / slice);
        const int cols = dv < slice ? dv : slice, nc = (cols + (v4 ? 4 : 1) - 1) / (v4 ? 4 : 1), RG = DS_THREADS / nc, need = (d + RG - 1) / RG;
#define DS_RUN(V, R) decay_memory_step_kernel<TA, V, R><<<grid, DS_THREADS, 0, st>>>(out, (const TA*)q, (const TA*)k, (const TA*)v, (const TA*)gate, m)
        SPY_REQUIRE(need <= (v4 ? 32 : 8), "spy_decay_memory: heads of %d x %d", d, dv);
        SPY_DISPATCH(dtype, TA, {
            if (!v4) DS_RUN(1, 8);
            else if (need <= 4) DS_RUN(4, 4);
            else if (need <= 8) DS_RUN(4, 8);
            else if (need <= 16) DS_RUN(4, 16);
            else DS_RUN(4, 32);
        });
#undef DS_RUN
        SPY_CHECK_LAUNCH("spy_decay_memory (single tokens)");
        return 0;
    }
    SPY_REQUIRE(pieces && n_pieces > 0 && work && decay, "spy_decay_memory: longer entries need their pieces and scratch memory");
    const int* pe = pieces;
    const int* p0 = pieces + n_pieces;
    const int* p1 = pieces + 2 * (size_t)n_pieces;
    const int* pf = pieces + 3 * (size_t)n_pieces;
    const dim3 pgrid(n_pieces, H, ((d + 63) / 64) * ((dv + 63) / 64));
    SPY_DISPATCH(dtype, TA, (decay_memory_pieces_kernel<TA><<<pgrid, DP_THREADS, 0, st>>>(work, decay, (const TA*)k, (const TA*)v, m, p0, p1)));
    SPY_CHECK_LAUNCH("spy_decay_memory (pieces)");
    const size_t size = (size_t)d * dv;
    const dim3 fgrid((unsigned)((size / (v4 ? 4 : 1) + 255) / 256), H, n_pieces);
    SPY_REQUIRE(n_pieces <= 65535, "spy_decay_memory: %d pieces are too many", n_pieces);
    if (v4) decay_memory_fold_kernel<4><<<fgrid, 256, 0, st>>>(work, decay, m, pe, pf, n_pieces);
    else decay_memory_fold_kernel<1><<<fgrid, 256, 0, st>>>(work, decay, m, pe, pf, n_pieces);
    SPY_CHECK_LAUNCH("spy_decay_memory (fold)");
    const int nj = dv <= 64 ? 4 : 8;
    const dim3 rgrid(n_pieces, H, (dv + 16 * nj - 1) / (16 * nj));
    SPY_DISPATCH(dtype, TA, {
        if (nj == 4) decay_memory_results_kernel<TA, 4><<<rgrid, DP_THREADS, 0, st>>>(out, work, (const TA*)q, (const TA*)k, (const TA*)v, (const TA*)gate, m, pe, p0, p1);
        else decay_memory_results_kernel<TA, 8><<<rgrid, DP_THREADS, 0, st>>>(out, work, (const TA*)q, (const TA*)k, (const TA*)v, (const TA*)gate, m, pe, p0, p1);
    });
    SPY_CHECK_LAUNCH("spy_decay_memory (results)");
    return 0;
}
