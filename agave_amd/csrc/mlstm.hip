// The matrix memory of xLSTM (Beck et al., "xLSTM: Extended Long Short-Term Memory") for gfx950.  Per sequence and head a
// matrix S [dk][dv], a vector n [dk] and a running maximum m, all 32-bit, advanced token by token from m = 0:
//
//   i = cap(i_in + i_bias),  f = logsigmoid(cap(f_in + f_bias)),  cap(z) = c tanh(z / c)
//   m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n <- exp(f + m - m') n + exp(i - m') k
//   o = S^T q / (max(|n . q|, exp(-m')) + floor)           (q times a scale)
//   y = o / rms(o) * w * sigmoid(gate)                     (rms over the head's dv elements)
//
// S is stored with a column's rows together, [slot][head][dv][dk]; n is one more column to every kernel.
//
// Steps of one token a sequence: mlstm_step updates the state (a group of lanes per column, the column in registers) and
// leaves S^T q and n . q; mlstm_readout divides, norms and gates, and stores the new m (which mlstm_step's workgroups all
// still read).
//
// Steps of more tokens run in chunks of CHUNK tokens.  With F_t the sum of a chunk's log forget gates up to t, a_j = i_j -
// F_j and b_t = max(m_0, max_{j <= t} a_j) (m_0: the maximum the chunk starts with) the recurrence says m_t = F_t + b_t and
//   S_t = exp(m_0 - b_t) S_0 + sum_{j <= t} exp(a_j - b_t) k_j v_j^T,
// so that every exponent is at most 0.  F, a and b are kept in double: they are differences of sums over the chunk.
//   mlstm_gates   F, a and the running maximum of a, per chunk and head, and the chunk's totals;
//   mlstm_chunk   what a chunk adds to the state, relative to its own maximum: all chunks at once;
//   mlstm_carry   the states the chunks start from: elementwise, chunk after chunk; the sequence's state at the end;
//   mlstm_read    the outputs: q against the chunk's starting state, plus q k^T inside the chunk weighted by exp(a_j - b_t)
//                 against v; division, norm and gate on the way out.
// The products are 32-bit ones (v_mfma_f32_16x16x4_f32: A[i][k] in lane i + 16 k, B[k][j] in lane j + 16 k, D[i][j] in lane
// j + 16 (i / 4) as element i % 4).  Which numbers a product's four k-places hold is free as long as both operands agree:
// a lane loads four neighbours along the summed dimension at once and uses them in four instructions.
#include "common_impl.h"
#include "mfma.h"
#include <math.h>

#define CHUNK 128
#define KEY_BLOCKS (CHUNK / 16)
#define MAX_DK 1024
#define MAX_DV 1024

struct MlstmArgs {
    const float *q, *k, *v, *gate, *i_in, *f_in;    // column slices of the same rows
    long ld;
    const float *i_bias, *f_bias, *weight;          // [nh], [nh], [nh * dv]
    float cap, floor_eps, norm_eps, q_scale;
    float *S, *n, *m;                               // [slots][nh][dv][dk], [slots][nh][dk], [slots][nh]
    const int *cu, *slots;
    int nh, dk, dv, n_seqs;
};

__device__ __forceinline__ float capped(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float sigmoid_of(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float exp_of_difference(double a, double b) { return expf((float)(a - b)); }

__device__ __forceinline__ void log_gates(const MlstmArgs& A, long row, int h, float& i, float& f) {
    i = capped(A.i_in[row * A.ld + h] + A.i_bias[h], A.cap);
    f = log_sigmoid(capped(A.f_in[row * A.ld + h] + A.f_bias[h], A.cap));
}

__device__ __forceinline__ f32x4_t mfma_16x16x4(float a, float b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// four neighbours x[d .. d + 3] of a row of n elements, zeros past its end (VEC: n is a multiple of 4 and rows are aligned)
template <bool VEC> __device__ __forceinline__ f32x4_t four(const float* x, int d, int n) {
    f32x4_t r;
    if (VEC) {
        r = *reinterpret_cast<const f32x4_t*>(x + (d < n ? d : 0));
        if (d >= n) r = f32x4_t{0.f, 0.f, 0.f, 0.f};
    } else {
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const float got = x[d + u < n ? d + u : 0];
            r[u] = d + u < n ? got : 0.f;
        }
    }
    return r;
}

// ------------------------------------------------------------------ one token a sequence
// A column of dk elements is shared by L lanes, each with R groups of V neighbours; a wave takes 64 / L columns at a time,
// UN times, with all of its loads under way before the first is used.  Column dv is n.
template <int L, int V, int R, int UN>
__global__ __launch_bounds__(256) void mlstm_step_kernel(MlstmArgs A, float* __restrict__ num, float* __restrict__ nq) {
    constexpr int CW = 64 / L;
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, part = lane % L;
    const int h = blockIdx.y, s = blockIdx.z, dk = A.dk, dv = A.dv;
    const long row = A.cu[s], sh = (long)A.slots[s] * A.nh + h;
    const int col0 = ((int)blockIdx.x * 4 + wv) * CW * UN + lane / L;
    float i, f;
    log_gates(A, row, h, i, f);
    const float m0 = A.m[sh];
    float* cols[UN];
    float S[UN][R][V], vv[UN], kx[R][V], qx[R][V];
#pragma unroll
    for (int u = 0; u < UN; ++u) {
        const int col = col0 + u * CW;
        cols[u] = col < dv ? A.S + (sh * dv + col) * dk : A.n + sh * dk;
        vv[u] = A.v[row * A.ld + (long)h * dv + (col < dv ? col : 0)];
        if (col >= dv) vv[u] = 1.f;
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = (r * L + part) * V, dd = d < dk ? d : 0;
        if (V == 4) {
            *reinterpret_cast<f32x4_t*>(kx[r]) = *reinterpret_cast<const f32x4_t*>(A.k + row * A.ld + (long)h * dk + dd);
            *reinterpret_cast<f32x4_t*>(qx[r]) = *reinterpret_cast<const f32x4_t*>(A.q + row * A.ld + (long)h * dk + dd);
        } else {
            kx[r][0] = A.k[row * A.ld + (long)h * dk + dd];
            qx[r][0] = A.q[row * A.ld + (long)h * dk + dd];
        }
#pragma unroll
        for (int u = 0; u < UN; ++u) {
            if (V == 4) *reinterpret_cast<f32x4_t*>(S[u][r]) = *reinterpret_cast<const f32x4_t*>(cols[u] + dd);
            else S[u][r][0] = cols[u][dd];
        }
    }
    const double kept = (double)f + (double)m0;              // (in double, so that a small f is not lost beside m)
    const float m1 = (float)fmax(kept, (double)i), keep = exp_of_difference(kept, m1), write = exp_of_difference(i, m1);
    float kq = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const bool in = (r * L + part) * V < dk;
#pragma unroll
        for (int e = 0; e < V; ++e) {
            qx[r][e] = in ? qx[r][e] * A.q_scale : 0.f;
            kq = fmaf(kx[r][e], qx[r][e], kq);
        }
    }
#pragma unroll
    for (int off = 1; off < L; off *= 2) kq += __shfl_xor(kq, off);
#pragma unroll
    for (int u = 0; u < UN; ++u) {
        const int col = col0 + u * CW;
        float dot = 0.f;
#pragma unroll
        for (int r = 0; r < R; ++r)
#pragma unroll
            for (int e = 0; e < V; ++e) dot = fmaf(S[u][r][e], qx[r][e], dot);
#pragma unroll
        for (int off = 1; off < L; off *= 2) dot += __shfl_xor(dot, off);
        if (col > dv) continue;
        const float w = write * vv[u];
        const float o = fmaf(w, kq, keep * dot);
        if (part == 0) {
            if (col < dv) num[row * ((long)A.nh * dv) + (long)h * dv + col] = o;
            else nq[row * A.nh + h] = o;
        }
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int d = (r * L + part) * V;
            if (d >= dk) continue;
#pragma unroll
            for (int e = 0; e < V; ++e) S[u][r][e] = fmaf(w, kx[r][e], keep * S[u][r][e]);
            if (V == 4) *reinterpret_cast<f32x4_t*>(cols[u] + d) = *reinterpret_cast<const f32x4_t*>(S[u][r]);
            else cols[u][d] = S[u][r][0];
        }
    }
}

// A workgroup per (sequence, head): division, norm, weight and gate; the new maximum.
template <typename T>
__global__ __launch_bounds__(256) void mlstm_readout_kernel(MlstmArgs A, const float* __restrict__ num, const float* __restrict__ nq,
                                                            T* __restrict__ out, long ldo) {
    __shared__ float red[16];
    constexpr int KEEP = MAX_DV / 64;
    const int s = blockIdx.x, h = blockIdx.y, dv = A.dv, nt = blockDim.x;
    const long row = A.cu[s], sh = (long)A.slots[s] * A.nh + h;
    const float* x = num + row * ((long)A.nh * dv) + (long)h * dv;
    const float* g = A.gate + row * A.ld + (long)h * dv;
    const float* w = A.weight + (long)h * dv;
    float i, f;
    log_gates(A, row, h, i, f);
    const float m1 = (float)fmax((double)f + (double)A.m[sh], (double)i);
    const float inv_den = 1.0f / (fmaxf(fabsf(nq[row * A.nh + h]), expf(-m1)) + A.floor_eps);
    float o[KEEP], ss = 0.f;
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const int e = (int)threadIdx.x + u * nt;
        if (u * nt >= dv) break;
        o[u] = e < dv ? x[e] * inv_den : 0.f;
        ss = fmaf(o[u], o[u], ss);
    }
    ss = block_sum(ss, red);                        // (its barriers: every thread has read m)
    if (threadIdx.x == 0) A.m[sh] = m1;
    const float inv = 1.0f / sqrtf(ss / (float)dv + A.norm_eps);
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const int e = (int)threadIdx.x + u * nt;
        if (u * nt >= dv) break;
        if (e < dv) st(out + row * ldo + (long)h * dv + e, o[u] * inv * w[e] * sigmoid_of(g[e]));
    }
}

// ------------------------------------------------------------------ chunks
// Chunk c of sequence b is number cu[b] / CHUNK + b + c of the step's: a sequence's numbers end before the next one's begin.
struct ChunkArgs {
    double *F, *a, *top;             // [number][nh][CHUNK]: sums of log forget gates, a, running maximum of a
    double *F_all, *top_all;         // [number][nh]: the chunk's totals
    float *m0;                       // [number][nh]: the maximum a chunk starts with
    float *m_end;                    // [sequence][nh]: the maximum behind the last chunk
    float *part;                     // [number][nh][dv + 1][dk]: what a chunk adds, then the state it starts from
};

struct ChunkPlace { int first, count; long number; };      // first row of the step, rows, number; count <= 0: no such chunk
__device__ __forceinline__ ChunkPlace chunk_of(const MlstmArgs& A, int s, int c) {
    const int r0 = A.cu[s], r1 = A.cu[s + 1];
    ChunkPlace p;
    p.first = r0 + c * CHUNK;
    p.count = min(CHUNK, r1 - p.first);
    p.number = (long)(r0 / CHUNK) + s + c;
    return p;
}

// What the `per` workgroups of one (chunk, head) read besides their own rows is the same for all of them, and every XCD has
// an L2 of its own: workgroup ids go round the XCDs, so the ids of a unit's workgroups are XCDS apart.
#define XCDS 8
struct UnitPlace { int sub, c, h, s; };          // s < 0: no such unit
__device__ __forceinline__ UnitPlace unit_of(int id, int per, int chunks, int nh, int n_seqs) {
    const int unit = id / (XCDS * per) * XCDS + id % XCDS;
    UnitPlace u{id / XCDS % per, unit % chunks, unit / chunks % nh, unit / (chunks * nh)};
    if (u.s >= n_seqs) u.s = -1;
    return u;
}
static long unit_workgroups(long units, long per) { return (units + XCDS - 1) / XCDS * XCDS * per; }

__global__ __launch_bounds__(CHUNK) void mlstm_gates_kernel(MlstmArgs A, ChunkArgs C) {
    __shared__ double tot[CHUNK / 64], most[CHUNK / 64];
    const int h = blockIdx.y, s = blockIdx.z, j = threadIdx.x, lane = j & 63, wv = j >> 6;
    const ChunkPlace P = chunk_of(A, s, blockIdx.x);
    if (P.count <= 0) return;                                // (the whole workgroup)
    float i, f;
    log_gates(A, P.first + (j < P.count ? j : 0), h, i, f);
    double F = j < P.count ? (double)f : 0.0;
#pragma unroll
    for (int off = 1; off < 64; off *= 2) {
        const double before = __shfl_up(F, off);
        if (lane >= off) F += before;
    }
    if (lane == 63) tot[wv] = F;
    __syncthreads();
    if (wv == 1) F += tot[0];
    const double a = j < P.count ? (double)i - F : -INFINITY;
    double top = a;
#pragma unroll
    for (int off = 1; off < 64; off *= 2) {
        const double before = __shfl_up(top, off);
        if (lane >= off) top = fmax(top, before);
    }
    if (lane == 63) most[wv] = top;
    __syncthreads();
    if (wv == 1) top = fmax(top, most[0]);
    const long at = (P.number * A.nh + h) * CHUNK + j;
    C.F[at] = F;
    C.a[at] = a;
    C.top[at] = top;
    if (j == CHUNK - 1) {                                    // (behind the last token F stays and a is -inf)
        C.F_all[P.number * A.nh + h] = F;
        C.top_all[P.number * A.nh + h] = top;
    }
}

// A wave's tile is 64 rows d by 64 columns e of sum_j exp(a_j - top) k_j v_j^T; four waves, four tiles a workgroup.
template <bool VEC>
__global__ __launch_bounds__(256) void mlstm_chunk_kernel(MlstmArgs A, ChunkArgs C, int chunks, int per) {
    __shared__ float w[CHUNK];
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, c16 = lane & 15, g = lane >> 4;
    const UnitPlace U0 = unit_of(blockIdx.x, per, chunks, A.nh, A.n_seqs);
    if (U0.s < 0) return;
    const int h = U0.h, dk = A.dk, dv = A.dv;
    const ChunkPlace P = chunk_of(A, U0.s, U0.c);
    if (P.count <= 0) return;                                // (the whole workgroup)
    const long nh_at = P.number * A.nh + h;
    if (threadIdx.x < CHUNK) w[threadIdx.x] = exp_of_difference(C.a[nh_at * CHUNK + threadIdx.x], C.top_all[nh_at]);
    __syncthreads();
    const int tiles_d = (dk + 63) / 64, tiles = tiles_d * ((dv + 63) / 64), tile = U0.sub * 4 + wv;
    if (tile >= tiles) return;                               // (no barrier follows)
    const int d0 = (tile % tiles_d) * 64, e0 = (tile / tiles_d) * 64;
    const float *kp[4], *vp[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) {
        kp[b] = A.k + (long)P.first * A.ld + (long)h * dk + min(d0 + 16 * b + c16, dk - 1);
        vp[b] = A.v + (long)P.first * A.ld + (long)h * dv + min(e0 + 16 * b + c16, dv - 1);
    }
    f32x4_t acc[4][4];                                       // [d block][e block]
    float n_sum[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int a = 0; a < 4; ++a)
#pragma unroll
        for (int b = 0; b < 4; ++b) acc[a][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int steps = (P.count + 3) / 4;                     // a token past the chunk's last: the last again, with weight 0
    constexpr int U = 4;
    float kx[2][U][4], vx[2][U][4];
    auto ask = [&](int buf, int s0) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const long r = (long)min(4 * (s0 + u) + g, P.count - 1) * A.ld;
#pragma unroll
            for (int b = 0; b < 4; ++b) {
                kx[buf][u][b] = kp[b][r];
                vx[buf][u][b] = vp[b][r];
            }
        }
    };
    auto use = [&](int buf, int s0) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (s0 + u >= steps) break;
            const float wj = w[4 * (s0 + u) + g];
            float wk[4];
#pragma unroll
            for (int a = 0; a < 4; ++a) {
                wk[a] = wj * kx[buf][u][a];
                n_sum[a] += wk[a];
            }
#pragma unroll
            for (int a = 0; a < 4; ++a)
#pragma unroll
                for (int b = 0; b < 4; ++b) acc[a][b] = mfma_16x16x4(wk[a], vx[buf][u][b], acc[a][b]);
        }
    };
    ask(0, 0);
    for (int s0 = 0; s0 < steps; s0 += 2 * U) {
        ask(1, s0 + U);
        use(0, s0);
        ask(0, s0 + 2 * U);
        use(1, s0 + U);
    }
    float* out = C.part + nh_at * (dv + 1) * (long)dk;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
        const int e = e0 + 16 * b + c16;
        if (e >= dv) continue;
#pragma unroll
        for (int a = 0; a < 4; ++a) {
            const int d = d0 + 16 * a + 4 * g;
            float* dst = out + (long)e * dk + d;
            if (VEC) {
                if (d < dk) *reinterpret_cast<f32x4_t*>(dst) = acc[a][b];
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (d + r < dk) dst[r] = acc[a][b][r];
            }
        }
    }
    if (e0 == 0) {
#pragma unroll
        for (int a = 0; a < 4; ++a) {
            float x = n_sum[a];
            x += __shfl_xor(x, 16);
            x += __shfl_xor(x, 32);
            const int d = d0 + 16 * a + c16;
            if (g == 0 && d < dk) out[(long)dv * dk + d] = x;
        }
    }
}

// A thread has V neighbouring elements of the state of one (sequence, head) and goes through the sequence's chunks.
template <int V>
__global__ __launch_bounds__(256) void mlstm_carry_kernel(MlstmArgs A, ChunkArgs C) {
    constexpr int P = 4;                                     // chunks asked for ahead
    const int h = blockIdx.y, s = blockIdx.z, dk = A.dk, dv = A.dv;
    const long count = (long)(dv + 1) * dk, at = ((long)blockIdx.x * 256 + threadIdx.x) * V, sh = (long)A.slots[s] * A.nh + h;
    const int r0 = A.cu[s], chunks = (A.cu[s + 1] - r0 + CHUNK - 1) / CHUNK;
    const long first = chunk_of(A, s, 0).number;
    const bool writer = blockIdx.x == 0 && threadIdx.x == 0;
    const bool live = at < count;
    const long here = live ? at : 0;
    float* home = here < (long)dv * dk ? A.S + sh * dv * dk + here : A.n + sh * dk + (here - (long)dv * dk);
    float* part = C.part + (first * A.nh + h) * count + here;
    const long stride = (long)A.nh * count;
    float S[V], got[P][V];
    double F[P], top[P];
    auto load = [&](float* x, const float* p) {
        if (V == 4) *reinterpret_cast<f32x4_t*>(x) = *reinterpret_cast<const f32x4_t*>(p);
        else x[0] = p[0];
    };
    auto store = [&](float* p, const float* x) {
        if (!live) return;
        if (V == 4) *reinterpret_cast<f32x4_t*>(p) = *reinterpret_cast<const f32x4_t*>(x);
        else p[0] = x[0];
    };
    load(S, home);
    float m = A.m[sh];
    for (int c0 = 0; c0 < chunks; c0 += P) {
#pragma unroll
        for (int u = 0; u < P; ++u) {
            const int c = min(c0 + u, chunks - 1);
            load(got[u], part + c * stride);
            F[u] = C.F_all[(first + c) * A.nh + h];
            top[u] = C.top_all[(first + c) * A.nh + h];
        }
#pragma unroll
        for (int u = 0; u < P; ++u) {
            const int c = c0 + u;
            if (c >= chunks) break;
            store(part + c * stride, S);
            if (writer) C.m0[(first + c) * A.nh + h] = m;
            const double kept = F[u] + (double)m, made = F[u] + top[u];
            const float m1 = (float)fmax(kept, made);
            const float keep = exp_of_difference(kept, m1), write = exp_of_difference(made, m1);
#pragma unroll
            for (int e = 0; e < V; ++e) S[e] = fmaf(keep, S[e], write * got[u][e]);
            m = m1;
        }
    }
    store(home, S);
    if (writer) C.m_end[(long)s * A.nh + h] = m;             // (the state's own m is still read by the other workgroups)
}

// A workgroup of NW waves has TT tiles of 16 tokens of one chunk and head: the waves share out the keys of the scores, then the
// columns of the values (EB blocks of 16 each).
template <typename T, int TT, int EB, int NW, bool VEC>
__global__ __launch_bounds__(NW * 64) void mlstm_read_kernel(MlstmArgs A, ChunkArgs C, int chunks, T* __restrict__ out, long ldo) {
    constexpr int TILE = 16 * TT, PER = CHUNK / TILE;
    __shared__ __attribute__((aligned(16))) f32x4_t ps[TT][KEY_BLOCKS][64];      // weighted scores, as they are made and used
    __shared__ double a_s[CHUNK], b_s[TILE];
    __shared__ float from_start[TILE], floor_s[TILE], nq_s[TILE], row_part[NW][TILE], ss_part[NW][TILE];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, c16 = lane & 15, g = lane >> 4;
    const UnitPlace U = unit_of(blockIdx.x, PER, chunks, A.nh, A.n_seqs);
    if (U.s < 0) return;
    const int h = U.h, s = U.s, dk = A.dk, dv = A.dv;
    const ChunkPlace P = chunk_of(A, s, U.c);
    const int t0 = U.sub * TILE;                             // first token of the tile, in the chunk
    if (P.count <= t0) return;                               // (the whole workgroup)
    const long nh_at = P.number * A.nh + h, rows0 = P.first;
    const double m0 = (double)C.m0[nh_at];
    const float* start = C.part + nh_at * (dv + 1) * (long)dk;
    const int last = P.count - 1;
    for (int j = tid; j < CHUNK; j += NW * 64) a_s[j] = C.a[nh_at * CHUNK + j];
    if (tid < TILE) {
        const long at = nh_at * CHUNK + t0 + tid;            // (a place past the last token holds the last sums: finite)
        const double b = fmax(m0, C.top[at]);
        b_s[tid] = b;
        from_start[tid] = exp_of_difference(m0, b);
        floor_s[tid] = expf(-(float)(C.F[at] + b));
    }
    // n . q of the starting state: NW * 4 / TT threads a token, eight loads of each on their way at a time
    {
        constexpr int SH = NW * 4 / TT, AHEAD = 8;
        const int t = tid / SH, p = tid % SH;
        const float* qr = A.q + (rows0 + min(t0 + t, last)) * A.ld + (long)h * dk;
        const float* nr = start + (long)dv * dk;
        float x = 0.f;
        for (int d0 = 4 * p; d0 < dk; d0 += 4 * SH * AHEAD) {
            f32x4_t qx[AHEAD], nx[AHEAD];
#pragma unroll
            for (int u = 0; u < AHEAD; ++u) {
                qx[u] = four<VEC>(qr, d0 + 4 * SH * u, dk);
                nx[u] = four<VEC>(nr, d0 + 4 * SH * u, dk);
            }
#pragma unroll
            for (int u = 0; u < AHEAD; ++u)
#pragma unroll
                for (int e = 0; e < 4; ++e) x = fmaf(qx[u][e], nx[u][e], x);
        }
#pragma unroll
        for (int off = 1; off < SH; off *= 2) x += __shfl_xor(x, off);
        if (p == 0) nq_s[t] = x;
    }
    // the state behind the step's last token
    if (U.sub == 0 && tid == 0 && P.first + P.count == A.cu[s + 1])
        A.m[(long)A.slots[s] * A.nh + h] = C.m_end[(long)s * A.nh + h];
    __syncthreads();
    const float* qp[TT];
#pragma unroll
    for (int u = 0; u < TT; ++u) qp[u] = A.q + (rows0 + min(t0 + 16 * u + c16, last)) * A.ld + (long)h * dk;
    const int blocks = (min(t0 + TILE, P.count) + 15) / 16;  // blocks of 16 keys that the tile's tokens see
    const int steps = (dk + 15) / 16;                        // a lane takes elements 16 step + 4 g and its three neighbours
    // this wave's columns of the values are e0 + 16 b + c16 (a wave without columns reads the last one and stores nothing)
    const int e0 = wv * EB * 16;
    const float *sp[EB], *vp[EB];
#pragma unroll
    for (int b = 0; b < EB; ++b) {
        const int e = min(e0 + 16 * b + c16, dv - 1);
        sp[b] = start + (long)e * dk;
        vp[b] = A.v + rows0 * A.ld + (long)h * dv + e;
    }
    // two sets of operands take turns, so that one is on its way while the other is multiplied
    f32x4_t qf[2][TT], sf[2][EB];
    auto ask_state = [&](int buf, int step) {
        const int d = 16 * min(step, steps - 1) + 4 * g;
#pragma unroll
        for (int u = 0; u < TT; ++u) qf[buf][u] = four<VEC>(qp[u], d, dk);
#pragma unroll
        for (int b = 0; b < EB; ++b) sf[buf][b] = four<VEC>(sp[b], d, dk);
    };
    f32x4_t acc[TT][EB];
#pragma unroll
    for (int u = 0; u < TT; ++u)
#pragma unroll
        for (int b = 0; b < EB; ++b) acc[u][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    auto use_state = [&](int buf, int step) {
        if (step >= steps) return;
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int b = 0; b < EB; ++b)
#pragma unroll
                for (int u = 0; u < TT; ++u) acc[u][b] = mfma_16x16x4(qf[buf][u][r], sf[buf][b][r], acc[u][b]);
    };
    float vx[2][4][EB];
    auto ask_values = [&](int buf, int jb) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const long j = (long)min(16 * min(jb, blocks - 1) + 4 * g + r, last) * A.ld;
#pragma unroll
            for (int b = 0; b < EB; ++b) vx[buf][r][b] = vp[b][j];
        }
    };
    auto use_values = [&](int buf, int jb) {
        if (jb >= blocks) return;
        f32x4_t pf[TT];
#pragma unroll
        for (int u = 0; u < TT; ++u) pf[u] = ps[u][jb][lane];
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int b = 0; b < EB; ++b)
#pragma unroll
                for (int u = 0; u < TT; ++u) acc[u][b] = mfma_16x16x4(pf[u][r], vx[buf][r][b], acc[u][b]);
    };
    float row_sum[TT] = {};
    for (int jb = wv; jb < blocks; jb += NW) {
        const float* kr = A.k + (rows0 + min(16 * jb + c16, last)) * A.ld + (long)h * dk;
        f32x4_t sc[TT];
#pragma unroll
        for (int u = 0; u < TT; ++u) sc[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        constexpr int U4 = 4;
        f32x4_t kf[2][U4], qk[2][U4][TT];
        auto ask = [&](int buf, int s0) {
#pragma unroll
            for (int u = 0; u < U4; ++u) {
                const int d = 16 * min(s0 + u, steps - 1) + 4 * g;
                kf[buf][u] = four<VEC>(kr, d, dk);
#pragma unroll
                for (int x = 0; x < TT; ++x) qk[buf][u][x] = four<VEC>(qp[x], d, dk);
            }
        };
        auto use = [&](int buf, int s0) {
#pragma unroll
            for (int u = 0; u < U4; ++u) {
                if (s0 + u >= steps) break;
#pragma unroll
                for (int r = 0; r < 4; ++r)
#pragma unroll
                    for (int x = 0; x < TT; ++x) sc[x] = mfma_16x16x4(kf[buf][u][r], qk[buf][u][x][r], sc[x]);
            }
        };
        ask(0, 0);
        for (int s0 = 0; s0 < steps; s0 += 2 * U4) {
            ask(1, s0 + U4);
            use(0, s0);
            ask(0, s0 + 2 * U4);
            use(1, s0 + U4);
        }
        // the lane holds keys 16 jb + 4 g + r against token t0 + 16 u + c16
#pragma unroll
        for (int u = 0; u < TT; ++u) {
            const int t = t0 + 16 * u + c16;
            f32x4_t p;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int j = 16 * jb + 4 * g + r;
                p[r] = j <= t && j <= last ? sc[u][r] * A.q_scale * exp_of_difference(a_s[j], b_s[16 * u + c16]) : 0.f;
                row_sum[u] += p[r];
            }
            ps[u][jb][lane] = p;
        }
    }
    ask_state(0, 0);                                         // (on its way across the meeting of the waves)
#pragma unroll
    for (int u = 0; u < TT; ++u) {
        float x = row_sum[u];
        x += __shfl_xor(x, 16);
        x += __shfl_xor(x, 32);
        if (g == 0) row_part[wv][16 * u + c16] = x;
    }
    __syncthreads();
    for (int step = 0; step < steps; step += 2) {
        ask_state(1, step + 1);
        use_state(0, step);
        ask_state(0, step + 2);
        use_state(1, step + 1);
    }
    ask_values(0, 0);
    // the lane holds tokens 16 u + 4 g + r of the tile
#pragma unroll
    for (int u = 0; u < TT; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float x = A.q_scale * from_start[16 * u + 4 * g + r];
#pragma unroll
            for (int b = 0; b < EB; ++b) acc[u][b][r] *= x;
        }
    for (int jb = 0; jb < blocks; jb += 2) {
        ask_values(1, jb + 1);
        use_values(0, jb);
        ask_values(0, jb + 2);
        use_values(1, jb + 1);
    }
    // what the last step reads, asked for before the waves meet (without conditions, from inside the rows)
    float gt[TT][4][EB], wt[EB];
#pragma unroll
    for (int b = 0; b < EB; ++b) {
        const int e = min(e0 + 16 * b + c16, dv - 1);
        wt[b] = A.weight[(long)h * dv + e];
#pragma unroll
        for (int u = 0; u < TT; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) gt[u][r][b] = A.gate[(rows0 + min(t0 + 16 * u + 4 * g + r, last)) * A.ld + (long)h * dv + e];
    }
    // division and the norm's sum of squares
#pragma unroll
    for (int u = 0; u < TT; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = 16 * u + 4 * g + r;
            float nq = A.q_scale * from_start[t] * nq_s[t];
#pragma unroll
            for (int w = 0; w < NW; ++w) nq += row_part[w][t];
            const float inv_den = 1.0f / (fmaxf(fabsf(nq), floor_s[t]) + A.floor_eps);
            float ss = 0.f;
#pragma unroll
            for (int b = 0; b < EB; ++b) {
                acc[u][b][r] *= inv_den;
                if (e0 + 16 * b + c16 < dv) ss = fmaf(acc[u][b][r], acc[u][b][r], ss);
            }
            ss += dpp_get<0xB1, 0xF>(0.f, ss);
            ss += dpp_get<0x4E, 0xF>(0.f, ss);
            ss += dpp_get<0x141, 0xF>(0.f, ss);
            ss += dpp_get<0x140, 0xF>(0.f, ss);
            if (c16 == 0) ss_part[wv][t] = ss;
        }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < TT; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = 16 * u + 4 * g + r;
            if (t0 + t > last) continue;
            float ss = 0.f;
#pragma unroll
            for (int w = 0; w < NW; ++w) ss += ss_part[w][t];
            const float inv = 1.0f / sqrtf(ss / (float)dv + A.norm_eps);
            const long row = rows0 + t0 + t;
#pragma unroll
            for (int b = 0; b < EB; ++b) {
                const int e = e0 + 16 * b + c16;
                if (e >= dv) continue;
                st(out + row * ldo + (long)h * dv + e, acc[u][b][r] * inv * wt[b] * sigmoid_of(gt[u][r][b]));
            }
        }
}

// ------------------------------------------------------------------ host
static int check_mlstm(const MlstmArgs& A, const void* out, long ldo, int n_tokens, int dtype) {
    AGAVE_CHECK(n_tokens >= 0 && A.n_seqs >= 0 && A.nh > 0 && A.dk > 0 && A.dv > 0, "mlstm: bad sizes N=%d B=%d heads=%d dk=%d dv=%d", n_tokens, A.n_seqs, A.nh, A.dk, A.dv);
    AGAVE_CHECK(A.dk <= MAX_DK && A.dv <= MAX_DV, "mlstm: heads of %d key and %d value elements (at most %d and %d)", A.dk, A.dv, MAX_DK, MAX_DV);
    AGAVE_CHECK(A.q && A.k && A.v && A.gate && A.i_in && A.f_in && A.i_bias && A.f_bias && A.weight && A.S && A.n && A.m && A.cu && A.slots && out, "mlstm: null buffer");
    AGAVE_CHECK(A.ld >= (long)A.nh * A.dk && A.ld >= (long)A.nh * A.dv && ldo >= (long)A.nh * A.dv, "mlstm: a row stride is too small");
    AGAVE_CHECK(A.cap > 0.f, "mlstm: the gates' cap must be positive");
    AGAVE_CHECK(A.nh <= 65535 && A.n_seqs <= 65535, "mlstm: too many heads or sequences");
    AGAVE_CHECK(dtype == AGAVE_F32 || dtype == AGAVE_BF16, "mlstm: unknown dtype %d", dtype);
    return 0;
}
static bool by_fours(const MlstmArgs& A) {
    return A.dk % 4 == 0 && A.ld % 4 == 0 && ((uintptr_t)A.q % 16) == 0 && ((uintptr_t)A.k % 16) == 0 && ((uintptr_t)A.S % 16) == 0 && ((uintptr_t)A.n % 16) == 0;
}

template <int L, int V, int R, int UN>
static void launch_step(const MlstmArgs& A, float* num, float* nq, hipStream_t stream) {
    constexpr int COLS = 4 * (64 / L) * UN;
    mlstm_step_kernel<L, V, R, UN><<<dim3((A.dv + 1 + COLS - 1) / COLS, A.nh, A.n_seqs), 256, 0, stream>>>(A, num, nq);
}

// num: [n_seqs][nh * dv], nq: [n_seqs][nh], both 32-bit scratch
extern "C" int agave_mlstm_step(int dtype, const float* q, const float* k, const float* v, const float* gate, const float* i_in,
                                const float* f_in, long ld, const float* i_bias, const float* f_bias, const float* weight, float cap,
                                float floor_eps, float norm_eps, float q_scale, float* S, float* n, float* m, const int* cu,
                                const int* slots, int n_seqs, int nh, int dk, int dv, float* num, float* nq, void* out, long ldo,
                                hipStream_t stream) {
    const MlstmArgs A{q, k, v, gate, i_in, f_in, ld, i_bias, f_bias, weight, cap, floor_eps, norm_eps, q_scale, S, n, m, cu, slots, nh, dk, dv, n_seqs};
    if (check_mlstm(A, out, ldo, n_seqs, dtype)) return -1;
    AGAVE_CHECK(num && nq, "mlstm_step: null scratch");
    if (n_seqs == 0) return 0;
    if (by_fours(A)) {
        if (dk <= 32) launch_step<8, 4, 1, 4>(A, num, nq, stream);
        else if (dk <= 64) launch_step<16, 4, 1, 4>(A, num, nq, stream);
        else if (dk <= 128) launch_step<32, 4, 1, 4>(A, num, nq, stream);
        else if (dk <= 256) launch_step<64, 4, 1, 4>(A, num, nq, stream);
        else if (dk <= 512) launch_step<64, 4, 2, 4>(A, num, nq, stream);
        else launch_step<64, 4, 4, 2>(A, num, nq, stream);
    } else if (dk <= 64) {
        launch_step<64, 1, 1, 4>(A, num, nq, stream);
    } else if (dk <= 256) {
        launch_step<64, 1, 4, 4>(A, num, nq, stream);
    } else {
        launch_step<64, 1, 16, 1>(A, num, nq, stream);
    }
    AGAVE_LAUNCH_CHECK("mlstm_step");
    const int threads = dv <= 64 ? 64 : dv <= 128 ? 128 : 256;
    if (dtype == AGAVE_F32) mlstm_readout_kernel<float><<<dim3(n_seqs, nh), threads, 0, stream>>>(A, num, nq, (float*)out, ldo);
    else mlstm_readout_kernel<bf16><<<dim3(n_seqs, nh), threads, 0, stream>>>(A, num, nq, (bf16*)out, ldo);
    AGAVE_LAUNCH_CHECK("mlstm_readout");
    return 0;
}

extern "C" int agave_mlstm_chunk_size() { return CHUNK; }

// (two tiles of 16 tokens a workgroup read the chunk's starting state half as often; one tile where two would leave
// compute units idle)
template <typename T, int TT, bool VEC>
static void launch_read(const MlstmArgs& A, const ChunkArgs& C, T* out, long ldo, int chunks, hipStream_t stream) {
    const unsigned grid = (unsigned)unit_workgroups((long)chunks * A.nh * A.n_seqs, CHUNK / (16 * TT));
    if (A.dv <= 64) mlstm_read_kernel<T, TT, 1, 4, VEC><<<grid, 256, 0, stream>>>(A, C, chunks, out, ldo);
    else if (A.dv <= 128) mlstm_read_kernel<T, TT, 2, 4, VEC><<<grid, 256, 0, stream>>>(A, C, chunks, out, ldo);
    else if (A.dv <= 256) mlstm_read_kernel<T, TT, 4, 4, VEC><<<grid, 256, 0, stream>>>(A, C, chunks, out, ldo);
    else if (A.dv <= 512) mlstm_read_kernel<T, TT, 8, 4, VEC><<<grid, 256, 0, stream>>>(A, C, chunks, out, ldo);
    else mlstm_read_kernel<T, TT, 8, 8, VEC><<<grid, 512, 0, stream>>>(A, C, chunks, out, ldo);
}

template <typename T, bool VEC>
static void choose_read(const MlstmArgs& A, const ChunkArgs& C, T* out, long ldo, int chunks, hipStream_t stream) {
    if ((long)chunks * A.nh * A.n_seqs * (CHUNK / 32) < 256) launch_read<T, 1, VEC>(A, C, out, ldo, chunks, stream);
    else launch_read<T, 2, VEC>(A, C, out, ldo, chunks, stream);
}

// gates: double [3][numbers][nh][CHUNK]; totals: double [2][numbers][nh]; m0: float [numbers + n_seqs][nh];
// part: float [numbers][nh][dv + 1][dk]; numbers is at least n_tokens / CHUNK + n_seqs
extern "C" int agave_mlstm_chunks(int dtype, const float* q, const float* k, const float* v, const float* gate, const float* i_in,
                                  const float* f_in, long ld, const float* i_bias, const float* f_bias, const float* weight, float cap,
                                  float floor_eps, float norm_eps, float q_scale, float* S, float* n, float* m, const int* cu,
                                  const int* slots, int n_tokens, int n_seqs, int max_rows, int nh, int dk, int dv, double* gates,
                                  double* totals, float* m0, float* part, long numbers, void* out, long ldo, hipStream_t stream) {
    const MlstmArgs A{q, k, v, gate, i_in, f_in, ld, i_bias, f_bias, weight, cap, floor_eps, norm_eps, q_scale, S, n, m, cu, slots, nh, dk, dv, n_seqs};
    if (check_mlstm(A, out, ldo, n_tokens, dtype)) return -1;
    AGAVE_CHECK(gates && totals && m0 && part && numbers >= (long)n_tokens / CHUNK + n_seqs, "mlstm_chunks: scratch for %ld chunks", numbers);
    AGAVE_CHECK(max_rows >= 0 && max_rows <= n_tokens, "mlstm_chunks: a sequence of %d rows in a step of %d", max_rows, n_tokens);
    if (n_tokens == 0 || n_seqs == 0 || max_rows == 0) return 0;
    const int chunks = (max_rows + CHUNK - 1) / CHUNK;
    const long per = numbers * nh;
    const ChunkArgs C{gates, gates + per * CHUNK, gates + 2 * per * CHUNK, totals, totals + per, m0, m0 + per, part};
    const bool vec = by_fours(A) && ((uintptr_t)part % 16) == 0;
    mlstm_gates_kernel<<<dim3(chunks, nh, n_seqs), CHUNK, 0, stream>>>(A, C);
    AGAVE_LAUNCH_CHECK("mlstm_gates");
    const int tiles = ((dk + 63) / 64) * ((dv + 63) / 64);
    const int wgs = (tiles + 3) / 4;
    const long units = (long)chunks * nh * n_seqs;
    AGAVE_CHECK(unit_workgroups(units, wgs > CHUNK / 16 ? wgs : CHUNK / 16) < (1L << 31), "mlstm_chunks: too many chunks, heads and sequences");
    if (vec) mlstm_chunk_kernel<true><<<(unsigned)unit_workgroups(units, wgs), 256, 0, stream>>>(A, C, chunks, wgs);
    else mlstm_chunk_kernel<false><<<(unsigned)unit_workgroups(units, wgs), 256, 0, stream>>>(A, C, chunks, wgs);
    AGAVE_LAUNCH_CHECK("mlstm_chunk");
    const long count = (long)(dv + 1) * dk;
    if (vec) mlstm_carry_kernel<4><<<dim3((unsigned)((count / 4 + 255) / 256), nh, n_seqs), 256, 0, stream>>>(A, C);
    else mlstm_carry_kernel<1><<<dim3((unsigned)((count + 255) / 256), nh, n_seqs), 256, 0, stream>>>(A, C);
    AGAVE_LAUNCH_CHECK("mlstm_carry");
    if (dtype == AGAVE_F32) {
        if (vec) choose_read<float, true>(A, C, (float*)out, ldo, chunks, stream);
        else choose_read<float, false>(A, C, (float*)out, ldo, chunks, stream);
    } else {
        if (vec) choose_read<bf16, true>(A, C, (bf16*)out, ldo, chunks, stream);
        else choose_read<bf16, false>(A, C, (bf16*)out, ldo, chunks, stream);
    }
    AGAVE_LAUNCH_CHECK("mlstm_read");
    return 0;
}
