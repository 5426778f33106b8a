// Kernels of the attention whose keys and values come from one small latent row per position, for gfx950:
//
//   latent_prepare   what a token's first product left becomes what the later steps read: the query latent divided by
//                    its root mean square times a weight (where queries come from a latent), or the query rows
//                    themselves with their trailing elements rotated (where they do not); and the key/value latent,
//                    normed likewise, with its last elements, which are not normed, rotated by the position: the row
//                    [c | r], put into its place in the cache page on the way;
//   heads_product    a small product per (token, head): y[t][h] = W[h] x[t][h], for the step that folds a head's key
//                    matrix into its query (so that scores are taken against the cached rows themselves) and for the
//                    step that makes a head's values from the attention's sum over latent rows; it can copy a
//                    head's trailing elements behind the product while rotating them, and multiply the result by
//                    the sigmoid of a gate;
//   latent_decode_rows   a decode step's fold and key/value rows side by side in one launch (neither needs the other);
//   latent_fresh_pages   for a prompt that starts at its first position, where every head's own keys and values are made
//                    from the latent rows instead (fewer multiplications than the folded form when rows are many):
//                    keys [k | r] and values of a page of tokens into pages that live as long as the step;
//   latent_turn_queries  the queries' trailing elements rotated, rows to rows or in place;
//   gate_rows        rows times the sigmoid of 32-bit logits, in place.
//
// A rotation turns the first 2 * half of its elements, in pairs (e, e + half) or (2e, 2e + 1), and multiplies the turned
// pairs by a magnitude (1 where it is a pure rotation).  Angles are made in double
// (trig.h); sines, norm sums and the products' sums are 32-bit; T is the element type of the rows between products.
#include "common_impl.h"
#include "mfma.h"
#include "row_pages.h"
#include "trig.h"
#include <math.h>

#define MAX_TURNED 256           // pairs a rotation turns at most (their sines wait in LDS)

struct Turn { const double* freq; int half; int neighbours; float magnitude; };     // neighbours: pairs (2e, 2e + 1)

// the sines and cosines of position `pos`, by the threads that share cs (a barrier is the caller's)
__device__ __forceinline__ void turn_table(const Turn& R, int pos, float (*cs)[MAX_TURNED], int tid, int n_threads) {
    for (int i = tid; i < R.half; i += n_threads) {
        float s, c;
        sincos_of_angle((double)pos * R.freq[i], s, c);
        cs[0][i] = c * R.magnitude;
        cs[1][i] = s * R.magnitude;
    }
}
__device__ __forceinline__ int first_of_pair(const Turn& R, int i) { return R.neighbours ? 2 * i : i; }
__device__ __forceinline__ int second_of_pair(const Turn& R, int i) { return R.neighbours ? 2 * i + 1 : i + R.half; }

// element e of a row x of which the first 2 * half are turned
template <typename T>
__device__ __forceinline__ float turned_element(const Turn& R, const T* x, int e, const float (*cs)[MAX_TURNED]) {
    if (e >= 2 * R.half) return ld(x + e);
    const int i = R.neighbours ? e >> 1 : (e < R.half ? e : e - R.half);
    const bool second = R.neighbours ? (e & 1) : e >= R.half;
    const float u = ld(x + first_of_pair(R, i)), v = ld(x + second_of_pair(R, i)), c = cs[0][i], s = cs[1][i];
    return second ? v * c + u * s : u * c - v * s;
}

// ------------------------------------------------------------------ a token's rows
struct LatentKv {                 // the key/value side of a token (raw null: none)
    const float* raw; long ldraw; const float* weight;
    void* row; long ldrow;        // [c | r] in the activations' type (null: only into the page)
    int rank, rot_dim;
    void* k_pages; void* v_pages; const int* table; int width; const int* base; int n_pages; int packed;      // null: no page
    const int* tok_seq;
};
struct LatentQ {                  // the query side: a latent to be normed (heads 0), or query rows (heads > 0)
    const void* raw; long ldraw; const float* weight;
    void* out; long ldout;
    int rank;
    int heads, dim, rot_dim;
};

// One workgroup of 256 threads: the key/value row of token t
template <typename T>
__device__ __forceinline__ void latent_kv_row(const LatentKv& A, const Turn& R, int t, int pos, float eps, float* red,
                                              float (*cs)[MAX_TURNED]) {
    const int tid = threadIdx.x, rank = A.rank, kd = A.rank + A.rot_dim;
    const float* x = A.raw + (size_t)t * A.ldraw;
    turn_table(R, pos, cs, tid, 256);
    PagePlace at{-1, 0};
    if (A.k_pages) at = place_of(pos, A.tok_seq[t], A.table, A.width, A.base, 0, A.n_pages);
    float ss = 0.f;
    for (int e = tid; e < rank; e += 256) ss = fmaf(x[e], x[e], ss);
    ss = block_sum(ss, red);                                    // (its barriers complete the table too)
    const float inv = 1.0f / sqrtf(ss / (float)rank + eps);
    const int ksl = (kd + 31) / 32;
    T* kp = (T*)A.k_pages + (size_t)at.page * (A.packed ? (size_t)AGAVE_PAGE * ksl * 32 : (size_t)AGAVE_PAGE * kd);
    T* vp = (T*)A.v_pages + (size_t)at.page * rank * AGAVE_PAGE;
    for (int e = tid; e < kd; e += 256) {
        const float y = e < rank ? x[e] * inv * A.weight[e] : turned_element(R, x + rank, e - rank, cs);
        if (A.row) st((T*)A.row + (size_t)t * A.ldrow + e, y);
        if (at.page >= 0) {
            st(kp + (A.packed ? k_operand_at(at.row, e, ksl) : (size_t)at.row * kd + e), y);
            if (e < rank) st(vp + (A.packed ? v_operand_at(e, at.row) : (size_t)e * AGAVE_PAGE + at.row), y);
        }
    }
}

// One workgroup of 256 threads: the query rows of token t with their trailing elements turned
template <typename XT, typename T>
__device__ __forceinline__ void latent_q_rows(const LatentQ& A, const Turn& R, int t, int pos, float (*cs)[MAX_TURNED]) {
    const int tid = threadIdx.x, qd = A.dim + A.rot_dim;
    const XT* x = (const XT*)A.raw + (size_t)t * A.ldraw;
    T* y = (T*)A.out + (size_t)t * A.ldout;
    turn_table(R, pos, cs, tid, 256);
    __syncthreads();
    if ((const void*)x != (const void*)y) {                     // (in place only the pairs move)
        const int still = A.dim, tail0 = A.dim + 2 * R.half;
        for (int i = tid; i < A.heads * still; i += 256) {
            const int at = (i / still) * qd + i % still;
            st(y + at, ld(x + at));
        }
        const int rest = qd - tail0;
        for (int i = tid; i < A.heads * rest; i += 256) {
            const int at = (i / rest) * qd + tail0 + i % rest;
            st(y + at, ld(x + at));
        }
    }
    // (a thread takes a whole pair, so nothing is read after it was written)
    for (int i = tid; i < A.heads * R.half; i += 256) {
        const int e = i % R.half, h0 = (i / R.half) * qd + A.dim;
        const int p = h0 + first_of_pair(R, e), q = h0 + second_of_pair(R, e);
        const float u = ld(x + p), v = ld(x + q), c = cs[0][e], s = cs[1][e];
        st(y + p, u * c - v * s);
        st(y + q, v * c + u * s);
    }
}

// grid (tokens, sides): the query side first where there is one
template <typename T>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentQ Q, LatentKv K, Turn R, const int* __restrict__ tok_pos, float eps) {
    __shared__ float red[16];
    __shared__ float cs[2][MAX_TURNED];
    const int t = blockIdx.x, tid = threadIdx.x;
    if (Q.raw && blockIdx.y == 0) {
        if (Q.heads) {
            latent_q_rows<float, T>(Q, R, t, tok_pos[t], cs);
            return;
        }
        const float* x = (const float*)Q.raw + (size_t)t * Q.ldraw;
        float ss = 0.f;
        for (int e = tid; e < Q.rank; e += 256) ss = fmaf(x[e], x[e], ss);
        ss = block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)Q.rank + eps);
        for (int e = tid; e < Q.rank; e += 256) st((T*)Q.out + (size_t)t * Q.ldout + e, x[e] * inv * Q.weight[e]);
        return;
    }
    latent_kv_row<T>(K, R, t, tok_pos[t], eps, red, cs);
}

static int check_turn(const char* what, const Turn& R, int rot_dim) {
    AGAVE_CHECK(R.half >= 0 && R.half <= MAX_TURNED && 2 * R.half <= rot_dim && (R.freq || R.half == 0),
                "%s: %d rotated pairs in %d elements (at most %d, with their frequencies)", what, R.half, rot_dim, MAX_TURNED);
    return 0;
}

static int check_kv(const char* what, const LatentKv& K, int dtype) {
    AGAVE_CHECK(K.rank > 0 && K.rot_dim >= 0 && K.weight && K.ldraw >= K.rank + K.rot_dim, "%s: bad key/value sizes or buffers", what);
    AGAVE_CHECK(K.row ? K.ldrow >= K.rank + K.rot_dim : K.k_pages != nullptr, "%s: no place for the key/value row", what);
    AGAVE_CHECK(!K.k_pages || (K.v_pages && K.table && K.base && K.tok_seq && K.width > 0 && K.n_pages > 0), "%s: cache pages without their table", what);
    AGAVE_CHECK(!K.packed || (dtype == AGAVE_BF16 && (K.rank + K.rot_dim) % 8 == 0 && K.rank % 16 == 0), "%s: pages in operand order hold bfloat16, rows in steps of 8 and values in steps of 16", what);
    return 0;
}

// q_heads 0: qraw is a query latent of q_rank; > 0: query rows of q_heads x (q_dim + rot_dim)
extern "C" int agave_latent_prepare(int dtype, const float* qraw, long ldq, const float* qw, void* qout, long ldqo, int q_rank,
                                    int q_heads, int q_dim, const float* kvraw, long ldkv, const float* kvw, void* krow, long ldkr,
                                    int kv_rank, int rot_dim, const double* freq, int half, int neighbours, float magnitude, void* k_pages,
                                    void* v_pages, const int* table, int width, const int* base, int n_pages, int packed,
                                    const int* tok_seq, const int* tok_pos, int n_tokens, float eps, hipStream_t stream) {
    AGAVE_CHECK(n_tokens >= 0 && (qraw || kvraw) && tok_pos, "latent_prepare: bad sizes N=%d or nothing to prepare", n_tokens);
    const Turn R{freq, half, neighbours, magnitude};
    if (check_turn("latent_prepare", R, rot_dim)) return -1;
    const LatentQ Q{qraw, ldq, qw, qout, ldqo, q_rank, q_heads, q_dim, rot_dim};
    if (qraw) {
        const long cols = q_heads ? (long)q_heads * (q_dim + rot_dim) : q_rank;
        AGAVE_CHECK(cols > 0 && qout && (q_heads ? q_dim >= 0 : qw != nullptr) && ldq >= cols && ldqo >= cols, "latent_prepare: bad query buffers");
    }
    const LatentKv K{kvraw, ldkv, kvw, krow, ldkr, kv_rank, rot_dim, k_pages, v_pages, table, width, base, n_pages, packed, tok_seq};
    if (kvraw && check_kv("latent_prepare", K, dtype)) return -1;
    if (n_tokens == 0) return 0;
    const dim3 grid(n_tokens, (qraw ? 1 : 0) + (kvraw ? 1 : 0));
    if (dtype == AGAVE_F32) latent_prepare_kernel<float><<<grid, 256, 0, stream>>>(Q, K, R, tok_pos, eps);
    else if (dtype == AGAVE_BF16) latent_prepare_kernel<bf16><<<grid, 256, 0, stream>>>(Q, K, R, tok_pos, eps);
    else AGAVE_CHECK(false, "latent_prepare: unknown dtype %d", dtype);
    AGAVE_LAUNCH_CHECK("latent_prepare");
    return 0;
}

template <typename T>
__global__ __launch_bounds__(256) void latent_turn_queries_kernel(LatentQ Q, Turn R, const int* __restrict__ tok_pos) {
    __shared__ float cs[2][MAX_TURNED];
    latent_q_rows<T, T>(Q, R, blockIdx.x, tok_pos[blockIdx.x], cs);
}

// rows of the activations' type; q_out may be q (in place)
extern "C" int agave_latent_turn_queries(int dtype, const void* q, long ldq, void* q_out, long ldqo, int heads, int dim, int rot_dim,
                                         const double* freq, int half, int neighbours, float magnitude, const int* tok_pos, int n_tokens, hipStream_t stream) {
    AGAVE_CHECK(n_tokens >= 0 && heads > 0 && dim >= 0 && rot_dim >= 0 && dim + rot_dim > 0 && q && q_out && tok_pos, "latent_turn_queries: bad sizes or buffers");
    AGAVE_CHECK(ldq >= (long)heads * (dim + rot_dim) && ldqo >= (long)heads * (dim + rot_dim) && (q != q_out || ldq == ldqo), "latent_turn_queries: bad row strides");
    const Turn R{freq, half, neighbours, magnitude};
    if (check_turn("latent_turn_queries", R, rot_dim)) return -1;
    if (n_tokens == 0) return 0;
    const LatentQ Q{q, ldq, nullptr, q_out, ldqo, 0, heads, dim, rot_dim};
    if (dtype == AGAVE_F32) latent_turn_queries_kernel<float><<<n_tokens, 256, 0, stream>>>(Q, R, tok_pos);
    else if (dtype == AGAVE_BF16) latent_turn_queries_kernel<bf16><<<n_tokens, 256, 0, stream>>>(Q, R, tok_pos);
    else AGAVE_CHECK(false, "latent_turn_queries: unknown dtype %d", dtype);
    AGAVE_LAUNCH_CHECK("latent_turn_queries");
    return 0;
}

// ------------------------------------------------------------------ a product per (token, head)
//   y[t][h][c] = sum_k W[h][c][k] x[t][h * xs + k]        (c < n_out, k < K;  W is [heads][n_out][K])
//   y[t][h][n_out + e] = the head's elements x[t][h * xs + K + e], e < tail, the first 2 * half of them turned
//   y[t][h][c] *= sigmoid(gate[t][h * n_out + c])          (where a gate is given; it is 32-bit)
// y's head h starts at column h * ys.  x's rows are of y's type or 32-bit.
struct HeadsProductArgs {
    const void* x; long ldx; int xs;
    const void* w;
    void* y; long ldy; int ys;
    const float* gate; long ldg;
    Turn turn; int tail;
    const int* tok_pos;
    int n_tokens, heads, n_out, K;
};

// The plain form: a workgroup per (token, head), the head's input in LDS, a wave per output column in turn with
// the lanes along K.  Any sizes, both element types.
template <typename XT, typename T>
__global__ __launch_bounds__(256) void heads_product_plain_kernel(HeadsProductArgs A) {
    extern __shared__ float xh[];                       // [K + tail]
    __shared__ float cs[2][MAX_TURNED];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const XT* x = (const XT*)A.x + (size_t)t * A.ldx + (size_t)h * A.xs;
    for (int k = tid; k < A.K + A.tail; k += 256) xh[k] = ld(x + k);
    if (A.tail) turn_table(A.turn, A.tok_pos[t], cs, tid, 256);
    __syncthreads();
    T* y = (T*)A.y + (size_t)t * A.ldy + (size_t)h * A.ys;
    const T* w = (const T*)A.w + (size_t)h * A.n_out * A.K;
    for (int c = wv; c < A.n_out; c += 4) {
        const T* wr = w + (size_t)c * A.K;
        float acc = 0.f;
        for (int k = lane; k < A.K; k += 64) acc = fmaf(ld(wr + k), xh[k], acc);
        acc = wave_sum(acc);
        if (lane == 0) {
            if (A.gate) acc *= 1.0f / (1.0f + expf(-A.gate[(size_t)t * A.ldg + (size_t)h * A.n_out + c]));
            st(y + c, acc);
        }
    }
    for (int e = tid; e < A.tail; e += 256) st(y + A.n_out + e, turned_element(A.turn, xh + A.K, e, cs));
}

__device__ __forceinline__ frag16 eight(const bf16* p) {
    frag16 f;
    f.u = *reinterpret_cast<const uint4*>(p);
    return f;
}
__device__ __forceinline__ frag16 eight(const float* p) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    frag16 f;
    f.u = make_uint4(f32x2_to_bf16x2(a.x, a.y), f32x2_to_bf16x2(a.z, a.w), f32x2_to_bf16x2(b.x, b.y), f32x2_to_bf16x2(b.z, b.w));
    return f;
}

// The matrix cores' form (bfloat16; K a multiple of 8, aligned rows): a workgroup takes 64 tokens of one head and 64
// output columns (or, in a step of up to 16 tokens, those tokens and 256 columns); each of its four waves 16 tokens
// against 64 columns, both operands straight from memory in the order v_mfma_f32_16x16x32_bf16 reads them (a lane's
// eight neighbours along K are 16 bytes of a row; a 32-bit row is rounded on the way in).  The head's weights are small
// and stay in the caches; what the kernel moves is the rows.  The trailing elements are copied, turned, by the
// workgroups of the first column block, a thread a pair.
template <typename XT>
__device__ __forceinline__ void heads_product_tile(const HeadsProductArgs& A, int bx, int h, int bz) {
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
    const int c = lane & 15, g = lane >> 4;
    // up to 16 tokens (a decode step): the four waves take four blocks of columns of the same 16 rows
    const bool few = A.n_tokens <= 16;
    const int wg_row0 = few ? 0 : bx * 64, wg_rows = few ? 16 : 64;
    const int row0 = few ? 0 : wg_row0 + wv * 16;
    const int col0 = few ? (bz * 4 + wv) * 64 : bz * 64;
    const int K = A.K, n_out = A.n_out;
    const XT* x = (const XT*)A.x;
    const bf16* w = (const bf16*)A.w + (size_t)h * n_out * K;
    bf16* y = (bf16*)A.y;
    if (col0 < n_out && row0 < A.n_tokens) {
        int trow = row0 + c;
        trow = trow < A.n_tokens ? trow : A.n_tokens - 1;
        const XT* arow = x + (size_t)trow * A.ldx + (size_t)h * A.xs + 8 * g;
        const bf16* brow[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            int col = col0 + 16 * j + c;
            col = col < n_out ? col : n_out - 1;
            brow[j] = w + (size_t)col * K + 8 * g;
        }
        f32x4_t acc[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        // four steps along K at a time: their loads leave together (without conditions, from inside the row; a lane past the
        // row's end reads its start and is emptied), so a product is a few round trips to memory and not one per step
        for (int k0 = 0; k0 < K; k0 += 128) {
            frag16 a[4], b[4][4];
            bool in[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                in[u] = k0 + 32 * u + 8 * g < K;
                const int at = in[u] ? k0 + 32 * u : -8 * g;
#pragma unroll
                for (int j = 0; j < 4; ++j) b[u][j].u = *reinterpret_cast<const uint4*>(brow[j] + at);
                a[u] = eight(arow + at);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                if (!in[u]) a[u].u = make_uint4(0, 0, 0, 0);
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[j] = mfma_16x16x32(a[u], b[u][j], acc[j]);
            }
        }
        // D[j]: the lane holds tokens row0 + 4 g + e4, column col0 + 16 j + c
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int col = col0 + 16 * j + c;
            if (col >= n_out) continue;
#pragma unroll
            for (int e4 = 0; e4 < 4; ++e4) {
                const int t = row0 + 4 * g + e4;
                if (t >= A.n_tokens) continue;
                float v = acc[j][e4];
                if (A.gate) v *= 1.0f / (1.0f + expf(-A.gate[(size_t)t * A.ldg + (size_t)h * n_out + col]));
                y[(size_t)t * A.ldy + (size_t)h * A.ys + col] = f32_to_bf16(v);
            }
        }
    }
    if (A.tail && bz == 0) {
        const Turn R = A.turn;
        const int rows = min(wg_rows, A.n_tokens - wg_row0), rest = A.tail - 2 * R.half;
        for (int i = threadIdx.x; i < rows * R.half; i += 256) {
            const int t = wg_row0 + i / R.half, e = i % R.half;
            const XT* r = x + (size_t)t * A.ldx + (size_t)h * A.xs + K;
            bf16* o = y + (size_t)t * A.ldy + (size_t)h * A.ys + n_out;
            const int p = first_of_pair(R, e), q = second_of_pair(R, e);
            const float u = ld(r + p), v = ld(r + q);
            float sn, cn;
            sincos_of_angle((double)A.tok_pos[t] * R.freq[e], sn, cn);
            sn *= R.magnitude;
            cn *= R.magnitude;
            o[p] = f32_to_bf16(u * cn - v * sn);
            o[q] = f32_to_bf16(v * cn + u * sn);
        }
        for (int i = threadIdx.x; i < rows * rest; i += 256) {
            const int t = wg_row0 + i / rest, e = 2 * R.half + i % rest;
            y[(size_t)t * A.ldy + (size_t)h * A.ys + n_out + e] = f32_to_bf16(ld(x + (size_t)t * A.ldx + (size_t)h * A.xs + K + e));
        }
    }
}

template <typename XT>
__global__ __launch_bounds__(256) void heads_product_mfma_kernel(HeadsProductArgs A) {
    heads_product_tile<XT>(A, blockIdx.x, blockIdx.y, blockIdx.z);
}

// A decode step of up to 16 tokens: grid (1, heads + tokens, column blocks).  The first `heads` rows of workgroups fold
// the queries, the others (first column block) make the tokens' key/value rows.
template <typename XT>
__global__ __launch_bounds__(256) void latent_decode_rows_kernel(HeadsProductArgs A, LatentKv K, Turn R, float eps) {
    __shared__ float red[16];
    __shared__ float cs[2][MAX_TURNED];
    if ((int)blockIdx.y < A.heads) {
        heads_product_tile<XT>(A, 0, blockIdx.y, blockIdx.z);
    } else if (blockIdx.z == 0) {
        const int t = blockIdx.y - A.heads;
        latent_kv_row<bf16>(K, R, t, A.tok_pos[t], eps, red, cs);
    }
}

static int check_heads_product(const HeadsProductArgs& A) {
    AGAVE_CHECK(A.n_tokens >= 0 && A.heads > 0 && A.n_out > 0 && A.K > 0 && A.tail >= 0, "heads_product: bad sizes N=%d heads=%d out=%d K=%d", A.n_tokens, A.heads, A.n_out, A.K);
    AGAVE_CHECK(A.x && A.w && A.y, "heads_product: null buffer");
    AGAVE_CHECK(A.xs >= A.K + A.tail && A.ldx >= (long)(A.heads - 1) * A.xs + A.K + A.tail, "heads_product: the input's rows are too short");
    AGAVE_CHECK(A.ys >= A.n_out + A.tail && A.ldy >= (long)(A.heads - 1) * A.ys + A.n_out + A.tail, "heads_product: the output's rows are too short");
    AGAVE_CHECK(!A.gate || A.ldg >= (long)A.heads * A.n_out, "heads_product: the gate's rows are too short");
    AGAVE_CHECK(A.tail == 0 || A.tok_pos, "heads_product: trailing elements need the tokens' positions");
    if (check_turn("heads_product", A.turn, A.tail)) return -1;
    AGAVE_CHECK(A.heads <= 65535 && (A.K + A.tail) * sizeof(float) <= 60 * 1024, "heads_product: too many heads or too long a head");
    return 0;
}

static bool heads_product_on_matrix_cores(int dtype, int x_f32, const HeadsProductArgs& A) {
    const int step = x_f32 ? 4 : 8;                     // elements of x in 16 bytes
    return dtype == AGAVE_BF16 && A.K % 8 == 0 && A.xs % step == 0 && A.ldx % step == 0 && ((uintptr_t)A.x % 16) == 0 && ((uintptr_t)A.w % 16) == 0;
}

extern "C" int agave_heads_product(int dtype, int x_f32, const void* x, long ldx, int xs, const void* w, void* y, long ldy, int ys,
                                   const float* gate, long ldg, const double* freq, int half, int neighbours, float magnitude, int tail,
                                   const int* tok_pos, int n_tokens, int heads, int n_out, int K, int plain, hipStream_t stream) {
    HeadsProductArgs A{x, ldx, xs, w, y, ldy, ys, gate, ldg, Turn{freq, half, neighbours, magnitude}, tail, tok_pos, n_tokens, heads, n_out, K};
    if (check_heads_product(A)) return -1;
    if (n_tokens == 0) return 0;
    if (!plain && heads_product_on_matrix_cores(dtype, x_f32, A)) {
        const dim3 grid = n_tokens <= 16 ? dim3(1, heads, (n_out + 255) / 256) : dim3((n_tokens + 63) / 64, heads, (n_out + 63) / 64);
        AGAVE_CHECK(grid.z <= 65535, "heads_product: too many columns");
        if (x_f32) heads_product_mfma_kernel<float><<<grid, 256, 0, stream>>>(A);
        else heads_product_mfma_kernel<bf16><<<grid, 256, 0, stream>>>(A);
    } else {
        const dim3 grid(n_tokens, heads);
        const size_t lds = (size_t)(K + tail) * sizeof(float);
        if (dtype == AGAVE_F32) heads_product_plain_kernel<float, float><<<grid, 256, lds, stream>>>(A);
        else if (dtype == AGAVE_BF16 && x_f32) heads_product_plain_kernel<float, bf16><<<grid, 256, lds, stream>>>(A);
        else if (dtype == AGAVE_BF16) heads_product_plain_kernel<bf16, bf16><<<grid, 256, lds, stream>>>(A);
        else AGAVE_CHECK(false, "heads_product: unknown dtype %d", dtype);
    }
    AGAVE_LAUNCH_CHECK("heads_product");
    return 0;
}

// 1 if a decode step of these sizes may use agave_latent_decode_rows (q: 32-bit rows)
extern "C" int agave_latent_decode_rows_ok(int n_tokens, int dim, int rot_dim, int ldq) {
    return n_tokens >= 1 && n_tokens <= 16 && dim > 0 && dim % 8 == 0 && (dim + rot_dim) % 4 == 0 && ldq % 4 == 0;
}

// A bfloat16 decode step of up to 16 tokens: folded[t][h] = [fold[h] q[t][h][: dim] | q's trailing elements turned], and the
// key/value rows into their pages.  q and kvraw are 32-bit rows of the first product.
extern "C" int agave_latent_decode_rows(const float* q, long ldq, const void* fold, void* folded, long ldf, int heads, int dim,
                                        const float* kvraw, long ldkv, const float* kvw, void* krow, long ldkr, int kv_rank, int rot_dim,
                                        const double* freq, int half, int neighbours, float magnitude, void* k_pages, void* v_pages, const int* table,
                                        int width, const int* base, int n_pages, int packed, const int* tok_seq, const int* tok_pos,
                                        int n_tokens, float eps, hipStream_t stream) {
    const Turn R{freq, half, neighbours, magnitude};
    HeadsProductArgs A{q, ldq, dim + rot_dim, fold, folded, ldf, kv_rank + rot_dim, nullptr, 0, R, rot_dim, tok_pos, n_tokens, heads, kv_rank, dim};
    const LatentKv K{kvraw, ldkv, kvw, krow, ldkr, kv_rank, rot_dim, k_pages, v_pages, table, width, base, n_pages, packed, tok_seq};
    if (check_heads_product(A) || check_turn("latent_decode_rows", R, rot_dim) || check_kv("latent_decode_rows", K, AGAVE_BF16)) return -1;
    AGAVE_CHECK(agave_latent_decode_rows_ok(n_tokens, dim, rot_dim, (int)(ldq % 4)) && heads_product_on_matrix_cores(AGAVE_BF16, 1, A) && kvraw && tok_pos,
                "latent_decode_rows: sizes or alignment that it does not take");
    const dim3 grid(1, heads + n_tokens, (kv_rank + 255) / 256);
    AGAVE_CHECK(grid.y <= 65535, "latent_decode_rows: too many heads");
    latent_decode_rows_kernel<float><<<grid, 256, 0, stream>>>(A, K, R, eps);
    AGAVE_LAUNCH_CHECK("latent_decode_rows");
    return 0;
}

// ------------------------------------------------------------------ every head's keys and values, a page of tokens at a time
// Keys [up_k[t][h] (dim) | krow[t][kv_rank ..] (rot_dim, turned already)] and values up_v[t][h] (vd) of the tokens of page i of
// sequence b, in operand order; places past the sequence's end are written as zeros, so a page needs no clearing.
// A workgroup per (page, sequence, head); a wave takes a key block, all waves the values through LDS (which turns them).
struct FreshArgs {
    const bf16* up; long ldu; int v_off;        // [tokens][heads * dim | ... at v_off: heads * vd]
    const bf16* krow; long ldkr; int kv_rank;
    bf16* k_pages; bf16* v_pages; const int* table; int width; int n_pages;
    const int* cu;
    int heads, dim, rot_dim, vd;
};
__global__ __launch_bounds__(256) void latent_fresh_pages_kernel(FreshArgs A) {
    extern __shared__ bf16 vt[];                // [64 tokens][vd + 2]
    const int i = blockIdx.x, b = blockIdx.y, h = blockIdx.z, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int c = lane & 15, g = lane >> 4;
    const int t0 = A.cu[b] + i * AGAVE_PAGE, n = min(AGAVE_PAGE, A.cu[b + 1] - t0);
    if (n <= 0 || i >= A.width) return;         // (the whole workgroup)
    const long pg = A.table[(size_t)b * A.width + i];
    if (pg < 0 || pg >= A.n_pages) return;
    const int qd = A.dim + A.rot_dim, ksl = (qd + 31) / 32, vd = A.vd, vs = vd + 2;
    const uint4 zero = make_uint4(0, 0, 0, 0);
    // values into LDS, 16 bytes a thread
    const int vp = vd / 8;
    for (int x = threadIdx.x; x < AGAVE_PAGE * vp; x += 256) {
        const int r = x / vp, d = (x % vp) * 8;
        const uint4 got = *reinterpret_cast<const uint4*>(A.up + (size_t)(t0 + (r < n ? r : 0)) * A.ldu + A.v_off + (size_t)h * vd + d);
        const uint4 v = r < n ? got : zero;
        uint32_t* dst = reinterpret_cast<uint32_t*>(vt + r * vs + d);
        dst[0] = v.x;
        dst[1] = v.y;
        dst[2] = v.z;
        dst[3] = v.w;
    }
    // keys: operand (w, ks) of the page
    {
        const int r = key_of(w, c), t = t0 + (r < n ? r : 0);
        const bf16* kn = A.up + (size_t)t * A.ldu + (size_t)h * A.dim;
        const bf16* kr = A.krow + (size_t)t * A.ldkr + A.kv_rank;
        uint4* dst = reinterpret_cast<uint4*>(A.k_pages) + ((size_t)pg * A.heads + h) * 4 * ksl * 64 + (size_t)w * ksl * 64 + lane;
        for (int ks = 0; ks < ksl; ++ks) {
            const int e = 32 * ks + 8 * g;
            const bf16* src = e < A.dim ? kn + e : kr + (e < qd ? e - A.dim : 0);
            const uint4 got = e < qd ? *reinterpret_cast<const uint4*>(src) : zero;
            dst[(size_t)ks * 64] = r < n ? got : zero;
        }
    }
    __syncthreads();
    uint4* vdst = reinterpret_cast<uint4*>(A.v_pages) + ((size_t)pg * A.heads + h) * (vd / 16) * 2 * 64;
    for (int tile = w; tile < (vd / 16) * 2; tile += 4) {
        const int d = (tile >> 1) * 16 + c, r0 = (tile & 1) * 32 + 8 * g;
        frag16 f;
#pragma unroll
        for (int j = 0; j < 8; ++j) f.h[j] = vt[(r0 + j) * vs + d];
        vdst[(size_t)tile * 64 + lane] = f.u;
    }
}

extern "C" int agave_latent_fresh_pages(const void* up, long ldu, int v_off, const void* krow, long ldkr, int kv_rank, void* k_pages,
                                        void* v_pages, const int* table, int width, int n_pages, const int* cu, int n_seqs, int max_rows,
                                        int heads, int dim, int rot_dim, int vd, hipStream_t stream) {
    AGAVE_CHECK(n_seqs > 0 && max_rows > 0 && heads > 0 && dim > 0 && rot_dim >= 0 && vd > 0 && kv_rank > 0 && width > 0 && n_pages > 0, "latent_fresh_pages: bad sizes");
    AGAVE_CHECK(up && krow && k_pages && v_pages && table && cu, "latent_fresh_pages: null buffer");
    AGAVE_CHECK(dim % 8 == 0 && rot_dim % 8 == 0 && vd % 16 == 0 && kv_rank % 8 == 0 && ldu % 8 == 0 && ldkr % 8 == 0 && v_off % 8 == 0 &&
                ((uintptr_t)up % 16) == 0 && ((uintptr_t)krow % 16) == 0, "latent_fresh_pages: heads in steps of 8 and values of 16, rows aligned to 16 bytes");
    AGAVE_CHECK(v_off >= heads * dim && ldu >= (long)v_off + (long)heads * vd && ldkr >= kv_rank + rot_dim, "latent_fresh_pages: a row stride is too small");
    const size_t lds = (size_t)AGAVE_PAGE * (vd + 2) * sizeof(bf16);
    AGAVE_CHECK(lds <= 64 * 1024 && n_seqs <= 65535 && heads <= 65535, "latent_fresh_pages: values of %d or too many heads or sequences", vd);
    FreshArgs A{(const bf16*)up, ldu, v_off, (const bf16*)krow, ldkr, kv_rank, (bf16*)k_pages, (bf16*)v_pages, table, width, n_pages, cu, heads, dim, rot_dim, vd};
    latent_fresh_pages_kernel<<<dim3((max_rows + AGAVE_PAGE - 1) / AGAVE_PAGE, n_seqs, heads), 256, lds, stream>>>(A);
    AGAVE_LAUNCH_CHECK("latent_fresh_pages");
    return 0;
}

// ------------------------------------------------------------------ x *= sigmoid(gate), gate in 32-bit
template <typename T>
__global__ void gate_rows_kernel(T* __restrict__ x, long ldx, const float* __restrict__ gate, long ldg, long total, int cols) {
    for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total; idx += (long)gridDim.x * blockDim.x) {
        const long r = idx / cols;
        const int c = (int)(idx % cols);
        T* at = x + r * ldx + c;
        st(at, ld(at) * (1.0f / (1.0f + expf(-gate[r * ldg + c]))));
    }
}

extern "C" int agave_gate_rows(int dtype, void* x, long ldx, const float* gate, long ldg, int rows, int cols, hipStream_t stream) {
    AGAVE_CHECK(rows >= 0 && cols > 0 && ldx >= cols && ldg >= cols && x && gate, "gate_rows: bad sizes rows=%d cols=%d", rows, cols);
    if (rows == 0) return 0;
    const long total = (long)rows * cols;
    long blocks = (total + 255) / 256;
    if (blocks > 65536) blocks = 65536;
    if (dtype == AGAVE_F32) gate_rows_kernel<float><<<(int)blocks, 256, 0, stream>>>((float*)x, ldx, gate, ldg, total, cols);
    else if (dtype == AGAVE_BF16) gate_rows_kernel<bf16><<<(int)blocks, 256, 0, stream>>>((bf16*)x, ldx, gate, ldg, total, cols);
    else AGAVE_CHECK(false, "gate_rows: unknown dtype %d", dtype);
    AGAVE_LAUNCH_CHECK("gate_rows");
    return 0;
}
