// The gated delta rule with a decay per key channel.  Per head, with state S [N, P] (N the key size, P the value size):
//
//   S <- diag(g_t) S;   u = beta_t (v_t - S^T k_t);   S <- S + k_t u^T;   o_t = S^T q_t
//
// q and k come from fewer heads than there are states (head h reads q/k head h / (heads / kv_heads)).  Everything here is
// 32-bit whatever the compute type; a sequence's state is a row of a state table per slot.
//
// pta_delta_prep makes what the recurrence reads: q, k and v through a short causal convolution per channel and silu, q and
// k to unit length per head (q times a constant), g = exp(-exp(A_log) softplus(a + dt_bias)), beta = sigmoid(b).
//
// pta_delta_scan runs the recurrence.  A workgroup of four waves owns (sequence, head, 64 * CPL columns p of the state) and
// a run of tokens; a wave owns 16 * CPL columns, and its four groups of sixteen lanes hold NPT consecutive rows n each in
// registers; sums over rows end with two exchanges between the groups.  A piece of the run's g, k, q, v and beta is staged
// in LDS by the whole workgroup, then walked in order.  Columns never meet, so a workgroup may take any of them.
//
// Short steps are one launch from each sequence's state to its state (DELTA_WHOLE).  A long prompt is cut into chunks that
// run side by side.  The recurrence is affine in the state: over chunk c, S_out = A_c S_in + B_c, with B_c the result from a
// zero state and A_c (N x N) that of the unit matrix with values of zero, so:
//   DELTA_LOCAL   every chunk from [0 | I]: columns 0 .. P - 1 leave B_c, columns P .. P + N - 1 leave A_c;
//   delta_carry   chunk after chunk, S_in(c + 1) = A_c S_in(c) + B_c, from the sequence's state to its state (32-bit matrix
//                 products; A_c is a product of contractions, so nothing grows);
//   DELTA_OUTPUT  every chunk again from its S_in, with the outputs.
#include "common.h"
#include "pta_kernels.h"

#define DELTA_PIECE 16
#define DELTA_MAX_TAPS 16
enum { DELTA_WHOLE = 0, DELTA_LOCAL = 1, DELTA_OUTPUT = 2 };

__device__ __forceinline__ float softplus_32(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// One wave per (token, unit): units are the q heads, the k heads, the value heads and the heads' decays (with beta).
template <typename T>
__global__ __launch_bounds__(64) void delta_prep_kernel(
    float* __restrict__ qkv, float* __restrict__ g, float* __restrict__ beta, const T* __restrict__ q, const T* __restrict__ k,
    const T* __restrict__ v, long ld, const float* __restrict__ conv, const T* __restrict__ a, long a_ld,
    const T* __restrict__ b, long b_ld, const float* __restrict__ A_log, const float* __restrict__ dt_bias,
    float* __restrict__ tail, long tail_ld, const int* __restrict__ cu_tokens, const int* __restrict__ token_seq,
    const int* __restrict__ seq_slot, int move_tail, int heads, int G, int N, int P, int K, float q_scale, float norm_eps) {
    const int m = blockIdx.x, unit = blockIdx.y, lane = threadIdx.x;
    if (unit >= 2 * G + heads) {  // a head's decays and step size
        const int h = unit - 2 * G - heads;
        const float rate = expf(A_log[h]);
        for (int e = lane; e < N; e += PTA_WAVE) {
            const int at = h * N + e;
            g[(long)m * heads * N + at] = expf(-rate * softplus_32(Io<T>::ld(a + (long)m * a_ld + at) + dt_bias[at]));
        }
        if (lane == 0) beta[(long)m * heads + h] = 1.0f / (1.0f + expf(-Io<T>::ld(b + (long)m * b_ld + h)));
        return;
    }
    const bool is_v = unit >= 2 * G, is_q = unit < G;
    const int len = is_v ? P : N, local = is_v ? unit - 2 * G : is_q ? unit : unit - G;  // the head within its tensor
    const T* src = (is_v ? v : is_q ? q : k) + (long)local * len;
    const int c0 = is_v ? 2 * G * N + local * P : unit * N;  // first channel of the head in q | k | v
    const int C = 2 * G * N + heads * P;
    const int s = token_seq[m], first = cu_tokens[s], j = m - first;
    float* tl = tail + (K > 1 ? (long)seq_slot[s] * tail_ld : 0L);
    float y[4], ss = 0.f;
    for (int e0 = 0; e0 < len; e0 += 4 * PTA_WAVE) {  // (heads of q and k fit one round)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int e = e0 + lane + r * PTA_WAVE, c = c0 + e;
            y[r] = 0.f;
            if (e >= len) continue;
            const float now = Io<T>::ld(src + (long)m * ld + e);
            float acc = 0.f;
            for (int kk = 0; kk + 1 < K; ++kk) {
                const int jj = j - (K - 1 - kk);
                const float before = jj >= 0 ? Io<T>::ld(src + (long)(first + jj) * ld + e) : tl[(long)(K - 1 + jj) * C + c];
                acc += conv[(long)kk * C + c] * before;
                if (move_tail && kk > 0) tl[(long)(kk - 1) * C + c] = before;  // (the sequence's one token: before is tail[kk])
            }
            if (move_tail && K > 1) tl[(long)(K - 2) * C + c] = now;
            acc += conv[(long)(K - 1) * C + c] * now;
            y[r] = acc / (1.0f + expf(-acc));
            ss += y[r] * y[r];
            if (is_v) qkv[(long)m * C + c] = y[r];
        }
    }
    if (is_v) return;
    const float inv = (is_q ? q_scale : 1.0f) / sqrtf(wave_sum(ss) + norm_eps);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int e = lane + r * PTA_WAVE;
        if (e < len) qkv[(long)m * C + c0 + e] = y[r] * inv;
    }
}

// qkv [M, 2 * kv_heads * N + heads * P], g [M, heads * N], beta [M, heads]: 32-bit, dense.  q, k, v: blocks of columns of rows
// ld apart; conv [taps, channels], channels in the order q | k | v; a [M, heads * N] and b [M, heads] with rows of their own.
// several: some sequence brings more than one token (the tails are then moved on by a launch of their own, for which
// q, k and v must lie side by side).
extern "C" int pta_delta_prep(float* qkv, float* g, float* beta, const void* q, const void* k, const void* v, long ld,
                              const float* conv, const void* a, long a_ld, const void* b, long b_ld, const float* A_log,
                              const float* dt_bias, float* tail, long tail_ld, const int* cu_tokens, const int* token_seq,
                              const int* seq_slot, int several, int n_seqs, int M, int heads, int kv_heads, int N, int P,
                              int taps, float q_scale, float norm_eps, int dtype, void* stream) {
    PTA_REQUIRE(M > 0 && n_seqs > 0 && heads > 0 && kv_heads > 0 && N > 0 && P > 0, "delta_prep: sizes must be positive");
    PTA_REQUIRE(heads % kv_heads == 0, "delta_prep: %d heads are no multiple of %d key heads", heads, kv_heads);
    PTA_REQUIRE(N <= 256, "delta_prep: keys of %d elements are more than the 256 the kernel holds", N);
    PTA_REQUIRE(taps >= 1 && taps <= DELTA_MAX_TAPS, "delta_prep: %d taps are outside 1..%d", taps, DELTA_MAX_TAPS);
    PTA_REQUIRE(2 * kv_heads + 2 * heads <= 65535, "delta_prep: too many heads for one launch");
    PTA_REQUIRE(qkv && g && beta && q && k && v && conv && a && b && A_log && dt_bias && cu_tokens && token_seq && seq_slot && (tail || taps == 1),
                "delta_prep: null pointer");
    const long C = 2L * kv_heads * N + (long)heads * P;
    PTA_REQUIRE(ld >= (long)kv_heads * N && ld >= (long)heads * P && a_ld >= (long)heads * N && b_ld >= heads && (taps == 1 || tail_ld >= (taps - 1) * C),
                "delta_prep: rows lie closer together than they are long");
    PTA_REQUIRE(dtype == PTA_F32 || dtype == PTA_BF16, "delta_prep: unknown dtype %d", dtype);
    const long size = dtype == PTA_F32 ? 4 : 2;
    PTA_REQUIRE(!several || ((const char*)k - (const char*)q == kv_heads * N * size && (const char*)v - (const char*)k == kv_heads * N * size && ld >= C),
                "delta_prep: q, k and v must lie side by side");
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(M, 2 * kv_heads + 2 * heads);
    const int move = several ? 0 : 1;
    if (dtype == PTA_F32)
        hipLaunchKernelGGL(delta_prep_kernel<float>, grid, dim3(64), 0, s, qkv, g, beta, (const float*)q, (const float*)k,
                           (const float*)v, ld, conv, (const float*)a, a_ld, (const float*)b, b_ld, A_log, dt_bias, tail, tail_ld,
                           cu_tokens, token_seq, seq_slot, move, heads, kv_heads, N, P, taps, q_scale, norm_eps);
    else
        hipLaunchKernelGGL(delta_prep_kernel<bf16_t>, grid, dim3(64), 0, s, qkv, g, beta, (const bf16_t*)q, (const bf16_t*)k,
                           (const bf16_t*)v, ld, conv, (const bf16_t*)a, a_ld, (const bf16_t*)b, b_ld, A_log, dt_bias, tail, tail_ld,
                           cu_tokens, token_seq, seq_slot, move, heads, kv_heads, N, P, taps, q_scale, norm_eps);
    if (several && taps > 1) {
        if (pta_check_launch("delta_prep")) return 1;
        return pta_conv_tail(q, ld, tail, tail_ld, cu_tokens, seq_slot, n_seqs, (int)C, taps, dtype, stream);
    }
    return pta_check_launch("delta_prep");
}

template <int NPT, int CPL, int MODE>
__global__ __launch_bounds__(256) void delta_scan_kernel(
    float* __restrict__ y, const float* __restrict__ qkv, const float* __restrict__ g, const float* __restrict__ beta,
    float* __restrict__ state, long state_ld, float* __restrict__ chunk_state, const int* __restrict__ cu_tokens,
    const int* __restrict__ seq_slot, int heads, int G, int P, int N, int chunk, int max_chunks) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    constexpr int GS = NPT + 4;      // a lane group's rows of a token in LDS, padded so that the four groups' banks differ
    constexpr int NP = 4 * GS;
    constexpr int COLS = 64 * CPL;   // columns of a workgroup
    const int h = blockIdx.y, kh = h / (heads / G);
    const int s = MODE == DELTA_WHOLE ? blockIdx.z : blockIdx.z / max_chunks;
    const int c = MODE == DELTA_WHOLE ? 0 : blockIdx.z - s * max_chunks;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int pl = lane & 15, g4 = lane >> 4;
    const int p0 = blockIdx.x * COLS;
    const int pw = (wave * 16 + pl) * CPL;  // the lane's first column within the workgroup's
    const int W = MODE == DELTA_WHOLE ? P : P + N;  // columns of the stored state
    const int used = MODE == DELTA_LOCAL ? P + N : P;
    int t0 = cu_tokens[s];
    int t1 = cu_tokens[s + 1];
    if (MODE != DELTA_WHOLE) {
        t0 += c * chunk;
        if (t0 >= t1) return;  // the sequence has fewer chunks
        t1 = min(t1, t0 + chunk);
    }
    float* sb = MODE == DELTA_WHOLE ? state + (long)seq_slot[s] * state_ld + (long)h * N * P
                                    : chunk_state + ((long)blockIdx.z * heads + h) * N * W;
    float* g_s = lds;                          // [DELTA_PIECE][NP]
    float* k_s = g_s + DELTA_PIECE * NP;       // [DELTA_PIECE][NP]
    float* q_s = k_s + DELTA_PIECE * NP;       // [DELTA_PIECE][NP]
    float* v_s = q_s + DELTA_PIECE * NP;       // [DELTA_PIECE][COLS]
    float* b_s = v_s + DELTA_PIECE * COLS;     // [DELTA_PIECE]
    const int C = 2 * G * N + heads * P;
    float S[CPL][NPT];
#pragma unroll
    for (int j = 0; j < CPL; ++j) {
        const int p = p0 + pw + j;
#pragma unroll
        for (int i = 0; i < NPT; ++i) {
            const int n = g4 * NPT + i;
            if (MODE == DELTA_LOCAL) S[j][i] = (p >= P && n == p - P) ? 1.f : 0.f;
            else S[j][i] = (n < N && p < P) ? sb[(long)n * W + p] : 0.f;
        }
    }
    for (int c0 = t0; c0 < t1; c0 += DELTA_PIECE) {
        const int cnt = min(DELTA_PIECE, t1 - c0);
        __syncthreads();
        for (int i = threadIdx.x; i < cnt * 4 * NPT; i += 256) {
            const int tt = i / (4 * NPT), n = i - tt * (4 * NPT);
            const int at = tt * NP + (n / NPT) * GS + n % NPT;
            const float* row = qkv + (long)(c0 + tt) * C + kh * N + n;
            g_s[at] = n < N ? g[((long)(c0 + tt) * heads + h) * N + n] : 0.f;
            k_s[at] = n < N ? row[(long)G * N] : 0.f;
            if (MODE != DELTA_LOCAL) q_s[at] = n < N ? row[0] : 0.f;
        }
        for (int i = threadIdx.x; i < cnt * COLS; i += 256) {
            const int tt = i / COLS, pp = i % COLS;
            v_s[i] = p0 + pp < P ? qkv[(long)(c0 + tt) * C + 2 * G * N + h * P + p0 + pp] : 0.f;
        }
        if (threadIdx.x < cnt) b_s[threadIdx.x] = beta[(long)(c0 + threadIdx.x) * heads + h];
        __syncthreads();
        for (int tt = 0; tt < cnt; ++tt) {
            const float4* gv = reinterpret_cast<const float4*>(g_s + tt * NP + g4 * GS);
            const float4* kv = reinterpret_cast<const float4*>(k_s + tt * NP + g4 * GS);
            const float4* qv = reinterpret_cast<const float4*>(q_s + tt * NP + g4 * GS);
            const float b = b_s[tt];
            float kk[NPT], u[CPL], o[CPL];
#pragma unroll
            for (int j = 0; j < CPL; ++j) u[j] = 0.f, o[j] = 0.f;
#pragma unroll
            for (int i = 0; i < NPT; i += 4) {
                const float4 gg = gv[i >> 2], k4 = kv[i >> 2];
                kk[i] = k4.x; kk[i + 1] = k4.y; kk[i + 2] = k4.z; kk[i + 3] = k4.w;
#pragma unroll
                for (int j = 0; j < CPL; ++j) {
                    S[j][i] *= gg.x; S[j][i + 1] *= gg.y; S[j][i + 2] *= gg.z; S[j][i + 3] *= gg.w;
                    u[j] += S[j][i] * k4.x;
                    u[j] += S[j][i + 1] * k4.y;
                    u[j] += S[j][i + 2] * k4.z;
                    u[j] += S[j][i + 3] * k4.w;
                }
            }
#pragma unroll
            for (int j = 0; j < CPL; ++j) {
                u[j] += __shfl_xor(u[j], 16, 64);
                u[j] += __shfl_xor(u[j], 32, 64);
                u[j] = b * (v_s[tt * COLS + pw + j] - u[j]);
            }
#pragma unroll
            for (int i = 0; i < NPT; i += 4) {
                float4 q4 = make_float4(0.f, 0.f, 0.f, 0.f);
                if (MODE != DELTA_LOCAL) q4 = qv[i >> 2];
#pragma unroll
                for (int j = 0; j < CPL; ++j) {
                    S[j][i] += kk[i] * u[j]; S[j][i + 1] += kk[i + 1] * u[j];
                    S[j][i + 2] += kk[i + 2] * u[j]; S[j][i + 3] += kk[i + 3] * u[j];
                    if (MODE != DELTA_LOCAL) {
                        o[j] += S[j][i] * q4.x;
                        o[j] += S[j][i + 1] * q4.y;
                        o[j] += S[j][i + 2] * q4.z;
                        o[j] += S[j][i + 3] * q4.w;
                    }
                }
            }
            if (MODE != DELTA_LOCAL) {
#pragma unroll
                for (int j = 0; j < CPL; ++j) {
                    o[j] += __shfl_xor(o[j], 16, 64);
                    o[j] += __shfl_xor(o[j], 32, 64);
                    const int p = p0 + pw + j;
                    if (g4 == 0 && p < P) y[((long)(c0 + tt) * heads + h) * P + p] = o[j];
                }
            }
        }
    }
    if (MODE != DELTA_OUTPUT) {
#pragma unroll
        for (int j = 0; j < CPL; ++j) {
            const int p = p0 + pw + j;
#pragma unroll
            for (int i = 0; i < NPT; ++i) {
                const int n = g4 * NPT + i;
                if (n < N && p < used) sb[(long)n * W + p] = S[j][i];
            }
        }
    }
}

// chunk after chunk: what a chunk starts from takes the place of B_c, the sequence's state moves to its end.  A workgroup
// owns (sequence, head, sixteen columns); the state stands in LDS between two chunks.  N a multiple of 16: products on the
// matrix cores in 32-bit, a wave a tile of sixteen rows in turn; a lane's four consecutive elements of a row of A_c are
// four products' operands (the order of a sum over rows of the state is that of the products).
typedef float delta_f4 __attribute__((ext_vector_type(4)));

template <bool MFMA>
__global__ __launch_bounds__(256) void delta_carry_kernel(float* __restrict__ state, long state_ld, float* __restrict__ chunk_state,
                                                          const int* __restrict__ cu_tokens, const int* __restrict__ seq_slot,
                                                          int heads, int P, int N, int chunk, int max_chunks) {
    __shared__ float S_s[256 * 17];  // [N][16 + 1]
    const int h = blockIdx.y, s = blockIdx.z, p0 = blockIdx.x * 16;
    const int n_chunks = (cu_tokens[s + 1] - cu_tokens[s] + chunk - 1) / chunk;
    const int W = P + N;
    const int col = threadIdx.x & 15, rg = threadIdx.x >> 4;  // sixteen groups of rows
    const bool in = p0 + col < P;
    float* sp = state + (long)seq_slot[s] * state_ld + (long)h * N * P + p0 + col;
    for (int n = rg; n < N; n += 16) S_s[n * 17 + col] = in ? sp[(long)n * P] : 0.f;
    __syncthreads();
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lk = lane >> 4;
    for (int c = 0; c < n_chunks; ++c) {
        float* cs = chunk_state + (((long)s * max_chunks + c) * heads + h) * (long)N * W;
        float next[16];  // rows this thread forms: (wave-tile rows) or rg, rg + 16, ...
        if constexpr (MFMA) {
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int r0 = (wave + 4 * j) * 16;
                if (r0 >= N) continue;
                delta_f4 acc;
#pragma unroll
                for (int e = 0; e < 4; ++e) acc[e] = p0 + lr < P ? cs[(long)(r0 + lk * 4 + e) * W + p0 + lr] : 0.f;
                const float* arow = cs + (long)(r0 + lr) * W + P + lk * 4;
                for (int m0 = 0; m0 < N; m0 += 16) {
                    float a[4];
#pragma unroll
                    for (int e = 0; e < 4; ++e) a[e] = arow[m0 + e];
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], S_s[(m0 + lk * 4 + e) * 17 + lr], acc, 0, 0, 0);
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) next[j * 4 + e] = acc[e];
            }
        } else {
#pragma unroll
            for (int j = 0; j < 16; ++j) {
                const int n = rg + 16 * j;
                if (n >= N) continue;
                const float* arow = cs + (long)n * W + P;
                float acc = in ? cs[(long)n * W + p0 + col] : 0.f;
                for (int m = 0; m < N; ++m) acc += arow[m] * S_s[m * 17 + col];
                next[j] = acc;
            }
        }
        __syncthreads();  // every sum has been formed: B_c and the state may be replaced
        for (int n = rg; n < N; n += 16)
            if (in) cs[(long)n * W + p0 + col] = S_s[n * 17 + col];
        __syncthreads();
        if constexpr (MFMA) {
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int r0 = (wave + 4 * j) * 16;
                if (r0 >= N) continue;
#pragma unroll
                for (int e = 0; e < 4; ++e) S_s[(r0 + lk * 4 + e) * 17 + lr] = next[j * 4 + e];
            }
        } else {
#pragma unroll
            for (int j = 0; j < 16; ++j)
                if (rg + 16 * j < N) S_s[(rg + 16 * j) * 17 + col] = next[j];
        }
        __syncthreads();
    }
    if (n_chunks > 0)
        for (int n = rg; n < N; n += 16)
            if (in) sp[(long)n * P] = S_s[n * 17 + col];
}

template <int NPT, int CPL, int MODE>
static void launch_delta_mode(const dim3& grid, float* y, const float* qkv, const float* g, const float* beta, float* state,
                              long state_ld, float* chunk_state, const int* cu_tokens, const int* seq_slot, int heads, int G, int P,
                              int N, int chunk, int max_chunks, hipStream_t s) {
    constexpr size_t lds = (size_t)DELTA_PIECE * (3 * 4 * (NPT + 4) + 64 * CPL + 1) * sizeof(float);
    static_assert(lds <= 64 * 1024, "the piece's rows fit the LDS a launch may ask for without saying so");
    hipLaunchKernelGGL((delta_scan_kernel<NPT, CPL, MODE>), grid, dim3(256), lds, s, y, qkv, g, beta, state, state_ld, chunk_state,
                       cu_tokens, seq_slot, heads, G, P, N, chunk, max_chunks);
}

template <int NPT>
static int launch_delta(float* y, const float* qkv, const float* g, const float* beta, float* state, long state_ld,
                        float* chunk_state, const int* cu_tokens, const int* seq_slot, int n_seqs, int max_new, int heads, int G,
                        int P, int N, int chunk, int max_chunks, hipStream_t s) {
#define DELTA_ARGS y, qkv, g, beta, state, state_ld, chunk_state, cu_tokens, seq_slot, heads, G, P, N, chunk, max_chunks, s
    constexpr int WIDE = NPT <= 32 ? 2 : 1;  // columns a lane where a launch is bound by its reads of LDS, not by its length
    auto tiles = [](int cols, int per) { return (unsigned)((cols + per - 1) / per); };
    if (max_chunks <= 1) {
        launch_delta_mode<NPT, 1, DELTA_WHOLE>(dim3(tiles(P, 64), heads, n_seqs), DELTA_ARGS);
        return pta_check_launch("delta_scan");
    }
    const unsigned runs = (unsigned)(n_seqs * max_chunks);
    if (P + N > 64) launch_delta_mode<NPT, WIDE, DELTA_LOCAL>(dim3(tiles(P + N, 64 * WIDE), heads, runs), DELTA_ARGS);
    else launch_delta_mode<NPT, 1, DELTA_LOCAL>(dim3(tiles(P + N, 64), heads, runs), DELTA_ARGS);
    const dim3 carry((P + 15) / 16, heads, n_seqs);
    if (N % 16 == 0)
        hipLaunchKernelGGL(delta_carry_kernel<true>, carry, dim3(256), 0, s, state, state_ld, chunk_state, cu_tokens, seq_slot, heads,
                           P, N, chunk, max_chunks);
    else
        hipLaunchKernelGGL(delta_carry_kernel<false>, carry, dim3(256), 0, s, state, state_ld, chunk_state, cu_tokens, seq_slot, heads,
                           P, N, chunk, max_chunks);
    if (P > 64) launch_delta_mode<NPT, WIDE, DELTA_OUTPUT>(dim3(tiles(P, 64 * WIDE), heads, runs), DELTA_ARGS);
    else launch_delta_mode<NPT, 1, DELTA_OUTPUT>(dim3(tiles(P, 64), heads, runs), DELTA_ARGS);
#undef DELTA_ARGS
    return pta_check_launch("delta_scan");
}

// y [M, heads * P], qkv [M, 2 * kv_heads * N + heads * P], g [M, heads * N], beta [M, heads], all 32-bit and dense; state
// [slots, >= heads * N * P] rows state_ld apart.  chunk_state [n_seqs * max_chunks, heads, N, P + N] is scratch for steps whose
// longest sequence is cut into max_chunks > 1 chunks of `chunk` tokens; else unused.
extern "C" int pta_delta_scan(float* y, const float* qkv, const float* g, const float* beta, float* state, long state_ld,
                              float* chunk_state, const int* cu_tokens, const int* seq_slot, int n_seqs, int max_new, int heads,
                              int kv_heads, int P, int N, int chunk, int max_chunks, void* stream) {
    PTA_REQUIRE(n_seqs > 0 && max_new > 0 && heads > 0 && kv_heads > 0 && P > 0 && N > 0, "delta_scan: sizes must be positive");
    PTA_REQUIRE(heads % kv_heads == 0, "delta_scan: %d heads are no multiple of %d key heads", heads, kv_heads);
    PTA_REQUIRE(N <= 256, "delta_scan: keys of %d elements are more than the 256 rows of state the kernel holds", N);
    PTA_REQUIRE(heads <= 65535 && n_seqs <= 65535, "delta_scan: too many heads or sequences for one launch");
    PTA_REQUIRE(y && qkv && g && beta && state && cu_tokens && seq_slot, "delta_scan: null pointer");
    PTA_REQUIRE(state_ld >= (long)heads * N * P, "delta_scan: state rows lie closer together than they are long");
    PTA_REQUIRE(max_chunks >= 1 && (max_chunks == 1 || (chunk > 0 && chunk_state && (long)max_chunks * chunk >= max_new)),
                "delta_scan: chunks need their size, enough of them and scratch memory");
    PTA_REQUIRE((long)n_seqs * max_chunks <= 65535, "delta_scan: %ld chunks are more than one launch takes", (long)n_seqs * max_chunks);
    hipStream_t s = (hipStream_t)stream;
#define DELTA_LAUNCH(NPT_) return launch_delta<NPT_>(y, qkv, g, beta, state, state_ld, chunk_state, cu_tokens, seq_slot, n_seqs, \
                                                     max_new, heads, kv_heads, P, N, chunk, max_chunks, s)
    const int npt = (N + 3) / 4;
    if (npt <= 4) DELTA_LAUNCH(4);
    if (npt <= 8) DELTA_LAUNCH(8);
    if (npt <= 16) DELTA_LAUNCH(16);
    if (npt <= 32) DELTA_LAUNCH(32);
    DELTA_LAUNCH(64);
#undef DELTA_LAUNCH
}
