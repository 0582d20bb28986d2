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
// pta_delta_scan runs the recurrence, in one of two ways.
//
// Few tokens a sequence (decoding, short portions): delta_step_kernel walks each sequence's tokens from its state to its
// state.  A workgroup of four waves owns (sequence, head, 64 columns p of the state); a wave owns sixteen columns, and its
// four groups of sixteen lanes hold NPT consecutive rows n each in registers; sums over rows end with two exchanges between
// the groups.  A piece of the tokens' g, k, q, v and beta is staged in LDS by the whole workgroup, then walked in order.
//
// Prompts: blocks of sixteen tokens as 32-bit matrix products.  With b_t = g_1 * ... * g_t inside a block (element by
// element) and S the block's first state, the recurrence says
//   R   = V - K^ S                        K^_t = b_t * k_t
//   U   = (I + diag(beta) L)^-1 diag(beta) R      L_ts = sum_n k_t k_s (g_(s+1) ... g_t), s < t
//   O   = Q^ S + A U                      Q^_t = b_t * q_t,  A_ts = sum_n q_t k_s (g_(s+1) ... g_t), s <= t
//   S  <- diag(b_16) S + Kd^T U           Kd_s = k_s * (g_(s+1) ... g_16)
// Every product of decays runs forward from a token to a later one, so nothing is divided by a decay and nothing can
// overflow.  delta_block_kernel makes K^, Q^, Kd, A and the triangular inverse for all blocks at once; delta_scan_kernel walks the
// blocks: a wave owns sixteen columns of the state as the accumulators of its row tiles, which are the second operand of the
// products with K^ and Q^ as they lie (a lane's four rows are the four products' rows of the state).
//
// A long prompt of few sequences and heads is also cut into chunks that run side by side.  The recurrence is affine in the
// state: over chunk c, S_out = A_c S_in + B_c, with B_c the result from a zero state and A_c (N x N) that of the unit matrix
// with values of zero, so:
//   DELTA_LOCAL   every chunk from [0 | I]: columns 0 .. P - 1 leave B_c, columns P .. P + N - 1 leave A_c;
//   delta_carry   chunk after chunk, S_in(c + 1) = A_c S_in(c) + B_c, from the sequence's state to its state (A_c is a
//                 product of contractions, so nothing grows);
//   DELTA_OUTPUT  every chunk again from its S_in, with the outputs.
#include "common.h"
#include "pta_kernels.h"

#include <algorithm>

#define DELTA_PIECE 16
#define DELTA_MAX_TAPS 16
enum { DELTA_WHOLE = 0, DELTA_LOCAL = 1, DELTA_OUTPUT = 2 };

__device__ __forceinline__ float softplus_32(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// One wave per (TOK tokens, unit): units are the q heads, the k heads, the value heads and the heads' decays (with
// beta); a unit's convolution weights stay in registers over its tokens.
#define PREP_TOKENS 4

template <typename T, int KMAX, int TOK>
__global__ __launch_bounds__(256) void delta_prep_kernel(
    float* __restrict__ qkv, float* __restrict__ g, float* __restrict__ beta, const T* __restrict__ q, const T* __restrict__ k,
    const T* __restrict__ v, long ld, const float* __restrict__ conv, const T* __restrict__ a, long a_ld,
    const T* __restrict__ b, long b_ld, const float* __restrict__ A_log, const float* __restrict__ dt_bias,
    float* __restrict__ tail, long tail_ld, const int* __restrict__ cu_tokens, const int* __restrict__ token_seq,
    const int* __restrict__ seq_slot, int move_tail, int M, int heads, int G, int N, int P, int K, float q_scale, float norm_eps) {
    const int unit = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int m0 = blockIdx.x * TOK, m1 = min(M, m0 + TOK);
    if (unit >= 2 * G + 2 * heads) return;
    if (unit >= 2 * G + heads) {  // a head's decays and step size
        const int h = unit - 2 * G - heads;
        const float rate = expf(A_log[h]);
        for (int e = lane; e < N; e += PTA_WAVE) {
            const int at = h * N + e;
            const float bias = dt_bias[at];
            for (int m = m0; m < m1; ++m)
                g[(long)m * heads * N + at] = expf(-rate * softplus_32(Io<T>::ld(a + (long)m * a_ld + at) + bias));
        }
        if (lane < m1 - m0) beta[(long)(m0 + lane) * heads + h] = 1.0f / (1.0f + expf(-Io<T>::ld(b + (long)(m0 + lane) * b_ld + h)));
        return;
    }
    const bool is_v = unit >= 2 * G, is_q = unit < G;
    const int len = is_v ? P : N, local = is_v ? unit - 2 * G : is_q ? unit : unit - G;  // the head within its tensor
    const T* src = (is_v ? v : is_q ? q : k) + (long)local * len;
    const int c0 = is_v ? 2 * G * N + local * P : unit * N;  // first channel of the head in q | k | v
    const int C = 2 * G * N + heads * P;
    // whether every input of these tokens is a row of this step: they are then asked for all at once
    const bool inside = TOK > 1 && m1 - m0 == TOK && token_seq[m0] == token_seq[m1 - 1] && m0 - cu_tokens[token_seq[m0]] >= K - 1;
    for (int e0 = 0; e0 < len; e0 += 4 * PTA_WAVE) {  // (heads of q and k fit one round)
        float w[4][KMAX];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int e = e0 + lane + r * PTA_WAVE;
#pragma unroll
            for (int kk = 0; kk < KMAX; ++kk)  // (fewer taps: zeros in front)
                w[r][kk] = (e < len && kk >= KMAX - K) ? conv[(long)(kk - (KMAX - K)) * C + c0 + e] : 0.f;
        }
        float x[4][TOK + KMAX - 1];  // row m0 - (KMAX - 1) + i
        if (TOK > 1 && KMAX <= 4 && inside) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int e = e0 + lane + r * PTA_WAVE;
                if (e0 + r * PTA_WAVE >= len) continue;
#pragma unroll
                for (int i = 0; i < TOK + KMAX - 1; ++i)
                    x[r][i] = Io<T>::ld(src + (long)max(m0 - (KMAX - 1) + i, 0) * ld + min(e, len - 1));
            }
#pragma unroll
            for (int t = 0; t < TOK; ++t) {
                float y[4], ss = 0.f;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    y[r] = 0.f;
                    if (e0 + lane + r * PTA_WAVE >= len) continue;
                    float acc = 0.f;
#pragma unroll
                    for (int kk = 0; kk < KMAX; ++kk) acc += w[r][kk] * x[r][t + kk];
                    y[r] = acc / (1.0f + expf(-acc));
                    ss += y[r] * y[r];
                }
                const float by = is_v ? 1.0f : (is_q ? q_scale : 1.0f) / sqrtf(wave_sum(ss) + norm_eps);
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int e = e0 + lane + r * PTA_WAVE;
                    if (e < len) qkv[(long)(m0 + t) * C + c0 + e] = y[r] * by;
                }
            }
            continue;
        }
        for (int m = m0; m < m1; ++m) {
            const int s = token_seq[m], first = cu_tokens[s], j = m - first;
            float* tl = tail + (K > 1 ? (long)seq_slot[s] * tail_ld : 0L);
            float y[4], ss = 0.f;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int e = e0 + lane + r * PTA_WAVE, c = c0 + e;
                y[r] = 0.f;
                if (e >= len) continue;
                float acc = 0.f;
#pragma unroll
                for (int kk = 0; kk < KMAX; ++kk) {
                    if (kk < KMAX - K) continue;
                    const int jj = j - (KMAX - 1 - kk);
                    const float x = jj >= 0 ? Io<T>::ld(src + (long)(first + jj) * ld + e) : tl[(long)(K - 1 + jj) * C + c];
                    acc += w[r][kk] * x;
                    if (move_tail && kk > KMAX - K) tl[(long)(kk - 1 - (KMAX - K)) * C + c] = x;  // (the one token: x is the tail's next, or its own)
                }
                y[r] = acc / (1.0f + expf(-acc));
                ss += y[r] * y[r];
            }
            const float by = is_v ? 1.0f : (is_q ? q_scale : 1.0f) / sqrtf(wave_sum(ss) + norm_eps);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int e = e0 + lane + r * PTA_WAVE;
                if (e < len) qkv[(long)m * C + c0 + e] = y[r] * by;
            }
        }
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
    const int each = several ? PREP_TOKENS : 1;  // (steps of one token per sequence are short of waves, not of registers)
    const dim3 grid((M + each - 1) / each, (2 * kv_heads + 2 * heads + 3) / 4);
    const int move = several ? 0 : 1;
#define DELTA_PREP_EACH(T_, KMAX_, TOK_)                                                                                                    \
    hipLaunchKernelGGL((delta_prep_kernel<T_, KMAX_, TOK_>), grid, dim3(256), 0, s, qkv, g, beta, (const T_*)q, (const T_*)k, (const T_*)v, \
                       ld, conv, (const T_*)a, a_ld, (const T_*)b, b_ld, A_log, dt_bias, tail, tail_ld, cu_tokens, token_seq,         \
                       seq_slot, move, M, heads, kv_heads, N, P, taps, q_scale, norm_eps)
#define DELTA_PREP(T_, KMAX_)                                   \
    do {                                                        \
        if (several) DELTA_PREP_EACH(T_, KMAX_, PREP_TOKENS);   \
        else DELTA_PREP_EACH(T_, KMAX_, 1);                     \
    } while (0)
    if (dtype == PTA_F32) {
        if (taps <= 4) DELTA_PREP(float, 4);
        else DELTA_PREP(float, DELTA_MAX_TAPS);
    } else {
        if (taps <= 4) DELTA_PREP(bf16_t, 4);
        else DELTA_PREP(bf16_t, DELTA_MAX_TAPS);
    }
#undef DELTA_PREP
#undef DELTA_PREP_EACH
    if (several && taps > 1) {
        if (pta_check_launch("delta_prep")) return 1;
        return pta_conv_tail(q, ld, tail, tail_ld, cu_tokens, seq_slot, n_seqs, (int)C, taps, dtype, stream);
    }
    return pta_check_launch("delta_prep");
}

// y, state as pta_delta_scan has them: every sequence's tokens in order, from its state to its state
template <int NPT>
__global__ __launch_bounds__(256) void delta_step_kernel(
    float* __restrict__ y, const float* __restrict__ qkv, const float* __restrict__ g, const float* __restrict__ beta,
    float* __restrict__ state, long state_ld, const int* __restrict__ cu_tokens, const int* __restrict__ seq_slot, int heads,
    int G, int P, int N) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    constexpr int GS = NPT + 4;      // a lane group's rows of a token in LDS, padded so that the four groups' banks differ
    constexpr int NP = 4 * GS;
    const int h = blockIdx.y, kh = h / (heads / G), s = blockIdx.z;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int pl = lane & 15, g4 = lane >> 4;
    const int p0 = blockIdx.x * 64, pw = wave * 16 + pl, p = p0 + pw;
    const int t0 = cu_tokens[s], t1 = cu_tokens[s + 1];
    float* sb = state + (long)seq_slot[s] * state_ld + (long)h * N * P;
    float* g_s = lds;                          // [DELTA_PIECE][NP]
    float* k_s = g_s + DELTA_PIECE * NP;       // [DELTA_PIECE][NP]
    float* q_s = k_s + DELTA_PIECE * NP;       // [DELTA_PIECE][NP]
    float* v_s = q_s + DELTA_PIECE * NP;       // [DELTA_PIECE][64]
    float* b_s = v_s + DELTA_PIECE * 64;       // [DELTA_PIECE]
    const int C = 2 * G * N + heads * P;
    float S[NPT];
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
        const int n = g4 * NPT + i;
        S[i] = (n < N && p < P) ? sb[(long)n * P + p] : 0.f;
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
            q_s[at] = n < N ? row[0] : 0.f;
        }
        for (int i = threadIdx.x; i < cnt * 64; i += 256) {
            const int tt = i >> 6, pp = i & 63;
            v_s[i] = p0 + pp < P ? qkv[(long)(c0 + tt) * C + 2 * G * N + h * P + p0 + pp] : 0.f;
        }
        if (threadIdx.x < cnt) b_s[threadIdx.x] = beta[(long)(c0 + threadIdx.x) * heads + h];
        __syncthreads();
        for (int tt = 0; tt < cnt; ++tt) {
            const float4* gv = reinterpret_cast<const float4*>(g_s + tt * NP + g4 * GS);
            const float4* kv = reinterpret_cast<const float4*>(k_s + tt * NP + g4 * GS);
            const float4* qv = reinterpret_cast<const float4*>(q_s + tt * NP + g4 * GS);
            float u = 0.f, o = 0.f;
#pragma unroll
            for (int i = 0; i < NPT; i += 4) {
                const float4 gg = gv[i >> 2], kk = kv[i >> 2];
                S[i] *= gg.x; S[i + 1] *= gg.y; S[i + 2] *= gg.z; S[i + 3] *= gg.w;
                u += S[i] * kk.x; u += S[i + 1] * kk.y; u += S[i + 2] * kk.z; u += S[i + 3] * kk.w;
            }
            u += __shfl_xor(u, 16, 64);
            u += __shfl_xor(u, 32, 64);
            u = b_s[tt] * (v_s[tt * 64 + pw] - u);
#pragma unroll
            for (int i = 0; i < NPT; i += 4) {
                const float4 kk = kv[i >> 2], qq = qv[i >> 2];
                S[i] += kk.x * u; S[i + 1] += kk.y * u; S[i + 2] += kk.z * u; S[i + 3] += kk.w * u;
                o += S[i] * qq.x; o += S[i + 1] * qq.y; o += S[i + 2] * qq.z; o += S[i + 3] * qq.w;
            }
            o += __shfl_xor(o, 16, 64);
            o += __shfl_xor(o, 32, 64);
            if (g4 == 0 && p < P) y[((long)(c0 + tt) * heads + h) * P + p] = o;
        }
    }
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
        const int n = g4 * NPT + i;
        if (n < N && p < P) sb[(long)n * P + p] = S[i];
    }
}

// ---- blocks of sixteen tokens ------------------------------------------------------------------------------------------
typedef float delta_f4 __attribute__((ext_vector_type(4)));
#define DELTA_BLOCK 16

template <int V>
__device__ __forceinline__ void delta_load(const float* p, float (&v)[V]) {
    if constexpr (V == 2) {
        const float2 q = *reinterpret_cast<const float2*>(p);
        v[0] = q.x; v[1] = q.y;
    } else {
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] = p[i];
    }
}

// One workgroup per (block, head, sequence).  hat [M, heads, 3, N]: K^, Q^ and Kd of every token; ta [M, heads, 2, 16]: its row of
// the inverse times diag(beta), and of A; the decays over the whole block take the place of its first token's row of g.
// Thread (token s, group of RT channels): k_s carried forward over the later tokens, channel by channel, gives a column of L
// and of A, summed over the channels by exchanges and through LDS in wave order.
template <int RT>
__global__ __launch_bounds__(256) void delta_block_kernel(float* __restrict__ hat, float* __restrict__ ta, float* __restrict__ g,
                                                          const float* __restrict__ qkv, const float* __restrict__ beta,
                                                          const int* __restrict__ cu_tokens, int heads, int G, int P, int N) {
    constexpr int NP = 16 * RT, ROW = NP + 4;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* g_s = lds;                    // [16][ROW]
    float* k_s = g_s + 16 * ROW;         // [16][ROW]
    float* q_s = k_s + 16 * ROW;         // [16][ROW]
    float* kd_s = q_s + 16 * ROW;        // [16][ROW]; later the waves' sums [4][2][16 t][16 s]
    float* red = kd_s;
    __shared__ float L_s[16][17];
    __shared__ float b_s[16];
    const int h = blockIdx.y, kh = h / (heads / G), s = blockIdx.z;
    const int m0 = cu_tokens[s] + blockIdx.x * DELTA_BLOCK, t1 = cu_tokens[s + 1];
    if (m0 >= t1) return;
    const int cnt = min(DELTA_BLOCK, t1 - m0);
    const int C = 2 * G * N + heads * P;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    {
        float gr[RT], kr[RT], qr[RT];  // all loads in flight at once; what lies past an end is read from inside and put down as nothing
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            const int t = (tid + j * 256) / NP, n = (tid + j * 256) % NP;
            const long m = m0 + min(t, cnt - 1);
            const float* row = qkv + m * C + kh * N + min(n, N - 1);
            gr[j] = g[(m * heads + h) * N + min(n, N - 1)];
            kr[j] = row[(long)G * N];
            qr[j] = row[0];
        }
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            const int t = (tid + j * 256) / NP, n = (tid + j * 256) % NP;
            const bool in = t < cnt && n < N;
            g_s[t * ROW + n] = in ? gr[j] : 1.f;  // (a token past the end changes nothing)
            k_s[t * ROW + n] = in ? kr[j] : 0.f;
            q_s[t * ROW + n] = in ? qr[j] : 0.f;
        }
    }
    if (tid < 16) b_s[tid] = tid < cnt ? beta[(long)(m0 + tid) * heads + h] : 0.f;
    __syncthreads();
    const int st = lane & 15, ch = (wave * 4 + (lane >> 4)) * RT;
    float lk[16], aq[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) lk[t] = 0.f, aq[t] = 0.f;
    constexpr int VN = RT < 2 ? RT : 2;  // channels at a time (the compiler asks for all sixteen tokens' rows at once)
#pragma unroll 1
    for (int c0 = 0; c0 < RT; c0 += VN) {
        const float* gp = g_s + ch + c0;
        const float* kp = k_s + ch + c0;
        const float* qp = q_s + ch + c0;
        float r[VN];
#pragma unroll
        for (int i = 0; i < VN; ++i) r[i] = 0.f;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float gt[VN], kt[VN], qt[VN];
            delta_load<VN>(gp + t * ROW, gt);
            delta_load<VN>(kp + t * ROW, kt);
            delta_load<VN>(qp + t * ROW, qt);
#pragma unroll
            for (int i = 0; i < VN; ++i) {
                r[i] = t == st ? kt[i] : r[i] * gt[i];
                lk[t] += kt[i] * r[i];
                aq[t] += qt[i] * r[i];
            }
        }
#pragma unroll
        for (int i = 0; i < VN; ++i) kd_s[st * ROW + ch + c0 + i] = r[i];
    }
    __syncthreads();
    for (int i = tid; i < cnt * N; i += 256) {
        const int t = i / N, n = i - t * N;
        hat[(((long)(m0 + t) * heads + h) * 3 + 2) * N + n] = kd_s[t * ROW + n];
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < 16; ++t) {
        lk[t] += __shfl_xor(lk[t], 16, 64);
        lk[t] += __shfl_xor(lk[t], 32, 64);
        aq[t] += __shfl_xor(aq[t], 16, 64);
        aq[t] += __shfl_xor(aq[t], 32, 64);
        if (lane < 16) {
            red[((wave * 2 + 0) * 16 + t) * 16 + st] = lk[t];
            red[((wave * 2 + 1) * 16 + t) * 16 + st] = aq[t];
        }
    }
    if (tid < N) {  // forward products from the block's start
        float b = 1.f;
        for (int t = 0; t < cnt; ++t) {
            b *= g_s[t * ROW + tid];
            float* to = hat + ((long)(m0 + t) * heads + h) * 3 * N + tid;
            to[0] = b * k_s[t * ROW + tid];
            to[N] = b * q_s[t * ROW + tid];
        }
        g[((long)m0 * heads + h) * N + tid] = b;
    }
    __syncthreads();
    {
        const int t = tid >> 4, sc = tid & 15;
        float l = 0.f, a = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            l += red[((w * 2 + 0) * 16 + t) * 16 + sc];
            a += red[((w * 2 + 1) * 16 + t) * 16 + sc];
        }
        L_s[t][sc] = sc < t ? l * b_s[t] : 0.f;
        if (t < cnt) ta[((long)(m0 + t) * heads + h) * 32 + 16 + sc] = sc <= t ? a : 0.f;
    }
    __syncthreads();
    if (tid < 16) {  // column tid of (I + diag(beta) L)^-1, times beta of its token
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float acc = t == tid ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < t; ++j) acc -= L_s[t][j] * x[j];
            x[t] = acc;
            if (t < cnt) ta[((long)(m0 + t) * heads + h) * 32 + tid] = acc * b_s[tid];
        }
    }
}

// VEC: N is a multiple of four.  hat and ta are readable for a block past their last token (hat for 256 elements more).
template <int RT, int MODE, bool VEC>
__global__ __launch_bounds__(256) void delta_scan_kernel(
    float* __restrict__ y, const float* __restrict__ qkv, const float* __restrict__ hat, const float* __restrict__ ta,
    const float* __restrict__ g, float* __restrict__ state, long state_ld, float* __restrict__ chunk_state,
    const int* __restrict__ cu_tokens, const int* __restrict__ seq_slot, int heads, int G, int P, int N, int chunk,
    int max_chunks) {
    constexpr int NP = 16 * RT, ROW = NP + 4, TROW = 36;
    constexpr int PIECES = 16 * 3 * NP / 4;                 // four elements of K^, Q^ or Kd each
    constexpr int PER = (PIECES + 255) / 256;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* hat_s = lds;                      // [3][16][ROW]
    float* ta_s = hat_s + 3 * 16 * ROW;      // [16][TROW]
    float* b_s = ta_s + 16 * TROW;           // [NP]
    const int h = blockIdx.y;
    const int s = MODE == DELTA_WHOLE ? blockIdx.z : blockIdx.z / max_chunks;
    const int c = MODE == DELTA_WHOLE ? 0 : blockIdx.z - s * max_chunks;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, lr = lane & 15, lk = lane >> 4;
    const int p = blockIdx.x * 64 + wave * 16 + lr;
    const int W = MODE == DELTA_WHOLE ? P : P + N;  // columns of the stored state
    int t0 = cu_tokens[s], t1 = cu_tokens[s + 1];
    if (MODE != DELTA_WHOLE) {
        t0 += c * chunk;
        if (t0 >= t1) return;  // the sequence has fewer chunks
        t1 = min(t1, t0 + chunk);
    }
    float* sb = MODE == DELTA_WHOLE ? state + (long)seq_slot[s] * state_ld + (long)h * N * P
                                    : chunk_state + ((long)blockIdx.z * heads + h) * N * W;
    const int C = 2 * G * N + heads * P;
    delta_f4 S[RT];
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = r * 16 + lk * 4 + e;
            if (MODE == DELTA_LOCAL) S[r][e] = (p >= P && n == p - P) ? 1.f : 0.f;
            else S[r][e] = (n < N && p < P) ? sb[(long)n * W + p] : 0.f;
        }
    // What a block needs is asked for one block ahead.  The loads branch on nothing: rows past the sequence's end are read
    // (they lie within the buffers) and elements past a row's end are read from inside the row, and both are put down as zeros.
    float4 ph[PER];
    float pt[2], pb, pv[4];
    int off[PER];
    bool keep[PER];
#pragma unroll
    for (int j = 0; j < PER; ++j) {
        const int i = min(tid + j * 256, PIECES - 1);
        const int t = i / (3 * NP / 4), rest = i - t * (3 * NP / 4), which = rest / (NP / 4), n = (rest - which * (NP / 4)) * 4;
        keep[j] = n < N;
        off[j] = (t * heads * 3 + which) * N + (VEC ? min(n, N - 4) : n);
    }
    auto fetch = [&](int m0) {
        const long first = (long)m0 * heads + h;
        const float* hb = hat + first * 3 * N;
        const float* tb = ta + first * 32;
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            if constexpr (VEC) ph[j] = *reinterpret_cast<const float4*>(hb + off[j]);
            else {  // (off[j] + 3 may lie in the next vector of the token, or in the next token's first)
                ph[j] = make_float4(hb[off[j]], hb[off[j] + 1], hb[off[j] + 2], hb[off[j] + 3]);
            }
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) pt[j] = tb[((tid >> 5) + 8 * j) * heads * 32 + (tid & 31)];
        pb = g[first * N + min(tid, N - 1)];
        const float* vb = qkv + (long)m0 * C + 2 * G * N + h * P + min(p, P - 1);
#pragma unroll
        for (int e = 0; e < 4; ++e) pv[e] = vb[(long)min(lk * 4 + e, t1 - 1 - m0) * C];
    };
    fetch(t0);
    for (int m0 = t0; m0 < t1; m0 += DELTA_BLOCK) {
        const int cnt = t1 - m0;  // (from sixteen on: a whole block)
        __syncthreads();
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            const int i = tid + j * 256;
            const int t = i / (3 * NP / 4), rest = i - t * (3 * NP / 4), which = rest / (NP / 4), n = (rest - which * (NP / 4)) * 4;
            const bool in = keep[j] && t < cnt;
            const float4 f = make_float4(in ? ph[j].x : 0.f, in && (VEC || n + 1 < N) ? ph[j].y : 0.f,
                                         in && (VEC || n + 2 < N) ? ph[j].z : 0.f, in && (VEC || n + 3 < N) ? ph[j].w : 0.f);
            if (PIECES % 256 == 0 || i < PIECES) *reinterpret_cast<float4*>(hat_s + (which * 16 + t) * ROW + n) = f;
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) ta_s[((tid >> 5) + 8 * j) * TROW + (tid & 31)] = (tid >> 5) + 8 * j < cnt ? pt[j] : 0.f;
        if (tid < NP) b_s[tid] = tid < N ? pb : 0.f;
        delta_f4 R0, R1 = {0.f, 0.f, 0.f, 0.f}, O0 = {0.f, 0.f, 0.f, 0.f}, O1 = {0.f, 0.f, 0.f, 0.f}, U = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) R0[e] = lk * 4 + e < cnt && p < P ? pv[e] : 0.f;
        __syncthreads();
        if (cnt > DELTA_BLOCK) fetch(m0 + DELTA_BLOCK);
        const float* kh_row = hat_s + lr * ROW + lk * 4;
        const float* qh_row = kh_row + 16 * ROW;
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const float4 a4 = *reinterpret_cast<const float4*>(kh_row + r * 16);
            const float a[4] = {-a4.x, -a4.y, -a4.z, -a4.w};
            delta_f4& R = (r & 1) ? R1 : R0;
#pragma unroll
            for (int e = 0; e < 4; ++e) R = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], S[r][e], R, 0, 0, 0);
        }
        if (MODE != DELTA_LOCAL) {
#pragma unroll
            for (int r = 0; r < RT; ++r) {
                const float4 a4 = *reinterpret_cast<const float4*>(qh_row + r * 16);
                const float a[4] = {a4.x, a4.y, a4.z, a4.w};
                delta_f4& O = (r & 1) ? O1 : O0;
#pragma unroll
                for (int e = 0; e < 4; ++e) O = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], S[r][e], O, 0, 0, 0);
            }
        }
        {
            const float4 a4 = *reinterpret_cast<const float4*>(ta_s + lr * TROW + lk * 4);
            const float a[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) U = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], R0[e] + R1[e], U, 0, 0, 0);
        }
        const float* kd = hat_s + 32 * ROW + lk * 4 * ROW + lr;
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const float4 b4 = *reinterpret_cast<const float4*>(b_s + r * 16 + lk * 4);
            S[r][0] *= b4.x; S[r][1] *= b4.y; S[r][2] *= b4.z; S[r][3] *= b4.w;
#pragma unroll
            for (int e = 0; e < 4; ++e) S[r] = __builtin_amdgcn_mfma_f32_16x16x4f32(kd[e * ROW + r * 16], U[e], S[r], 0, 0, 0);
        }
        if (MODE != DELTA_LOCAL) {
            const float4 a4 = *reinterpret_cast<const float4*>(ta_s + lr * TROW + 16 + lk * 4);
            const float a[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) O0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], U[e], O0, 0, 0, 0);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int m = m0 + lk * 4 + e;
                if (m < t1 && p < P) y[((long)m * heads + h) * P + p] = O0[e] + O1[e];
            }
        }
    }
    if (MODE != DELTA_OUTPUT) {
        const int used = MODE == DELTA_LOCAL ? P + N : P;
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = r * 16 + lk * 4 + e;
                if (n < N && p < used) sb[(long)n * W + p] = S[r][e];
            }
    }
}

// chunk after chunk: what a chunk starts from takes the place of B_c, the sequence's state moves to its end.  A workgroup of
// eight waves owns (sequence, head, sixteen columns); a wave forms RTW tiles of sixteen rows; the state stands in LDS between
// two chunks, and the next chunk's A_c and B_c are asked for while this one's products run.  VEC: A_c's rows can be loaded
// four elements at a time.
template <int RTW, bool VEC>
__global__ __launch_bounds__(512) void delta_carry_kernel(float* __restrict__ state, long state_ld, float* __restrict__ chunk_state,
                                                          const int* __restrict__ cu_tokens, const int* __restrict__ seq_slot,
                                                          int heads, int P, int N, int chunk, int max_chunks) {
    constexpr int RT = 8 * RTW;      // row tiles, and pieces of sixteen elements of a row of A_c
    __shared__ float S_s[RT * 16 * 17];
    const int h = blockIdx.y, s = blockIdx.z, p0 = blockIdx.x * 16;
    const int n_chunks = (cu_tokens[s + 1] - cu_tokens[s] + chunk - 1) / chunk;
    if (n_chunks <= 0) return;
    const long W = P + N;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lk = lane >> 4;
    const bool in = p0 + lr < P;
    float* sp = state + (long)seq_slot[s] * state_ld + (long)h * N * P + p0 + lr;
    float4 a[RTW][RT];
    delta_f4 S[RTW], B[RTW];
    auto base = [&](int c) { return chunk_state + (((long)s * max_chunks + c) * heads + h) * (long)N * W; };
    auto fetch = [&](int c) {
        const float* cs = base(c);
#pragma unroll
        for (int j = 0; j < RTW; ++j) {
            const int r0 = (wave + 8 * j) * 16;
            const float* row = cs + (long)min(r0 + lr, N - 1) * W + P;
#pragma unroll
            for (int m = 0; m < RT; ++m) {
                const int k = m * 16 + lk * 4;
                if (VEC) a[j][m] = *reinterpret_cast<const float4*>(row + min(k, N - 4));
                else a[j][m] = make_float4(row[min(k, N - 1)], row[min(k + 1, N - 1)], row[min(k + 2, N - 1)], row[min(k + 3, N - 1)]);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = r0 + lk * 4 + e;
                B[j][e] = cs[(long)min(n, N - 1) * W + min(p0 + lr, P - 1)];
            }
        }
    };
#pragma unroll
    for (int j = 0; j < RTW; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = (wave + 8 * j) * 16 + lk * 4 + e;
            S[j][e] = (in && n < N) ? sp[(long)n * P] : 0.f;
        }
    fetch(0);
    for (int c = 0; c < n_chunks; ++c) {
        float* cs = base(c);
#pragma unroll
        for (int j = 0; j < RTW; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = (wave + 8 * j) * 16 + lk * 4 + e;
                S_s[n * 17 + lr] = S[j][e];
                if (in && n < N) cs[(long)n * W + p0 + lr] = S[j][e];  // (B_c of these elements is this lane's own, already here)
            }
        __syncthreads();
        delta_f4 acc[RTW][2];
#pragma unroll
        for (int j = 0; j < RTW; ++j) acc[j][0] = B[j], acc[j][1] = delta_f4{0.f, 0.f, 0.f, 0.f};
        // (what stands in LDS beyond row N - 1 is zero, so A_c's elements beyond column N - 1 count for nothing, whatever they are)
#pragma unroll
        for (int m = 0; m < RT; ++m) {
            float b[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) b[e] = S_s[(m * 16 + lk * 4 + e) * 17 + lr];
#pragma unroll
            for (int j = 0; j < RTW; ++j) {
                const float av[4] = {a[j][m].x, a[j][m].y, a[j][m].z, a[j][m].w};
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    acc[j][m & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[e], b[e], acc[j][m & 1], 0, 0, 0);
            }
        }
        if (c + 1 < n_chunks) fetch(c + 1);
#pragma unroll
        for (int j = 0; j < RTW; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e)
                S[j][e] = (wave + 8 * j) * 16 + lk * 4 + e < N ? acc[j][0][e] + acc[j][1][e] : 0.f;
        __syncthreads();  // everyone has read the state that the next turn replaces
    }
#pragma unroll
    for (int j = 0; j < RTW; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = (wave + 8 * j) * 16 + lk * 4 + e;
            if (in && n < N) sp[(long)n * P] = S[j][e];
        }
}

struct DeltaLaunch {
    float* y; const float* qkv; float* g; const float* beta; float* state; long state_ld;
    float *hat, *ta, *chunk_state;
    const int *cu_tokens, *seq_slot;
    int n_seqs, max_new, heads, G, P, N, chunk, max_chunks;
    hipStream_t s;
};

template <int NPT>
static int launch_delta_steps(const DeltaLaunch& d) {
    constexpr size_t lds = (size_t)DELTA_PIECE * (3 * 4 * (NPT + 4) + 64 + 1) * sizeof(float);
    static_assert(lds <= 64 * 1024, "a piece's rows fit the LDS a launch may ask for without saying so");
    hipLaunchKernelGGL(delta_step_kernel<NPT>, dim3((d.P + 63) / 64, d.heads, d.n_seqs), dim3(256), lds, d.s, d.y, d.qkv, d.g, d.beta,
                       d.state, d.state_ld, d.cu_tokens, d.seq_slot, d.heads, d.G, d.P, d.N);
    return pta_check_launch("delta_scan");
}

template <int RT>
static int launch_delta_blocks(const DeltaLaunch& d) {
    constexpr size_t block_lds = (size_t)(3 * 16 * (16 * RT + 4) + std::max(16 * (16 * RT + 4), 4 * 2 * 256)) * sizeof(float);
    constexpr size_t scan_lds = (size_t)(3 * 16 * (16 * RT + 4) + 16 * 36 + 16 * RT) * sizeof(float);
    static_assert(block_lds <= 80 * 1024 && scan_lds <= 64 * 1024, "a block's rows fit the LDS");
    if (block_lds > 62 * 1024)  // more than a launch may ask for unless the kernel has been told
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(delta_block_kernel<RT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)block_lds);
    hipLaunchKernelGGL(delta_block_kernel<RT>, dim3((d.max_new + DELTA_BLOCK - 1) / DELTA_BLOCK, d.heads, d.n_seqs), dim3(256), block_lds,
                       d.s, d.hat, d.ta, d.g, d.qkv, d.beta, d.cu_tokens, d.heads, d.G, d.P, d.N);
#define DELTA_SCAN(MODE_, COLS_, RUNS_)                                                                                          \
    hipLaunchKernelGGL((d.N % 4 ? delta_scan_kernel<RT, MODE_, false> : delta_scan_kernel<RT, MODE_, true>),                       \
                       dim3(((COLS_) + 63) / 64, d.heads, (RUNS_)), dim3(256), scan_lds, d.s, d.y, d.qkv, d.hat, d.ta, d.g, d.state, \
                        d.state_ld, d.chunk_state, d.cu_tokens, d.seq_slot, d.heads, d.G, d.P, d.N, d.chunk, d.max_chunks)
    if (d.max_chunks <= 1) {
        DELTA_SCAN(DELTA_WHOLE, d.P, d.n_seqs);
        return pta_check_launch("delta_scan");
    }
    DELTA_SCAN(DELTA_LOCAL, d.P + d.N, d.n_seqs * d.max_chunks);
    const dim3 carry((d.P + 15) / 16, d.heads, d.n_seqs);
    const bool vec = d.N % 4 == 0 && d.P % 4 == 0;
    auto kern = d.N <= 128 ? (vec ? delta_carry_kernel<1, true> : delta_carry_kernel<1, false>)
                           : (vec ? delta_carry_kernel<2, true> : delta_carry_kernel<2, false>);
    hipLaunchKernelGGL(kern, carry, dim3(512), 0, d.s, d.state, d.state_ld, d.chunk_state, d.cu_tokens, d.seq_slot, d.heads, d.P, d.N,
                       d.chunk, d.max_chunks);
    DELTA_SCAN(DELTA_OUTPUT, d.P, d.n_seqs * d.max_chunks);
#undef DELTA_SCAN
    return pta_check_launch("delta_scan");
}

// y [M, heads * P], qkv [M, 2 * kv_heads * N + heads * P], g [M, heads * N], beta [M, heads], all 32-bit and dense; state
// [slots, >= heads * N * P] rows state_ld apart.  hat [M + 16, heads, 3, N] with 256 elements behind it and ta [M + 16, heads, 2, 16] given
// (scratch): blocks of sixteen tokens; g is then written over.  Without them the tokens are walked one by one.  chunk_state [n_seqs * max_chunks, heads, N,
// P + N] is scratch for steps whose longest sequence is cut into max_chunks > 1 chunks of `chunk` tokens (a multiple of 16).
extern "C" int pta_delta_scan(float* y, const float* qkv, float* g, const float* beta, float* state, long state_ld, float* hat,
                              float* ta, float* chunk_state, const int* cu_tokens, const int* seq_slot, int n_seqs, int max_new,
                              int heads, int kv_heads, int P, int N, int chunk, int max_chunks, void* stream) {
    PTA_REQUIRE(n_seqs > 0 && max_new > 0 && heads > 0 && kv_heads > 0 && P > 0 && N > 0, "delta_scan: sizes must be positive");
    PTA_REQUIRE(heads % kv_heads == 0, "delta_scan: %d heads are no multiple of %d key heads", heads, kv_heads);
    PTA_REQUIRE(N <= 256, "delta_scan: keys of %d elements are more than the 256 rows of state the kernel holds", N);
    PTA_REQUIRE(heads <= 65535 && n_seqs <= 65535, "delta_scan: too many heads or sequences for one launch");
    PTA_REQUIRE(y && qkv && g && beta && state && cu_tokens && seq_slot, "delta_scan: null pointer");
    PTA_REQUIRE(state_ld >= (long)heads * N * P, "delta_scan: state rows lie closer together than they are long");
    PTA_REQUIRE((hat == nullptr) == (ta == nullptr), "delta_scan: blocks need all of their scratch memory");
    PTA_REQUIRE(max_chunks >= 1 && (max_chunks == 1 || (hat && chunk > 0 && chunk % DELTA_BLOCK == 0 && chunk_state &&
                                                        (long)max_chunks * chunk >= max_new)),
                "delta_scan: chunks need their size, a multiple of %d, enough of them and scratch memory", DELTA_BLOCK);
    PTA_REQUIRE((long)n_seqs * max_chunks <= 65535, "delta_scan: %ld chunks are more than one launch takes", (long)n_seqs * max_chunks);
    PTA_REQUIRE(((uintptr_t)hat % 16) == 0 && ((uintptr_t)chunk_state % 16) == 0, "delta_scan: scratch memory must be 16-byte aligned");
    const DeltaLaunch d{y, qkv, g, beta, state, state_ld, hat, ta, chunk_state, cu_tokens, seq_slot, n_seqs, max_new, heads, kv_heads,
                        P, N, chunk, max_chunks, (hipStream_t)stream};
    if (hat) {
        if (N <= 16) return launch_delta_blocks<1>(d);
        if (N <= 32) return launch_delta_blocks<2>(d);
        if (N <= 64) return launch_delta_blocks<4>(d);
        if (N <= 128) return launch_delta_blocks<8>(d);
        return launch_delta_blocks<16>(d);
    }
    if (N <= 16) return launch_delta_steps<4>(d);
    if (N <= 32) return launch_delta_steps<8>(d);
    if (N <= 64) return launch_delta_steps<16>(d);
    if (N <= 128) return launch_delta_steps<32>(d);
    return launch_delta_steps<64>(d);
}
