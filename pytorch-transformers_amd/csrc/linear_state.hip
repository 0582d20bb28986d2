// Linear attention whose state decays, per head (a constant) or per head and key channel (from the token):
//
//   q' = rotate(q) * q_scale, k' = rotate(k) * k_scale       by position, over the head's first elements (or not at all)
//   a  = decay[h], or sigmoid(z)^inv_tau with z = A2 low + bias: one number per key channel, low a short vector per token
//   S <- diag(a) S + k' v^T;  o = S^T q'                      S: [N, P] per head, N the key size, P the value size
//   out = o / sqrt(mean(o^2) + eps) * w * silu(g) * mult      per head, w [P] for all heads or none
//
// q, k, v, g and low are blocks of columns of one product (compute type, rows ld apart); everything between them and out is
// 32-bit; a sequence's state is a row of a state table per slot.
//
// pta_linear_state runs it in one of two ways.
//
// Few tokens a sequence (decoding, short portions): lin_step_kernel, one launch from the product to out.  A workgroup owns
// (head, sequence); a wave owns sixteen columns p of the state, and its four groups of sixteen lanes hold NPT consecutive
// rows n each in registers; a sum over rows ends with two exchanges between the groups.  The tokens' q', k', a and v are staged
// in LDS piece by piece, walked in order, and the piece's results are normed and gated from LDS.
//
// Prompts: blocks of sixteen tokens as 32-bit matrix products.  With b_t = a_1 ... a_t inside a block and S its first state:
//   O = Q^ S + A V      Q^_t = b_t q'_t,  A_ts = sum_n q'_t k'_s (a_(s+1) ... a_t), s <= t
//   S <- diag(b_16) S + Kd^T V            Kd_s = k'_s (a_(s+1) ... a_16)
// Every product of decays runs forward from a token to a later one, so nothing is divided by a decay and nothing overflows.
// lin_block_kernel makes Q^, Kd, A and b_16 of all blocks at once; lin_scan_kernel walks the blocks: a wave owns sixteen columns
// of the state as the accumulators of its row tiles, which are the second operand of the product with Q^ as they lie.
// Long prompts of few sequences and heads are cut into chunks that run side by side: LIN_LOCAL (every chunk from a zero
// state: what it adds, and the product of its decays), lin_carry_kernel (chunk after chunk, S_in(c + 1) = diag(d_c) S_in(c) +
// S_c, from the sequence's state to its state), LIN_OUTPUT (every chunk again from its S_in, with the outputs).
#include "common.h"
#include "pta_kernels.h"
#include "qkv_tail.h"

#include <algorithm>

#define LIN_PIECE 16   // most tokens a step launch stages at once
#define LIN_BLOCK 16
#define LIN_LOW 32     // elements of the short vector that a block launch stages at once
enum { LIN_WHOLE = 0, LIN_LOCAL = 1, LIN_OUTPUT = 2 };

typedef float lin_f4 __attribute__((ext_vector_type(4)));

// sigmoid(z)^inv_tau = exp(-inv_tau softplus(-z))
__device__ __forceinline__ float channel_decay(float z, float inv_tau) {
    const float sp = z < -20.f ? -z : log1pf(expf(-z));
    return expf(-inv_tau * sp);
}

struct LinIn {  // what both ways read
    const void *q, *k, *v, *g, *low, *a2;
    long ld;
    float q_scale, k_scale, inv_tau;
    PtaRotation rot;
    const int *token_pos, *token_seq, *cu_tokens, *seq_slot;
    const float *decay, *a2_bias;
    int rank, heads, P, N;
};

// element n of a head's row, rotated by the token's position
template <typename T>
__device__ __forceinline__ float lin_rotated(const T* row, int n, const PtaRotation& rot, const float* freq, float pos) {
    const float x = Io<T>::ld(row + n);
    if (!freq || n >= rot.rotary_dim) return x;
    const int half = rot.rotary_dim >> 1;
    int p, other;
    float sign;
    if (rot.pairing == PTA_PAIR_INTERLEAVED) { p = n >> 1; other = n ^ 1; sign = (n & 1) ? 1.f : -1.f; }
    else { p = n < half ? n : n - half; other = n < half ? n + half : n - half; sign = n < half ? -1.f : 1.f; }
    const float ang = pos * freq[p];
    return x * (cosf(ang) * rot.cs_scale) + sign * Io<T>::ld(row + other) * (sinf(ang) * rot.cs_scale);
}

__device__ __forceinline__ const float* lin_freq(const LinIn& in, int m) {
    return in.rot.inv_freq ? in.rot.inv_freq + (in.rot.inv_freq_ld ? (long)in.token_seq[m] * in.rot.inv_freq_ld : 0L) : nullptr;
}

// sum over the short vector: A2 row . low
template <typename T>
__device__ __forceinline__ float lin_low_dot(const T* a, const T* low, int rank) {
    float acc = 0.f;
    int r = 0;
    if (sizeof(T) == 2 && ((uintptr_t)a & 15) == 0 && ((uintptr_t)low & 15) == 0) {
        for (; r + 8 <= rank; r += 8) {
            float x[8], y[8];
            unpack8(*reinterpret_cast<const uint4*>((const bf16_t*)a + r), x);
            unpack8(*reinterpret_cast<const uint4*>((const bf16_t*)low + r), y);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc += x[e] * y[e];
        }
    }
    for (; r < rank; ++r) acc += Io<T>::ld(a + r) * Io<T>::ld(low + r);
    return acc;
}

// What an element of the first tokens needs, asked for before anything is waited for: q and k with the elements they are
// rotated with, and up to LIN_AHEAD sixteen-byte pieces of the channel's row of A2 and of the short vector.
#define LIN_AHEAD 4
template <typename T>
struct LinAhead {
    float k, q, k2, q2;
    uint4 a[LIN_AHEAD], l[LIN_AHEAD];
};

// ---- tokens one by one --------------------------------------------------------------------------------------------------
// (MOST: threads of the largest workgroup, which the registers a lane may use follow from)
template <typename T, int NPT, bool CHANNEL, int MOST>
__global__ __launch_bounds__(MOST) void lin_step_kernel(T* __restrict__ out, long out_ld, LinIn in, const float* __restrict__ w,
                                                        float eps, float mult, float* __restrict__ state, long state_ld, int piece) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    constexpr int GS = NPT + 4;  // a lane group's rows of a token in LDS, padded so that the four groups' banks differ
    constexpr int NP = 4 * GS;
    const int N = in.N, P = in.P, h = blockIdx.x, s = blockIdx.y;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, waves = blockDim.x >> 6;
    const int pl = lane & 15, g4 = lane >> 4;
    const int pw = wave * 16 + pl, PP = waves * 16;
    const int t0 = in.cu_tokens[s], t1 = in.cu_tokens[s + 1];
    float* sb = state + (long)in.seq_slot[s] * state_ld + (long)h * N * P;
    float* k_s = lds;                    // [piece][NP]
    float* q_s = k_s + piece * NP;       // [piece][NP]
    float* a_s = q_s + piece * NP;       // [piece][NP] (decays per channel only)
    float* v_s = a_s + (CHANNEL ? piece * NP : 0);  // [piece][PP]; then the piece's results
    const float a_h = CHANNEL ? 1.f : in.decay[h];
    const T *q = (const T*)in.q + (long)h * N, *k = (const T*)in.k + (long)h * N, *v = (const T*)in.v + (long)h * P;
    const T *a2 = (const T*)in.a2 + (long)h * N * in.rank, *low = (const T*)in.low;
    // whether the short vector's products are of so few whole pieces that they are asked for ahead
    const bool pieces = CHANNEL && sizeof(T) == 2 && in.rank % 8 == 0 && in.rank <= 8 * LIN_AHEAD && ((uintptr_t)in.a2 & 15) == 0 &&
                        ((uintptr_t)in.low & 15) == 0 && in.ld % 8 == 0;
    const bool turned = in.rot.inv_freq != nullptr;
    // element i of a piece's tokens: (token, key element)
    auto ask = [&](int c0, int cnt, int i, LinAhead<T>& e) {
        const int tt = min(i / (4 * NPT), cnt - 1), n = min(i % (4 * NPT), N - 1);
        const long m = c0 + tt;
        const int half = in.rot.rotary_dim >> 1;
        const int other = !turned || n >= in.rot.rotary_dim ? n : in.rot.pairing == PTA_PAIR_INTERLEAVED ? n ^ 1 : n < half ? n + half : n - half;
        e.k = Io<T>::ld(k + m * in.ld + n);
        e.q = Io<T>::ld(q + m * in.ld + n);
        if (turned) {
            e.k2 = Io<T>::ld(k + m * in.ld + other);
            e.q2 = Io<T>::ld(q + m * in.ld + other);
        }
        if (pieces) {
#pragma unroll
            for (int r = 0; r < LIN_AHEAD; ++r) {
                const int at = min(r * 8, in.rank - 8);
                e.a[r] = *reinterpret_cast<const uint4*>((const bf16_t*)a2 + (long)n * in.rank + at);
                e.l[r] = *reinterpret_cast<const uint4*>((const bf16_t*)low + m * in.ld + at);
            }
        }
    };
    auto put = [&](int c0, int cnt, int i, const LinAhead<T>& e) {
        const int tt = i / (4 * NPT), n = i - tt * (4 * NPT), m = c0 + tt;
        if (tt >= cnt) return;
        const int at = tt * NP + (n / NPT) * GS + n % NPT;
        float kv = 0.f, qv = 0.f, av = 0.f;
        if (n < N) {
            kv = e.k, qv = e.q;
            if (turned && n < in.rot.rotary_dim) {
                const int half = in.rot.rotary_dim >> 1;
                const bool inter = in.rot.pairing == PTA_PAIR_INTERLEAVED;
                const float ang = (float)in.token_pos[m] * lin_freq(in, m)[inter ? n >> 1 : n < half ? n : n - half];
                const float sign = (inter ? (n & 1) != 0 : n >= half) ? 1.f : -1.f;
                const float cs = cosf(ang) * in.rot.cs_scale, sn = sinf(ang) * in.rot.cs_scale;
                kv = kv * cs + sign * e.k2 * sn;
                qv = qv * cs + sign * e.q2 * sn;
            }
            kv *= in.k_scale;
            qv *= in.q_scale;
            if constexpr (CHANNEL) {
                float z = 0.f;
                if (pieces) {
#pragma unroll
                    for (int r = 0; r < LIN_AHEAD; ++r) {
                        if (r * 8 >= in.rank) continue;
                        float x[8], y[8];
                        unpack8(e.a[r], x);
                        unpack8(e.l[r], y);
#pragma unroll
                        for (int c = 0; c < 8; ++c) z += x[c] * y[c];
                    }
                } else {
                    z = lin_low_dot(a2 + (long)n * in.rank, low + m * in.ld, in.rank);
                }
                av = channel_decay(z + in.a2_bias[h * N + n], in.inv_tau);
            }
        }
        k_s[at] = kv;
        q_s[at] = qv;
        if constexpr (CHANNEL) a_s[at] = av;
    };
    LinAhead<T> ahead;
    ask(t0, min(piece, t1 - t0), threadIdx.x, ahead);
    float S[NPT];
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
        const int n = g4 * NPT + i;
        S[i] = (n < N && pw < P) ? sb[(long)n * P + pw] : 0.f;
    }
    for (int c0 = t0; c0 < t1; c0 += piece) {
        const int cnt = min(piece, t1 - c0);
        __syncthreads();
        for (int i = threadIdx.x; i < cnt * 4 * NPT; i += blockDim.x) {
            if (c0 != t0 || i >= (int)blockDim.x) ask(c0, cnt, i, ahead);
            put(c0, cnt, i, ahead);
        }
        for (int i = threadIdx.x; i < cnt * PP; i += blockDim.x) {
            const int tt = i / PP, pp = i - tt * PP;
            v_s[i] = pp < P ? Io<T>::ld(v + (long)(c0 + tt) * in.ld + pp) : 0.f;
        }
        __syncthreads();
        for (int tt = 0; tt < cnt; ++tt) {
            const float4* kv = reinterpret_cast<const float4*>(k_s + tt * NP + g4 * GS);
            const float4* qv = reinterpret_cast<const float4*>(q_s + tt * NP + g4 * GS);
            const float4* av = reinterpret_cast<const float4*>(a_s + tt * NP + g4 * GS);
            const float x = v_s[tt * PP + pw];
            float o = 0.f;
#pragma unroll
            for (int i = 0; i < NPT; i += 4) {
                const float4 kk = kv[i >> 2], qq = qv[i >> 2];
                float4 aa = make_float4(a_h, a_h, a_h, a_h);
                if constexpr (CHANNEL) aa = av[i >> 2];
                S[i] = aa.x * S[i] + kk.x * x;
                S[i + 1] = aa.y * S[i + 1] + kk.y * x;
                S[i + 2] = aa.z * S[i + 2] + kk.z * x;
                S[i + 3] = aa.w * S[i + 3] + kk.w * x;
                o += S[i] * qq.x; o += S[i + 1] * qq.y; o += S[i + 2] * qq.z; o += S[i + 3] * qq.w;
            }
            o += __shfl_xor(o, 16, 64);
            o += __shfl_xor(o, 32, 64);
            if (g4 == 0) v_s[tt * PP + pw] = pw < P ? o : 0.f;  // (this wave alone has read that value, and its lanes run together)
        }
        __syncthreads();
        for (int tt = wave; tt < cnt; tt += waves) {  // a wave a token: norm and gate
            const long m = c0 + tt;
            const T* gr = (const T*)in.g + m * in.ld + (long)h * P;
            T* to = out + m * out_ld + (long)h * P;
            float ss = 0.f;
            for (int e = lane; e < P; e += PTA_WAVE) ss += v_s[tt * PP + e] * v_s[tt * PP + e];
            const float inv = mult / sqrtf(wave_sum(ss) / (float)P + eps);
            for (int e = lane; e < P; e += PTA_WAVE) {
                const float gv = Io<T>::ld(gr + e);
                Io<T>::st(to + e, v_s[tt * PP + e] * inv * (w ? w[e] : 1.f) * (gv / (1.0f + expf(-gv))));
            }
        }
    }
#pragma unroll
    for (int i = 0; i < NPT; ++i) {
        const int n = g4 * NPT + i;
        if (n < N && pw < P) sb[(long)n * P + pw] = S[i];
    }
}

// ---- blocks of sixteen tokens --------------------------------------------------------------------------------------------
// hat [M + 16, heads, 2, N]: Q^ and Kd of every token; ta [M + 16, heads, 16]: its row of A; bd [blocks, heads, N]: the decays over
// a whole block, blocks counted through all sequences (block b of sequence s is block cu[s] / 16 + s + b).
__device__ __forceinline__ long lin_block_index(int first_token, int s, int b) { return first_token / LIN_BLOCK + s + b; }

template <typename T, int RT, bool CHANNEL>
__global__ __launch_bounds__(256) void lin_block_kernel(float* __restrict__ hat, float* __restrict__ ta, float* __restrict__ bd, LinIn in) {
    constexpr int NP = 16 * RT, ROW = NP + 4;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* k_s = lds;                  // [16][ROW]
    float* q_s = k_s + 16 * ROW;       // [16][ROW]
    float* a_s = q_s + 16 * ROW;       // [16][ROW] (decays per channel only)
    float* red = a_s + (CHANNEL ? 16 * ROW : 0);  // [4 waves][16 t][16 s]; before that the short vectors [16][LIN_LOW]
    __shared__ float pw_s[LIN_BLOCK + 1];
    const int N = in.N, h = blockIdx.y, s = blockIdx.z, first = in.cu_tokens[s];
    const int m0 = first + blockIdx.x * LIN_BLOCK, t1 = in.cu_tokens[s + 1];
    if (m0 >= t1) return;
    const int cnt = min(LIN_BLOCK, t1 - m0);
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const long blk = lin_block_index(first, s, blockIdx.x);
    const T *q = (const T*)in.q + (long)h * N, *k = (const T*)in.k + (long)h * N;
    if (in.rot.inv_freq) {
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            const int t = (tid + j * 256) / NP, n = (tid + j * 256) % NP;
            float kv = 0.f, qv = 0.f;
            if (t < cnt && n < N) {
                const int m = m0 + t;
                const float* freq = lin_freq(in, m);
                const float pos = (float)in.token_pos[m];
                kv = lin_rotated(k + (long)m * in.ld, n, in.rot, freq, pos) * in.k_scale;
                qv = lin_rotated(q + (long)m * in.ld, n, in.rot, freq, pos) * in.q_scale;
            }
            k_s[t * ROW + n] = kv;
            q_s[t * ROW + n] = qv;
        }
    } else {
        float kr[RT], qr[RT];  // all loads in flight at once; what lies past an end is read from inside and put down as nothing
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            const int t = (tid + j * 256) / NP, n = (tid + j * 256) % NP;
            const long at = (long)(m0 + min(t, cnt - 1)) * in.ld + min(n, N - 1);
            kr[j] = Io<T>::ld(k + at);
            qr[j] = Io<T>::ld(q + at);
        }
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            const int t = (tid + j * 256) / NP, n = (tid + j * 256) % NP;
            const bool inside = t < cnt && n < N;
            k_s[t * ROW + n] = inside ? kr[j] * in.k_scale : 0.f;
            q_s[t * ROW + n] = inside ? qr[j] * in.q_scale : 0.f;
        }
    }
    if constexpr (CHANNEL) {
        // z of RT tokens of one channel a thread: the channel's row of A2 against the tokens' short vectors
        const int n = tid % NP, ts = tid / NP * RT;
        const T* a2 = (const T*)in.a2 + ((long)h * N + min(n, N - 1)) * in.rank;
        float z[RT];
#pragma unroll
        for (int j = 0; j < RT; ++j) z[j] = 0.f;
        for (int r0 = 0; r0 < in.rank; r0 += LIN_LOW) {
            const int len = min(LIN_LOW, in.rank - r0);
            __syncthreads();
            for (int i = tid; i < 16 * LIN_LOW; i += 256) {
                const int t = i / LIN_LOW, r = i % LIN_LOW;
                red[i] = r < len ? Io<T>::ld((const T*)in.low + (long)(m0 + min(t, cnt - 1)) * in.ld + r0 + r) : 0.f;
            }
            // (elements past the row's end are read from inside it, and meet zeros)
            float c[LIN_LOW];
            if (sizeof(T) == 2 && in.rank % 8 == 0 && ((uintptr_t)in.a2 & 15) == 0) {
#pragma unroll
                for (int r = 0; r < LIN_LOW; r += 8) {
                    float x[8];
                    unpack8(*reinterpret_cast<const uint4*>((const bf16_t*)a2 + r0 + min(r, len - 8)), x);
#pragma unroll
                    for (int e = 0; e < 8; ++e) c[r + e] = x[e];
                }
            } else {
#pragma unroll
                for (int r = 0; r < LIN_LOW; ++r) c[r] = Io<T>::ld(a2 + r0 + min(r, len - 1));
            }
            __syncthreads();
#pragma unroll
            for (int r = 0; r < LIN_LOW; r += 4) {
                if (r >= len) continue;
#pragma unroll
                for (int j = 0; j < RT; ++j) {
                    const float4 l4 = *reinterpret_cast<const float4*>(red + (ts + j) * LIN_LOW + r);
                    z[j] += c[r] * l4.x + c[r + 1] * l4.y + c[r + 2] * l4.z + c[r + 3] * l4.w;
                }
            }
        }
        const float bias = in.a2_bias[h * N + min(n, N - 1)];
#pragma unroll
        for (int j = 0; j < RT; ++j)
            a_s[(ts + j) * ROW + n] = ts + j < cnt && n < N ? channel_decay(z[j] + bias, in.inv_tau) : 1.f;  // (past an end: nothing changes)
    } else if (tid == 0) {
        const float a = in.decay[h];
        float p = 1.f;
        for (int i = 0; i <= LIN_BLOCK; ++i) { pw_s[i] = p; p *= a; }
    }
    __syncthreads();
    if constexpr (CHANNEL) {
        // thread (token s, RT channels): k'_s carried forward over the later tokens, channel by channel, gives a column of A,
        // summed over the channels by exchanges and through LDS in wave order; what it has become at the end is Kd
        const int st = lane & 15, ch = (wave * 4 + (lane >> 4)) * RT;
        float aq[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) aq[t] = 0.f;
        constexpr int VN = RT < 2 ? RT : 2;
        // (a column of k' is read by its sixteen lanes alone, all of one wave, so Kd can take its place at once; two channels at a
        // time, because the compiler asks for all sixteen tokens' rows at once)
#pragma unroll 1
        for (int c0 = 0; c0 < RT; c0 += VN) {
            float r[VN];
#pragma unroll
            for (int i = 0; i < VN; ++i) r[i] = 0.f;
#pragma unroll
            for (int t = 0; t < 16; ++t) {
#pragma unroll
                for (int i = 0; i < VN; ++i) {
                    const int at = t * ROW + ch + c0 + i;
                    r[i] = t == st ? k_s[at] : r[i] * a_s[at];
                    aq[t] += q_s[at] * r[i];
                }
            }
#pragma unroll
            for (int i = 0; i < VN; ++i) k_s[st * ROW + ch + c0 + i] = r[i];
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            aq[t] += __shfl_xor(aq[t], 16, 64);
            aq[t] += __shfl_xor(aq[t], 32, 64);
            if (lane < 16) red[(wave * 16 + t) * 16 + st] = aq[t];
        }
        __syncthreads();  // q' has been read by all: Q^ takes its place
        if (tid < N) {
            float b = 1.f;
#pragma unroll
            for (int t = 0; t < 16; ++t) {
                b *= a_s[t * ROW + tid];
                q_s[t * ROW + tid] *= b;
            }
            bd[(blk * in.heads + h) * N + tid] = b;
        }
    } else {
        // A without its decays is a product of q' and k' over the channels, a quarter of them a wave
        const int lr = lane & 15, lk = lane >> 4;
        lin_f4 acc = {0.f, 0.f, 0.f, 0.f};
        for (int r = wave; r < RT; r += 4) {
            const float4 a4 = *reinterpret_cast<const float4*>(q_s + lr * ROW + r * 16 + lk * 4);
            const float4 b4 = *reinterpret_cast<const float4*>(k_s + lr * ROW + r * 16 + lk * 4);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.x, b4.x, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.y, b4.y, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.z, b4.z, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a4.w, b4.w, acc, 0, 0, 0);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int t = lk * 4 + e;
            red[(wave * 16 + t) * 16 + lr] = lr <= t ? acc[e] * pw_s[t - lr] : 0.f;
        }
        if (tid < N) bd[(blk * in.heads + h) * N + tid] = pw_s[cnt];
    }
    __syncthreads();
    {
        const int t = tid >> 4, sc = tid & 15;
        float a = 0.f;
#pragma unroll
        for (int wv = 0; wv < 4; ++wv) a += red[(wv * 16 + t) * 16 + sc];
        if (t < cnt) ta[((long)(m0 + t) * in.heads + h) * 16 + sc] = sc <= t ? a : 0.f;
    }
    for (int i = tid; i < cnt * N; i += 256) {
        const int t = i / N, n = i - t * N;
        float* to = hat + ((long)(m0 + t) * in.heads + h) * 2 * N + n;
        to[0] = q_s[t * ROW + n] * (CHANNEL ? 1.f : pw_s[t + 1]);
        to[N] = k_s[t * ROW + n] * (CHANNEL ? 1.f : pw_s[cnt - 1 - t]);
    }
}

// VEC: N is a multiple of four.  hat and ta are readable for a block past their last token (hat for 256 elements more).  A
// workgroup's waves take neighbouring sixteens of columns.
template <typename T, int RT, int MODE, bool VEC>
__global__ __launch_bounds__(512) void lin_scan_kernel(float* __restrict__ y, LinIn in, const float* __restrict__ hat,
                                                       const float* __restrict__ ta, const float* __restrict__ bd,
                                                       float* __restrict__ state, long state_ld, float* __restrict__ chunk_state,
                                                       float* __restrict__ chunk_decay, int chunk, int max_chunks) {
    constexpr int NP = 16 * RT, ROW = NP + 4, TROW = 20;
    constexpr int FIRST = MODE == LIN_LOCAL ? 1 : 0, KINDS = 2 - FIRST;  // (a chunk that makes no outputs needs no Q^)
    constexpr int PIECES = 16 * KINDS * NP / 4;                 // four elements of Q^ or Kd each
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* hat_s = lds;                          // [KINDS][16][ROW]
    float* ta_s = hat_s + KINDS * 16 * ROW;      // [16][TROW]
    float* b_s = ta_s + 16 * TROW;               // [NP]
    const int N = in.N, P = in.P, heads = in.heads, h = blockIdx.y;
    const int s = MODE == LIN_WHOLE ? blockIdx.z : blockIdx.z / max_chunks;
    const int c = MODE == LIN_WHOLE ? 0 : blockIdx.z - s * max_chunks;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, lr = lane & 15, lk = lane >> 4, threads = blockDim.x;
    const int p = (blockIdx.x * (threads >> 6) + wave) * 16 + lr;
    const int first = in.cu_tokens[s];
    int t0 = first, t1 = in.cu_tokens[s + 1];
    if (MODE != LIN_WHOLE) {
        t0 += c * chunk;
        if (t0 >= t1) return;  // the sequence has fewer chunks
        t1 = min(t1, t0 + chunk);
    }
    float* sb = MODE == LIN_WHOLE ? state + (long)in.seq_slot[s] * state_ld + (long)h * N * P
                                  : chunk_state + ((long)blockIdx.z * heads + h) * N * P;
    lin_f4 S[RT];
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = r * 16 + lk * 4 + e;
            S[r][e] = (MODE != LIN_LOCAL && n < N && p < P) ? sb[(long)n * P + p] : 0.f;
        }
    float decay = 1.f;  // of row tid over the chunk
    // What a block needs is asked for one block ahead.  The loads branch on nothing: rows past the sequence's end are read
    // (they lie within the buffers) and elements past a row's end are read from inside the row, and both are put down as zeros.
    constexpr int MOST = (PIECES + 255) / 256;  // (a workgroup has at least four waves)
    float4 ph[MOST];
    float pt = 0.f, pb = 1.f, pv[4];
    const int per = (PIECES + threads - 1) / threads;
    auto piece = [&](int j, int& which, int& t, int& n) {
        const int i = min(tid + j * threads, PIECES - 1);
        t = i / (KINDS * NP / 4);
        const int rest = i - t * (KINDS * NP / 4);
        which = rest / (NP / 4);
        n = (rest - which * (NP / 4)) * 4;
    };
    auto fetch = [&](int m0) {
        const float* hb = hat + ((long)m0 * heads + h) * 2 * N;
#pragma unroll
        for (int j = 0; j < MOST; ++j) {
            if (j >= per) break;
            int which, t, n;
            piece(j, which, t, n);
            const float* from = hb + (long)t * heads * 2 * N + (which + FIRST) * N;
            if constexpr (VEC) ph[j] = *reinterpret_cast<const float4*>(from + min(n, N - 4));
            else ph[j] = make_float4(from[n], from[n + 1], from[n + 2], from[n + 3]);  // (may lie in the next vector or token)
        }
        if (MODE != LIN_LOCAL && tid < 256) pt = ta[((long)(m0 + (tid >> 4)) * heads + h) * 16 + (tid & 15)];
        pb = tid < NP ? bd[(lin_block_index(first, s, (m0 - first) / LIN_BLOCK) * heads + h) * N + min(tid, N - 1)] : 1.f;
        const T* vb = (const T*)in.v + (long)m0 * in.ld + (long)h * P + min(p, P - 1);
#pragma unroll
        for (int e = 0; e < 4; ++e) pv[e] = Io<T>::ld(vb + (long)min(lk * 4 + e, t1 - 1 - m0) * in.ld);
    };
    fetch(t0);
    for (int m0 = t0; m0 < t1; m0 += LIN_BLOCK) {
        const int cnt = t1 - m0;  // (from sixteen on: a whole block)
        __syncthreads();
#pragma unroll
        for (int j = 0; j < MOST; ++j) {
            if (j >= per) break;
            int which, t, n;
            piece(j, which, t, n);
            const bool inside = n < N && t < cnt;
            const float4 f = make_float4(inside ? ph[j].x : 0.f, inside && (VEC || n + 1 < N) ? ph[j].y : 0.f,
                                         inside && (VEC || n + 2 < N) ? ph[j].z : 0.f, inside && (VEC || n + 3 < N) ? ph[j].w : 0.f);
            if (tid + j * threads < PIECES) *reinterpret_cast<float4*>(hat_s + (which * 16 + t) * ROW + n) = f;
        }
        if (MODE != LIN_LOCAL && tid < 256) ta_s[(tid >> 4) * TROW + (tid & 15)] = (tid >> 4) < cnt ? pt : 0.f;
        if (tid < NP) {
            b_s[tid] = tid < N ? pb : 0.f;
            decay *= pb;
        }
        lin_f4 O0 = {0.f, 0.f, 0.f, 0.f}, O1 = {0.f, 0.f, 0.f, 0.f};
        float V[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) V[e] = lk * 4 + e < cnt && p < P ? pv[e] : 0.f;
        __syncthreads();
        if (cnt > LIN_BLOCK) fetch(m0 + LIN_BLOCK);
        if (MODE != LIN_LOCAL) {
            const float* qh_row = hat_s + lr * ROW + lk * 4;
#pragma unroll
            for (int r = 0; r < RT; ++r) {
                const float4 a4 = *reinterpret_cast<const float4*>(qh_row + r * 16);
                const float a[4] = {a4.x, a4.y, a4.z, a4.w};
                lin_f4& O = (r & 1) ? O1 : O0;
#pragma unroll
                for (int e = 0; e < 4; ++e) O = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], S[r][e], O, 0, 0, 0);
            }
            const float4 a4 = *reinterpret_cast<const float4*>(ta_s + lr * TROW + lk * 4);
            const float a[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) O0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], V[e], O0, 0, 0, 0);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int m = m0 + lk * 4 + e;
                if (m < t1 && p < P) y[((long)m * heads + h) * P + p] = O0[e] + O1[e];
            }
        }
        const float* kd = hat_s + (1 - FIRST) * 16 * ROW + lk * 4 * ROW + lr;
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const float4 b4 = *reinterpret_cast<const float4*>(b_s + r * 16 + lk * 4);
            S[r][0] *= b4.x; S[r][1] *= b4.y; S[r][2] *= b4.z; S[r][3] *= b4.w;
#pragma unroll
            for (int e = 0; e < 4; ++e) S[r] = __builtin_amdgcn_mfma_f32_16x16x4f32(kd[e * ROW + r * 16], V[e], S[r], 0, 0, 0);
        }
    }
    if (MODE != LIN_OUTPUT) {
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = r * 16 + lk * 4 + e;
                if (n < N && p < P) sb[(long)n * P + p] = S[r][e];
            }
    }
    if (MODE == LIN_LOCAL && blockIdx.x == 0 && tid < N) chunk_decay[((long)blockIdx.z * heads + h) * N + tid] = decay;
}

// chunk after chunk: what a chunk starts from takes the place of what it adds; the sequence's state moves to its end
__global__ void lin_carry_kernel(float* __restrict__ state, long state_ld, float* __restrict__ chunk_state,
                                 const float* __restrict__ chunk_decay, const int* __restrict__ cu_tokens,
                                 const int* __restrict__ seq_slot, int heads, int P, int N, int chunk, int max_chunks) {
    const long e = (long)blockIdx.x * blockDim.x + threadIdx.x;  // element of the sequence's state
    const int s = blockIdx.y;
    const long step = (long)heads * N * P;  // from a chunk's element to the next chunk's
    if (e >= step) return;
    const long row = e / P;  // (head, key channel)
    const int n_chunks = (cu_tokens[s + 1] - cu_tokens[s] + chunk - 1) / chunk;
    float* sp = state + (long)seq_slot[s] * state_ld + e;
    float S = *sp;
    float* cs = chunk_state + (long)s * max_chunks * step + e;
    const float* cd = chunk_decay + (long)s * max_chunks * heads * N + row;
    // eight chunks' additions are asked for at once: the walk itself is a chain, its loads need not be
    for (int c0 = 0; c0 < n_chunks; c0 += 8) {
        float add[8], dec[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int c = min(c0 + j, n_chunks - 1);
            add[j] = cs[(long)c * step];
            dec[j] = cd[(long)c * heads * N];
        }
#pragma unroll
        for (int j = 0; j < 8; ++j)
            if (c0 + j < n_chunks) {
                cs[(long)(c0 + j) * step] = S;
                S = dec[j] * S + add[j];
            }
    }
    *sp = S;
}

struct LinLaunch {
    void* out; long out_ld; float* y; LinIn in;
    const float* w; float eps, mult;
    float* state; long state_ld;
    float *hat, *ta, *bd, *chunk_state, *chunk_decay;
    int n_seqs, max_new, chunk, max_chunks, M, dtype;
    hipStream_t s;
};

template <typename T, int NPT, bool CHANNEL>
static int launch_lin_steps(const LinLaunch& d) {
    const int piece = std::min(d.max_new, LIN_PIECE), waves = (d.in.P + 15) / 16;
    const size_t lds = (size_t)piece * ((CHANNEL ? 3 : 2) * 4 * (NPT + 4) + waves * 16) * sizeof(float);
    static_assert(LIN_PIECE * (3 * 4 * (NPT + 4) + 256) * 4 <= 80 * 1024, "a piece's rows fit the LDS");
    auto kern = waves <= 8 ? lin_step_kernel<T, NPT, CHANNEL, 512> : lin_step_kernel<T, NPT, CHANNEL, 1024>;
    if (lds > 62 * 1024)  // more than a launch may ask for unless the kernel has been told
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(kern, dim3(d.in.heads, d.n_seqs), dim3(64 * waves), lds, d.s, (T*)d.out, d.out_ld, d.in,
                       d.w, d.eps, d.mult, d.state, d.state_ld, piece);
    return pta_check_launch("linear_state");
}

template <typename T, int RT, bool CHANNEL>
static int launch_lin_blocks(const LinLaunch& d) {
    constexpr size_t block_lds = (size_t)((CHANNEL ? 3 : 2) * 16 * (16 * RT + 4) + 4 * 256) * sizeof(float);
    constexpr size_t scan_lds = (size_t)(2 * 16 * (16 * RT + 4) + 16 * 20 + 16 * RT) * sizeof(float);
    static_assert(block_lds <= 62 * 1024 && scan_lds <= 62 * 1024, "a block's rows fit the LDS that a launch may ask for without saying so");
    hipLaunchKernelGGL((lin_block_kernel<T, RT, CHANNEL>), dim3((d.max_new + LIN_BLOCK - 1) / LIN_BLOCK, d.in.heads, d.n_seqs), dim3(256), block_lds,
                       d.s, d.hat, d.ta, d.bd, d.in);
    // waves of a workgroup: all columns of a head if there are at most 128; at least four, which stage what a block needs
    const int waves = std::min(8, std::max(4, (d.in.P + 15) / 16));
    const int cols = (d.in.P + waves * 16 - 1) / (waves * 16);
#define LIN_SCAN(MODE_, RUNS_)                                                                                                        \
    hipLaunchKernelGGL((d.in.N % 4 ? lin_scan_kernel<T, RT, MODE_, false> : lin_scan_kernel<T, RT, MODE_, true>),                       \
                       dim3(cols, d.in.heads, (RUNS_)), dim3(64 * waves), scan_lds, d.s, d.y, d.in, d.hat, d.ta, d.bd, d.state, d.state_ld, \
                       d.chunk_state, d.chunk_decay, d.chunk, d.max_chunks)
    if (d.max_chunks <= 1) {
        LIN_SCAN(LIN_WHOLE, d.n_seqs);
        return pta_check_launch("linear_state");
    }
    LIN_SCAN(LIN_LOCAL, d.n_seqs * d.max_chunks);
    const long elements = (long)d.in.heads * d.in.N * d.in.P;
    hipLaunchKernelGGL(lin_carry_kernel, dim3((unsigned)((elements + 255) / 256), d.n_seqs), dim3(256), 0, d.s, d.state, d.state_ld, d.chunk_state,
                       d.chunk_decay, d.in.cu_tokens, d.in.seq_slot, d.in.heads, d.in.P, d.in.N, d.chunk, d.max_chunks);
    LIN_SCAN(LIN_OUTPUT, d.n_seqs * d.max_chunks);
#undef LIN_SCAN
    return pta_check_launch("linear_state");
}

template <typename T, bool CHANNEL>
static int launch_lin(const LinLaunch& d) {
    const int N = d.in.N;
    if (d.hat) {
        if (N <= 16) return launch_lin_blocks<T, 1, CHANNEL>(d);
        if (N <= 32) return launch_lin_blocks<T, 2, CHANNEL>(d);
        if (N <= 64) return launch_lin_blocks<T, 4, CHANNEL>(d);
        if (N <= 128) return launch_lin_blocks<T, 8, CHANNEL>(d);
        return launch_lin_blocks<T, 16, CHANNEL>(d);
    }
    if (N <= 16) return launch_lin_steps<T, 4, CHANNEL>(d);
    if (N <= 32) return launch_lin_steps<T, 8, CHANNEL>(d);
    if (N <= 64) return launch_lin_steps<T, 16, CHANNEL>(d);
    if (N <= 128) return launch_lin_steps<T, 32, CHANNEL>(d);
    return launch_lin_steps<T, 64, CHANNEL>(d);
}

// out [M, heads * P] (compute type, rows out_ld apart).  decay [heads], or low [M, rank] with a2 [heads * N, rank] (compute type)
// and a2_bias [heads * N].  hat [(M + 16) * heads * 2 * N + 256], ta [M + 16, heads, 16], bd [M / 16 + n_seqs + 1, heads, N] and y [M,
// heads * P] given (scratch, 32-bit): blocks of sixteen tokens; without them the tokens are walked one by one.  chunk_state [n_seqs
// * max_chunks, heads, N, P] and chunk_decay [n_seqs * max_chunks, heads, N] are scratch for steps whose longest sequence is cut
// into max_chunks > 1 chunks of `chunk` tokens (a multiple of 16).
extern "C" int pta_linear_state(void* out, long out_ld, float* y, const void* q, const void* k, const void* v, const void* g, long ld,
                                float q_scale, float k_scale, const PtaRotation* rotation, const float* decay, const void* low,
                                const void* a2, const float* a2_bias, int rank, float inv_tau, const float* w, float eps, float mult,
                                float* state, long state_ld, float* hat, float* ta, float* bd, float* chunk_state, float* chunk_decay,
                                const int* token_pos, const int* token_seq, const int* cu_tokens, const int* seq_slot, int n_seqs,
                                int max_new, int M, int heads, int P, int N, int chunk, int max_chunks, int dtype, void* stream) {
    PTA_REQUIRE(n_seqs > 0 && max_new > 0 && M > 0 && heads > 0 && P > 0 && N > 0, "linear_state: sizes must be positive");
    PTA_REQUIRE(N <= 256 && P <= 256, "linear_state: keys of %d and values of %d elements are more than the 256 the kernels hold", N, P);
    PTA_REQUIRE(heads <= 65535 && n_seqs <= 65535, "linear_state: too many heads or sequences for one launch");
    PTA_REQUIRE(out && q && k && v && g && state && token_pos && token_seq && cu_tokens && seq_slot, "linear_state: null pointer");
    PTA_REQUIRE((decay != nullptr) != (low != nullptr) && (!low || (a2 && a2_bias && rank > 0 && ld >= rank)),
                "linear_state: a constant per head, or a short vector with its matrix and bias");
    PTA_REQUIRE(ld >= (long)heads * N && ld >= (long)heads * P && out_ld >= (long)heads * P && state_ld >= (long)heads * N * P,
                "linear_state: rows lie closer together than they are long");
    PTA_REQUIRE((hat == nullptr) == (ta == nullptr) && (hat == nullptr) == (bd == nullptr) && (hat == nullptr) == (y == nullptr),
                "linear_state: blocks need all of their scratch memory");
    PTA_REQUIRE(max_chunks >= 1 && (max_chunks == 1 || (hat && chunk > 0 && chunk % LIN_BLOCK == 0 && chunk_state && chunk_decay &&
                                                        (long)max_chunks * chunk >= max_new)),
                "linear_state: chunks need their size, a multiple of %d, enough of them and scratch memory", LIN_BLOCK);
    PTA_REQUIRE((long)n_seqs * max_chunks <= 65535, "linear_state: %ld chunks are more than one launch takes", (long)n_seqs * max_chunks);
    PTA_REQUIRE(((uintptr_t)hat % 16) == 0, "linear_state: scratch memory must be 16-byte aligned");
    PTA_REQUIRE(dtype == PTA_F32 || dtype == PTA_BF16, "linear_state: unknown dtype %d", dtype);
    const PtaRotation rot = pta_rotation_of(rotation);
    if (pta_check_rotation("linear_state", rot, N, token_seq)) return 1;
    LinLaunch d{out, out_ld, y,
                LinIn{q, k, v, g, low, a2, ld, q_scale, k_scale, inv_tau, rot, token_pos, token_seq, cu_tokens, seq_slot, decay, a2_bias, rank, heads, P, N},
                w, eps, mult, state, state_ld, hat, ta, bd, chunk_state, chunk_decay, n_seqs, max_new, chunk, max_chunks, M, dtype,
                (hipStream_t)stream};
    int rc;
    if (dtype == PTA_F32) rc = low ? launch_lin<float, true>(d) : launch_lin<float, false>(d);
    else rc = low ? launch_lin<bf16_t, true>(d) : launch_lin<bf16_t, false>(d);
    if (rc || !hat) return rc;
    return pta_head_norm_gate(out, out_ld, y, g, ld, w, eps, PTA_ACT_SILU, mult, M, heads, P, dtype, stream);
}
