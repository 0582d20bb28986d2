// A real-gated linear recurrent unit with its convolution and gates, per channel of `blocks` equal parts of W channels:
//
//   u = conv_b + sum_k conv[k] * (x + x_b) of taps - 1 - k tokens ago        (the last tap is the token's own; zeros before the start)
//   r = sigmoid(Wr u_part + br), i = sigmoid(Wi u_part + bi)                 square matrices of a part's size, one pair a part
//   log a = rate * r * softplus(lam);  S <- a S + sqrt(1 - a^2) * i * u
//   out = S * gelu_tanh(y + y_b)
//
// x and y are blocks of columns of one product (compute type); everything between them and out is 32-bit, the gates' products
// included: in bfloat16 models u is split into three bfloat16 numbers whose sum it is to the last bit, each multiplied with the
// (bfloat16) gate matrices on the matrix cores; in 32-bit models the products are 32-bit matrix products.
//
// The convolution's earlier inputs of a sequence are a ring of `taps` rows of W channels (the input at position p lies in row p
// mod taps): in a step of one token per sequence the rows that are read and the one that is written differ, so many
// workgroups can read them while one writes.
//
// rglru_gates_kernel: a workgroup of four waves owns a tile of tokens and 64 channels of a part; a wave sixteen of them, both
// gates.  u of the tile is formed 64 channels of the part at a time in LDS.  The launch leaves a and sqrt(1 - a^2) i u per (token,
// channel) for the recurrence, which runs whole (RGLRU_WHOLE) or in chunks side by side (RGLRU_LOCAL: each from zero, with the
// product of its a; carry; RGLRU_OUTPUT).
// rglru_step_kernel: the same for steps of one token per sequence, through to the states, the rings and the output in one launch;
// u is formed 256 channels at a time, every load branching on nothing so that all are in flight together.
#include "common.h"
#include "pta_kernels.h"

#define RGLRU_MAX_TAPS 16
#define RGLRU_K 64   // channels of a part that are staged at once
enum { RGLRU_WHOLE = 0, RGLRU_LOCAL = 1, RGLRU_OUTPUT = 2 };

typedef __bf16 rg_bf16x8 __attribute__((ext_vector_type(8)));
typedef float rg_f4 __attribute__((ext_vector_type(4)));
union RgFrag { uint4 u; rg_bf16x8 v; };

__device__ __forceinline__ float rg_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float rg_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float rg_gelu(float x) { return apply_act(x, PTA_ACT_GELU_TANH); }

struct RgIn {
    const void *y, *x, *gates;
    long ld, state_ld;
    const float *y_bias, *x_bias, *conv, *conv_bias, *r_bias, *i_bias, *lam;
    float rate;
    float *state, *ring;
    const int *token_pos, *token_seq, *cu_tokens, *seq_slot;
    int n_seqs, M, W, part, padded, taps;
};

// u of token m, channel ch
template <typename T, int KMAX>
__device__ __forceinline__ float rg_conv(const RgIn& in, int m, int ch, const float (&w)[KMAX], float xb, float cb) {
    const T* x = (const T*)in.x + ch;
    const int s = in.token_seq[m];
    const int pos = in.token_pos[m], j = m - in.cu_tokens[s];
    const float* ring = in.ring + (long)in.seq_slot[s] * in.state_ld + ch;
    float acc = cb;
#pragma unroll
    for (int kk = 0; kk < KMAX; ++kk) {  // (fewer taps: nothing in front)
        const int back = KMAX - 1 - kk;
        if (back >= in.taps) continue;
        float v = 0.f;
        if (back <= j) v = Io<T>::ld(x + (long)(m - back) * in.ld) + xb;
        else if (back <= pos) v = ring[(long)((pos - back) % in.taps) * in.W];
        acc += w[kk] * v;
    }
    return acc;
}

// a number as three bfloat16 numbers whose sum it is
__device__ __forceinline__ void rg_split(float v, bf16_t& hi, bf16_t& mid, bf16_t& lo) {
    hi = f32_to_bf16_bits(v);
    const float rest = v - bf16_bits_to_f32(hi);
    mid = f32_to_bf16_bits(rest);
    lo = f32_to_bf16_bits(rest - bf16_bits_to_f32(mid));
}

// what the two gates of a channel make of u: the decay and the addend
__device__ __forceinline__ void rg_coefficients(float r, float i, float u, float slope, float& a, float& add) {
    const float log_a = slope * rg_sigmoid(r);
    a = expf(log_a);
    add = sqrtf(-expm1f(2.f * log_a)) * rg_sigmoid(i) * u;
}

// TG: groups of sixteen tokens a workgroup takes
template <typename T, int TG, int KMAX>
__global__ __launch_bounds__(256) void rglru_gates_kernel(float* __restrict__ coef, RgIn in) {
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int TT = TG * 16, UROW = RGLRU_K + 4, PROW = RGLRU_K + 8;
    // 32-bit: u [TT][UROW]; bfloat16: three planes [TT][PROW]
    constexpr int LDS_BYTES = F32 ? TT * UROW * 4 : 3 * TT * PROW * 2;
    __shared__ __attribute__((aligned(16))) char lds[LDS_BYTES];
    __shared__ __attribute__((aligned(16))) float own_s[TT * UROW];  // u of the workgroup's own channels
    float* u_s = reinterpret_cast<float*>(lds);
    bf16_t* p_s = reinterpret_cast<bf16_t*>(lds);
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = lane & 15, gq = lane >> 4;
    const int b = blockIdx.y, m0 = blockIdx.z * TT, m1 = min(in.M, m0 + TT);
    const int row0 = blockIdx.x * 64 + wave * 16;   // first of the wave's channels within the part
    const bool live = row0 < in.padded;             // (the padded rows of the gate matrices are zeros)
    const T* G = (const T*)in.gates + (long)b * 2 * in.padded * in.padded;
    const T* rrow = G + (long)min(row0 + c, in.padded - 1) * in.padded + gq * (F32 ? 4 : 8);
    const T* irow = rrow + (long)in.padded * in.padded;
    rg_f4 ar[TG], ai[TG];
#pragma unroll
    for (int g = 0; g < TG; ++g) ar[g] = ai[g] = rg_f4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < in.padded; k0 += RGLRU_K) {
        const int kn = min(RGLRU_K, in.padded - k0);  // a multiple of 32
        // the gate rows' pieces are asked for before u is formed
        RgFrag wr[2], wi[2];
        float4 fr[4], fi[4];
        if constexpr (!F32) {
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                const int at = k0 + min(ks * 32, kn - 32);
                wr[ks].u = *reinterpret_cast<const uint4*>((const bf16_t*)rrow + at);
                wi[ks].u = *reinterpret_cast<const uint4*>((const bf16_t*)irow + at);
            }
        } else {
#pragma unroll
            for (int ks = 0; ks < 4; ++ks) {
                const int at = k0 + min(ks * 16, kn - 16);
                fr[ks] = *reinterpret_cast<const float4*>((const float*)rrow + at);
                fi[ks] = *reinterpret_cast<const float4*>((const float*)irow + at);
            }
        }
        __syncthreads();
        {   // a thread forms u of one channel for TT / 4 neighbouring tokens
            const int kk = tid & 63, tq = (tid >> 6) * (TT / 4), ch = k0 + kk;
            const bool in_part = ch < in.part;
            const int gch = b * in.part + min(ch, in.part - 1);
            float w[KMAX];
#pragma unroll
            for (int k = 0; k < KMAX; ++k) w[k] = k >= KMAX - in.taps ? in.conv[(long)(k - (KMAX - in.taps)) * in.W + gch] : 0.f;
            const float xb = in.x_bias ? in.x_bias[gch] : 0.f, cb = in.conv_bias ? in.conv_bias[gch] : 0.f;
            constexpr int U = TT / 4 < 8 ? TT / 4 : 8;  // tokens whose inputs are held at once
#pragma unroll 1
            for (int t0 = 0; t0 < TT / 4; t0 += U) {
                float u[U];
                const int ma = m0 + tq + t0;
                bool inside = false;  // every input of these tokens is a row of this step: they are then asked for all at once
                if (KMAX <= 4 && ma + U <= m1) {
                    const int s = in.token_seq[ma];
                    inside = s == in.token_seq[ma + U - 1] && ma - in.cu_tokens[s] >= KMAX - 1;
                }
                if (inside) {
                    float x[U + KMAX - 1];
#pragma unroll
                    for (int i = 0; i < U + KMAX - 1; ++i)
                        x[i] = Io<T>::ld((const T*)in.x + (long)(ma - (KMAX - 1) + i) * in.ld + gch) + xb;
#pragma unroll
                    for (int t = 0; t < U; ++t) {
                        u[t] = cb;
#pragma unroll
                        for (int k = 0; k < KMAX; ++k) u[t] += w[k] * x[t + k];
                    }
                } else {
#pragma unroll
                    for (int t = 0; t < U; ++t) u[t] = ma + t < m1 ? rg_conv<T, KMAX>(in, ma + t, gch, w, xb, cb) : 0.f;
                }
#pragma unroll
                for (int t = 0; t < U; ++t) {
                    const float v = in_part ? u[t] : 0.f;
                    const int row = tq + t0 + t;
                    if (k0 == (int)blockIdx.x * RGLRU_K) own_s[row * UROW + kk] = v;
                    if constexpr (F32) {
                        u_s[row * UROW + kk] = v;
                    } else {
                        bf16_t* to = p_s + row * PROW + kk;
                        rg_split(v, to[0], to[TT * PROW], to[2 * TT * PROW]);
                    }
                }
            }
        }
        __syncthreads();
        if (live) {
            if constexpr (!F32) {
#pragma unroll
                for (int ks = 0; ks < 2; ++ks) {
                    if (ks * 32 >= kn) continue;
#pragma unroll
                    for (int pl = 2; pl >= 0; --pl)  // the small parts first
#pragma unroll
                        for (int g = 0; g < TG; ++g) {
                            RgFrag f;
                            f.u = *reinterpret_cast<const uint4*>(p_s + (pl * TT + g * 16 + c) * PROW + ks * 32 + gq * 8);
                            ar[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wr[ks].v, f.v, ar[g], 0, 0, 0);
                            ai[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wi[ks].v, f.v, ai[g], 0, 0, 0);
                        }
                }
            } else {
#pragma unroll
                for (int ks = 0; ks < 4; ++ks) {
                    if (ks * 16 >= kn) continue;
                    const float r4[4] = {fr[ks].x, fr[ks].y, fr[ks].z, fr[ks].w}, i4[4] = {fi[ks].x, fi[ks].y, fi[ks].z, fi[ks].w};
#pragma unroll
                    for (int g = 0; g < TG; ++g) {
                        const float4 f = *reinterpret_cast<const float4*>(u_s + (g * 16 + c) * UROW + ks * 16 + gq * 4);
                        const float f4[4] = {f.x, f.y, f.z, f.w};
#pragma unroll
                        for (int e = 0; e < 4; ++e) {
                            ar[g] = __builtin_amdgcn_mfma_f32_16x16x4f32(r4[e], f4[e], ar[g], 0, 0, 0);
                            ai[g] = __builtin_amdgcn_mfma_f32_16x16x4f32(i4[e], f4[e], ai[g], 0, 0, 0);
                        }
                    }
                }
            }
        }
    }
    // acc[g][j]: channel row0 + 4 gq + j of the token in column c of group g
    const int row = row0 + 4 * gq, many = min(4, in.part - row);
    if (many <= 0) return;
    const int ch = b * in.part + row;
    float slope[4], br[4], bi[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int at = ch + min(j, many - 1);
        slope[j] = in.rate * rg_softplus(in.lam[at]), br[j] = in.r_bias[at], bi[j] = in.i_bias[at];
    }
#pragma unroll
    for (int g = 0; g < TG; ++g) {
        const int m = m0 + g * 16 + c;
        if (m >= m1) continue;
        const float4 u4 = *reinterpret_cast<const float4*>(own_s + (g * 16 + c) * UROW + wave * 16 + 4 * gq);
        const float u[4] = {u4.x, u4.y, u4.z, u4.w};
        float a[4], add[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) rg_coefficients(ar[g][j] + br[j], ai[g][j] + bi[j], u[j], slope[j], a[j], add[j]);
        float* to = coef + ((long)m * in.W + ch) * 2;
        if (many == 4 && ((uintptr_t)to & 15) == 0) {
            *reinterpret_cast<float4*>(to) = make_float4(a[0], add[0], a[1], add[1]);
            *reinterpret_cast<float4*>(to + 4) = make_float4(a[2], add[2], a[3], add[3]);
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (j < many) *reinterpret_cast<float2*>(to + 2 * j) = make_float2(a[j], add[j]);
        }
    }
}

// One token per sequence, sixteen sequences and 64 channels of a part a workgroup.
#define RGLRU_STEP_K 256

template <typename T, int KMAX>
__global__ __launch_bounds__(256) void rglru_step_kernel(T* __restrict__ out, RgIn in) {
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int TT = 16, UROW = RGLRU_STEP_K + 4, PROW = RGLRU_STEP_K + 8, OROW = 64 + 4;
    constexpr int LDS_BYTES = F32 ? TT * UROW * 4 : 3 * TT * PROW * 2;
    __shared__ __attribute__((aligned(16))) char lds[LDS_BYTES];
    __shared__ __attribute__((aligned(16))) float own_s[TT * OROW];  // u of the workgroup's own channels
    float* u_s = reinterpret_cast<float*>(lds);
    bf16_t* p_s = reinterpret_cast<bf16_t*>(lds);
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = lane & 15, gq = lane >> 4;
    const int b = blockIdx.y, m0 = blockIdx.z * TT, cnt = min(TT, in.M - m0);
    const int row0 = blockIdx.x * 64 + wave * 16;
    const bool live = row0 < in.padded;
    const T* G = (const T*)in.gates + (long)b * 2 * in.padded * in.padded;
    const T* rrow = G + (long)min(row0 + c, in.padded - 1) * in.padded + gq * (F32 ? 4 : 8);
    const T* irow = rrow + (long)in.padded * in.padded;
    // what the end of the launch needs of this lane's four channels and token is asked for at its beginning (lanes past an end
    // ask for what their neighbours do)
    const int row = row0 + 4 * gq, many = min(4, in.part - row);
    const int ch0 = b * in.part + min(row, in.part - 1), m = m0 + min(c, cnt - 1);
    float* sp = in.state + (long)in.seq_slot[m] * in.state_ld + ch0;
    float* ring_to = in.ring + (long)in.seq_slot[m] * in.state_ld + (long)(in.token_pos[m] % in.taps) * in.W + ch0;
    float S[4], xv[4], yv[4], slope[4], br[4], bi[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int at = max(min(j, many - 1), 0);
        S[j] = sp[at];
        xv[j] = Io<T>::ld((const T*)in.x + (long)m * in.ld + ch0 + at);
        yv[j] = Io<T>::ld((const T*)in.y + (long)m * in.ld + ch0 + at);
        slope[j] = in.lam[ch0 + at], br[j] = in.r_bias[ch0 + at], bi[j] = in.i_bias[ch0 + at];
        if (in.x_bias) xv[j] += in.x_bias[ch0 + at];
        if (in.y_bias) yv[j] += in.y_bias[ch0 + at];
    }
    rg_f4 ar = {0.f, 0.f, 0.f, 0.f}, ai = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < in.padded; k0 += RGLRU_STEP_K) {
        const int kn = min(RGLRU_STEP_K, in.padded - k0);
        RgFrag wr[F32 ? 1 : 8], wi[F32 ? 1 : 8];
        if constexpr (!F32) {  // the gate rows' pieces are asked for before u is formed
#pragma unroll
            for (int ks = 0; ks < 8; ++ks) {
                const int at = k0 + min(ks * 32, kn - 32);
                wr[ks].u = *reinterpret_cast<const uint4*>((const bf16_t*)rrow + at);
                wi[ks].u = *reinterpret_cast<const uint4*>((const bf16_t*)irow + at);
            }
        }
        const int ch = k0 + tid, gch = b * in.part + min(ch, in.part - 1);
        const bool in_part = ch < in.part;
        float w[KMAX];
#pragma unroll
        for (int k = 0; k < KMAX; ++k) w[k] = in.conv[(long)max(k - (KMAX - in.taps), 0) * in.W + gch];
        const float xb = in.x_bias ? in.x_bias[gch] : 0.f, cb = in.conv_bias ? in.conv_bias[gch] : 0.f;
        __syncthreads();
        constexpr int U = KMAX <= 4 ? 8 : 2;  // tokens whose loads are in flight together
#pragma unroll 1
        for (int t0 = 0; t0 < TT; t0 += U) {
            float x[U], r[U][KMAX];
            int pos[U];
            if (t0 < cnt) {
#pragma unroll
                for (int i = 0; i < U; ++i) {
                    const int mi = m0 + min(t0 + i, cnt - 1);
                    pos[i] = in.token_pos[mi];
                    const int p0 = pos[i] % in.taps;
                    const float* ring = in.ring + (long)in.seq_slot[mi] * in.state_ld + gch;
                    x[i] = Io<T>::ld((const T*)in.x + (long)mi * in.ld + gch);
#pragma unroll
                    for (int back = 1; back < KMAX; ++back) {
                        const int at = p0 - back + (p0 < back ? in.taps : 0);
                        r[i][back] = ring[(long)max(at, 0) * in.W];
                    }
                }
            }
#pragma unroll
            for (int i = 0; i < U; ++i) {
                float v = 0.f;
                if (t0 + i < cnt && in_part) {
                    v = cb;
#pragma unroll
                    for (int back = KMAX - 1; back >= 1; --back)
                        v += (back < in.taps && back <= pos[i]) ? w[KMAX - 1 - back] * r[i][back] : 0.f;
                    v += w[KMAX - 1] * (x[i] + xb);
                }
                if (ch >= (int)blockIdx.x * 64 && ch < (int)blockIdx.x * 64 + 64) own_s[(t0 + i) * OROW + (ch & 63)] = v;
                if constexpr (F32) {
                    u_s[(t0 + i) * UROW + tid] = v;
                } else {
                    bf16_t* to = p_s + (t0 + i) * PROW + tid;
                    rg_split(v, to[0], to[TT * PROW], to[2 * TT * PROW]);
                }
            }
        }
        __syncthreads();
        if (live) {
            if constexpr (!F32) {
#pragma unroll
                for (int pl = 2; pl >= 0; --pl)  // the small parts first
#pragma unroll
                    for (int ks = 0; ks < 8; ++ks) {
                        if (ks * 32 >= kn) continue;
                        RgFrag f;
                        f.u = *reinterpret_cast<const uint4*>(p_s + (pl * TT + c) * PROW + ks * 32 + gq * 8);
                        ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wr[ks].v, f.v, ar, 0, 0, 0);
                        ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wi[ks].v, f.v, ai, 0, 0, 0);
                    }
            } else {
                for (int k = 0; k < kn; k += 16) {
                    const float4 r = *reinterpret_cast<const float4*>((const float*)rrow + k0 + k), i = *reinterpret_cast<const float4*>((const float*)irow + k0 + k);
                    const float4 f = *reinterpret_cast<const float4*>(u_s + c * UROW + k + gq * 4);
                    const float r4[4] = {r.x, r.y, r.z, r.w}, i4[4] = {i.x, i.y, i.z, i.w}, f4[4] = {f.x, f.y, f.z, f.w};
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        ar = __builtin_amdgcn_mfma_f32_16x16x4f32(r4[e], f4[e], ar, 0, 0, 0);
                        ai = __builtin_amdgcn_mfma_f32_16x16x4f32(i4[e], f4[e], ai, 0, 0, 0);
                    }
                }
            }
        }
    }
    if (many <= 0 || c >= cnt) return;
    T* o = out + (long)m * in.W + ch0;
    const float4 u4 = *reinterpret_cast<const float4*>(own_s + c * OROW + wave * 16 + 4 * gq);
    const float u[4] = {u4.x, u4.y, u4.z, u4.w};
#pragma unroll
    for (int j = 0; j < 4; ++j)
        if (j < many) {
            float a, add;
            rg_coefficients(ar[j] + br[j], ai[j] + bi[j], u[j], in.rate * rg_softplus(slope[j]), a, add);
            S[j] = a * S[j] + add;
            sp[j] = S[j];
            ring_to[j] = xv[j];
            Io<T>::st(o + j, S[j] * rg_gelu(yv[j]));
        }
}

// the last taps - 1 inputs of every sequence's tokens of the step into its ring (the others' places are not read again)
template <typename T>
__global__ void rglru_ring_kernel(RgIn in) {
    const int ch = blockIdx.x * blockDim.x + threadIdx.x, s = blockIdx.y;
    if (ch >= in.W) return;
    const int first = in.cu_tokens[s], end = in.cu_tokens[s + 1];
    const float xb = in.x_bias ? in.x_bias[ch] : 0.f;
    float* ring = in.ring + (long)in.seq_slot[s] * in.state_ld + ch;
    for (int m = max(first, end - (in.taps - 1)); m < end; ++m)
        ring[(long)(in.token_pos[m] % in.taps) * in.W] = Io<T>::ld((const T*)in.x + (long)m * in.ld + ch) + xb;
}

// coef [M, W, 2]: a and the addend.  A thread per (run of tokens, channel); UNROLL tokens' loads are in flight together.
template <typename T, int UNROLL, int MODE>
__global__ void rglru_scan_kernel(T* __restrict__ out, const float* __restrict__ coef, RgIn in, float* __restrict__ chunk_state,
                                  float* __restrict__ chunk_decay, int chunk, int max_chunks) {
    const int ch = blockIdx.x * blockDim.x + threadIdx.x;
    const int s = MODE == RGLRU_WHOLE ? blockIdx.y : blockIdx.y / max_chunks;
    if (ch >= in.W) return;
    int t0 = in.cu_tokens[s], t1 = in.cu_tokens[s + 1];
    if (MODE != RGLRU_WHOLE) {
        t0 += (blockIdx.y - s * max_chunks) * chunk;
        if (t0 >= t1) return;
        t1 = min(t1, t0 + chunk);
    }
    float* sp = MODE == RGLRU_WHOLE ? in.state + (long)in.seq_slot[s] * in.state_ld + ch : chunk_state + (long)blockIdx.y * in.W + ch;
    float S = MODE == RGLRU_LOCAL ? 0.f : *sp, decay = 1.f;
    const float yb = in.y_bias ? in.y_bias[ch] : 0.f;
    for (int t = t0; t < t1; t += UNROLL) {
        float2 ab[UNROLL];
        float yr[UNROLL];
#pragma unroll
        for (int i = 0; i < UNROLL; ++i) {
            const long m = min(t + i, t1 - 1);
            ab[i] = *reinterpret_cast<const float2*>(coef + (m * in.W + ch) * 2);
            if (MODE != RGLRU_LOCAL) yr[i] = Io<T>::ld((const T*)in.y + m * in.ld + ch);
        }
#pragma unroll
        for (int i = 0; i < UNROLL; ++i) {
            if (t + i < t1) {
                S = ab[i].x * S + ab[i].y;
                decay *= ab[i].x;
                if (MODE != RGLRU_LOCAL) Io<T>::st(out + (long)(t + i) * in.W + ch, S * rg_gelu(yr[i] + yb));
            }
        }
    }
    if (MODE != RGLRU_OUTPUT) *sp = S;
    if (MODE == RGLRU_LOCAL) chunk_decay[(long)blockIdx.y * in.W + ch] = decay;
}

__global__ void rglru_carry_kernel(RgIn in, float* __restrict__ chunk_state, const float* __restrict__ chunk_decay, int chunk,
                                   int max_chunks) {
    const int ch = blockIdx.x * blockDim.x + threadIdx.x, s = blockIdx.y;
    if (ch >= in.W) return;
    const int n_chunks = (in.cu_tokens[s + 1] - in.cu_tokens[s] + chunk - 1) / chunk;
    float* sp = in.state + (long)in.seq_slot[s] * in.state_ld + ch;
    float S = *sp;
    const long at = (long)s * max_chunks * in.W + ch;
    for (int c0 = 0; c0 < n_chunks; c0 += 8) {  // eight chunks' loads at once
        float add[8], dec[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const long k = at + (long)min(c0 + j, n_chunks - 1) * in.W;
            add[j] = chunk_state[k];
            dec[j] = chunk_decay[k];
        }
#pragma unroll
        for (int j = 0; j < 8; ++j)
            if (c0 + j < n_chunks) {
                chunk_state[at + (long)(c0 + j) * in.W] = S;
                S = dec[j] * S + add[j];
            }
    }
    *sp = S;
}

template <typename T, int KMAX>
static int launch_rglru(T* out, float* coef, const RgIn& in, int blocks, int one_each, float* chunk_state, float* chunk_decay, int chunk,
                        int max_chunks, hipStream_t s) {
    const unsigned tiles = (in.part + 63) / 64;
    if (one_each) {
        hipLaunchKernelGGL((rglru_step_kernel<T, KMAX>), dim3(tiles, blocks, (in.M + 15) / 16), dim3(256), 0, s, out, in);
        return pta_check_launch("rglru");
    }
    if (in.M >= 256)
        hipLaunchKernelGGL((rglru_gates_kernel<T, 4, KMAX>), dim3(tiles, blocks, (in.M + 63) / 64), dim3(256), 0, s, coef, in);
    else
        hipLaunchKernelGGL((rglru_gates_kernel<T, 1, KMAX>), dim3(tiles, blocks, (in.M + 15) / 16), dim3(256), 0, s, coef, in);
    const dim3 block(64);
    const unsigned cb = (in.W + 63) / 64;
    if (in.taps > 1) hipLaunchKernelGGL(rglru_ring_kernel<T>, dim3(cb, in.n_seqs), block, 0, s, in);
#define RGLRU_SCAN(MODE_, RUNS_) \
    hipLaunchKernelGGL((rglru_scan_kernel<T, 8, MODE_>), dim3(cb, RUNS_), block, 0, s, out, coef, in, chunk_state, chunk_decay, chunk, max_chunks)
    if (max_chunks <= 1) {
        RGLRU_SCAN(RGLRU_WHOLE, in.n_seqs);
        return pta_check_launch("rglru");
    }
    RGLRU_SCAN(RGLRU_LOCAL, in.n_seqs * max_chunks);
    hipLaunchKernelGGL(rglru_carry_kernel, dim3(cb, in.n_seqs), block, 0, s, in, chunk_state, chunk_decay, chunk, max_chunks);
    RGLRU_SCAN(RGLRU_OUTPUT, in.n_seqs * max_chunks);
#undef RGLRU_SCAN
    return pta_check_launch("rglru");
}

// out [M, W] (compute type, dense); y, x [M, W] blocks of columns, rows ld apart; conv [taps, W]; gates [blocks, 2, padded, padded] in
// the compute type: a part's Wr and Wi, rows and columns filled up with zeros to a multiple of 32; the vectors [W].  state (W
// numbers) and ring (taps * W) are columns of one state table with rows state_ld apart.  one_each: every sequence brings exactly
// one token, row m being sequence m's.  Else coef [M, W, 2] is scratch, and chunk_state and chunk_decay [n_seqs * max_chunks, W]
// for steps whose longest sequence is cut into max_chunks > 1 chunks of `chunk` tokens.
extern "C" int pta_rglru(void* out, const void* y, const void* x, long ld, const float* y_bias, const float* x_bias, const float* conv,
                         const float* conv_bias, const void* gates, const float* r_bias, const float* i_bias, const float* lam, float rate,
                         float* state, float* ring, long state_ld, float* coef, float* chunk_state, float* chunk_decay, const int* token_pos,
                         const int* token_seq, const int* cu_tokens, const int* seq_slot, int n_seqs, int one_each, int M, int W, int blocks,
                         int padded, int taps, int chunk, int max_chunks, int dtype, void* stream) {
    PTA_REQUIRE(n_seqs > 0 && M > 0 && W > 0 && blocks > 0 && W % blocks == 0, "rglru: %d channels in %d parts", W, blocks);
    PTA_REQUIRE(padded % 32 == 0 && padded >= W / blocks, "rglru: gate matrices of %d rows for parts of %d channels", padded, W / blocks);
    PTA_REQUIRE(taps >= 1 && taps <= RGLRU_MAX_TAPS, "rglru: %d taps are outside 1..%d", taps, RGLRU_MAX_TAPS);
    PTA_REQUIRE(out && y && x && conv && gates && r_bias && i_bias && lam && state && ring && token_pos && token_seq && cu_tokens && seq_slot,
                "rglru: null pointer");
    PTA_REQUIRE(ld >= W && state_ld >= (long)(taps + 1) * W, "rglru: rows lie closer together than they are long");
    PTA_REQUIRE(!one_each || M == n_seqs, "rglru: %d tokens of %d sequences are not one each", M, n_seqs);
    PTA_REQUIRE(one_each || coef, "rglru: steps of several tokens need their scratch memory");
    PTA_REQUIRE(max_chunks >= 1 && (max_chunks == 1 || (chunk > 0 && chunk_state && chunk_decay)), "rglru: chunks need their size and scratch memory");
    PTA_REQUIRE((long)n_seqs * max_chunks <= 65535 && blocks <= 65535 && (M + 15) / 16 <= 65535, "rglru: more than one launch takes");
    PTA_REQUIRE(((uintptr_t)gates % 16) == 0 && ((uintptr_t)coef % 8) == 0, "rglru: gate matrices must be aligned to sixteen bytes");
    PTA_REQUIRE(dtype == PTA_F32 || dtype == PTA_BF16, "rglru: unknown dtype %d", dtype);
    const RgIn in{y, x, gates, ld, state_ld, y_bias, x_bias, conv, conv_bias, r_bias, i_bias, lam, rate, state, ring, token_pos, token_seq,
                  cu_tokens, seq_slot, n_seqs, M, W, W / blocks, padded, taps};
    hipStream_t s = (hipStream_t)stream;
    if (dtype == PTA_F32)
        return taps <= 4 ? launch_rglru<float, 4>((float*)out, coef, in, blocks, one_each, chunk_state, chunk_decay, chunk, max_chunks, s)
                         : launch_rglru<float, RGLRU_MAX_TAPS>((float*)out, coef, in, blocks, one_each, chunk_state, chunk_decay, chunk, max_chunks, s);
    return taps <= 4 ? launch_rglru<bf16_t, 4>((bf16_t*)out, coef, in, blocks, one_each, chunk_state, chunk_decay, chunk, max_chunks, s)
                     : launch_rglru<bf16_t, RGLRU_MAX_TAPS>((bf16_t*)out, coef, in, blocks, one_each, chunk_state, chunk_decay, chunk, max_chunks, s);
}
