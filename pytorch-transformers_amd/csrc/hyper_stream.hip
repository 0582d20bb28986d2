// Several residual streams in place of one (hyper-connections), held in 32-bit: per token S vectors x_1 .. x_S.
//
//   x_t <- sum_s mix[s, t] x_s + out[t] * y        (y: what a sublayer left; all streams at once from the old ones)
//   u    = sum_t in[t] x_t                         (what the next sublayer reads; in null: the plain sum)
//   n    = u / sqrt(mean(u^2) + eps) * (offset + w)
//   h    = n + sum_k c[k] * n of K - 1 - k tokens ago   (optional: a causal convolution per channel on the norm's output)
//
// One launch does all of it.  A workgroup owns a token: it forms the new streams feature by feature, leaves u in LDS
// for the second pass, and writes h in the compute type.  The convolution rides in it where every sequence brings one
// token: the inputs from before are then all in the sequence's tail (the last K - 1 norm outputs, oldest first, 32-bit),
// which the same threads move on.  Where sequences bring several tokens the launch leaves n in 32-bit (n_out) for the
// convolution's own launch (pta_conv_add).
#include "common.h"
#include "pta_kernels.h"

#include <algorithm>

#define HYPER_MAX_STREAMS 8

template <int V> struct Vec;
template <> struct Vec<4> {
    static __device__ __forceinline__ void ld(const float* p, float (&v)[4]) {
        const float4 q = *reinterpret_cast<const float4*>(p);
        v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
    }
    static __device__ __forceinline__ void ld(const bf16_t* p, float (&v)[4]) {
        const uint2 q = *reinterpret_cast<const uint2*>(p);
        v[0] = bf16_bits_to_f32((bf16_t)(q.x & 0xffffu)); v[1] = bf16_bits_to_f32((bf16_t)(q.x >> 16));
        v[2] = bf16_bits_to_f32((bf16_t)(q.y & 0xffffu)); v[3] = bf16_bits_to_f32((bf16_t)(q.y >> 16));
    }
    static __device__ __forceinline__ void st(float* p, const float (&v)[4]) {
        *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    }
    static __device__ __forceinline__ void st(bf16_t* p, const float (&v)[4]) {
        bf16_t r[4] = {f32_to_bf16_bits(v[0]), f32_to_bf16_bits(v[1]), f32_to_bf16_bits(v[2]), f32_to_bf16_bits(v[3])};
        *reinterpret_cast<uint2*>(p) = make_uint2((uint32_t)r[0] | ((uint32_t)r[1] << 16), (uint32_t)r[2] | ((uint32_t)r[3] << 16));
    }
};
template <> struct Vec<1> {
    template <typename T> static __device__ __forceinline__ void ld(const T* p, float (&v)[1]) { v[0] = Io<T>::ld(p); }
    template <typename T> static __device__ __forceinline__ void st(T* p, const float (&v)[1]) { Io<T>::st(p, v[0]); }
};

struct HyperArgs {
    void* h;              // [M, H] in the compute type, or null
    float* n_out;         // [M, H], or null
    float* u_out;         // [M, H], or null
    float* x_out;         // [M, S, H], or null
    const float* x;       // row m, stream s at x + m * x_row + s * x_stream
    long x_row, x_stream; // x_stream 0: the streams are all equal, one vector
    const void* y;        // [M, H] rows y_ld apart in the compute type, or null
    long y_ld;
    const float *mix, *out, *in;
    const float* w;
    float offset, eps;
    const int* rows;
    const float* conv;    // [K, H], or null
    int K;
    float* tail;
    long tail_ld;
    const int *token_seq, *seq_slot;
    int H;
};

template <typename T, int S, int V>
__global__ __launch_bounds__(1024) void hyper_norm_kernel(HyperArgs a) {
    extern __shared__ __attribute__((aligned(16))) float u_s[];
    __shared__ float red[16];
    const int m = blockIdx.x, H = a.H;
    const long src = a.rows ? a.rows[m] : m;
    const float* x = a.x + src * a.x_row;
    const T* y = a.y ? (const T*)a.y + src * a.y_ld : nullptr;
    float ss = 0.f;
    for (int i = threadIdx.x * V; i < H; i += blockDim.x * V) {
        float xs[S][V], yv[V], u[V];
#pragma unroll
        for (int s = 0; s < S; ++s) Vec<V>::ld(x + s * a.x_stream + i, xs[s]);
#pragma unroll
        for (int v = 0; v < V; ++v) u[v] = 0.f;
        if (y) Vec<V>::ld(y + i, yv);
#pragma unroll
        for (int t = 0; t < S; ++t) {
            float xt[V];
            if (y) {
                const float o = a.out[t];
#pragma unroll
                for (int v = 0; v < V; ++v) xt[v] = 0.f;
#pragma unroll
                for (int s = 0; s < S; ++s) {
                    const float c = a.mix[s * S + t];
#pragma unroll
                    for (int v = 0; v < V; ++v) xt[v] += c * xs[s][v];
                }
#pragma unroll
                for (int v = 0; v < V; ++v) xt[v] += o * yv[v];
                if (a.x_out) Vec<V>::st(a.x_out + ((long)m * S + t) * H + i, xt);
            } else {
#pragma unroll
                for (int v = 0; v < V; ++v) xt[v] = xs[t][v];
            }
            const float c = a.in ? a.in[t] : 1.f;
#pragma unroll
            for (int v = 0; v < V; ++v) u[v] += c * xt[v];
        }
        Vec<V>::st(u_s + i, u);
        if (a.u_out) Vec<V>::st(a.u_out + (long)m * H + i, u);
#pragma unroll
        for (int v = 0; v < V; ++v) ss += u[v] * u[v];
    }
    if (!a.h && !a.n_out) return;
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)H + a.eps);
    float* tl = a.conv && a.K > 1 ? a.tail + (long)a.seq_slot[a.token_seq[m]] * a.tail_ld : nullptr;
    for (int i = threadIdx.x * V; i < H; i += blockDim.x * V) {
        float n[V], w[V], h[V];
        Vec<V>::ld(u_s + i, n);
        Vec<V>::ld(a.w + i, w);
#pragma unroll
        for (int v = 0; v < V; ++v) n[v] = n[v] * inv * (a.offset + w[v]);
        if (a.n_out) Vec<V>::st(a.n_out + (long)m * H + i, n);
        if (!a.h) continue;
#pragma unroll
        for (int v = 0; v < V; ++v) h[v] = n[v];
        if (a.conv) {
            float acc[V], c[V];
#pragma unroll
            for (int v = 0; v < V; ++v) acc[v] = 0.f;
            for (int k = 0; k + 1 < a.K; ++k) {
                float before[V];
                Vec<V>::ld(tl + (long)k * H + i, before);
                Vec<V>::ld(a.conv + (long)k * H + i, c);
#pragma unroll
                for (int v = 0; v < V; ++v) acc[v] += c[v] * before[v];
                if (k > 0) Vec<V>::st(tl + (long)(k - 1) * H + i, before);  // each input moves one place towards the oldest
            }
            if (a.K > 1) Vec<V>::st(tl + (long)(a.K - 2) * H + i, n);
            Vec<V>::ld(a.conv + (long)(a.K - 1) * H + i, c);
#pragma unroll
            for (int v = 0; v < V; ++v) h[v] += acc[v] + c[v] * n[v];
        }
        Vec<V>::st((T*)a.h + (long)m * H + i, h);
    }
}

template <typename T, int S>
static int hyper_launch_s(const HyperArgs& a, int M, bool wide, hipStream_t s) {
    const int per = wide ? 4 : 1;
    const dim3 block(std::min(1024, std::max(64, ((a.H + per - 1) / per + 63) / 64 * 64)));
    const size_t lds = (size_t)a.H * sizeof(float);
    if (wide) hipLaunchKernelGGL((hyper_norm_kernel<T, S, 4>), dim3(M), block, lds, s, a);
    else hipLaunchKernelGGL((hyper_norm_kernel<T, S, 1>), dim3(M), block, lds, s, a);
    return pta_check_launch("hyper_norm");
}

template <typename T>
static int hyper_launch(const HyperArgs& a, int M, int S, bool wide, hipStream_t s) {
    switch (S) {
        case 1: return hyper_launch_s<T, 1>(a, M, wide, s);
        case 2: return hyper_launch_s<T, 2>(a, M, wide, s);
        case 3: return hyper_launch_s<T, 3>(a, M, wide, s);
        case 4: return hyper_launch_s<T, 4>(a, M, wide, s);
        case 5: return hyper_launch_s<T, 5>(a, M, wide, s);
        case 6: return hyper_launch_s<T, 6>(a, M, wide, s);
        case 7: return hyper_launch_s<T, 7>(a, M, wide, s);
        default: return hyper_launch_s<T, 8>(a, M, wide, s);
    }
}

extern "C" int pta_hyper_norm(void* h, float* n_out, float* u_out, float* x_out, const float* x, long x_row, long x_stream,
                              const void* y, long y_ld, const float* mix, const float* out, const float* in, const float* w,
                              float offset, float eps, const int* rows, const float* conv, int taps, float* tail, long tail_ld,
                              const int* token_seq, const int* seq_slot, int M, int H, int streams, int dtype, void* stream) {
    PTA_REQUIRE(M > 0 && H > 0, "hyper_norm: M=%d H=%d must be positive", M, H);
    PTA_REQUIRE(streams >= 1 && streams <= HYPER_MAX_STREAMS, "hyper_norm: %d streams are outside 1..%d", streams, HYPER_MAX_STREAMS);
    PTA_REQUIRE(H <= 16384, "hyper_norm: rows of %d features are more than the 16384 that fit the kernel's LDS", H);
    PTA_REQUIRE(x && (h || n_out || u_out || x_out), "hyper_norm: null pointer");
    PTA_REQUIRE((h == nullptr && n_out == nullptr) || w, "hyper_norm: a norm needs its weight");
    PTA_REQUIRE(!y || (mix && out && y_ld >= H), "hyper_norm: a sublayer's result needs the streams' mix and its weights");
    PTA_REQUIRE(x_stream == 0 || x_stream >= H, "hyper_norm: streams of %d features cannot lie %ld apart", H, x_stream);
    PTA_REQUIRE(x_row >= (x_stream ? (streams - 1) * x_stream + H : (long)H), "hyper_norm: a token's streams do not fit its row");
    PTA_REQUIRE(!x_out || (y && x_out != x && !rows), "hyper_norm: new streams need a sublayer's result and a buffer of their own");
    PTA_REQUIRE(!conv || (h && taps >= 1 && !rows && token_seq && seq_slot && (taps == 1 || (tail && tail_ld >= (long)(taps - 1) * H))),
                "hyper_norm: the convolution needs its inputs from before the step");
    PTA_REQUIRE(dtype == PTA_F32 || dtype == PTA_BF16, "hyper_norm: unknown dtype %d", dtype);
    const HyperArgs a{h, n_out, u_out, x_out, x, x_row, x_stream, y, y_ld, mix, out, in, w, offset, eps, rows, conv, taps, tail,
                      tail_ld, token_seq, seq_slot, H};
    auto at16 = [](const void* p) { return ((uintptr_t)p % 16) == 0; };
    const bool wide = H % 4 == 0 && x_row % 4 == 0 && x_stream % 4 == 0 && y_ld % 4 == 0 && tail_ld % 4 == 0 && at16(h) && at16(n_out) &&
                      at16(u_out) && at16(x_out) && at16(x) && at16(y) && at16(w) && at16(conv) && at16(tail);
    if (dtype == PTA_F32) return hyper_launch<float>(a, M, streams, wide, (hipStream_t)stream);
    return hyper_launch<bf16_t>(a, M, streams, wide, (hipStream_t)stream);
}
