// Row-wise ops of designs whose residual stream is kept in fp32 and whose sizes come at run time (storage type bf16 or fp32):
// embedding with learned positions, the residual update behind a projection with its norms on either side, the gate of a feed-forward
// with biases, and the scaled output product.  One kernel per row where a norm needs the whole row; a row stays in registers between
// the reductions.
#include "gh_product.h"

#include <algorithm>
#include <type_traits>

namespace gh {
namespace {

bool aligned16( const void* p ) { return ( reinterpret_cast<uintptr_t>( p ) & 15u ) == 0; }

// ---- embedding ---------------------------------------------------------------------------------
template<typename E>
__global__ __launch_bounds__( 256 ) void embed_positions_kernel( float* __restrict__ x,
                                                                 const uint32_t* __restrict__ tokens,
                                                                 const uint32_t* __restrict__ start_pos,
                                                                 uint32_t n_tokens,
                                                                 const E* __restrict__ embed,
                                                                 const E* __restrict__ pos_table,
                                                                 uint32_t width,
                                                                 uint32_t vocab,
                                                                 uint32_t max_pos,
                                                                 E* __restrict__ copy,
                                                                 uint64_t copy_stride )
{
  const uint32_t row = blockIdx.x;
  const uint64_t token = min( tokens[row], vocab - 1 ); // rows without a context may hold anything
  const E* e = embed + token * width;
  const E* p = pos_table != nullptr ? pos_table + (uint64_t)min( start_pos[row / n_tokens] + row % n_tokens, max_pos - 1 ) * width : nullptr;
  for ( uint32_t c = threadIdx.x; c < width; c += blockDim.x ) {
    const float v = to_f32( e[c] ) + ( p != nullptr ? to_f32( p[c] ) : 0.0f );
    x[(uint64_t)row * width + c] = v;
    if ( copy != nullptr ) {
      copy[(uint64_t)row * copy_stride + c] = from_f32<E>( v );
    }
  }
}

// four columns a thread: width, strides and tables in groups of four
template<typename E>
__global__ __launch_bounds__( 256 ) void embed_positions4_kernel( float* __restrict__ x, const uint32_t* __restrict__ tokens, const uint32_t* __restrict__ start_pos,
                                                                  uint32_t n_tokens, const E* __restrict__ embed, const E* __restrict__ pos_table, uint32_t width,
                                                                  uint32_t vocab, uint32_t max_pos, E* __restrict__ copy, uint64_t copy_stride )
{
  const uint32_t row = blockIdx.x;
  const uint64_t token = min( tokens[row], vocab - 1 );
  const E* p = pos_table != nullptr ? pos_table + (uint64_t)min( start_pos[row / n_tokens] + row % n_tokens, max_pos - 1 ) * width : nullptr;
  for ( uint32_t c = 4 * threadIdx.x; c < width; c += 4 * blockDim.x ) {
    float4 v = ProductView<E>::load4( embed + token * width + c );
    if ( p != nullptr ) {
      const float4 a = ProductView<E>::load4( p + c );
      v = make_float4( v.x + a.x, v.y + a.y, v.z + a.z, v.w + a.w );
    }
    *reinterpret_cast<float4*>( x + (uint64_t)row * width + c ) = v;
    if ( copy != nullptr ) {
      E* to = copy + (uint64_t)row * copy_stride + c;
      to[0] = from_f32<E>( v.x ), to[1] = from_f32<E>( v.y ), to[2] = from_f32<E>( v.z ), to[3] = from_f32<E>( v.w );
    }
  }
}

// ---- residual update ---------------------------------------------------------------------------
struct StepPtrs
{
  const void *bias, *post_norm, *add, *next_norm;
  void* out;
  uint64_t out_stride;
  float eps;
  int accumulate;
  float norm_base; // added to the weights of the norms
};

__device__ __forceinline__ float row_sum( float v, float* smem )
{
  v = wave_sum( v );
  if ( ( threadIdx.x & 63 ) == 0 ) {
    smem[threadIdx.x >> 6] = v;
  }
  __syncthreads();
  float total = 0.0f;
  for ( uint32_t w = 0; w < blockDim.x / WAVE; w++ ) {
    total += smem[w];
  }
  return total;
}

template<typename E>
__device__ __forceinline__ float4 load4_e( const void* p, uint32_t c )
{
  return ProductView<E>::load4( static_cast<const E*>( p ) + c );
}

// A thread owns NV groups of four columns.  A group past the row's end reads group 0 and stores nothing: no load sits under a branch.
template<typename E, typename View, bool PRODUCT, int NV>
__global__ __launch_bounds__( 1024 ) void stream_step_kernel( float* __restrict__ x, View y, uint32_t width, StepPtrs p )
{
  __shared__ float s_post[16], s_next[16];
  const uint64_t row = blockIdx.x;
  float* xr = x + row * width;
  uint32_t col[NV];
  bool live[NV];
  float4 v[NV], old[NV];
#pragma unroll
  for ( int g = 0; g < NV; g++ ) {
    const uint32_t c = ( g * blockDim.x + threadIdx.x ) * 4;
    live[g] = c < width;
    col[g] = live[g] ? c : 0;
    old[g] = *reinterpret_cast<const float4*>( xr + col[g] );
  }
  if constexpr ( PRODUCT ) {
#pragma unroll
    for ( int g = 0; g < NV; g++ ) {
      v[g] = y.at4( row, col[g] );
    }
    if ( p.bias != nullptr ) {
#pragma unroll
      for ( int g = 0; g < NV; g++ ) {
        const float4 b = load4_e<E>( p.bias, col[g] );
        v[g] = make_float4( v[g].x + b.x, v[g].y + b.y, v[g].z + b.z, v[g].w + b.w );
      }
    }
    if ( p.post_norm != nullptr ) {
      float ss = 0.0f;
#pragma unroll
      for ( int g = 0; g < NV; g++ ) {
        ss += live[g] ? v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w : 0.0f;
      }
      const float inv = 1.0f / sqrtf( row_sum( ss, s_post ) / (float)width + p.eps );
#pragma unroll
      for ( int g = 0; g < NV; g++ ) {
        const float4 w = load4_e<E>( p.post_norm, col[g] );
        v[g] = make_float4( v[g].x * inv * ( p.norm_base + w.x ), v[g].y * inv * ( p.norm_base + w.y ), v[g].z * inv * ( p.norm_base + w.z ),
                            v[g].w * inv * ( p.norm_base + w.w ) );
      }
    }
#pragma unroll
    for ( int g = 0; g < NV; g++ ) {
      if ( p.accumulate ) {
        v[g] = make_float4( old[g].x + v[g].x, old[g].y + v[g].y, old[g].z + v[g].z, old[g].w + v[g].w );
      }
      if ( p.add != nullptr ) {
        const float4 a = load4_e<E>( p.add, col[g] );
        v[g] = make_float4( v[g].x + a.x, v[g].y + a.y, v[g].z + a.z, v[g].w + a.w );
      }
      if ( live[g] ) {
        *reinterpret_cast<float4*>( xr + col[g] ) = v[g];
      }
    }
  } else {
#pragma unroll
    for ( int g = 0; g < NV; g++ ) {
      v[g] = old[g];
    }
  }
  if ( p.out == nullptr ) {
    return;
  }
  float inv = 1.0f;
  if ( p.next_norm != nullptr ) {
    float ss = 0.0f;
#pragma unroll
    for ( int g = 0; g < NV; g++ ) {
      ss += live[g] ? v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w : 0.0f;
    }
    inv = 1.0f / sqrtf( row_sum( ss, s_next ) / (float)width + p.eps );
  }
  E* out = static_cast<E*>( p.out ) + row * p.out_stride;
#pragma unroll
  for ( int g = 0; g < NV; g++ ) {
    float4 w = make_float4( 1.0f, 1.0f, 1.0f, 1.0f );
    if ( p.next_norm != nullptr ) {
      w = load4_e<E>( p.next_norm, col[g] );
      w = make_float4( p.norm_base + w.x, p.norm_base + w.y, p.norm_base + w.z, p.norm_base + w.w );
    }
    union
    {
      E e[4];
      uint2 half;
      uint4 full;
    } o;
    o.e[0] = from_f32<E>( v[g].x * inv * w.x );
    o.e[1] = from_f32<E>( v[g].y * inv * w.y );
    o.e[2] = from_f32<E>( v[g].z * inv * w.z );
    o.e[3] = from_f32<E>( v[g].w * inv * w.w );
    if ( live[g] ) {
      if constexpr ( sizeof( E ) == 2 ) {
        *reinterpret_cast<uint2*>( out + col[g] ) = o.half;
      } else {
        *reinterpret_cast<uint4*>( out + col[g] ) = o.full;
      }
    }
  }
}

// any width: the row goes through memory between the passes (each thread re-reads only what it wrote)
template<typename E, typename View, bool PRODUCT>
__global__ __launch_bounds__( 256 ) void stream_step_any_kernel( float* __restrict__ x, View y, uint32_t width, StepPtrs p )
{
  __shared__ float s_post[16], s_next[16];
  const uint64_t row = blockIdx.x;
  float* xr = x + row * width;
  const E *bias = static_cast<const E*>( p.bias ), *post = static_cast<const E*>( p.post_norm ), *add = static_cast<const E*>( p.add ),
          *next = static_cast<const E*>( p.next_norm );
  if constexpr ( PRODUCT ) {
    float inv = 1.0f;
    if ( post != nullptr ) {
      float ss = 0.0f;
      for ( uint32_t c = threadIdx.x; c < width; c += blockDim.x ) {
        const float v = y.at( row, c ) + ( bias != nullptr ? to_f32( bias[c] ) : 0.0f );
        ss += v * v;
      }
      inv = 1.0f / sqrtf( row_sum( ss, s_post ) / (float)width + p.eps );
    }
    for ( uint32_t c = threadIdx.x; c < width; c += blockDim.x ) {
      float v = y.at( row, c ) + ( bias != nullptr ? to_f32( bias[c] ) : 0.0f );
      if ( post != nullptr ) {
        v = v * inv * ( p.norm_base + to_f32( post[c] ) );
      }
      v = ( p.accumulate ? xr[c] : 0.0f ) + v;
      if ( add != nullptr ) {
        v += to_f32( add[c] );
      }
      xr[c] = v;
    }
  }
  if ( p.out == nullptr ) {
    return;
  }
  float inv = 1.0f;
  if ( next != nullptr ) {
    float ss = 0.0f;
    for ( uint32_t c = threadIdx.x; c < width; c += blockDim.x ) {
      ss += xr[c] * xr[c];
    }
    inv = 1.0f / sqrtf( row_sum( ss, s_next ) / (float)width + p.eps );
  }
  E* out = static_cast<E*>( p.out ) + row * p.out_stride;
  for ( uint32_t c = threadIdx.x; c < width; c += blockDim.x ) {
    out[c] = from_f32<E>( xr[c] * inv * ( next != nullptr ? p.norm_base + to_f32( next[c] ) : 1.0f ) );
  }
}

template<typename E, bool PRODUCT, typename View>
int launch_step( float* x, const View& y, uint64_t width, uint64_t rows, const StepPtrs& p, hipStream_t st )
{
  const bool vec = width % 4 == 0 && width <= 32768 && y.stride % 4 == 0 && p.out_stride % 4 == 0 && aligned16( x ) && aligned16( p.out ) && aligned16( p.bias )
                   && aligned16( p.post_norm ) && aligned16( p.add ) && aligned16( p.next_norm );
  const uint32_t w = (uint32_t)width;
  if ( !vec ) {
    stream_step_any_kernel<E, View, PRODUCT><<<(unsigned)rows, 256, 0, st>>>( x, y, w, p );
    GH_LAUNCH_CHECK();
    return GH_OK;
  }
  const uint32_t groups = w / 4;
  // many rows: fewer threads with more of the row each; few rows: the row over as many threads as it has groups
  const uint32_t want = rows >= 1024 ? ( groups + 3 ) / 4 : groups;
  uint32_t threads = std::min<uint32_t>( 1024, std::max<uint32_t>( 64, ( want + 63 ) / 64 * 64 ) );
  const uint32_t nv = ( groups + threads - 1 ) / threads;
  if ( nv <= 1 ) {
    stream_step_kernel<E, View, PRODUCT, 1><<<(unsigned)rows, threads, 0, st>>>( x, y, w, p );
  } else if ( nv <= 2 ) {
    stream_step_kernel<E, View, PRODUCT, 2><<<(unsigned)rows, threads, 0, st>>>( x, y, w, p );
  } else if ( nv <= 4 ) {
    stream_step_kernel<E, View, PRODUCT, 4><<<(unsigned)rows, threads, 0, st>>>( x, y, w, p );
  } else {
    stream_step_kernel<E, View, PRODUCT, 8><<<(unsigned)rows, threads, 0, st>>>( x, y, w, p );
  }
  GH_LAUNCH_CHECK();
  return GH_OK;
}

StepPtrs step_ptrs( const gh_stream_step* s )
{
  return StepPtrs { s->bias, s->post_norm, s->add, s->next_norm, s->out, s->out_stride, s->eps, s->accumulate, s->norm_base };
}

// ---- gate of a feed-forward --------------------------------------------------------------------
// grid: (column groups of a row / 256, rows); V columns a thread: 8 (rounded products), 4 or 1
template<typename E, typename View, int V>
__global__ __launch_bounds__( 256 ) void gate_rows_kernel( E* __restrict__ hb, View y, const E* __restrict__ bias, uint32_t hidden, int act )
{
  const uint64_t row = blockIdx.y;
  const uint32_t c = ( blockIdx.x * 256 + threadIdx.x ) * V;
  if ( c >= hidden ) {
    return;
  }
  if constexpr ( V == 1 ) {
    float g = y.at( row, c ), u = y.at( row, hidden + c );
    if ( bias != nullptr ) {
      g += to_f32( bias[c] );
      u += to_f32( bias[hidden + c] );
    }
    hb[row * hidden + c] = from_f32<E>( activate<E>( g, act ) * u );
  } else {
    float g[V], u[V];
#pragma unroll
    for ( int k = 0; k < V; k += 4 ) {
      const float4 a = y.at4( row, c + k ), b = y.at4( row, hidden + c + k );
      g[k] = a.x, g[k + 1] = a.y, g[k + 2] = a.z, g[k + 3] = a.w;
      u[k] = b.x, u[k + 1] = b.y, u[k + 2] = b.z, u[k + 3] = b.w;
    }
    if ( bias != nullptr ) {
#pragma unroll
      for ( int k = 0; k < V; k += 4 ) {
        const float4 a = load4_e<E>( bias, c + k ), b = load4_e<E>( bias, hidden + c + k );
        g[k] += a.x, g[k + 1] += a.y, g[k + 2] += a.z, g[k + 3] += a.w;
        u[k] += b.x, u[k + 1] += b.y, u[k + 2] += b.z, u[k + 3] += b.w;
      }
    }
    union
    {
      E e[V];
      uint2 half[V * sizeof( E ) / 8];
      uint4 full[( V * sizeof( E ) + 15 ) / 16];
    } o;
#pragma unroll
    for ( int k = 0; k < V; k++ ) {
      o.e[k] = from_f32<E>( activate<E>( g[k], act ) * u[k] );
    }
    if constexpr ( V * sizeof( E ) == 8 ) {
      *reinterpret_cast<uint2*>( hb + row * hidden + c ) = o.half[0];
    } else {
#pragma unroll
      for ( uint32_t k = 0; k < V * sizeof( E ) / 16; k++ ) {
        reinterpret_cast<uint4*>( hb + row * hidden + c )[k] = o.full[k];
      }
    }
  }
}

// ---- fp32 output of a product ------------------------------------------------------------------
template<typename View>
__global__ __launch_bounds__( 256 ) void scale_rows_kernel( float* __restrict__ out, View y, uint32_t r, uint64_t rows, float scale )
{
  const uint64_t total = rows * r, stride = (uint64_t)gridDim.x * blockDim.x;
  for ( uint64_t i = (uint64_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += stride ) {
    out[i] = y.at( i / r, i % r ) * scale;
  }
}

unsigned grid_for( uint64_t items ) { return (unsigned)std::min<uint64_t>( std::max<uint64_t>( 1, ( items + 255 ) / 256 ), 16384 ); }

// ---- gather of rows ----------------------------------------------------------------------------
__global__ __launch_bounds__( 256 ) void gather_rows_kernel( float* __restrict__ out, const float* __restrict__ x, const uint32_t* __restrict__ rows, uint32_t n_rows,
                                                             uint32_t width )
{
  const uint32_t src = min( rows[blockIdx.x], n_rows - 1 );
  for ( uint32_t c = threadIdx.x; c < width; c += blockDim.x ) {
    out[(uint64_t)blockIdx.x * width + c] = x[(uint64_t)src * width + c];
  }
}

} // namespace
} // namespace gh

using namespace gh;

extern "C" {

int gh_embed_positions( float* x, const uint32_t* tokens_dev, const uint32_t* start_pos_dev, uint64_t batch, uint32_t n_tokens, const void* embed,
                        const void* pos_table, uint64_t width, uint64_t vocab, uint64_t max_pos, void* copy, uint64_t copy_stride, gh_dtype dt, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  const uint64_t rows = batch * n_tokens;
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( x && tokens_dev && start_pos_dev && embed && width > 0 && vocab > 0 && max_pos > 0, "gh_embed_positions: bad argument" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_embed_positions: unsupported dtype %d", (int)dt );
  GH_REQUIRE( rows < ( 1ull << 31 ) && width < ( 1ull << 31 ), "gh_embed_positions: too large" );
  auto launch = [&]( auto tag ) {
    using E = decltype( tag );
    const E *e = static_cast<const E*>( embed ), *p = static_cast<const E*>( pos_table );
    const bool vec = width % 4 == 0 && aligned16( x ) && aligned16( embed ) && aligned16( pos_table );
    const uint32_t threads = vec ? (uint32_t)std::min<uint64_t>( 256, ( width / 4 + 63 ) / 64 * 64 ) : 256;
    ( vec ? embed_positions4_kernel<E> : embed_positions_kernel<E> )<<<(unsigned)rows, threads, 0, as_stream( stream )>>>(
      x, tokens_dev, start_pos_dev, n_tokens, e, p, (uint32_t)width, (uint32_t)vocab, (uint32_t)max_pos, static_cast<E*>( copy ), copy_stride );
  };
  if ( dt == GH_F32 ) {
    launch( float {} );
  } else {
    launch( __bf16 {} );
  }
  GH_LAUNCH_CHECK();
  return GH_OK;
}

int gh_stream_out( float* x, uint64_t width, uint64_t rows, const gh_stream_step* step, gh_dtype dt, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( x && step && step->out && width > 0 && width < ( 1ull << 31 ) && rows < ( 1ull << 31 ), "gh_stream_out: bad argument" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_stream_out: unsupported dtype %d", (int)dt );
  const Product none;
  const ProductView<float> view( none );
  if ( dt == GH_F32 ) {
    return launch_step<float, false>( x, view, width, rows, step_ptrs( step ), as_stream( stream ) );
  }
  return launch_step<__bf16, false>( x, view, width, rows, step_ptrs( step ), as_stream( stream ) );
}

int gh_matmul_stream( float* x, const void* in, const void* w, uint64_t s, uint64_t width, uint64_t rows, const gh_stream_step* step, gh_dtype dt,
                      gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( x && in && w && step, "gh_matmul_stream: NULL pointer" );
  GH_REQUIRE( s > 0 && s < ( 1ull << 31 ) && width > 0 && width < ( 1ull << 31 ) && rows < ( 1ull << 31 ), "gh_matmul_stream: bad shape" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_matmul_stream: unsupported dtype %d", (int)dt );
  hipStream_t st = as_stream( stream );
  Product y;
  if ( int rc = make_product( in, w, s, width, rows, dt, false, st, &y ) ) {
    return rc;
  }
  return with_product( dt, y, [&]( auto tag, auto view ) { return launch_step<decltype( tag ), true>( x, view, width, rows, step_ptrs( step ), st ); } );
}

int gh_matmul_gate( void* hb, const void* x, const void* w_gate_up, const void* bias, uint64_t s, uint64_t hidden, uint64_t rows, int activation, gh_dtype dt,
                    gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( hb && x && w_gate_up, "gh_matmul_gate: NULL pointer" );
  GH_REQUIRE( s > 0 && s < ( 1ull << 31 ) && hidden > 0 && hidden < ( 1ull << 30 ) && rows < ( 1ull << 31 ), "gh_matmul_gate: bad shape" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_matmul_gate: unsupported dtype %d", (int)dt );
  GH_REQUIRE( activation == GH_ACT_SILU || activation == GH_ACT_GELU_TANH, "gh_matmul_gate: unknown activation %d", activation );
  hipStream_t st = as_stream( stream );
  Product y;
  if ( int rc = make_product( x, w_gate_up, s, 2 * hidden, rows, dt, false, st, &y ) ) {
    return rc;
  }
  return with_product( dt, y, [&]( auto tag, auto view ) -> int {
    using E = decltype( tag );
    using View = decltype( view );
    const E* b = static_cast<const E*>( bias );
    const bool vec = aligned16( hb ) && aligned16( bias );
    auto launch = [&]( auto v_tag ) {
      constexpr int V = decltype( v_tag )::value;
      for ( uint64_t r0 = 0; r0 < rows; r0 += 65535 ) { // a grid's second dimension ends there
        View part = view;
        part.data += r0 * view.stride;
        const dim3 grid( (unsigned)( ( hidden + 256 * V - 1 ) / ( 256 * V ) ), (unsigned)std::min<uint64_t>( 65535, rows - r0 ) );
        gate_rows_kernel<E, View, V><<<grid, 256, 0, st>>>( static_cast<E*>( hb ) + r0 * hidden, part, b, (uint32_t)hidden, activation );
      }
    };
    if ( vec && hidden % 8 == 0 && std::is_same_v<View, ProductView<__bf16>> ) {
      launch( std::integral_constant<int, 8> {} );
    } else if ( vec && hidden % 4 == 0 ) {
      launch( std::integral_constant<int, 4> {} );
    } else {
      launch( std::integral_constant<int, 1> {} );
    }
    GH_LAUNCH_CHECK();
    return GH_OK;
  } );
}

int gh_matmul_scaled( float* out, const void* x, const void* w, uint64_t s, uint64_t r, uint64_t rows, float scale, gh_dtype dt, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( out && x && w, "gh_matmul_scaled: NULL pointer" );
  GH_REQUIRE( s > 0 && s < ( 1ull << 31 ) && r > 0 && r < ( 1ull << 31 ) && rows < ( 1ull << 31 ), "gh_matmul_scaled: bad shape" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_matmul_scaled: unsupported dtype %d", (int)dt );
  hipStream_t st = as_stream( stream );
  Product y;
  if ( int rc = make_product( x, w, s, r, rows, dt, true, st, &y ) ) {
    return rc;
  }
  const ProductView<float> view( y );
  scale_rows_kernel<<<grid_for( rows * r ), 256, 0, st>>>( out, view, (uint32_t)r, rows, scale );
  GH_LAUNCH_CHECK();
  return GH_OK;
}

int gh_gather_rows( float* out, const float* x, const uint32_t* rows_dev, uint64_t n, uint64_t n_rows, uint64_t width, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( n == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( out && x && rows_dev && n_rows > 0 && width > 0 && n < ( 1ull << 31 ) && n_rows < ( 1ull << 31 ) && width < ( 1ull << 31 ),
              "gh_gather_rows: bad argument" );
  gather_rows_kernel<<<(unsigned)n, 256, 0, as_stream( stream )>>>( out, x, rows_dev, (uint32_t)n_rows, (uint32_t)width );
  GH_LAUNCH_CHECK();
  return GH_OK;
}

} // extern "C"
