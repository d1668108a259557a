// What the drivers of the run-time sized designs share: weights out of one allocation and a safetensors file, the tables of a step, the
// residual stream and logits, and the two ways a step is asked for.  A step is `n_tokens` consecutive tokens of every context of a batch;
// decode is a step of one token, prefill a step of many, over the same ops.  A design adds its weights, its scratch and its layers.
#pragma once

#include <algorithm>
#include <cstdio>
#include <filesystem>
#include <functional>
#include <memory>
#include <string>
#include <vector>

#include "glint/hip/ops.hh"
#include "glint/layered_context.hh"
#include "glint/model_options.hh"
#include "glint/safetensors.hh"
#include "glint/span_timer.hh"
#include "glint/state.hh"

namespace glint {

// One tensor of a design and where it goes.  The rows of a matrix may lie farther apart than they are long: matrices side by side form
// one for a product that adds theirs up.
template<typename DType>
struct DesignTensor
{
  std::string name;
  std::vector<uint64_t> shape;
  DType* dst;
  uint64_t stride; // elements from row to row
  float mean;      // of a random initialisation
  uint64_t cols() const { return shape.back(); }
  uint64_t elements() const
  {
    uint64_t n = 1;
    for ( const uint64_t d : shape ) {
      n *= d;
    }
    return n;
  }
};

// Walks over the weights of a design in the order they lie in memory.  Run twice: first with no memory behind it, to size it.
template<typename DType>
class WeightCursor
{
  DType* base_;
  std::vector<DesignTensor<DType>>& tensors_;
  uint64_t at_ { 0 };

public:
  WeightCursor( DType* base, std::vector<DesignTensor<DType>>& tensors )
    : base_( base )
    , tensors_( tensors )
  {
    tensors_.clear();
  }
  uint64_t elements() const { return at_; }
  void align() { at_ = ( at_ + 127 ) / 128 * 128; }
  // room for n elements; what no tensor is loaded into stays zero
  DType* take( const uint64_t n )
  {
    DType* p = base_ == nullptr ? nullptr : base_ + at_;
    at_ += n;
    return p;
  }
  // right behind the last one: tensors that form one matrix for a product
  DType* tensor( std::string name, std::vector<uint64_t> shape, const float mean = 0.0f )
  {
    tensors_.push_back( { std::move( name ), std::move( shape ), nullptr, 0, mean } );
    auto& t = tensors_.back();
    t.stride = t.cols();
    return t.dst = take( t.elements() );
  }
  DType* alone( std::string name, std::vector<uint64_t> shape, const float mean = 0.0f )
  {
    align();
    return tensor( std::move( name ), std::move( shape ), mean );
  }
  // columns [first, first + shape[1]) of the matrix at `matrix`, whose rows are `stride` elements long
  void columns( std::string name, std::vector<uint64_t> shape, DType* matrix, const uint64_t first, const uint64_t stride )
  {
    tensors_.push_back( { std::move( name ), std::move( shape ), matrix == nullptr ? nullptr : matrix + first, stride, 0.0f } );
  }
};

template<typename Tag, typename DType, typename Context>
class DesignDriver
{
public:
  using ConfigType = Tag;
  using DataTypeT = DType;
  using ContextType = Context;
  using SettingsType = DesignSettings;
  using StateType = BatchedInferenceState<ConfigType>;
  using ContextVector = std::vector<std::shared_ptr<Context>>;
  using Operations = hip::Operations<DType>;
  static constexpr gh_dtype DT = hip::gh_type<DType>();

  struct Sizes
  {
    uint32_t width, vocab, max_positions;
    float eps;       // of every norm over the stream
    float norm_base; // what a norm's stored weights are added to
  };

  virtual ~DesignDriver()
  {
    if ( tables_host_ != nullptr ) {
      (void)gh_host_free( tables_host_ );
    }
  }
  DesignDriver( const DesignDriver& ) = delete;
  DesignDriver& operator=( const DesignDriver& ) = delete;

  const SettingsType& settings() const { return settings_; }
  Operations& ops() { return ops_; }
  uint32_t vocab_size() const { return sizes_.vocab; }
  uint32_t max_positions() const { return sizes_.max_positions; }
  virtual size_t n_runs() const = 0;

  void time_device_spans( const bool on ) { spans_.enable( on ); }
  std::pair<double, uint64_t> device_spans() { return spans_.take(); }

  // every tensor of the design out of a safetensors file; empty string on success
  std::string load( const std::filesystem::path& model_dir )
  {
    SafeTensors file;
    if ( auto err = file.open( model_dir / "model.safetensors" ); !err.empty() ) {
      return err;
    }
    std::vector<DType> host;
    for ( const auto& t : tensors_ ) {
      const auto* src = file.find( t.name );
      if ( src == nullptr ) {
        return "tensor " + t.name + " is missing";
      }
      if ( src->shape != t.shape || src->dtype == "I32" ) {
        return "tensor " + t.name + " has another shape or type than config.json implies";
      }
      host.resize( src->elements() );
      for ( uint64_t i = 0; i < host.size(); i++ ) {
        host[i] = static_cast<DType>( SafeTensors::value( *src, i ) );
      }
      GLINT_GH( gh_memcpy_rows( t.dst, t.stride * sizeof( DType ), host.data(), t.cols() * sizeof( DType ), t.cols() * sizeof( DType ), host.size() / t.cols(),
                                GH_HOST_TO_DEVICE, ops_.stream() ) );
    }
    return load_tables( file );
  }

  // Whether a batch can be run at these positions: inside the model's positions, every context at the length it has, and none twice
  // (a context takes its tokens one after the other).
  bool positions_fit( const ContextVector& contexts, const uint32_t* start_pos, const uint32_t n_tokens ) const
  {
    std::vector<const void*> seen;
    for ( const auto& c : contexts ) {
      if ( !c->empty() ) {
        seen.push_back( c->data() );
      }
    }
    std::sort( seen.begin(), seen.end() );
    if ( std::adjacent_find( seen.begin(), seen.end() ) != seen.end() ) {
      return false;
    }
    for ( size_t i = 0; i < contexts.size(); i++ ) {
      if ( !contexts[i]->empty() && ( (uint64_t)start_pos[i] + n_tokens > sizes_.max_positions || !contexts[i]->takes( start_pos[i] ) ) ) {
        return false;
      }
    }
    return true;
  }
  bool positions_fit( const StateType& states, const ContextVector& contexts ) const
  {
    std::vector<uint32_t> pos( states.batch_size() );
    for ( size_t i = 0; i < pos.size(); i++ ) {
      pos[i] = states.token_pos( i );
    }
    return contexts.size() == pos.size() && positions_fit( contexts, pos.data(), 1 );
  }

  // one token of every active row: the next token of each is sampled into the state
  void forward( StateType& states, const ContextVector& contexts )
  {
    const size_t batch = states.batch_size();
    GLINT_CHECK( batch > 0 && batch <= settings_.concurrency_limit && contexts.size() == batch );
    GLINT_CHECK( states.next_stage() == InferenceStage::PreAttention && states.next_layer() == 0 );
    GLINT_CHECK( states.dtype() == dtype_of<DType>() );
    GLINT_CHECK( positions_fit( states, contexts ) );
    ensure_scratch( batch, batch );
    begin_tables( batch, batch, 0 );
    for ( size_t i = 0; i < batch; i++ ) {
      const bool live = states.active( i );
      GLINT_CHECK( !live || states.token( i ) < sizes_.vocab );
      put_context( i, *contexts[i], live ? states.token_pos( i ) : 0, 1 );
      table_tokens()[i] = live ? states.token( i ) : 0;
    }
    upload_tables();
    spans_.mark( 0, ops_.stream() );
    run_layers( batch, 1, true, nullptr );
    classify( batch );
    spans_.mark( 1, ops_.stream() );

    std::vector<float> temperatures;
    for ( size_t i = 0; i < batch; i++ ) {
      temperatures.push_back( states.temperature( i ) );
    }
    if ( std::any_of( temperatures.begin(), temperatures.end(), []( float t ) { return t > 0; } ) ) {
      logit_ops_.soft_sample( logits_.get(), temperatures, sizes_.vocab );
    }
    sample( batch );
    spans_.close();
    states.set_next_layer( 0 );
    states.set_next_stage( InferenceStage::PreAttention );
    for ( size_t i = 0; i < batch; i++ ) {
      if ( !contexts[i]->empty() ) {
        contexts[i]->set_length( states.token_pos( i ) + 1 );
      }
      if ( states.active( i ) ) {
        states.set_token( i, argmax_[i] );
        states.set_token_pos( i, states.token_pos( i ) + 1 );
        if ( states.check_finished( i ) || states.token_pos( i ) >= sizes_.max_positions ) {
          states.set_finished( i );
        }
      }
    }
  }

  // `n_tokens` consecutive tokens per context, context i from start_pos[i] on (row = context * n_tokens + token).
  //   want          rows whose logits are asked for, ascending; they go to logits_out (host, (want.size(), vocab) fp32)
  //   next_tokens   (batch) greedy token behind each context's last row, or nullptr
  //   residuals_out the residual stream behind every layer run (host, (runs, rows, width) fp32), or nullptr: for tests
  void prefill( const ContextVector& contexts,
                const uint32_t* start_pos,
                const uint32_t n_tokens,
                const uint32_t* token_ids,
                const std::vector<uint32_t>& want,
                float* logits_out,
                uint32_t* next_tokens,
                float* residuals_out = nullptr )
  {
    const size_t batch = contexts.size();
    const uint64_t rows = (uint64_t)batch * n_tokens;
    GLINT_CHECK( batch > 0 && batch <= settings_.concurrency_limit && n_tokens > 0 && rows <= 0x7fffffffull );
    GLINT_CHECK( positions_fit( contexts, start_pos, n_tokens ) );
    std::vector<uint32_t> picked = want;
    if ( next_tokens != nullptr ) {
      for ( size_t i = 0; i < batch; i++ ) {
        picked.push_back( static_cast<uint32_t>( ( i + 1 ) * n_tokens - 1 ) );
      }
    }
    ensure_scratch( rows, std::max<uint64_t>( 1, std::min<uint64_t>( picked.size(), LOGIT_ROWS ) ) );
    begin_tables( batch, rows, picked.size() );
    for ( size_t i = 0; i < batch; i++ ) {
      put_context( i, *contexts[i], start_pos[i], n_tokens );
    }
    for ( uint64_t r = 0; r < rows; r++ ) {
      GLINT_CHECK( token_ids[r] < sizes_.vocab );
      table_tokens()[r] = token_ids[r];
    }
    for ( size_t k = 0; k < picked.size(); k++ ) {
      GLINT_CHECK( picked[k] < rows );
      table_picked()[k] = picked[k];
    }
    upload_tables();
    run_layers( batch, n_tokens, false, residuals_out );
    // the wanted rows, at most LOGIT_ROWS of them at a time
    for ( size_t k = 0; k < picked.size(); k += LOGIT_ROWS ) {
      const size_t n = std::min<size_t>( LOGIT_ROWS, picked.size() - k );
      GLINT_GH( gh_gather_rows( picked_x_.get(), x_.get(), picked_dev() + k, n, rows, sizes_.width, ops_.stream() ) );
      gh_stream_step step = no_step();
      lead_out( step );
      GLINT_GH( gh_stream_out( picked_x_.get(), sizes_.width, n, &step, DT, ops_.stream() ) );
      classify( n );
      const size_t plain = k < want.size() ? std::min( n, want.size() - k ) : 0;
      if ( plain > 0 ) {
        logit_ops_.copy( logits_out + k * sizes_.vocab, logits_.get(), plain * sizes_.vocab * sizeof( float ), CopyType::DeviceToHost );
      }
      if ( plain < n ) {
        sample( n );
        for ( size_t j = plain; j < n; j++ ) {
          next_tokens[k + j - want.size()] = argmax_[j];
        }
      }
    }
    ops_.synchronize();
    for ( size_t i = 0; i < batch; i++ ) {
      if ( !contexts[i]->empty() ) {
        contexts[i]->set_length( start_pos[i] + n_tokens );
      }
    }
  }

  // logits of the last forward(): (batch, vocab) fp32, on the device
  float* logits() const { return logits_.get(); }
  void copy_logits( float* host, const uint64_t rows )
  {
    logit_ops_.copy( host, logits_.get(), rows * sizes_.vocab * sizeof( float ), CopyType::DeviceToHost );
  }

protected:
  static constexpr uint64_t LOGIT_ROWS = 256;

  DesignDriver( const Sizes& sizes, SettingsType settings, const ModelOptions& options, ContextPlan plan )
    : sizes_( sizes )
    , settings_( std::move( settings ) )
    , options_( options )
  {
    GLINT_CHECK( settings_.concurrency_limit > 0 && settings_.concurrency_limit <= MAX_BATCH_SIZE );
    settings_.plan = std::make_shared<const ContextPlan>( std::move( plan ) );
  }
  // the last thing a design's constructor does: weights are left for load(), or drawn N(0, weight_std) around each tensor's mean when
  // settings.randomize_parameters
  void allocate()
  {
    WeightCursor<DType> sizing( nullptr, tensors_ );
    lay_out( sizing );
    sizing.align();
    weights_ = ops_.device_allocate( sizing.elements() * sizeof( DType ) );
    GLINT_GH( gh_memset_zero( weights_.get(), sizing.elements() * sizeof( DType ), ops_.stream() ) );
    WeightCursor<DType> placing( weights_.get(), tensors_ );
    lay_out( placing );
    grow_tables( settings_.concurrency_limit, settings_.concurrency_limit, 0 );
    if ( settings_.randomize_parameters ) {
      uint64_t seed = options_.seed * 1000003ull;
      for ( const auto& t : tensors_ ) {
        const bool dense = t.stride == t.cols();
        for ( uint64_t r = 0; r < ( dense ? 1 : t.elements() / t.cols() ); r++ ) {
          GLINT_GH( gh_fill_normal( t.dst + r * t.stride, dense ? t.elements() : t.cols(), t.mean, options_.weight_std, seed++, DT, ops_.stream() ) );
        }
      }
      randomize_tables( seed );
      ops_.synchronize();
    }
  }

  // ---- what a design brings --------------------------------------------------------------------
  virtual void lay_out( WeightCursor<DType>& cursor ) = 0;
  // scratch of the layers for steps of up to `rows` rows; the device is idle
  virtual void allocate_layer_scratch( uint64_t rows ) = 0;
  // embedding and all layers, over the tables of this step; `all_rows_classified`: the output's norm of every row ends up in h.
  // residuals_out as prefill()'s
  virtual void run_layers( uint64_t batch, uint32_t n_tokens, bool all_rows_classified, float* residuals_out ) = 0;
  // logits of the first n rows of h
  virtual void classify( uint64_t n ) = 0;
  // tensors that are not copied as they are
  virtual std::string load_tables( const SafeTensors& ) { return {}; }
  virtual void randomize_tables( uint64_t ) {}

  // ---- scratch and tables: scratch grows to the largest step seen ------------------------------
  void ensure_scratch( const uint64_t rows, const uint64_t logit_rows )
  {
    if ( rows > rows_ ) {
      ops_.synchronize();
      x_ = logit_ops_.device_allocate( rows * sizes_.width * sizeof( float ) );
      h_ = ops_.device_allocate( std::max( rows, LOGIT_ROWS ) * sizes_.width * sizeof( DType ) );
      allocate_layer_scratch( rows );
      rows_ = rows;
    }
    if ( logit_rows > logit_rows_ ) {
      ops_.synchronize();
      logits_ = logit_ops_.device_allocate( logit_rows * sizes_.vocab * sizeof( float ) );
      picked_x_ = logit_ops_.device_allocate( logit_rows * sizes_.width * sizeof( float ) );
      argmax_dev_ = logit_ops_.device_allocate( logit_rows * sizeof( uint32_t ) );
      argmax_.resize( logit_rows );
      logit_rows_ = logit_rows;
    }
  }

  // one upload per step: [context base | start position | token | picked row], page-locked on the host
  void grow_tables( const uint64_t batch, const uint64_t rows, const uint64_t picked )
  {
    const uint64_t bytes = batch * ( sizeof( void* ) + sizeof( uint32_t ) ) + ( rows + picked ) * sizeof( uint32_t ) + 64;
    if ( bytes <= tables_bytes_ ) {
      return;
    }
    ops_.synchronize();
    if ( tables_host_ != nullptr ) {
      GLINT_GH( gh_host_free( tables_host_ ) );
    }
    tables_dev_ = ops_.device_allocate( bytes );
    void* pinned = nullptr;
    GLINT_GH( gh_host_malloc( &pinned, bytes ) );
    tables_host_ = static_cast<uint8_t*>( pinned );
    tables_bytes_ = bytes;
  }
  void begin_tables( const uint64_t batch, const uint64_t rows, const uint64_t picked )
  {
    // the last step ended with a wait for its results, so its upload has been read
    grow_tables( batch, rows, picked );
    t_batch_ = batch;
    t_rows_ = rows;
    t_picked_ = picked;
    max_start_ = 0;
  }
  uint64_t pos_off() const { return t_batch_ * sizeof( void* ); }
  uint64_t tokens_off() const { return pos_off() + t_batch_ * sizeof( uint32_t ); }
  uint64_t picked_off() const { return tokens_off() + t_rows_ * sizeof( uint32_t ); }
  uint32_t* table_tokens() { return reinterpret_cast<uint32_t*>( tables_host_ + tokens_off() ); }
  uint32_t* table_picked() { return reinterpret_cast<uint32_t*>( tables_host_ + picked_off() ); }
  void put_context( const size_t i, Context& ctx, const uint32_t pos, const uint32_t n_tokens )
  {
    GLINT_CHECK( ctx.prepare( pos, n_tokens ) );
    reinterpret_cast<void**>( tables_host_ )[i] = ctx.data();
    reinterpret_cast<uint32_t*>( tables_host_ + pos_off() )[i] = pos;
    max_start_ = std::max( max_start_, pos );
  }
  void upload_tables()
  {
    GLINT_GH( gh_memcpy( tables_dev_.get(), tables_host_, picked_off() + t_picked_ * sizeof( uint32_t ), GH_HOST_TO_DEVICE, 1, ops_.stream() ) );
  }
  const uint8_t* dev() const { return reinterpret_cast<const uint8_t*>( tables_dev_.get() ); }
  void* const* contexts_dev() const { return reinterpret_cast<void* const*>( tables_dev_.get() ); }
  const uint32_t* pos_dev() const { return reinterpret_cast<const uint32_t*>( dev() + pos_off() ); }
  const uint32_t* tokens_dev() const { return reinterpret_cast<const uint32_t*>( dev() + tokens_off() ); }
  const uint32_t* picked_dev() const { return reinterpret_cast<const uint32_t*>( dev() + picked_off() ); }

  // ---- steps of the residual stream --------------------------------------------------------------
  gh_stream_step no_step() const
  {
    gh_stream_step s {};
    s.eps = sizes_.eps;
    s.norm_base = sizes_.norm_base;
    return s;
  }
  // `norm` of the stream goes to h, the next product's input
  void lead_to( gh_stream_step& step, const DType* norm ) const
  {
    step.next_norm = norm;
    step.out = h_.get();
    step.out_stride = sizes_.width;
  }
  void lead_out( gh_stream_step& step ) const { lead_to( step, final_norm_ ); }
  void copy_residuals( float* out, const uint64_t run, const uint64_t rows )
  {
    if ( out != nullptr ) {
      logit_ops_.copy( out + run * rows * sizes_.width, x_.get(), rows * sizes_.width * sizeof( float ), CopyType::DeviceToHost );
    }
  }
  // greedy token of the first n rows of the logits, on the host
  void sample( const uint64_t n )
  {
    GLINT_GH( gh_argmax( argmax_.data(), reinterpret_cast<uint32_t*>( argmax_dev_.get() ), logits_.get(), sizes_.vocab, n, GH_F32, ops_.stream() ) );
  }

  Sizes sizes_;
  SettingsType settings_;
  ModelOptions options_;
  Operations ops_ {};
  hip::Operations<float> logit_ops_ {};
  DeviceSpans spans_ {};

  std::vector<DesignTensor<DType>> tensors_ {};
  typename Operations::DeviceUniquePtr weights_ {};
  DType* final_norm_ {}; // set by lay_out()

  typename Operations::DeviceUniquePtr h_ {}, tables_dev_ {};
  hip::Operations<float>::DeviceUniquePtr x_ {}, logits_ {}, picked_x_ {}, argmax_dev_ {};
  uint64_t rows_ { 0 }, logit_rows_ { 0 };
  std::vector<uint32_t> argmax_ {};
  uint8_t* tables_host_ { nullptr };
  uint64_t tables_bytes_ { 0 }, t_batch_ { 0 }, t_rows_ { 0 }, t_picked_ { 0 };
  uint32_t max_start_ { 0 };
};

} // namespace glint
